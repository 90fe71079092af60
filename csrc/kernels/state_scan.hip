// Matrix-state recurrences of linear-attention mixers, S [key channels, value channels] fp32 per
// (request slot, head), kept transposed as [slots, H, dv, dk]:
//
//   channel-decayed delta rule   S <- diag(g_t) S;  u = beta_t (v_t - S^T k_t);  S <- S + k_t u^T;  o_t = S^T q_t
//       q, k: causal depthwise convolution + SiLU, unit vector per head (q also / sqrt(dk)); v: convolution + SiLU;
//       g = exp(-exp(A_log_h) softplus(z + dt_bias)) per head and key channel; beta = sigmoid(b);
//       afterwards o / rms(o) * w * sigmoid(gate) per head
//   lightning attention          S <- decay_h S + k_t v_t^T;  o_t = S^T q_t,   q, k, v = silu(projection)
//
// Prompt rows run in chunks of 16: over a chunk the recurrence is a few small matrix products (for the
// delta rule with a 16 x 16 triangular solve for the writes).  `chunk_prep` does everything that does not
// need the state, parallel over (chunk, head): convolutions, unit norms, running decays, the 16 x 16
// matrices, the decayed operands.  `chunk_scan` then walks the chunks of every (sequence, head) with the state
// in MFMA accumulators, all products in fp32 (16 x 16 x 4).  `conv_tail` rewrites the convolution tails in a
// launch of its own, because the rows before it read the old ones.  Single rows (decoding): `state_step`, one
// launch from the projections to the normed, gated head output, tails included -- a workgroup owns
// all heads that share a key head, so nobody else reads what it rewrites.
#include "common.h"

namespace {

template <typename T>
__device__ __forceinline__ float ex(float x) {
  if constexpr (sizeof(T) == 4) return expf(x);
  else return __expf(x);
}
template <typename T>
__device__ __forceinline__ float sigm(float x) {
  if constexpr (sizeof(T) == 4) return 1.f / (1.f + expf(-x));
  else return __builtin_amdgcn_rcpf(1.f + __expf(-x));
}
template <typename T>
__device__ __forceinline__ float silu(float x) {
  return x * sigm<T>(x);
}
// (16-bit models: the hardware's log of 1 + e^-|x|, absolute error of an fp32 rounding of 1)
template <typename T>
__device__ __forceinline__ float softplus(float x) {
  if constexpr (sizeof(T) == 4) return x > 20.f ? x : log1pf(expf(x));
  else return fmaxf(x, 0.f) + __logf(1.f + __expf(-fabsf(x)));
}
// decay factor of a raw decay input (A = exp(A_log) of the head)
template <typename T>
__device__ __forceinline__ float decay_of(float z, float bias, float A) {
  return ex<T>(-A * softplus<T>(z + bias));
}

// sum over aligned groups of L lanes, result in all of them
template <int L>
__device__ __forceinline__ float lanes_sum(float v) {
#define DPP_ADD(ctrl) \
  v += __builtin_bit_cast(float, __builtin_amdgcn_update_dpp(0, __builtin_bit_cast(int, v), ctrl, 0xF, 0xF, false))
  if constexpr (L >= 2) DPP_ADD(0xB1);    // quad_perm: neighbour
  if constexpr (L >= 4) DPP_ADD(0x4E);    // quad_perm: other pair
  if constexpr (L >= 8) DPP_ADD(0x141);   // row_half_mirror
  if constexpr (L >= 16) DPP_ADD(0x140);  // row_mirror
#undef DPP_ADD
  if constexpr (L >= 32) v += __shfl_xor(v, 16);
  if constexpr (L >= 64) v += __shfl_xor(v, 32);
  return v;
}

// N neighbouring elements; VEC: one aligned access
template <typename T, int N, bool VEC>
__device__ __forceinline__ void ldn(const T* p, float (&f)[N]) {
  if constexpr (VEC && N > 1) {
    typedef T vec __attribute__((ext_vector_type(N)));
    const vec t = *reinterpret_cast<const vec*>(p);
#pragma unroll
    for (int i = 0; i < N; ++i) f[i] = (float)t[i];
  } else {
#pragma unroll
    for (int i = 0; i < N; ++i) f[i] = (float)p[i];
  }
}

// ------------------------------------------------------------------------------------------
// prompt rows, in chunks of CH rows of a sequence (counted from its first row of the step)
// ------------------------------------------------------------------------------------------
constexpr int CH = 16;

// grid row z -> (sequence, chunk of it); every wave scans the sequence lengths
__device__ __forceinline__ bool find_chunk(const int* __restrict__ cu, int S, int z, int& s, int& c) {
  const int lane = threadIdx.x & 63;
  int before = 0;
  for (int base = 0; base < S; base += 64) {
    const int i = base + lane;
    const int n = i < S ? (cu[i + 1] - cu[i] + CH - 1) / CH : 0;
    int incl = n;
#pragma unroll
    for (int o = 1; o < 64; o <<= 1) {
      const int t = __shfl_up(incl, o);
      if (lane >= o) incl += t;
    }
    const int total = __shfl(incl, 63);
    if (z < before + total) {
      const unsigned long long m = __ballot(z < before + incl);
      const int l = __ffsll(m) - 1;
      s = base + l;
      c = z - before - (__shfl(incl, l) - __shfl(n, l));
      return true;
    }
    before += total;
  }
  return false;
}
// chunks of the sequences before s
__device__ __forceinline__ int chunks_before(const int* __restrict__ cu, int s) {
  int n = 0;
  for (int i = threadIdx.x & 63; i < s; i += 64) n += (cu[i + 1] - cu[i] + CH - 1) / CH;
#pragma unroll
  for (int o = 32; o > 0; o >>= 1) n += __shfl_xor(n, o);
  return n;
}

enum { DELTA = 0, LIGHTNING = 1 };

__device__ __forceinline__ f32x4 mfma4(float a, float b, f32x4 c) {
  return __builtin_amdgcn_mfma_f32_16x16x4f32(a, b, c, 0, 0, 0);
}

// What `chunk_prep` leaves for `chunk_scan`, per (chunk, head), in floats: the operands of the state
// products [CH][DKP] each (delta only: -G k), G q, the write keys transposed [DKP][CH], the state's decay over
// the chunk [DKP], the CH x CH matrices (delta only: the solved write matrix), the read-out of the writes.
template <int DKP, int MODE>
struct ChunkLayout {
  static constexpr int GK = 0, GQ = MODE == DELTA ? CH * DKP : 0, KT = GQ + CH * DKP, GC = KT + CH * DKP, TB = GC + DKP,
                       BM = TB + (MODE == DELTA ? CH * CH : 0), SIZE = BM + CH * CH;
};

struct PrepArgs {
  int64_t stride, z_stride, b_stride;   // rows of the projection (q, k, v / lightning: q, k), z, b
  int K;                                // taps
  const float *A_log, *dt_bias, *decay;
  float* ws;                            // [H][chunks] chunk operands
  const int *cu, *slot, *reset;
  int S, H, Hk, dk, dv;
};

// SiLU(convolution) of channels ch .. ch + N - 1 at rows r .. r + RW - 1 (clamped to `last`) of a sequence whose
// step starts at row r0; st: the sequence's tail of channel ch, null when it starts in this step
template <typename T, int N, int RW, int KT, bool VEC>
__device__ __forceinline__ void conv_rows(const T* __restrict__ x, int64_t stride, const T* __restrict__ w,
                                          const T* __restrict__ st, int K, int r0, int r, int last, int ch,
                                          float (&y)[RW][N]) {
  if constexpr (KT > 0) {
    float xs[RW + KT - 1][N], wt[KT][N];
#pragma unroll
    for (int i = 0; i < RW + KT - 1; ++i) {
      const int rr = min(max(r - (KT - 1) + i, r0), last);
      ldn<T, N, VEC>(x + (int64_t)rr * stride + ch, xs[i]);
    }
    constexpr int W = N * KT;          // neighbouring taps of the lane's channels
    float wf[W];
    if constexpr (VEC && (W == 4 || W == 8)) {
      ldn<T, W, true>(w + (int64_t)ch * KT, wf);
    } else {
#pragma unroll
      for (int i = 0; i < W; ++i) wf[i] = (float)w[(int64_t)ch * KT + i];
    }
#pragma unroll
    for (int n = 0; n < N; ++n)
#pragma unroll
      for (int j = 0; j < KT; ++j) wt[j][n] = wf[n * KT + j];
    if (r - r0 < KT - 1) {      // rows before the step come from the tail
#pragma unroll
      for (int i = 0; i < KT - 1; ++i) {
        const int back = r0 - (r - (KT - 1) + i);   // this many rows before the step
        if (back > 0) {
#pragma unroll
          for (int n = 0; n < N; ++n) xs[i][n] = st == nullptr ? 0.f : (float)st[n * (KT - 1) + KT - 1 - back];
        }
      }
    }
#pragma unroll
    for (int i = 0; i < RW; ++i)
#pragma unroll
      for (int n = 0; n < N; ++n) {
        float acc = 0.f;
#pragma unroll
        for (int j = 0; j < KT; ++j) acc += wt[j][n] * xs[i + j][n];
        y[i][n] = silu<T>(acc);
      }
  } else {
#pragma unroll
    for (int i = 0; i < RW; ++i)
#pragma unroll
      for (int n = 0; n < N; ++n) {
        float acc = 0.f;
        const int row = min(r + i, last);
        for (int j = 0; j < K; ++j) {
          const int rr = row - (K - 1) + j;
          const float t = rr >= r0 ? (float)x[(int64_t)rr * stride + ch + n]
                                   : (st == nullptr ? 0.f : (float)st[n * (K - 1) + K - 1 - (r0 - rr)]);
          acc += (float)w[(int64_t)(ch + n) * K + j] * t;
        }
        y[i][n] = silu<T>(acc);
      }
  }
}

// One workgroup per (chunk, head).  N channels of q / k per lane (64 N >= DKP), four rows per wave.
//   delta      A_ts = beta_t sum_c k_t k_s G_t / G_s (s < t);  the chunk's writes solve (1 + A) u = beta (v - (G k) S)
//   both       B_ts = sum_c q_t k_s G_t / G_s (s <= t):        o = (G q) S + B u
// with G_t the product of the decays from the chunk's start.  Rows beyond the sequence are empty: no key, no decay, nothing written.
template <typename T, int DKP, int MODE, int KT, bool VEC>
__global__ __launch_bounds__(256) void chunk_prep_kernel(const T* __restrict__ x, const T* __restrict__ k_in,
                                                         const T* __restrict__ w, const T* __restrict__ conv_state,
                                                         const T* __restrict__ z, const T* __restrict__ b,
                                                         T* __restrict__ v, PrepArgs a) {
  constexpr int N = DKP > 64 ? DKP / 64 : 1, LD = DKP + 4, RW = CH / 4;
  typedef ChunkLayout<DKP, MODE> Lay;
  __shared__ __attribute__((aligned(16))) float sq[CH][LD], sk[CH][LD], sa[MODE == DELTA ? CH : 1][LD];
  __shared__ __attribute__((aligned(16))) float sA[CH][CH + 4];
  __shared__ float sb[CH + 1], part[2][4][CH * CH];
  int s = 0, c = 0;
  if (!find_chunk(a.cu, a.S, blockIdx.x, s, c)) return;   // uniform per block
  const int h = blockIdx.y, tid = threadIdx.x, lane = tid & 63, wv = tid >> 6;
  const int rep = a.H / a.Hk, hk = h / rep, dk = a.dk, dv = a.dv, kd = a.Hk * dk;
  const int r0 = a.cu[s], r1 = a.cu[s + 1], ra = r0 + c * CH, nr = min(CH, r1 - ra), last = r1 - 1;
  const int64_t slot = a.slot[s];
  const bool fresh = a.reset[s] != 0;
  float* ws = a.ws + ((int64_t)h * gridDim.x + blockIdx.x) * Lay::SIZE;
  const int ch0 = lane * N, row0 = wv * RW;
  constexpr int NZ = CH * DKP / 256;      // decays per thread, all of one channel
  T zr[NZ], br = (T)0.f;
  float dtb = 0.f;
  if constexpr (MODE == DELTA) {          // (requested first, needed last)
    const int cc = min(tid % DKP, dk - 1);
    dtb = a.dt_bias[(int64_t)h * dk + cc];
#pragma unroll
    for (int u = 0; u < NZ; ++u)
      zr[u] = z[(int64_t)min(ra + (tid + 256 * u) / DKP, last) * a.z_stride + (int64_t)h * dk + cc];
    br = b[(int64_t)min(ra + tid % CH, last) * a.b_stride + h];
  }

  // ---- queries and keys of the wave's rows into LDS
  float q[RW][N], k[RW][N];
#pragma unroll
  for (int i = 0; i < RW; ++i)
#pragma unroll
    for (int n = 0; n < N; ++n) q[i][n] = k[i][n] = 0.f;
  if constexpr (MODE == DELTA) {
    const int C = 2 * kd + a.H * dv;
    auto tail = [&](int ch) -> const T* { return fresh ? nullptr : conv_state + (slot * C + ch) * (a.K - 1); };
    const int cq = hk * dk + ch0, ck = kd + cq;
    if (row0 < nr) {
      if (ch0 + N <= dk) {
        conv_rows<T, N, RW, KT, VEC>(x, a.stride, w, tail(cq), a.K, r0, ra + row0, last, cq, q);
        conv_rows<T, N, RW, KT, VEC>(x, a.stride, w, tail(ck), a.K, r0, ra + row0, last, ck, k);
      } else if constexpr (N > 1) {
#pragma unroll
        for (int n = 0; n < N; ++n)
          if (ch0 + n < dk) {
            float t[RW][1];
            conv_rows<T, 1, RW, KT, false>(x, a.stride, w, tail(cq + n), a.K, r0, ra + row0, last, cq + n, t);
#pragma unroll
            for (int i = 0; i < RW; ++i) q[i][n] = t[i][0];
            conv_rows<T, 1, RW, KT, false>(x, a.stride, w, tail(ck + n), a.K, r0, ra + row0, last, ck + n, t);
#pragma unroll
            for (int i = 0; i < RW; ++i) k[i][n] = t[i][0];
          }
      }
    }
    const float rd = 1.f / sqrtf((float)dk);
#pragma unroll
    for (int i = 0; i < RW; ++i) {
      float ssq = 0.f, ssk = 0.f;
#pragma unroll
      for (int n = 0; n < N; ++n) {
        ssq += q[i][n] * q[i][n];
        ssk += k[i][n] * k[i][n];
      }
      const float iq = rd / sqrtf(lanes_sum<64>(ssq) + 1e-6f), ik = 1.f / sqrtf(lanes_sum<64>(ssk) + 1e-6f);
#pragma unroll
      for (int n = 0; n < N; ++n) {
        q[i][n] *= iq;
        k[i][n] *= ik;
      }
    }
  } else {
#pragma unroll
    for (int i = 0; i < RW; ++i)
#pragma unroll
      for (int n = 0; n < N; ++n)
        if (row0 + i < nr && ch0 + n < dk) {
          const int64_t o = (int64_t)(ra + row0 + i) * a.stride + h * dk + ch0 + n;
          q[i][n] = silu<T>((float)x[o]);
          k[i][n] = silu<T>((float)k_in[o]);
        }
  }
  if (ch0 < DKP)
#pragma unroll
    for (int i = 0; i < RW; ++i)
#pragma unroll
      for (int n = 0; n < N; ++n) {
        const bool on = row0 + i < nr;
        sq[row0 + i][ch0 + n] = on ? q[i][n] : 0.f;
        sk[row0 + i][ch0 + n] = on ? k[i][n] : 0.f;
      }

  // ---- decays (log2), write strengths, values
  if constexpr (MODE == DELTA) {
    constexpr int NV = VEC ? 2 : 1;
    const int C = 2 * kd + a.H * dv;
    for (int cv = lane * NV; cv < dv && row0 < nr; cv += 64 * NV) {
      const int ch = 2 * kd + h * dv + cv;
      float t[RW][NV];
      conv_rows<T, NV, RW, KT, VEC>(x, a.stride, w, fresh ? nullptr : conv_state + (slot * C + ch) * (a.K - 1), a.K, r0,
                                    ra + row0, last, ch, t);
#pragma unroll
      for (int i = 0; i < RW; ++i)
        if (row0 + i < nr) {
          T* vo = v + ((int64_t)(ra + row0 + i) * a.H + h) * dv + cv;
#pragma unroll
          for (int n = 0; n < NV; ++n) vo[n] = (T)t[i][n];
        }
    }
    const float A = expf(a.A_log[h]) * 1.44269504088896341f;
#pragma unroll
    for (int u = 0; u < NZ; ++u) {
      const int t = (tid + 256 * u) / DKP, cc = tid % DKP;
      sa[t][cc] = t < nr && cc < dk ? -A * softplus<T>((float)zr[u] + dtb) : 0.f;
    }
    if (tid < CH) sb[tid] = tid < nr ? sigm<float>((float)br) : 0.f;
    __syncthreads();
    for (int cc = tid; cc < DKP; cc += 256) {   // running sums over the chunk
      float acc = 0.f;
#pragma unroll
      for (int t = 0; t < CH; ++t) {
        acc += sa[t][cc];
        sa[t][cc] = acc;
      }
    }
  } else {
    if (tid <= CH) sb[tid] = powf(a.decay[h], (float)tid);
  }
  __syncthreads();

  // ---- the CH x CH products (on fp32 MFMA: K order permuted as in the scan, the waves split the channels)
  float kk = 0.f, qk = 0.f;
  const int pt = tid / CH, pu = tid % CH;     // this thread's pair of rows
  {
    constexpr int M = DKP / 16;
    const int g = lane >> 4, li = lane & 15;
    bool wide = false;      // decays of the chunk beyond what the factored form can hold
    if constexpr (MODE == DELTA) {
      for (int cc = lane; cc < DKP; cc += 64) wide |= sa[CH - 1][cc] < -110.f;
      wide = __ballot(wide) != 0;      // (every wave looks at all channels: uniform over the block)
    }
    if (!wide) {
      // G_t / G_u = 2^(a_t - a_mid) 2^(a_mid - a_u): either factor at most 2^110
      f32x4 ckk = f32x4{0.f, 0.f, 0.f, 0.f}, cqk = ckk;
      for (int m = wv; m < M; m += 4) {
        const int cc = 16 * m + 4 * g;
        const f32x4 kr = *reinterpret_cast<const f32x4*>(&sk[li][cc]);
        f32x4 ka = kr, kb = kr, qa = *reinterpret_cast<const f32x4*>(&sq[li][cc]);
        if constexpr (MODE == DELTA) {
          const f32x4 al = *reinterpret_cast<const f32x4*>(&sa[li][cc]), am = *reinterpret_cast<const f32x4*>(&sa[CH / 2 - 1][cc]);
#pragma unroll
          for (int r = 0; r < 4; ++r) {
            const float f = __builtin_amdgcn_exp2f(al[r] - am[r]);
            ka[r] *= f;
            qa[r] *= f;
            kb[r] *= __builtin_amdgcn_exp2f(am[r] - al[r]);
          }
        }
#pragma unroll
        for (int r = 0; r < 4; ++r) {
          if constexpr (MODE == DELTA) ckk = mfma4(ka[r], kb[r], ckk);
          cqk = mfma4(qa[r], kb[r], cqk);
        }
      }
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        if constexpr (MODE == DELTA) part[0][wv][(4 * g + r) * CH + li] = ckk[r];
        part[1][wv][(4 * g + r) * CH + li] = cqk[r];
      }
      __syncthreads();
#pragma unroll
      for (int u = 0; u < 4; ++u) {
        if constexpr (MODE == DELTA) kk += part[0][u][tid];
        qk += part[1][u][tid];
      }
    } else if constexpr (MODE == DELTA) {     // one pair of rows per thread, every ratio on its own
      for (int cc = 0; cc < DKP; ++cc) {
        const float f = sk[pu][cc] * __builtin_amdgcn_exp2f(fminf(sa[pt][cc] - sa[pu][cc], 0.f));
        kk += sk[pt][cc] * f;
        qk += sq[pt][cc] * f;
      }
    }
  }
  if constexpr (MODE == DELTA) {
    sA[pt][pu] = pu < pt ? sb[pt] * kk : 0.f;
    ws[Lay::BM + tid] = pu <= pt ? qk : 0.f;
    __syncthreads();
    if (wv == 0) {   // X = (1 + A)^-1 column by column; the write matrix is X diag(beta)
      float X[CH];
#pragma unroll
      for (int t = 0; t < CH; ++t) {
        float acc = t == lane ? 1.f : 0.f;
#pragma unroll
        for (int u = 0; u < t; ++u) acc -= sA[t][u] * X[u];
        X[t] = acc;
      }
      if (lane < CH)
#pragma unroll
        for (int t = 0; t < CH; ++t) ws[Lay::TB + t * CH + lane] = X[t] * sb[lane];
    }
  } else {
    ws[Lay::BM + tid] = pu <= pt ? qk * sb[pt - pu] : 0.f;
  }
  // ---- operands of the state products
  for (int e = 4 * tid; e < CH * DKP; e += 1024) {
    const int t = e / DKP, cc = e % DKP;
    f32x4 gq = *reinterpret_cast<const f32x4*>(&sq[t][cc]);
    if constexpr (MODE == DELTA) {
      f32x4 gk = *reinterpret_cast<const f32x4*>(&sk[t][cc]);
      const f32x4 al = *reinterpret_cast<const f32x4*>(&sa[t][cc]);
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const float f = __builtin_amdgcn_exp2f(al[r]);
        gq[r] *= f;
        gk[r] *= -f;
      }
      *reinterpret_cast<f32x4*>(ws + Lay::GK + e) = gk;
    } else {
      gq *= sb[min(t + 1, nr)];
    }
    *reinterpret_cast<f32x4*>(ws + Lay::GQ + e) = gq;
  }
  for (int e = 4 * tid; e < CH * DKP; e += 1024) {
    const int cc = e / CH, t = e % CH;
    f32x4 kt;
#pragma unroll
    for (int r = 0; r < 4; ++r)
      kt[r] = sk[t + r][cc] * (MODE == DELTA ? __builtin_amdgcn_exp2f(sa[CH - 1][cc] - sa[t + r][cc]) : sb[max(nr - 1 - t - r, 0)]);
    *reinterpret_cast<f32x4*>(ws + Lay::KT + e) = kt;
  }
  for (int cc = tid; cc < DKP; cc += 256) ws[Lay::GC + cc] = MODE == DELTA ? __builtin_amdgcn_exp2f(sa[CH - 1][cc]) : sb[nr];
}

// state[slot][c][j] <- the raw input of the j-th of a sequence's last K - 1 rows
template <typename T>
__global__ __launch_bounds__(256) void conv_tail_kernel(const T* __restrict__ x, int64_t stride, T* __restrict__ state,
                                                        const int* __restrict__ cu, const int* __restrict__ slot,
                                                        const int* __restrict__ reset, int C, int K) {
  const int c = blockIdx.x * 256 + threadIdx.x, s = blockIdx.y;
  if (c >= C) return;
  const int r0 = cu[s], r1 = cu[s + 1], n = r1 - r0;
  if (n <= 0) return;
  T* st = state + ((int64_t)slot[s] * C + c) * (K - 1);
  const bool fresh = reset[s] != 0;
  for (int j = 0; j < K - 1; ++j) {   // (ascending: entry j + n is still the old one when entry j takes it)
    const int rr = r1 - (K - 1) + j;
    st[j] = rr >= r0 ? x[(int64_t)rr * stride + c] : (fresh ? (T)0.f : st[j + n]);
  }
}

struct ScanArgs {
  const float* ws;
  int chunks;
  int64_t v_stride;
  float* state;
  const int *cu, *slot, *reset;
  int H, dk, dv;
};

// Walks the chunks of one (sequence, head); wave w owns 16 value columns.  Accumulator layout of the
// 16 x 16 x 4 product: lane (g = lane / 16, li = lane % 16) holds rows 4 g + r of column li; as the second
// operand lane (g, li) supplies row g.  The order of a dot product's terms is free, so product r of a tile takes
// the rows {4 g + r}: an accumulator's element r IS the second operand, and the first operand's four elements
// are neighbours in LDS.  The state (channels 16 m + 4 g + r of column li) never leaves its accumulators.
template <typename T, int DKP, int MODE>
__global__ __launch_bounds__(256, 2) void chunk_scan_kernel(const T* __restrict__ v, T* __restrict__ out, ScanArgs a) {
  typedef ChunkLayout<DKP, MODE> Lay;
  constexpr int M = DKP / 16, LD = DKP + 4, LT = CH + 4;
  constexpr int OGK = 0, OGQ = MODE == DELTA ? CH * LD : 0, OKT = OGQ + CH * LD, OGC = OKT + DKP * LT, OTB = OGC + DKP,
                OBM = OTB + (MODE == DELTA ? CH * LT : 0), OSZ = OBM + CH * LT + 4;   // the same operands with padded rows
  constexpr int NF = (Lay::SIZE / 4 + 255) / 256;   // 16-byte loads per thread and chunk
  extern __shared__ __attribute__((aligned(16))) float sm[];
  const int s = blockIdx.x, h = blockIdx.y, tid = threadIdx.x, lane = tid & 63, g = lane >> 4, li = lane & 15;
  const int r0 = a.cu[s], r1 = a.cu[s + 1];
  if (r1 <= r0) return;   // uniform per block
  const int col = blockIdx.z * 64 + (tid >> 6) * 16 + li, dk = a.dk, dv = a.dv;
  const bool on = col < dv;
  float* st = a.state + (((int64_t)a.slot[s] * a.H + h) * dv + (on ? col : 0)) * dk;
  const bool vec = dk % 4 == 0;
  f32x4 S[M];
  const bool fresh = a.reset[s] != 0;
#pragma unroll
  for (int m = 0; m < M; ++m) {
    S[m] = f32x4{0.f, 0.f, 0.f, 0.f};
    const int c = 16 * m + 4 * g;
    if (on && !fresh && c < dk) {
      if (vec) S[m] = *reinterpret_cast<const f32x4*>(st + c);
      else
#pragma unroll
        for (int r = 0; r < 4; ++r) S[m][r] = c + r < dk ? st[c + r] : 0.f;
    }
  }
  const int nc = (r1 - r0 + CH - 1) / CH;
  const float* ws = a.ws + ((int64_t)h * a.chunks + chunks_before(a.cu, s)) * Lay::SIZE;
  // operands and values of the next chunk in flight (values unconverted: a use would wait for the load)
  f32x4 pre[NF];
  T pv[4];
  const T* vp = v + (int64_t)h * dv + (on ? col : 0);
  int at[NF];          // where they go in LDS (the surplus of the last round: four unused floats)
#pragma unroll
  for (int u = 0; u < NF; ++u) {
    const int e = 4 * (tid + 256 * u);
    if (e >= Lay::SIZE) at[u] = OSZ - 4;
    else if (MODE == DELTA && e < Lay::GQ) at[u] = OGK + e / DKP * LD + e % DKP;
    else if (e < Lay::KT) at[u] = OGQ + (e - Lay::GQ) / DKP * LD + (e - Lay::GQ) % DKP;
    else if (e < Lay::GC) at[u] = OKT + (e - Lay::KT) / CH * LT + (e - Lay::KT) % CH;
    else if (e < Lay::TB) at[u] = OGC + e - Lay::GC;
    else if (e < Lay::BM) at[u] = OTB + (e - Lay::TB) / CH * LT + (e - Lay::TB) % CH;
    else at[u] = OBM + (e - Lay::BM) / CH * LT + (e - Lay::BM) % CH;
  }
  // loads i0 .. i1 - 1 of the NF + 4 of chunk c (beyond the sequence: its last chunk again)
  auto fetch_part = [&](int c, int i0, int i1) {
    c = min(c, nc - 1);
    const f32x4* p = reinterpret_cast<const f32x4*>(ws + (int64_t)c * Lay::SIZE);
#pragma unroll
    for (int u = 0; u < NF; ++u)
      if (u >= i0 && u < i1) pre[u] = p[min(tid + 256 * u, Lay::SIZE / 4 - 1)];
#pragma unroll
    for (int r = 0; r < 4; ++r)
      if (NF + r >= i0 && NF + r < i1) pv[r] = vp[(int64_t)min(r0 + c * CH + 4 * g + r, r1 - 1) * a.v_stride];
  };
  auto store = [&](float* p) {
#pragma unroll
    for (int u = 0; u < NF; ++u) *reinterpret_cast<f32x4*>(p + at[u]) = pre[u];
  };
  auto rd4 = [](const float* p) { return *reinterpret_cast<const f32x4*>(p); };
  auto values = [&](int c) {
    f32x4 R;
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const float t = MODE == LIGHTNING ? silu<T>((float)pv[r]) : (float)pv[r];
      R[r] = r0 + c * CH + 4 * g + r < r1 ? t : 0.f;
    }
    return R;
  };
  fetch_part(0, 0, NF + 4);
  store(sm);
  f32x4 R = values(0);
  fetch_part(1, 0, NF + 4);
  __syncthreads();
  for (int c = 0; c < nc; ++c) {
    const float* p = sm + (c & 1) * OSZ;
    f32x4 O = f32x4{0.f, 0.f, 0.f, 0.f}, Vn = O;
    if constexpr (MODE == DELTA) {
      f32x4 gk[2], gq[2];      // (the next tile's operands are read while this one's products run)
      gk[0] = rd4(p + OGK + li * LD + 4 * g);
      gq[0] = rd4(p + OGQ + li * LD + 4 * g);
#pragma unroll
      for (int m = 0; m < M; ++m) {
        if (m + 1 < M) {
          gk[(m + 1) & 1] = rd4(p + OGK + li * LD + 16 * (m + 1) + 4 * g);
          gq[(m + 1) & 1] = rd4(p + OGQ + li * LD + 16 * (m + 1) + 4 * g);
        }
#pragma unroll
        for (int r = 0; r < 4; ++r) {
          R = mfma4(gk[m & 1][r], S[m][r], R);
          O = mfma4(gq[m & 1][r], S[m][r], O);
        }
        __builtin_amdgcn_sched_barrier(0);
      }
      const f32x4 tb = rd4(p + OTB + li * LT + 4 * g);
      f32x4 U = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int r = 0; r < 4; ++r) U = mfma4(tb[r], R[r], U);
      R = U;
    } else {
      f32x4 O2 = f32x4{0.f, 0.f, 0.f, 0.f};
      f32x4 gq[M];
#pragma unroll
      for (int m = 0; m < M; ++m) gq[m] = rd4(p + OGQ + li * LD + 16 * m + 4 * g);
#pragma unroll
      for (int m = 0; m < M; ++m)
#pragma unroll
        for (int r = 0; r < 4; r += 2) {
          O = mfma4(gq[m][r], S[m][r], O);
          O2 = mfma4(gq[m][r + 1], S[m][r + 1], O2);
        }
      O += O2;
    }
    if (c + 1 < nc) {      // the other buffer was last read before the barrier; a whole chunk's time for the next loads
      store(sm + ((c + 1) & 1) * OSZ);
      Vn = values(c + 1);
    }
    const f32x4 bm = rd4(p + OBM + li * LT + 4 * g);
    f32x4 kt[M], gc[M];
#pragma unroll
    for (int m = 0; m < M; ++m) {
      gc[m] = rd4(p + OGC + 16 * m + 4 * g);
      kt[m] = rd4(p + OKT + (16 * m + li) * LT + 4 * g);
    }
#pragma unroll
    for (int m = 0; m < M; ++m) S[m] *= gc[m];
    __builtin_amdgcn_sched_barrier(0);
#pragma unroll
    for (int r = 0; r < 4; ++r) {     // the loads of the chunk after next go out between the products
      O = mfma4(bm[r], R[r], O);
#pragma unroll
      for (int m = 0; m < M; ++m) {
        S[m] = mfma4(kt[m][r], R[r], S[m]);
        constexpr int STEP = 4 * M / (NF + 4) > 0 ? 4 * M / (NF + 4) : 1;
        if ((r * M + m) % STEP == STEP - 1 || r * M + m == 4 * M - 1) {
          const int i = (r * M + m) / STEP;
          if (r * M + m < 4 * M - 1) fetch_part(c + 2, i, i + 1);
          else fetch_part(c + 2, i, NF + 4);
          __builtin_amdgcn_sched_barrier(0);
        }
      }
    }
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int row = r0 + c * CH + 4 * g + r;
      if (on && row < r1) out[((int64_t)row * a.H + h) * dv + col] = (T)O[r];
    }
    R = Vn;
    __syncthreads();
  }
  if (!on) return;
#pragma unroll
  for (int m = 0; m < M; ++m) {
    const int c = 16 * m + 4 * g;
    if (c < dk) {
      if (vec) *reinterpret_cast<f32x4*>(st + c) = S[m];
      else
#pragma unroll
        for (int r = 0; r < 4; ++r)
          if (c + r < dk) st[c + r] = S[m][r];
    }
  }
}

// ------------------------------------------------------------------------------------------
// single rows
// ------------------------------------------------------------------------------------------
struct StepArgs {
  int64_t x_stride, z_stride, b_stride;   // lightning: x_stride of q / k / v
  int K;
  const float *A_log, *dt_bias, *decay;
  float eps;
  float* state;
  const int *cu, *slot, *reset;
  int H, Hk, dk, dv;
};

// raw convolution input of the row -> SiLU(convolution); the channel's tail moves on by one
template <typename T>
__device__ __forceinline__ float conv_step(const T* __restrict__ x, const T* __restrict__ w, T* __restrict__ st, int K,
                                           bool fresh) {
  const T cur = *x;
  float acc = (float)w[K - 1] * (float)cur;
  if (K <= 5) {          // (loads side by side, then the stores)
    T t[4];
#pragma unroll
    for (int j = 0; j < 4; ++j) t[j] = j < K - 1 && !fresh ? st[j] : (T)0.f;
#pragma unroll
    for (int j = 0; j < 4; ++j)
      if (j < K - 1) acc += (float)w[j] * (float)t[j];
#pragma unroll
    for (int j = 0; j < 4; ++j)
      if (j < K - 1) st[j] = j + 1 < K - 1 ? t[j + 1 < 4 ? j + 1 : 3] : cur;
  } else {
    for (int j = 0; j < K - 1; ++j) {
      const T t = fresh ? (T)0.f : st[j];
      acc += (float)w[j] * (float)t;
      if (j > 0) st[j - 1] = t;
    }
    st[K - 2] = cur;
  }
  return silu<T>(acc);
}

// One workgroup per (sequence, key head).  NB column passes of the state are in flight together; the
// first ones are requested before anything else is computed.
template <typename T, int L, int MODE>
__global__ __launch_bounds__(256) void state_step_kernel(const T* __restrict__ q, const T* __restrict__ k,
                                                         const T* __restrict__ v, const T* __restrict__ conv_w,
                                                         T* __restrict__ conv_state, const T* __restrict__ z,
                                                         const T* __restrict__ b, const T* __restrict__ norm_w,
                                                         T* __restrict__ out, StepArgs a) {
  constexpr int DKP = 8 * L, CPP = 256 / L, NB = 8, NU = DKP > 64 ? DKP / 64 : 1;
  extern __shared__ __attribute__((aligned(16))) float sm[];
  float *sq = sm, *sk = sm + DKP, *sg = sm + 2 * DKP, *sv = sm + 3 * DKP, *so = sv + a.dv, *sc = so + a.dv;
  const int s = blockIdx.x, hk = blockIdx.y, tid = threadIdx.x, lane = tid & 63, wv = tid >> 6;
  const int row = a.cu[s];
  if (a.cu[s + 1] <= row) return;   // uniform per block
  const int slot = a.slot[s], dk = a.dk, dv = a.dv, rep = a.H / a.Hk, kd = a.Hk * dk;
  const bool fresh = a.reset[s] != 0;
  const int C = 2 * kd + a.H * dv;
  const int li = tid % L, cg = tid / L;          // channel group, column of a pass
  const bool vec = dk == DKP;
  f32x4 S0[NB], S1[NB];
  auto load = [&](const float* st, int j0) {
#pragma unroll
    for (int i = 0; i < NB; ++i) {
      const int j = j0 + i * CPP + cg;
      S0[i] = S1[i] = f32x4{0.f, 0.f, 0.f, 0.f};
      if (fresh || j >= dv) continue;
      const float* p = st + (int64_t)j * dk;
      if (vec) {
        S0[i] = *reinterpret_cast<const f32x4*>(p + 4 * li);
        S1[i] = *reinterpret_cast<const f32x4*>(p + 4 * (L + li));
      } else {
#pragma unroll
        for (int e = 0; e < 4; ++e) {
          S0[i][e] = 4 * li + e < dk ? p[4 * li + e] : 0.f;
          S1[i][e] = 4 * (L + li) + e < dk ? p[4 * (L + li) + e] : 0.f;
        }
      }
    }
  };
  for (int e = 0; e < rep; ++e) {
    const int h = hk * rep + e;
    float* st = a.state + ((int64_t)slot * a.H + h) * dv * dk;
    load(st, 0);
    // wave 0 / 1: q / k (first head of the group), 2: decays, 3: values and the write strength
    if (wv < 2) {
      if (e == 0) {
        float t[NU], ss = 0.f;
        const int ch0 = (MODE == DELTA ? wv * kd : 0) + hk * dk;
        const T* src = MODE == DELTA ? q : (wv == 0 ? q : k);
#pragma unroll
        for (int u = 0; u < NU; ++u) {
          const int c = lane + 64 * u;
          t[u] = 0.f;
          if (c < dk) {
            const T* xp = src + (int64_t)row * a.x_stride + ch0 + c;
            if constexpr (MODE == DELTA)
              t[u] = conv_step<T>(xp, conv_w + (int64_t)(ch0 + c) * a.K, conv_state + ((int64_t)slot * C + ch0 + c) * (a.K - 1),
                                  a.K, fresh);
            else
              t[u] = silu<T>((float)*xp);
          }
          ss += t[u] * t[u];
        }
        float f = 1.f;
        if constexpr (MODE == DELTA) {
          f = 1.f / sqrtf(wave_sum(ss) + 1e-6f);
          if (wv == 0) f *= 1.f / sqrtf((float)dk);
        }
#pragma unroll
        for (int u = 0; u < NU; ++u)
          if (lane + 64 * u < DKP) (wv == 0 ? sq : sk)[lane + 64 * u] = t[u] * f;
      }
    } else if (wv == 2) {
      if constexpr (MODE == DELTA) {
        const float A = expf(a.A_log[h]);
#pragma unroll
        for (int u = 0; u < NU; ++u) {
          const int c = lane + 64 * u;
          if (c < DKP)
            sg[c] = c < dk ? decay_of<T>((float)z[(int64_t)row * a.z_stride + (int64_t)h * dk + c], a.dt_bias[(int64_t)h * dk + c], A)
                           : 0.f;
        }
      }
    } else {
      for (int c = lane; c < dv; c += 64) {
        if constexpr (MODE == DELTA) {
          const int ch = 2 * kd + h * dv + c;
          sv[c] = conv_step<T>(q + (int64_t)row * a.x_stride + ch, conv_w + (int64_t)ch * a.K,
                               conv_state + ((int64_t)slot * C + ch) * (a.K - 1), a.K, fresh);
        } else {
          sv[c] = silu<T>((float)v[(int64_t)row * a.x_stride + (int64_t)h * dv + c]);
        }
      }
      if (MODE == DELTA && lane == 0) sc[0] = sigm<float>((float)b[(int64_t)row * a.b_stride + h]);
    }
    __syncthreads();
    const f32x4 q0 = *reinterpret_cast<const f32x4*>(sq + 4 * li), q1 = *reinterpret_cast<const f32x4*>(sq + 4 * (L + li));
    const f32x4 k0 = *reinterpret_cast<const f32x4*>(sk + 4 * li), k1 = *reinterpret_cast<const f32x4*>(sk + 4 * (L + li));
    f32x4 g0, g1;
    float beta = 0.f, kq = 0.f;
    if constexpr (MODE == DELTA) {
      g0 = *reinterpret_cast<const f32x4*>(sg + 4 * li);
      g1 = *reinterpret_cast<const f32x4*>(sg + 4 * (L + li));
      beta = sc[0];
#pragma unroll
      for (int i = 0; i < 4; ++i) kq += q0[i] * k0[i] + q1[i] * k1[i];
      kq = lanes_sum<L>(kq);
    } else {
      const float d = a.decay[h];
      g0 = g1 = f32x4{d, d, d, d};
    }
    for (int j0 = 0; j0 < dv; j0 += NB * CPP) {
      if (j0 > 0) load(st, j0);
      float x1[NB], x2[NB];
#pragma unroll
      for (int i = 0; i < NB; ++i) {
        x1[i] = x2[i] = 0.f;
        const int j = j0 + i * CPP + cg;
        const float vj = sv[j < dv ? j : dv - 1];
#pragma unroll
        for (int c = 0; c < 4; ++c) {
          S0[i][c] *= g0[c];
          S1[i][c] *= g1[c];
          if constexpr (MODE == LIGHTNING) {
            S0[i][c] += k0[c] * vj;
            S1[i][c] += k1[c] * vj;
          } else {
            x1[i] += S0[i][c] * k0[c] + S1[i][c] * k1[c];
          }
          x2[i] += S0[i][c] * q0[c] + S1[i][c] * q1[c];
        }
        if constexpr (MODE == DELTA) x1[i] = lanes_sum<L>(x1[i]);
        x2[i] = lanes_sum<L>(x2[i]);
        if constexpr (MODE == DELTA) {
          const float u = (vj - x1[i]) * beta;
          x2[i] += u * kq;
          S0[i] += k0 * u;
          S1[i] += k1 * u;
        }
        if (j < dv) {
          float* w = st + (int64_t)j * dk;
          if (vec) {
            *reinterpret_cast<f32x4*>(w + 4 * li) = S0[i];
            *reinterpret_cast<f32x4*>(w + 4 * (L + li)) = S1[i];
          } else {
#pragma unroll
            for (int c = 0; c < 4; ++c) {
              if (4 * li + c < dk) w[4 * li + c] = S0[i][c];
              if (4 * (L + li) + c < dk) w[4 * (L + li) + c] = S1[i][c];
            }
          }
          if (li == 0) so[j] = x2[i];
        }
      }
    }
    __syncthreads();
    T* orow = out + (int64_t)row * a.H * dv + (int64_t)h * dv;
    if constexpr (MODE == DELTA) {
      float ss = 0.f;
      for (int c = lane; c < dv; c += 64) ss += so[c] * so[c];
      const float rs = 1.f / sqrtf(wave_sum(ss) / (float)dv + a.eps);
      const T* gate = z + (int64_t)row * a.z_stride + (int64_t)a.H * dk + (int64_t)h * dv;
      for (int c = tid; c < dv; c += 256) orow[c] = (T)(so[c] * rs * (float)norm_w[c] * sigm<T>((float)gate[c]));
      __syncthreads();   // (the next head's waves overwrite sg, sv and so)
    } else {
      for (int c = tid; c < dv; c += 256) orow[c] = (T)so[c];
    }
  }
}

int padded_dk(int dk) {
  int p = 16;
  while (p < dk) p *= 2;
  return p;
}

template <typename T, int DKP, int MODE>
int chunked(const void* x, const void* k, const void* v_in, const void* w, const void* conv_state, const void* z, const void* b,
            void* v, const PrepArgs& p, const ScanArgs& a, void* out, int chunks, bool vec, hipStream_t stream) {
  typedef ChunkLayout<DKP, MODE> Lay;
  const dim3 pg(chunks, p.H);
#define PREP(KT, V)                                                                                             \
  chunk_prep_kernel<T, DKP, MODE, KT, V><<<pg, 256, 0, stream>>>((const T*)x, (const T*)k, (const T*)w,        \
                                                                 (const T*)conv_state, (const T*)z, (const T*)b, (T*)v, p)
  if constexpr (MODE == LIGHTNING) {
    PREP(0, false);
  } else if (vec) {
    if (p.K == 2) PREP(2, true);
    else if (p.K == 3) PREP(3, true);
    else if (p.K == 4) PREP(4, true);
    else PREP(0, true);
  } else {
    if (p.K == 2) PREP(2, false);
    else if (p.K == 3) PREP(3, false);
    else if (p.K == 4) PREP(4, false);
    else PREP(0, false);
  }
#undef PREP
  OME_CHECK_LAUNCH();
  constexpr int LD = DKP + 4, LT = CH + 4;
  constexpr int lds = 2 * ((MODE == DELTA ? 2 : 1) * CH * LD + DKP * LT + DKP + (MODE == DELTA ? 2 : 1) * CH * LT + 4) * 4;
  static_assert(lds <= 160 * 1024 && Lay::SIZE % 4 == 0, "chunk operands in LDS");
  if constexpr (lds > 64 * 1024) {
    static bool done = false;   // (per instantiation; repeating the call is harmless)
    if (!done) {
      const hipError_t e = hipFuncSetAttribute((const void*)chunk_scan_kernel<T, DKP, MODE>,
                                               hipFuncAttributeMaxDynamicSharedMemorySize, lds);
      if (e != hipSuccess) return (int)e;
      done = true;
    }
  }
  const dim3 sg(p.S, p.H, (p.dv + 63) / 64);
  chunk_scan_kernel<T, DKP, MODE><<<sg, 256, lds, stream>>>((const T*)v_in, (T*)out, a);
  OME_CHECK_LAUNCH();
  return 0;
}

template <typename T, int MODE>
int chunked_by_width(const void* x, const void* k, const void* v_in, const void* w, const void* conv_state, const void* z,
                     const void* b, void* v, const PrepArgs& p, const ScanArgs& a, void* out, int chunks, bool vec,
                     hipStream_t stream) {
#define GO(D) chunked<T, D, MODE>(x, k, v_in, w, conv_state, z, b, v, p, a, out, chunks, vec, stream)
  switch (padded_dk(p.dk)) {
    case 16: return GO(16);
    case 32: return GO(32);
    case 64: return GO(64);
    case 128: return GO(128);
    default: return GO(256);
  }
#undef GO
}

template <typename T, int MODE>
int step_by_width(const void* q, const void* k, const void* v, const void* conv_w, void* conv_state, const void* z,
                  const void* b, const void* norm_w, void* out, const StepArgs& a, int S, hipStream_t stream) {
  const int DKP = padded_dk(a.dk);
  const size_t lds = ((size_t)3 * DKP + 2 * a.dv + 4) * sizeof(float);
  if (lds > 64 * 1024) return -4;
  const dim3 grid(S, a.Hk);
#define STEP(L)                                                                                                        \
  state_step_kernel<T, L, MODE><<<grid, 256, lds, stream>>>((const T*)q, (const T*)k, (const T*)v, (const T*)conv_w, \
                                                            (T*)conv_state, (const T*)z, (const T*)b, (const T*)norm_w, \
                                                            (T*)out, a)
  switch (DKP) {
    case 16: STEP(2); break;
    case 32: STEP(4); break;
    case 64: STEP(8); break;
    case 128: STEP(16); break;
    default: STEP(32); break;
  }
#undef STEP
  OME_CHECK_LAUNCH();
  return 0;
}

bool bad_shape(int S, int H, int Hk, int dk, int dv) {
  return Hk <= 0 || H <= 0 || H % Hk || dk <= 0 || dk > 256 || dv <= 0 || H > 65535 || S > 0x7fffffff / 64;
}

}  // namespace

OME_API int ome_conv_tail(const void* x, int64_t stride, void* state, const int* cu, const int* slot, const int* reset,
                          int S, int C, int K, int f32, hipStream_t stream) {
  if (S <= 0 || C <= 0 || K <= 1) return 0;
  if (S > 65535) return -3;
  const dim3 grid((C + 255) / 256, S);
  if (f32) conv_tail_kernel<float><<<grid, 256, 0, stream>>>((const float*)x, stride, (float*)state, cu, slot, reset, C, K);
  else conv_tail_kernel<bf16><<<grid, 256, 0, stream>>>((const bf16*)x, stride, (bf16*)state, cu, slot, reset, C, K);
  OME_CHECK_LAUNCH();
  return 0;
}

// floats of workspace per (chunk of 16 rows, head)
OME_API int ome_state_chunk_floats(int dk, int delta) {
  const int DKP = padded_dk(dk);
  return (delta ? 3 : 2) * CH * DKP + DKP + (delta ? 2 : 1) * CH * CH;
}

// Delta rule over the rows of every sequence.  x: projection rows [q (Hk * dk) | k (Hk * dk) | v (H * dv)] (row stride in
// elements), conv_w [C, K], conv_state [slots, C, K - 1]; z rows [decay inputs (H * dk) | ..], b rows [H]; v: scratch
// [T, H * dv]; ws: ome_state_chunk_floats per (chunk, head), chunks >= sum over sequences of ceil(rows / 16);
// state fp32 [slots, H, dv, dk]; out [T, H * dv] (before the head norm).
OME_API int ome_delta_scan(const void* x, int64_t stride, const void* conv_w, const void* conv_state, int K, const void* z,
                           int64_t z_stride, const void* b, int64_t b_stride, const float* A_log, const float* dt_bias, void* v,
                           float* ws, int chunks, float* state, void* out, const int* cu, const int* slot, const int* reset,
                           int S, int H, int Hk, int dk, int dv, int f32, hipStream_t stream) {
  if (S <= 0 || chunks <= 0) return 0;
  if (bad_shape(S, H, Hk, dk, dv) || K < 1 || K > 32) return -2;
  const PrepArgs p{stride, z_stride, b_stride, K, A_log, dt_bias, nullptr, ws, cu, slot, reset, S, H, Hk, dk, dv};
  const ScanArgs a{ws, chunks, (int64_t)H * dv, state, cu, slot, reset, H, dk, dv};
  const int N = padded_dk(dk) > 64 ? padded_dk(dk) / 64 : 1, A = N > 2 ? N : 2;   // elements a vector access needs aligned
  const bool vec = N > 1 && dk % A == 0 && dv % 2 == 0 && stride % A == 0 && ((uintptr_t)x & (A * (f32 ? 4 : 2) - 1)) == 0;
  if (f32) return chunked_by_width<float, DELTA>(x, nullptr, v, conv_w, conv_state, z, b, v, p, a, out, chunks, vec, stream);
  return chunked_by_width<bf16, DELTA>(x, nullptr, v, conv_w, conv_state, z, b, v, p, a, out, chunks, vec, stream);
}

// q / k [T, H * dk], v [T, H * dv]: views of one projection (row stride in elements); decay fp32 [H].
OME_API int ome_lightning_scan(const void* q, const void* k, const void* v, int64_t stride, const float* decay, float* ws,
                               int chunks, float* state, void* out, const int* cu, const int* slot, const int* reset, int S,
                               int H, int dk, int dv, int f32, hipStream_t stream) {
  if (S <= 0 || chunks <= 0) return 0;
  if (bad_shape(S, H, H, dk, dv)) return -2;
  const PrepArgs p{stride, 0, 0, 1, nullptr, nullptr, decay, ws, cu, slot, reset, S, H, H, dk, dv};
  const ScanArgs a{ws, chunks, stride, state, cu, slot, reset, H, dk, dv};
  if (f32)
    return chunked_by_width<float, LIGHTNING>(q, k, v, nullptr, nullptr, nullptr, nullptr, nullptr, p, a, out, chunks, false, stream);
  return chunked_by_width<bf16, LIGHTNING>(q, k, v, nullptr, nullptr, nullptr, nullptr, nullptr, p, a, out, chunks, false, stream);
}

// The whole mixer core for sequences of one row each: z rows [decay inputs (H * dk) | output gate (H * dv)].
OME_API int ome_delta_step(const void* x, int64_t stride, const void* conv_w, void* conv_state, int K, const void* z,
                           int64_t z_stride, const void* b, int64_t b_stride, const float* A_log, const float* dt_bias,
                           const void* norm_w, float eps, float* state, void* out, const int* cu, const int* slot,
                           const int* reset, int S, int H, int Hk, int dk, int dv, int f32, hipStream_t stream) {
  if (S <= 0) return 0;
  if (bad_shape(S, H, Hk, dk, dv) || K < 1 || K > 32) return -2;
  const StepArgs a{stride, z_stride, b_stride, K, A_log, dt_bias, nullptr, eps, state, cu, slot, reset, H, Hk, dk, dv};
  if (f32) return step_by_width<float, DELTA>(x, nullptr, nullptr, conv_w, conv_state, z, b, norm_w, out, a, S, stream);
  return step_by_width<bf16, DELTA>(x, nullptr, nullptr, conv_w, conv_state, z, b, norm_w, out, a, S, stream);
}

OME_API int ome_lightning_step(const void* q, const void* k, const void* v, int64_t stride, const float* decay,
                               float* state, void* out, const int* cu, const int* slot, const int* reset, int S, int H,
                               int dk, int dv, int f32, hipStream_t stream) {
  if (S <= 0) return 0;
  if (bad_shape(S, H, H, dk, dv)) return -2;
  const StepArgs a{stride, 0, 0, 1, nullptr, nullptr, decay, 0.f, state, cu, slot, reset, H, H, dk, dv};
  if (f32) return step_by_width<float, LIGHTNING>(q, k, v, nullptr, nullptr, nullptr, nullptr, nullptr, out, a, S, stream);
  return step_by_width<bf16, LIGHTNING>(q, k, v, nullptr, nullptr, nullptr, nullptr, nullptr, out, a, S, stream);
}
