// Matrix-state recurrences of linear-attention mixers, S [key channels, value channels] fp32 per
// (request slot, head), kept transposed as [slots, H, dv, dk]:
//
//   channel-decayed delta rule   S <- diag(g_t) S;  u = beta_t (v_t - S^T k_t);  S <- S + k_t u^T;  o_t = S^T q_t
//       q, k: causal depthwise convolution + SiLU, unit vector per head (q also / sqrt(dk)); v: convolution + SiLU;
//       g = exp(-exp(A_log_h) softplus(z + dt_bias)) per head and key channel; beta = sigmoid(b);
//       afterwards o / rms(o) * w * sigmoid(gate) per head
//   lightning attention          S <- decay_h S + k_t v_t^T;  o_t = S^T q_t,   q, k, v = silu(projection)
//
// Prompt rows: `delta_prep` (parallel over rows: convolutions and unit norms, q / k in fp32), then
// `state_scan` walks every sequence; `conv_tail` rewrites the convolution tails in a launch of its
// own, because the rows before it read the old ones.  Single rows (decoding): `state_step`, one
// launch from the projections to the normed, gated head output, tails included -- a workgroup owns
// all heads that share a key head, so nobody else reads what it rewrites.
//
// Scan layout: column j of S (all key channels of one value channel) is spread over L = DKP / 8 lanes
// of a wave, two groups of 4 neighbouring channels each (DKP: key width padded to 16 .. 512); the
// dot products with k and q are in-lane sums and an L-lane DPP reduction, every lane carries NC
// columns.  A workgroup takes 4 * (64 / L) * NC columns of one (sequence, head) and stages RB rows of
// q, k, decays and values in LDS at a time: the next block's loads are in flight while the current one
// runs, activations are applied once on the way into LDS, one barrier per block.
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
__device__ __forceinline__ float softplus(float x) { return x > 20.f ? x : log1pf(expf(x)); }
// decay factor of a raw decay input (A = exp(A_log) of the head)
__device__ __forceinline__ float decay_of(float z, float bias, float A) { return expf(-A * softplus(z + bias)); }

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
// convolutions + unit norms of prompt rows
// ------------------------------------------------------------------------------------------
struct PrepArgs {
  int64_t stride;        // of the projection rows [q | k | v]
  int C, K;              // convolved channels, taps
  const int* first;      // [T] first row of the row's sequence in this step
  const int* slot;       // [T] state slot, bit 30: the sequence starts in this step
  float *qn, *kn, *qk;   // [T, Hk, DKP] x 2, [T, Hk]
  int T, Hk, rep, dk, dv, DKP;
};

constexpr int PREP_ROWS = 4;   // rows per wave

// SiLU(convolution) of channels ch .. ch + N - 1 at rows r .. r + PREP_ROWS - 1
template <typename T, int N, int KT, bool VEC>
__device__ __forceinline__ void conv_rows(const T* __restrict__ x, const T* __restrict__ w, const T* __restrict__ state,
                                          const PrepArgs& a, int r, int ch, float (&y)[PREP_ROWS][N]) {
  if constexpr (KT > 0) {
    float xs[PREP_ROWS + KT - 1][N], wt[KT][N];
#pragma unroll
    for (int i = 0; i < PREP_ROWS + KT - 1; ++i) {
      const int rr = min(max(r - (KT - 1) + i, 0), a.T - 1);
      ldn<T, N, VEC>(x + (int64_t)rr * a.stride + ch, xs[i]);
    }
#pragma unroll
    for (int n = 0; n < N; ++n)
#pragma unroll
      for (int j = 0; j < KT; ++j) wt[j][n] = (float)w[(int64_t)(ch + n) * KT + j];
#pragma unroll
    for (int i = 0; i < PREP_ROWS; ++i) {
      const int row = min(r + i, a.T - 1);
      const int back = row - a.first[row];          // rows of the sequence before this one in the step
#pragma unroll
      for (int n = 0; n < N; ++n) y[i][n] = wt[KT - 1][n] * xs[i + KT - 1][n];
      if (back >= KT - 1) {
#pragma unroll
        for (int j = 0; j < KT - 1; ++j)
#pragma unroll
          for (int n = 0; n < N; ++n) y[i][n] += wt[j][n] * xs[i + j][n];
      } else {
        const int sl = a.slot[row];
        const bool fresh = (sl >> 30) & 1;
        const T* st = state + ((int64_t)(sl & 0x3fffffff) * a.C + ch) * (KT - 1);
#pragma unroll
        for (int j = 0; j < KT - 1; ++j) {
          const int d = KT - 1 - j;                 // tap j reads d rows back
#pragma unroll
          for (int n = 0; n < N; ++n) {
            const float t = d <= back ? xs[i + j][n] : (fresh ? 0.f : (float)st[n * (KT - 1) + KT - 1 - (d - back)]);
            y[i][n] += wt[j][n] * t;
          }
        }
      }
#pragma unroll
      for (int n = 0; n < N; ++n) y[i][n] = silu<T>(y[i][n]);
    }
  } else {
    const int K = a.K;
    for (int i = 0; i < PREP_ROWS; ++i) {
      const int row = min(r + i, a.T - 1);
      const int back = row - a.first[row], sl = a.slot[row];
      const bool fresh = (sl >> 30) & 1;
#pragma unroll
      for (int n = 0; n < N; ++n) {
        const T* st = state + ((int64_t)(sl & 0x3fffffff) * a.C + ch + n) * (K - 1);
        float acc = 0.f;
        for (int j = 0; j < K; ++j) {
          const int d = K - 1 - j;
          const float t = d <= back ? (float)x[(int64_t)(row - d) * a.stride + ch + n]
                                    : (fresh ? 0.f : (float)st[K - 1 - (d - back)]);
          acc += (float)w[(int64_t)(ch + n) * K + j] * t;
        }
        y[i][n] = silu<T>(acc);
      }
    }
  }
}

// One wave per (PREP_ROWS rows, key head): N channels of q and of k per lane (N * 64 >= DKP), then the
// values of the head's `rep` value heads.
template <typename T, int N, int KT, bool VEC>
__global__ __launch_bounds__(256) void delta_prep_kernel(const T* __restrict__ x, const T* __restrict__ w,
                                                         const T* __restrict__ state, T* __restrict__ v, PrepArgs a) {
  const int lane = threadIdx.x & 63;
  const int wid = blockIdx.x * 4 + (threadIdx.x >> 6);
  const int hk = wid % a.Hk, r = (wid / a.Hk) * PREP_ROWS;
  if (r >= a.T) return;   // whole wave
  const int c = lane * N, kd = a.Hk * a.dk;
  float q[PREP_ROWS][N], k[PREP_ROWS][N];
#pragma unroll
  for (int i = 0; i < PREP_ROWS; ++i)
#pragma unroll
    for (int n = 0; n < N; ++n) q[i][n] = k[i][n] = 0.f;
  if (c + N <= a.dk) {
    conv_rows<T, N, KT, VEC>(x, w, state, a, r, hk * a.dk + c, q);
    conv_rows<T, N, KT, VEC>(x, w, state, a, r, kd + hk * a.dk + c, k);
  } else if (N > 1) {
#pragma unroll
    for (int n = 0; n < N; ++n)
      if (c + n < a.dk) {
        float t[PREP_ROWS][1];
        conv_rows<T, 1, KT, false>(x, w, state, a, r, hk * a.dk + c + n, t);
        for (int i = 0; i < PREP_ROWS; ++i) q[i][n] = t[i][0];
        conv_rows<T, 1, KT, false>(x, w, state, a, r, kd + hk * a.dk + c + n, t);
        for (int i = 0; i < PREP_ROWS; ++i) k[i][n] = t[i][0];
      }
  }
  const float rd = 1.f / sqrtf((float)a.dk);
#pragma unroll
  for (int i = 0; i < PREP_ROWS; ++i) {
    float sq = 0.f, sk = 0.f, sqk = 0.f;
#pragma unroll
    for (int n = 0; n < N; ++n) {
      sq += q[i][n] * q[i][n];
      sk += k[i][n] * k[i][n];
      sqk += q[i][n] * k[i][n];
    }
    sq = wave_sum(sq);
    sk = wave_sum(sk);
    sqk = wave_sum(sqk);
    const float iq = rd / sqrtf(sq + 1e-6f), ik = 1.f / sqrtf(sk + 1e-6f);
    if (r + i < a.T) {
      const int64_t o = ((int64_t)(r + i) * a.Hk + hk);
      if (c < a.DKP) {    // (N divides DKP: the padding is written as zeros)
        float* qo = a.qn + o * a.DKP + c;
        float* ko = a.kn + o * a.DKP + c;
#pragma unroll
        for (int n = 0; n < N; ++n) {
          qo[n] = q[i][n] * iq;
          ko[n] = k[i][n] * ik;
        }
      }
      if (lane == 0) a.qk[o] = sqk * iq * ik;
    }
  }
  // values: rep * dv channels of the group, two per lane where that divides
  const int nv = a.rep * a.dv, v0 = hk * nv, VD = a.Hk * nv;
  constexpr int NV = VEC ? 2 : 1;
  for (int cv = lane * NV; cv < nv; cv += 64 * NV) {
    float t[PREP_ROWS][NV];
    conv_rows<T, NV, KT, VEC>(x, w, state, a, r, 2 * kd + v0 + cv, t);
#pragma unroll
    for (int i = 0; i < PREP_ROWS; ++i)
      if (r + i < a.T) {
        T* vo = v + (int64_t)(r + i) * VD + v0 + cv;
#pragma unroll
        for (int n = 0; n < NV; ++n) vo[n] = (T)t[i][n];
      }
  }
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

// ------------------------------------------------------------------------------------------
// scan
// ------------------------------------------------------------------------------------------
struct ScanArgs {
  const float *qn, *kn, *qk;          // delta: [T, Hk, DKP] x 2, [T, Hk]
  int64_t q_stride, v_stride;         // lightning: rows of the projection (q, k, v); delta: rows of v
  const float *A_log, *dt_bias;       // delta: [H], [H * dk]
  int64_t z_stride, b_stride;
  const float* decay;                 // lightning: [H]
  float* state;
  const int *cu, *slot, *reset;
  int H, Hk, dk, dv;
};

enum { DELTA = 0, LIGHTNING = 1 };

template <typename T, int L, int NC, int MODE, int RB>
__global__ __launch_bounds__(256) void state_scan_kernel(const T* __restrict__ q, const T* __restrict__ k,
                                                         const T* __restrict__ v, const T* __restrict__ z,
                                                         const T* __restrict__ b, T* __restrict__ out, ScanArgs a) {
  constexpr int DKP = 8 * L, GPW = 64 / L, CPB = 4 * GPW * NC;
  constexpr int NK = (RB * DKP + 255) / 256, NV = (RB * CPB + 255) / 256;   // staged elements per thread
  constexpr int ROWF = (MODE == DELTA ? 3 : 2) * DKP + CPB + 4;             // floats of a staged row
  __shared__ __attribute__((aligned(16))) float sm[2][RB][ROWF];
  const int s = blockIdx.x, h = blockIdx.y, tid = threadIdx.x;
  const int r0 = a.cu[s], r1 = a.cu[s + 1];
  if (r1 <= r0) return;   // uniform per block
  const int lane = tid & 63, wv = tid >> 6, li = lane % L;
  const int cb = blockIdx.z * CPB, cl = (wv * GPW + lane / L) * NC;   // the block's / the lane's first column
  const int hk = h / (a.H / a.Hk), dk = a.dk, dv = a.dv;
  const bool fresh = a.reset[s] != 0;
  float* st = a.state + ((int64_t)a.slot[s] * a.H + h) * dv * dk;
  const bool vec = dk == DKP;
  f32x4 S0[NC], S1[NC];
#pragma unroll
  for (int c = 0; c < NC; ++c) {
    S0[c] = S1[c] = f32x4{0.f, 0.f, 0.f, 0.f};
    if (!fresh && cb + cl + c < dv) {
      const float* p = st + (int64_t)(cb + cl + c) * dk;
      if (vec) {
        S0[c] = *reinterpret_cast<const f32x4*>(p + 4 * li);
        S1[c] = *reinterpret_cast<const f32x4*>(p + 4 * (L + li));
      } else {
#pragma unroll
        for (int e = 0; e < 4; ++e) {
          S0[c][e] = 4 * li + e < dk ? p[4 * li + e] : 0.f;
          S1[c][e] = 4 * (L + li) + e < dk ? p[4 * (L + li) + e] : 0.f;
        }
      }
    }
  }
  const float A = MODE == DELTA ? expf(a.A_log[h]) : 0.f;
  const float dec = MODE == LIGHTNING ? a.decay[h] : 0.f;

  // raw operands of the rows rb .. rb + RB - 1 (addresses clamped to the sequence and the head)
  float rq[NK], rk[NK], rz[MODE == DELTA ? NK : 1], rv[NV], rs = 0.f;
  auto fetch = [&](int rb) {
#pragma unroll
    for (int u = 0; u < NK; ++u) {
      const int e = tid + 256 * u, r = min(rb + e / DKP, r1 - 1), c = e % DKP;
      if constexpr (MODE == DELTA) {
        const int64_t o = ((int64_t)r * a.Hk + hk) * DKP + c;
        rq[u] = a.qn[o];
        rk[u] = a.kn[o];
        rz[u] = (float)z[(int64_t)r * a.z_stride + (int64_t)h * dk + min(c, dk - 1)];
      } else {
        const int64_t o = (int64_t)r * a.q_stride + (int64_t)hk * dk + min(c, dk - 1);
        rq[u] = (float)q[o];
        rk[u] = (float)k[o];
      }
    }
#pragma unroll
    for (int u = 0; u < NV; ++u) {
      const int e = tid + 256 * u, r = min(rb + e / CPB, r1 - 1), c = min(cb + e % CPB, dv - 1);
      rv[u] = (float)v[(int64_t)r * a.v_stride + (int64_t)h * dv + c];
    }
    if (MODE == DELTA && tid < 2 * RB) {
      const int r = min(rb + tid / 2, r1 - 1);
      rs = tid & 1 ? a.qk[(int64_t)r * a.Hk + hk] : (float)b[(int64_t)r * a.b_stride + h];
    }
  };
  float db[MODE == DELTA ? NK : 1];
  if constexpr (MODE == DELTA) {
#pragma unroll
    for (int u = 0; u < NK; ++u) db[u] = a.dt_bias[(int64_t)h * dk + min((tid + 256 * u) % DKP, dk - 1)];
  }
  auto store = [&](int p) {
#pragma unroll
    for (int u = 0; u < NK; ++u) {
      const int e = tid + 256 * u, r = e / DKP, c = e % DKP;
      if (RB * DKP % 256 == 0 || e < RB * DKP) {
        if constexpr (MODE == DELTA) {
          sm[p][r][c] = rq[u];
          sm[p][r][DKP + c] = rk[u];
          sm[p][r][2 * DKP + c] = decay_of(rz[u], db[u], A);
        } else {
          sm[p][r][c] = c < dk ? silu<T>(rq[u]) : 0.f;
          sm[p][r][DKP + c] = c < dk ? silu<T>(rk[u]) : 0.f;
        }
      }
    }
    constexpr int VO = (MODE == DELTA ? 3 : 2) * DKP;
#pragma unroll
    for (int u = 0; u < NV; ++u) {
      const int e = tid + 256 * u;
      if (RB * CPB % 256 == 0 || e < RB * CPB) sm[p][e / CPB][VO + e % CPB] = MODE == LIGHTNING ? silu<T>(rv[u]) : rv[u];
    }
    if (MODE == DELTA && tid < 2 * RB) sm[p][tid / 2][VO + CPB + (tid & 1)] = tid & 1 ? rs : sigm<float>(rs);
  };

  fetch(r0);
  store(0);
  __syncthreads();
  int p = 0;
  for (int rb = r0; rb < r1; rb += RB, p ^= 1) {
    const bool more = rb + RB < r1;
    if (more) fetch(rb + RB);
    const int nb = min(RB, r1 - rb);
#pragma unroll 2
    for (int t = 0; t < nb; ++t) {
      const float* row = sm[p][t];
      const f32x4 q0 = *reinterpret_cast<const f32x4*>(row + 4 * li), q1 = *reinterpret_cast<const f32x4*>(row + 4 * (L + li));
      const f32x4 k0 = *reinterpret_cast<const f32x4*>(row + DKP + 4 * li),
                  k1 = *reinterpret_cast<const f32x4*>(row + DKP + 4 * (L + li));
      constexpr int VO = (MODE == DELTA ? 3 : 2) * DKP;
      float vj[NC], o[NC];
#pragma unroll
      for (int c = 0; c < NC; ++c) vj[c] = row[VO + cl + c];
      if constexpr (MODE == DELTA) {
        const f32x4 g0 = *reinterpret_cast<const f32x4*>(row + 2 * DKP + 4 * li),
                    g1 = *reinterpret_cast<const f32x4*>(row + 2 * DKP + 4 * (L + li));
        const float beta = row[VO + CPB], kq = row[VO + CPB + 1];
        float sk[NC], sq[NC];
#pragma unroll
        for (int c = 0; c < NC; ++c) {
          sk[c] = sq[c] = 0.f;
#pragma unroll
          for (int e = 0; e < 4; ++e) {
            S0[c][e] *= g0[e];
            S1[c][e] *= g1[e];
            sk[c] += S0[c][e] * k0[e] + S1[c][e] * k1[e];
            sq[c] += S0[c][e] * q0[e] + S1[c][e] * q1[e];
          }
        }
#pragma unroll
        for (int c = 0; c < NC; ++c) {
          sk[c] = lanes_sum<L>(sk[c]);
          sq[c] = lanes_sum<L>(sq[c]);
        }
#pragma unroll
        for (int c = 0; c < NC; ++c) {
          const float u = (vj[c] - sk[c]) * beta;
          o[c] = sq[c] + u * kq;
          S0[c] += k0 * u;
          S1[c] += k1 * u;
        }
      } else {
#pragma unroll
        for (int c = 0; c < NC; ++c) {
          o[c] = 0.f;
#pragma unroll
          for (int e = 0; e < 4; ++e) {
            S0[c][e] = S0[c][e] * dec + k0[e] * vj[c];
            S1[c][e] = S1[c][e] * dec + k1[e] * vj[c];
            o[c] += S0[c][e] * q0[e] + S1[c][e] * q1[e];
          }
        }
#pragma unroll
        for (int c = 0; c < NC; ++c) o[c] = lanes_sum<L>(o[c]);
      }
      if (li == 0) {
        T* oo = out + (int64_t)(rb + t) * a.H * dv + (int64_t)h * dv + cb + cl;
#pragma unroll
        for (int c = 0; c < NC; ++c)
          if (cb + cl + c < dv) oo[c] = (T)o[c];
      }
    }
    if (more) store(p ^ 1);   // (last read before the previous barrier)
    __syncthreads();
  }
#pragma unroll
  for (int c = 0; c < NC; ++c)
    if (cb + cl + c < dv) {
      float* w = st + (int64_t)(cb + cl + c) * dk;
      if (vec) {
        *reinterpret_cast<f32x4*>(w + 4 * li) = S0[c];
        *reinterpret_cast<f32x4*>(w + 4 * (L + li)) = S1[c];
      } else {
#pragma unroll
        for (int e = 0; e < 4; ++e) {
          if (4 * li + e < dk) w[4 * li + e] = S0[c][e];
          if (4 * (L + li) + e < dk) w[4 * (L + li) + e] = S1[c][e];
        }
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
            sg[c] = c < dk ? decay_of((float)z[(int64_t)row * a.z_stride + (int64_t)h * dk + c], a.dt_bias[(int64_t)h * dk + c], A)
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

template <typename T, int N, bool VEC>
int prep(const void* x, const void* w, const void* state, void* v, const PrepArgs& a, hipStream_t stream) {
  const int64_t waves = (int64_t)((a.T + PREP_ROWS - 1) / PREP_ROWS) * a.Hk;
  const int nblk = (int)((waves + 3) / 4);
#define PREP(KT) \
  delta_prep_kernel<T, N, KT, VEC><<<nblk, 256, 0, stream>>>((const T*)x, (const T*)w, (const T*)state, (T*)v, a)
  if (a.K == 2) PREP(2);
  else if (a.K == 3) PREP(3);
  else if (a.K == 4) PREP(4);
  else PREP(0);
#undef PREP
  OME_CHECK_LAUNCH();
  return 0;
}

template <typename T, int L, int MODE>
int scan(const void* q, const void* k, const void* v, const void* z, const void* b, void* out, const ScanArgs& a, int S,
         int nc, hipStream_t stream) {
  constexpr int RB = L <= 16 ? 8 : (L == 32 ? 4 : 2), GPW = 64 / L;
  const dim3 grid(S, a.H, (a.dv + 4 * GPW * nc - 1) / (4 * GPW * nc));
#define SCAN(NC)                                                                                                  \
  state_scan_kernel<T, L, NC, MODE, RB><<<grid, 256, 0, stream>>>((const T*)q, (const T*)k, (const T*)v, (const T*)z, \
                                                                  (const T*)b, (T*)out, a)
  if (nc == 1) SCAN(1);
  else if (nc == 2) SCAN(2);
  else SCAN(4);
#undef SCAN
  OME_CHECK_LAUNCH();
  return 0;
}

template <typename T, int MODE>
int scan_by_width(const void* q, const void* k, const void* v, const void* z, const void* b, void* out, const ScanArgs& a,
                  int S, hipStream_t stream) {
  const int DKP = padded_dk(a.dk), gpw = 64 / (DKP / 8);
  // columns per lane: more of them share a row's operands, fewer leave more workgroups
  int nc = 4;
  while (nc > 1 && (int64_t)S * a.H * ((a.dv + 4 * gpw * nc - 1) / (4 * gpw * nc)) < 512) nc /= 2;
  while (nc > 1 && 4 * gpw * (nc / 2) >= a.dv) nc /= 2;
  switch (DKP) {
    case 16: return scan<T, 2, MODE>(q, k, v, z, b, out, a, S, nc, stream);
    case 32: return scan<T, 4, MODE>(q, k, v, z, b, out, a, S, nc, stream);
    case 64: return scan<T, 8, MODE>(q, k, v, z, b, out, a, S, nc, stream);
    case 128: return scan<T, 16, MODE>(q, k, v, z, b, out, a, S, nc, stream);
    case 256: return scan<T, 32, MODE>(q, k, v, z, b, out, a, S, nc, stream);
    default: return scan<T, 64, MODE>(q, k, v, z, b, out, a, S, nc, stream);
  }
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
    case 256: STEP(32); break;
    default: STEP(64); break;
  }
#undef STEP
  OME_CHECK_LAUNCH();
  return 0;
}

bool bad_shape(int H, int Hk, int dk, int dv) { return Hk <= 0 || H <= 0 || H % Hk || dk <= 0 || dk > 512 || dv <= 0; }

}  // namespace

// x: projection rows [q (Hk * dk) | k (Hk * dk) | v (H * dv)] (row stride in elements), conv_w [C, K], conv_state
// [slots, C, K - 1]; first / slot [T]: see PrepArgs; qn / kn fp32 [T, Hk, DKP], qk fp32 [T, Hk], v [T, H * dv].
OME_API int ome_delta_prep(const void* x, int64_t stride, const void* conv_w, const void* conv_state, int K,
                           const int* first, const int* slot, float* qn, float* kn, float* qk, void* v, int T, int H,
                           int Hk, int dk, int dv, int f32, hipStream_t stream) {
  if (T <= 0) return 0;
  if (bad_shape(H, Hk, dk, dv) || K < 1 || K > 32) return -2;
  const int DKP = padded_dk(dk);
  const PrepArgs a{stride, 2 * Hk * dk + H * dv, K, first, slot, qn, kn, qk, T, Hk, H / Hk, dk, dv, DKP};
  const int esz = f32 ? 4 : 2;
  const int N = DKP <= 64 ? 1 : DKP / 64;
  const int A = N > 2 ? N : 2;   // elements a vector access needs aligned
  const bool vec = N > 1 && dk % A == 0 && (H / Hk * dv) % 2 == 0 && stride % A == 0 && ((uintptr_t)x & (A * esz - 1)) == 0;
#define PREP_N(TT, NN) (vec ? prep<TT, NN, true>(x, conv_w, conv_state, v, a, stream) : prep<TT, NN, false>(x, conv_w, conv_state, v, a, stream))
  if (f32) {
    if (N == 1) return prep<float, 1, false>(x, conv_w, conv_state, v, a, stream);
    if (N == 2) return PREP_N(float, 2);
    if (N == 4) return PREP_N(float, 4);
    return prep<float, 8, false>(x, conv_w, conv_state, v, a, stream);
  }
  if (N == 1) return prep<bf16, 1, false>(x, conv_w, conv_state, v, a, stream);
  if (N == 2) return PREP_N(bf16, 2);
  if (N == 4) return PREP_N(bf16, 4);
  return PREP_N(bf16, 8);
#undef PREP_N
}

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

// Delta rule over the rows of every sequence: operands of ome_delta_prep, z rows [decay inputs (H * dk) | ..], b rows
// [H]; state fp32 [slots, H, dv, dk]; out [T, H * dv] (before the head norm).
OME_API int ome_delta_scan(const float* qn, const float* kn, const float* qk, const void* v, const void* z,
                           int64_t z_stride, const void* b, int64_t b_stride, const float* A_log, const float* dt_bias,
                           float* state, void* out, const int* cu, const int* slot, const int* reset, int S, int H, int Hk,
                           int dk, int dv, int f32, hipStream_t stream) {
  if (S <= 0) return 0;
  if (bad_shape(H, Hk, dk, dv) || H > 65535) return -2;
  const ScanArgs a{qn, kn, qk, 0, (int64_t)H * dv, A_log, dt_bias, z_stride, b_stride, nullptr, state, cu, slot, reset, H, Hk, dk, dv};
  if (f32) return scan_by_width<float, DELTA>(nullptr, nullptr, v, z, b, out, a, S, stream);
  return scan_by_width<bf16, DELTA>(nullptr, nullptr, v, z, b, out, a, S, stream);
}

// q / k [T, H * dk], v [T, H * dv]: views of one projection (row stride in elements); decay fp32 [H].
OME_API int ome_lightning_scan(const void* q, const void* k, const void* v, int64_t stride, const float* decay, float* state,
                               void* out, const int* cu, const int* slot, const int* reset, int S, int H, int dk, int dv,
                               int f32, hipStream_t stream) {
  if (S <= 0) return 0;
  if (bad_shape(H, H, dk, dv) || H > 65535) return -2;
  const ScanArgs a{nullptr, nullptr, nullptr, stride, stride, nullptr, nullptr, 0, 0, decay, state, cu, slot, reset, H, H, dk, dv};
  if (f32) return scan_by_width<float, LIGHTNING>(q, k, v, nullptr, nullptr, out, a, S, stream);
  return scan_by_width<bf16, LIGHTNING>(q, k, v, nullptr, nullptr, out, a, S, stream);
}

// The whole mixer core for sequences of one row each: z rows [decay inputs (H * dk) | output gate (H * dv)].
OME_API int ome_delta_step(const void* x, int64_t stride, const void* conv_w, void* conv_state, int K, const void* z,
                           int64_t z_stride, const void* b, int64_t b_stride, const float* A_log, const float* dt_bias,
                           const void* norm_w, float eps, float* state, void* out, const int* cu, const int* slot,
                           const int* reset, int S, int H, int Hk, int dk, int dv, int f32, hipStream_t stream) {
  if (S <= 0) return 0;
  if (bad_shape(H, Hk, dk, dv) || Hk > 65535 || K < 1 || K > 32) return -2;
  const StepArgs a{stride, z_stride, b_stride, K, A_log, dt_bias, nullptr, eps, state, cu, slot, reset, H, Hk, dk, dv};
  if (f32) return step_by_width<float, DELTA>(x, nullptr, nullptr, conv_w, conv_state, z, b, norm_w, out, a, S, stream);
  return step_by_width<bf16, DELTA>(x, nullptr, nullptr, conv_w, conv_state, z, b, norm_w, out, a, S, stream);
}

OME_API int ome_lightning_step(const void* q, const void* k, const void* v, int64_t stride, const float* decay,
                               float* state, void* out, const int* cu, const int* slot, const int* reset, int S, int H,
                               int dk, int dv, int f32, hipStream_t stream) {
  if (S <= 0) return 0;
  if (bad_shape(H, H, dk, dv) || H > 65535) return -2;
  const StepArgs a{stride, 0, 0, 1, nullptr, nullptr, decay, 0.f, state, cu, slot, reset, H, H, dk, dv};
  if (f32) return step_by_width<float, LIGHTNING>(q, k, v, nullptr, nullptr, nullptr, nullptr, nullptr, out, a, S, stream);
  return step_by_width<bf16, LIGHTNING>(q, k, v, nullptr, nullptr, nullptr, nullptr, nullptr, out, a, S, stream);
}
