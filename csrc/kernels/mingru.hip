// Gated element-wise recurrence whose gates read only the current token (minGRU), fused with the
// activations before it and the output gate after it:
//
//   z_t = sigmoid(z_raw + bz),   c_t = u + 1/2 where u >= 0, sigmoid(u) where u < 0,  u = x_raw + bx
//   S_t = S_{t-1} + z_t (c_t - S_{t-1}),      out_t = S_t * silu(g_raw)
//
// z_raw / x_raw / g_raw are row-strided views of one fused projection; biases, gates, the recurrence
// and its state [slots, width] are fp32, `out` is rounded once.
//
// The recurrence is affine in S, so a sequence's rows of a step are cut into chunks of `CH` rows
// that run side by side.  Launch 1: the first chunk of every sequence runs in full from the slot's
// state (decode rows end here); every further chunk but the last leaves (A, B) = (product of 1 - z,
// the state it reaches from zero) per channel, the first one B = the state it reached.  Launch 2:
// the workgroups of the further chunks fold the summaries of the chunks before them into their start
// state and run in full; the last chunk of a sequence writes the slot's state.  No chunk reads
// anything another workgroup of the same launch writes.
#include "common.h"

namespace {

// V neighbouring channels of a thread
template <int V>
struct Vec {
  float f[V];
};
// the same as they lie in memory (kept unconverted while a load is in flight)
template <typename T, int V>
struct Raw {
  typedef T type __attribute__((ext_vector_type(V)));
};
template <typename T>
struct Raw<T, 1> {
  typedef T type;
};
template <typename T, int V>
using raw_t = typename Raw<T, V>::type;

template <typename T, int V>
__device__ __forceinline__ raw_t<T, V> ldr(const T* p) {
  return *reinterpret_cast<const raw_t<T, V>*>(p);
}
template <typename T, int V>
__device__ __forceinline__ Vec<V> widen(raw_t<T, V> t) {
  Vec<V> r;
  if constexpr (V == 1) {
    r.f[0] = (float)t;
  } else {
#pragma unroll
    for (int i = 0; i < V; ++i) r.f[i] = (float)t[i];
  }
  return r;
}
template <typename T, int V>
__device__ __forceinline__ Vec<V> ldv(const T* p) {
  return widen<T, V>(ldr<T, V>(p));
}
template <typename T, int V>
__device__ __forceinline__ void stv(T* p, const Vec<V>& v) {
  raw_t<T, V> t;
  if constexpr (V == 1) {
    t = (T)v.f[0];
  } else {
#pragma unroll
    for (int i = 0; i < V; ++i) t[i] = (T)v.f[i];
  }
  *reinterpret_cast<raw_t<T, V>*>(p) = t;
}

__device__ __forceinline__ float sig(float x) { return __builtin_amdgcn_rcpf(1.f + __expf(-x)); }

// workgroup row `z` of the grid -> (sequence, chunk of it); every wave scans the sequence lengths
__device__ __forceinline__ bool find_chunk(const int* __restrict__ cu, int S, int CH, int z, int& s, int& c) {
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

constexpr int64_t V4_MIN = 256 * 1024;
constexpr int RB = 8;   // rows whose loads are in flight together

template <typename T, int V, bool OUT>
struct Batch {
  raw_t<T, V> z[RB], x[RB], g[OUT ? RB : 1];
};

template <typename T, int V, bool OUT>
__device__ __forceinline__ void fetch(Batch<T, V, OUT>& b, const T* __restrict__ zr, const T* __restrict__ xr,
                                      const T* __restrict__ gr, int64_t stride, int t0, int e, int ch) {
#pragma unroll
  for (int r = 0; r < RB; ++r) {
    const int64_t o = (int64_t)min(t0 + r, e - 1) * stride + ch;
    b.z[r] = ldr<T, V>(zr + o);
    b.x[r] = ldr<T, V>(xr + o);
    if constexpr (OUT) b.g[r] = ldr<T, V>(gr + o);
  }
}

// rows [a, e): advance S; OUT: write the gated output, otherwise gather A = prod(1 - z)
template <typename T, int V, bool OUT>
__device__ __forceinline__ void run_rows(const T* __restrict__ zr, const T* __restrict__ xr, const T* __restrict__ gr,
                                         int64_t stride, T* __restrict__ out, int width, int a, int e, int ch,
                                         const Vec<V>& bz, const Vec<V>& bx, Vec<V>& S, Vec<V>& A) {
  for (int t0 = a; t0 < e; t0 += RB) {
    Batch<T, V, OUT> cur;
    fetch(cur, zr, xr, gr, stride, t0, e, ch);
#pragma unroll
    for (int r = 0; r < RB; ++r) {
      if (t0 + r >= e) break;
      const Vec<V> z = widen<T, V>(cur.z[r]), x = widen<T, V>(cur.x[r]);
      Vec<V> y;
      if constexpr (OUT) y = widen<T, V>(cur.g[r]);
#pragma unroll
      for (int i = 0; i < V; ++i) {
        const float zz = sig(z.f[i] + bz.f[i]);
        const float u = x.f[i] + bx.f[i];
        const float c = u >= 0.f ? u + 0.5f : sig(u);
        S.f[i] += zz * (c - S.f[i]);
        if constexpr (OUT) y.f[i] = S.f[i] * y.f[i] * sig(y.f[i]);
        else A.f[i] *= 1.f - zz;
      }
      if constexpr (OUT) stv<T, V>(out + (int64_t)(t0 + r) * width + ch, y);
    }
  }
}

// PASS 1 / 2: see the head of the file.  sum: [chunk][2][width]
template <typename T, int V, int PASS>
__global__ __launch_bounds__(256) void mingru_kernel(const T* __restrict__ zr, const T* __restrict__ xr,
                                                     const T* __restrict__ gr, int64_t stride,
                                                     const T* __restrict__ zb, const T* __restrict__ xb,
                                                     float* __restrict__ state, const int* __restrict__ cu,
                                                     const int* __restrict__ slot, const int* __restrict__ reset, int S,
                                                     float* __restrict__ sum, T* __restrict__ out, int width, int CH) {
  int s = 0, c = 0;
  if (!find_chunk(cu, S, CH, blockIdx.y, s, c)) return;
  const int ch = (blockIdx.x * 256 + threadIdx.x) * V;
  if (ch >= width) return;
  const int r0 = cu[s], r1 = cu[s + 1];
  const int a = r0 + c * CH, e = min(a + CH, r1);
  const bool first = c == 0, last = e == r1;
  if (PASS == 1 ? (!first && (last || sum == nullptr)) : first) return;
  const Vec<V> bz = ldv<T, V>(zb + ch), bx = ldv<T, V>(xb + ch);
  Vec<V> st, A;
#pragma unroll
  for (int i = 0; i < V; ++i) {
    st.f[i] = 0.f;
    A.f[i] = 1.f;
  }
  float* stp = state + (int64_t)slot[s] * width + ch;
  float* mine = sum + (int64_t)blockIdx.y * 2 * width + ch;
  if (PASS == 1 && !first) {
    run_rows<T, V, false>(zr, xr, gr, stride, out, width, a, e, ch, bz, bx, st, A);
    stv<float, V>(mine, A);
    stv<float, V>(mine + width, st);
    return;
  }
  if (PASS == 1) {
    if (reset[s] == 0) st = ldv<float, V>(stp);
  } else {   // chunks 0 .. c - 1 of the sequence sit right before this one
    const float* p = mine - (int64_t)c * 2 * width;
    st = ldv<float, V>(p + width);
#pragma unroll 8
    for (int j = 1; j < c; ++j) {
      const Vec<V> Aj = ldv<float, V>(p + (int64_t)j * 2 * width), Bj = ldv<float, V>(p + (int64_t)j * 2 * width + width);
#pragma unroll
      for (int i = 0; i < V; ++i) st.f[i] = Aj.f[i] * st.f[i] + Bj.f[i];
    }
  }
  run_rows<T, V, true>(zr, xr, gr, stride, out, width, a, e, ch, bz, bx, st, A);
  if (last) stv<float, V>(stp, st);
  else if (PASS == 1 && sum != nullptr) stv<float, V>(mine + width, st);
}

template <typename T, int V>
int launch(const void* z, const void* x, const void* g, int64_t stride, const void* zb, const void* xb, float* state,
           const int* cu, const int* slot, const int* reset, int S, float* sum, void* out, int T_, int width, int CH,
           int chunks, hipStream_t stream) {
  const dim3 grid((width + 256 * V - 1) / (256 * V), chunks);
  mingru_kernel<T, V, 1><<<grid, 256, 0, stream>>>((const T*)z, (const T*)x, (const T*)g, stride, (const T*)zb,
                                                   (const T*)xb, state, cu, slot, reset, S, sum, (T*)out, width, CH);
  OME_CHECK_LAUNCH();
  if (T_ > CH && sum != nullptr) {
    mingru_kernel<T, V, 2><<<grid, 256, 0, stream>>>((const T*)z, (const T*)x, (const T*)g, stride, (const T*)zb,
                                                     (const T*)xb, state, cu, slot, reset, S, sum, (T*)out, width, CH);
    OME_CHECK_LAUNCH();
  }
  return 0;
}

}  // namespace

// rows [cu[s], cu[s + 1]) of the step belong to state slot slot[s] (reset[s]: the sequence starts).
// CH: rows per chunk; chunks: grid rows, at least sum over s of ceil(rows of s / CH); sum: fp32
// scratch [chunks][2][width], null only when no sequence has more than CH rows.
OME_API int ome_mingru_scan(const void* z, const void* x, const void* g, int64_t stride, const void* zb, const void* xb,
                            float* state, const int* cu, const int* slot, const int* reset, int S, float* sum, void* out,
                            int T, int width, int CH, int chunks, int f32, hipStream_t stream) {
  if (T <= 0 || S <= 0) return 0;
  if (width <= 0 || CH <= 0 || chunks <= 0) return -2;
  if (chunks > 65535) return -3;
  const int esz = f32 ? 4 : 2;
  // channels per thread: as wide as the alignment allows (v: 2 or 4)
  auto ok = [&](int v) {
    auto al = [&](const void* p) { return ((uintptr_t)p & (v * esz - 1)) == 0; };
    return width % v == 0 && stride % v == 0 && al(z) && al(x) && al(g) && al(zb) && al(xb) && al(out) &&
           ((uintptr_t)state & (4 * v - 1)) == 0 && ((uintptr_t)sum & (4 * v - 1)) == 0;
  };
#define MG(TT, VV) \
  launch<TT, VV>(z, x, g, stride, zb, xb, state, cu, slot, reset, S, sum, out, T, width, CH, chunks, stream)
  // (four per thread only where that still leaves a workgroup for every CU)
  if (f32) return ok(2) ? MG(float, 2) : MG(float, 1);
  if (ok(4) && (int64_t)chunks * width >= V4_MIN) return MG(bf16, 4);
  return ok(2) ? MG(bf16, 2) : MG(bf16, 1);
#undef MG
}
