// Residual stream of post-norm decoders whose norm works on groups of channels and whose layers
// pass on a learned average over depth.  One step of row t:
//
//   n = w * y / rms_g(y)          (y: a sublayer's output, a gathered embedding row or the stream
//                                  itself; every one of `groups` equal consecutive parts is divided
//                                  by its own sqrt(mean(part^2) + eps))
//   X = res + n                   (res absent: X = n)
//   history[k] = X                (optional: entry k of the depth history [k + 1 .., T, H] fp32)
//   x = sum_{j < k} coef[j] * history[j] + coef[k] * X      (coef absent: x = X)
//   x_out = x (fp32),  out = x rounded to the model dtype (the next GEMM's input); either optional
//
// Everything is fp32 with one rounding at `out`.  One workgroup per row.
#include "common.h"

namespace {

template <typename T>
__device__ __forceinline__ f32x4 gs_ld4(const T* p) {
  if constexpr (sizeof(T) == 4) {
    return *reinterpret_cast<const f32x4*>(p);
  } else {
    const bf16x4 t = *reinterpret_cast<const bf16x4*>(p);
    return f32x4{(float)t[0], (float)t[1], (float)t[2], (float)t[3]};
  }
}
template <typename T>
__device__ __forceinline__ void gs_st4(T* p, f32x4 v) {
  if constexpr (sizeof(T) == 4) {
    *reinterpret_cast<f32x4*>(p) = v;
  } else {
    *reinterpret_cast<bf16x4*>(p) = bf16x4{(bf16)v[0], (bf16)v[1], (bf16)v[2], (bf16)v[3]};
  }
}

struct StreamArgs {
  const int* ids;          // gather rows of y by token (null: row t)
  int V;
  const float* res;
  int64_t res_stride;
  float* hist;             // entry j at hist + j * hist_stride, rows H apart
  int64_t hist_stride;
  int k;                   // the entry this step writes
  const float* coef;       // [k + 1]
  float* x_out;
  int64_t x_stride;
  int64_t out_stride;
  int H, groups;
  float eps;
};

__device__ __forceinline__ int64_t src_row(const StreamArgs& a, int64_t row) {
  if (a.ids == nullptr) return row;
  const int id = a.ids[row];
  return id < 0 ? 0 : (id >= a.V ? a.V - 1 : id);
}

// any width and group count, element by element
template <typename TI, typename T>
__global__ __launch_bounds__(256) void stream_step_kernel(const TI* __restrict__ y, int64_t y_stride,
                                                          const T* __restrict__ w, T* __restrict__ out,
                                                          StreamArgs a) {
  __shared__ float red[4];
  const int64_t row = blockIdx.x;
  const TI* yr = y + src_row(a, row) * y_stride;
  const int gw = a.H / a.groups;
  for (int g = 0; g < a.groups; ++g) {
    float ss = 0.f;
    for (int i = g * gw + threadIdx.x; i < (g + 1) * gw; i += 256) {
      const float v = (float)yr[i];
      ss += v * v;
    }
    const float rs = 1.f / sqrtf(block_sum<256>(ss, red) / (float)gw + a.eps);
    for (int i = g * gw + threadIdx.x; i < (g + 1) * gw; i += 256) {
      float v = (float)yr[i] * rs * (float)w[i];
      if (a.res != nullptr) v += a.res[row * a.res_stride + i];
      if (a.coef != nullptr) {
        float s = a.coef[a.k] * v;
        for (int j = 0; j < a.k; ++j) s += a.coef[j] * a.hist[j * a.hist_stride + row * a.H + i];
        if (a.hist != nullptr) a.hist[a.k * a.hist_stride + row * a.H + i] = v;
        v = s;
      } else if (a.hist != nullptr) {
        a.hist[a.k * a.hist_stride + row * a.H + i] = v;
      }
      if (a.x_out != nullptr) a.x_out[row * a.x_stride + i] = v;
      if (out != nullptr) out[row * a.out_stride + i] = (T)v;
    }
  }
}

// Rows of 4-element vectors held in registers (H <= 1024 * NCH; a vector never spans two groups):
// every input is read once, the history loads are in flight during the reduction.  Each wave leaves
// its partial square sum of every group in LDS, so one barrier serves all groups.
constexpr int GS_MAXG = 16;

template <typename TI, typename T, int NCH>
__global__ __launch_bounds__(256) void stream_step_vec_kernel(const TI* __restrict__ y, int64_t y_stride,
                                                              const T* __restrict__ w, T* __restrict__ out,
                                                              StreamArgs a) {
  __shared__ float red[GS_MAXG][4];
  const int64_t row = blockIdx.x;
  const TI* yr = y + src_row(a, row) * y_stride;
  const int gw = a.H / a.groups;
  f32x4 v[NCH], acc[NCH], rv[NCH];
  float cs[NCH];
  int gid[NCH];
#pragma unroll
  for (int c = 0; c < NCH; ++c) {
    const int i = (threadIdx.x + 256 * c) * 4;
    const bool on = i < a.H;
    v[c] = acc[c] = rv[c] = f32x4{0.f, 0.f, 0.f, 0.f};
    if (on) {
      v[c] = gs_ld4<TI>(yr + i);
      if (a.res != nullptr) rv[c] = *reinterpret_cast<const f32x4*>(a.res + row * a.res_stride + i);
    }
    gid[c] = on ? i / gw : -1;
  }
  if (a.coef != nullptr) {
    const float* h = a.hist + row * a.H;
    int j = 0;
    for (; j + 4 <= a.k; j += 4) {
      f32x4 t[4][NCH];
#pragma unroll
      for (int u = 0; u < 4; ++u)
#pragma unroll
        for (int c = 0; c < NCH; ++c) {
          const int i = (threadIdx.x + 256 * c) * 4;
          t[u][c] = i < a.H ? *reinterpret_cast<const f32x4*>(h + (j + u) * a.hist_stride + i) : f32x4{0.f, 0.f, 0.f, 0.f};
        }
#pragma unroll
      for (int u = 0; u < 4; ++u) {
        const float cf = a.coef[j + u];
#pragma unroll
        for (int c = 0; c < NCH; ++c) acc[c] += cf * t[u][c];
      }
    }
    for (; j < a.k; ++j) {
      const float cf = a.coef[j];
#pragma unroll
      for (int c = 0; c < NCH; ++c) {
        const int i = (threadIdx.x + 256 * c) * 4;
        if (i < a.H) acc[c] += cf * *reinterpret_cast<const f32x4*>(h + j * a.hist_stride + i);
      }
    }
  }
#pragma unroll
  for (int c = 0; c < NCH; ++c) cs[c] = v[c][0] * v[c][0] + v[c][1] * v[c][1] + v[c][2] * v[c][2] + v[c][3] * v[c][3];
  for (int g = 0; g < a.groups; ++g) {
    float s = 0.f;
#pragma unroll
    for (int c = 0; c < NCH; ++c) s += gid[c] == g ? cs[c] : 0.f;
    s = wave_sum(s);
    if ((threadIdx.x & 63) == 0) red[g][threadIdx.x >> 6] = s;
  }
  __syncthreads();
  const float ck = a.coef != nullptr ? a.coef[a.k] : 1.f;
#pragma unroll
  for (int c = 0; c < NCH; ++c) {
    const int i = (threadIdx.x + 256 * c) * 4;
    if (i < a.H) {
      const float ss = red[gid[c]][0] + red[gid[c]][1] + red[gid[c]][2] + red[gid[c]][3];
      const float rs = 1.f / sqrtf(ss / (float)gw + a.eps);
      f32x4 X = v[c] * rs * gs_ld4<T>(w + i) + rv[c];
      if (a.hist != nullptr) *reinterpret_cast<f32x4*>(a.hist + a.k * a.hist_stride + row * a.H + i) = X;
      if (a.coef != nullptr) X = acc[c] + ck * X;
      if (a.x_out != nullptr) *reinterpret_cast<f32x4*>(a.x_out + row * a.x_stride + i) = X;
      if (out != nullptr) gs_st4<T>(out + row * a.out_stride + i, X);
    }
  }
}

template <typename TI, typename T>
int stream_step(const void* y, int64_t y_stride, const void* w, void* out, const StreamArgs& a, int rows, bool vec,
                hipStream_t stream) {
#define GS_VEC(N)                                                                                              \
  stream_step_vec_kernel<TI, T, N><<<rows, 256, 0, stream>>>((const TI*)y, y_stride, (const T*)w, (T*)out, a)
  if (!vec) stream_step_kernel<TI, T><<<rows, 256, 0, stream>>>((const TI*)y, y_stride, (const T*)w, (T*)out, a);
  else if (a.H <= 1024) GS_VEC(1);
  else if (a.H <= 2048) GS_VEC(2);
  else if (a.H <= 4096) GS_VEC(4);
  else GS_VEC(8);
#undef GS_VEC
  OME_CHECK_LAUNCH();
  return 0;
}

}  // namespace

// y_f32: y is fp32 (the stream itself) although the model dtype (w, out) is bf16
OME_API int ome_stream_step(const void* y, int64_t y_stride, int y_f32, const int* ids, int V, const float* res,
                            int64_t res_stride, const void* w, int groups, float eps, float* hist, int64_t hist_stride,
                            int k, const float* coef, float* x_out, int64_t x_stride, void* out, int64_t out_stride,
                            int rows, int H, int f32, hipStream_t stream) {
  if (rows <= 0) return 0;
  if (H <= 0 || groups <= 0 || H % groups || k < 0 || (coef != nullptr && hist == nullptr) || (f32 && !y_f32)) return -2;
  const StreamArgs a{ids, V, res, res_stride, hist, hist_stride, k, coef, x_out, x_stride, out_stride, H, groups, eps};
  const int esz = f32 ? 4 : 2, ysz = y_f32 ? 4 : 2;
  auto al = [](const void* p, int64_t stride, int e) { return (((uintptr_t)p | (uintptr_t)(stride * e)) & (4 * e - 1)) == 0; };
  const bool vec = (H / groups) % 4 == 0 && H <= 8192 && groups <= GS_MAXG && al(y, y_stride, ysz) && al(w, 0, esz) &&
                   al(res, res_stride, 4) && al(hist, hist_stride, 4) && al(x_out, x_stride, 4) && al(out, out_stride, esz);
  if (f32) return stream_step<float, float>(y, y_stride, w, out, a, rows, vec, stream);
  if (y_f32) return stream_step<float, bf16>(y, y_stride, w, out, a, rows, vec, stream);
  return stream_step<bf16, bf16>(y, y_stride, w, out, a, rows, vec, stream);
}
