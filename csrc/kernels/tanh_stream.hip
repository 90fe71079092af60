// Step of an fp32 residual stream whose norms are tanh curves, D(v) = tanh(alpha v) w + b (scalar
// alpha, vectors w and b; no statistics), before and after every sublayer:
//
//   y  = the sublayer's output, or, for two mixers side by side, (y1 / rms(y1) * w1 + y2 / rms(y2) * w2) / 2
//   x += mult * D_post(y)          (in place; no y: x stays)
//   out = D_pre(x)                 rounded once to the model dtype: the next GEMM's input
//
// One workgroup per row; rows of 4-element vectors are held in registers (H <= 1024 * NCH).
#include "common.h"

namespace {

template <typename T>
__device__ __forceinline__ f32x4 ts_ld4(const T* p) {
  if constexpr (sizeof(T) == 4) {
    return *reinterpret_cast<const f32x4*>(p);
  } else {
    const bf16x4 t = *reinterpret_cast<const bf16x4*>(p);
    return f32x4{(float)t[0], (float)t[1], (float)t[2], (float)t[3]};
  }
}
template <typename T>
__device__ __forceinline__ void ts_st4(T* p, f32x4 v) {
  if constexpr (sizeof(T) == 4) {
    *reinterpret_cast<f32x4*>(p) = v;
  } else {
    *reinterpret_cast<bf16x4*>(p) = bf16x4{(bf16)v[0], (bf16)v[1], (bf16)v[2], (bf16)v[3]};
  }
}

// fp32 models: the library's tanh; otherwise 1 - 2 / (e^2z + 1) on the hardware exponential, and the Taylor
// series up to z^11 where that difference would cancel (|z| < 0.35: next term 1e-8 of z)
template <typename T>
__device__ __forceinline__ float tanh_t(float z) {
  if constexpr (sizeof(T) == 4) {
    return tanhf(z);
  } else {
    const float s = z * z;
    const float p = 1.f + s * (-1.f / 3.f + s * (2.f / 15.f + s * (-17.f / 315.f + s * (62.f / 2835.f - s * (1382.f / 155925.f)))));
    const float e = __expf(2.f * fabsf(z));
    const float big = copysignf(1.f - 2.f * __builtin_amdgcn_rcpf(e + 1.f), z);
    return fabsf(z) < 0.35f ? z * p : big;
  }
}

template <typename T>
struct TanhArgs {
  float* x;
  int64_t x_stride;
  const T *y, *y2;
  int64_t y_stride, y2_stride;
  const T *jw1, *jw2;      // joined outputs: their norms' weights
  float eps, mult;
  float post_alpha;
  const T *post_w, *post_b;
  float pre_alpha;
  const T *pre_w, *pre_b;
  T* out;
  int64_t out_stride;
  int H;
};

template <typename T>
__device__ __forceinline__ f32x4 curve4(f32x4 v, float alpha, const T* w, const T* b) {
  const f32x4 wv = ts_ld4<T>(w), bv = ts_ld4<T>(b);
  f32x4 r;
#pragma unroll
  for (int e = 0; e < 4; ++e) r[e] = tanh_t<T>(alpha * v[e]) * wv[e] + bv[e];
  return r;
}

// any width and alignment, element by element
template <typename T>
__global__ __launch_bounds__(256) void tanh_stream_kernel(TanhArgs<T> a) {
  __shared__ float red[4];
  const int64_t row = blockIdx.x;
  float* xr = a.x + row * a.x_stride;
  const T* y1 = a.y == nullptr ? nullptr : a.y + row * a.y_stride;
  const T* y2 = a.y2 == nullptr ? nullptr : a.y2 + row * a.y2_stride;
  float r1 = 1.f, r2 = 0.f;
  if (y2 != nullptr) {
    float s1 = 0.f, s2 = 0.f;
    for (int i = threadIdx.x; i < a.H; i += 256) {
      s1 += (float)y1[i] * (float)y1[i];
      s2 += (float)y2[i] * (float)y2[i];
    }
    r1 = 0.5f / sqrtf(block_sum<256>(s1, red) / (float)a.H + a.eps);
    r2 = 0.5f / sqrtf(block_sum<256>(s2, red) / (float)a.H + a.eps);
  }
  for (int i = threadIdx.x; i < a.H; i += 256) {
    float x = xr[i];
    if (y1 != nullptr) {
      float v = (float)y1[i];
      if (y2 != nullptr) v = v * r1 * (float)a.jw1[i] + (float)y2[i] * r2 * (float)a.jw2[i];
      x += a.mult * (tanh_t<T>(a.post_alpha * v) * (float)a.post_w[i] + (float)a.post_b[i]);
      xr[i] = x;
    }
    a.out[row * a.out_stride + i] = (T)(tanh_t<T>(a.pre_alpha * x) * (float)a.pre_w[i] + (float)a.pre_b[i]);
  }
}

// USE: 0 no sublayer output, 1 one, 2 two joined
template <typename T, int NCH, int USE>
__global__ __launch_bounds__(256) void tanh_stream_vec_kernel(TanhArgs<T> a) {
  __shared__ float red[2][4];
  const int64_t row = blockIdx.x;
  float* xr = a.x + row * a.x_stride;
  f32x4 x[NCH], v[NCH], u[NCH];
#pragma unroll
  for (int c = 0; c < NCH; ++c) {
    const int i = (threadIdx.x + 256 * c) * 4;
    x[c] = v[c] = u[c] = f32x4{0.f, 0.f, 0.f, 0.f};
    if (i < a.H) {
      x[c] = *reinterpret_cast<const f32x4*>(xr + i);
      if constexpr (USE >= 1) v[c] = ts_ld4<T>(a.y + row * a.y_stride + i);
      if constexpr (USE == 2) u[c] = ts_ld4<T>(a.y2 + row * a.y2_stride + i);
    }
  }
  float r1 = 0.f, r2 = 0.f;
  if constexpr (USE == 2) {
    float s1 = 0.f, s2 = 0.f;
#pragma unroll
    for (int c = 0; c < NCH; ++c)
#pragma unroll
      for (int e = 0; e < 4; ++e) {
        s1 += v[c][e] * v[c][e];
        s2 += u[c][e] * u[c][e];
      }
    s1 = wave_sum(s1);
    s2 = wave_sum(s2);
    if ((threadIdx.x & 63) == 0) {
      red[0][threadIdx.x >> 6] = s1;
      red[1][threadIdx.x >> 6] = s2;
    }
    __syncthreads();
    r1 = 0.5f / sqrtf((red[0][0] + red[0][1] + red[0][2] + red[0][3]) / (float)a.H + a.eps);
    r2 = 0.5f / sqrtf((red[1][0] + red[1][1] + red[1][2] + red[1][3]) / (float)a.H + a.eps);
  }
#pragma unroll
  for (int c = 0; c < NCH; ++c) {
    const int i = (threadIdx.x + 256 * c) * 4;
    if (i < a.H) {
      if constexpr (USE == 2) v[c] = v[c] * r1 * ts_ld4<T>(a.jw1 + i) + u[c] * r2 * ts_ld4<T>(a.jw2 + i);
      if constexpr (USE >= 1) {
        x[c] += a.mult * curve4<T>(v[c], a.post_alpha, a.post_w + i, a.post_b + i);
        *reinterpret_cast<f32x4*>(xr + i) = x[c];
      }
      ts_st4<T>(a.out + row * a.out_stride + i, curve4<T>(x[c], a.pre_alpha, a.pre_w + i, a.pre_b + i));
    }
  }
}

template <typename T, int USE>
void launch_vec(const TanhArgs<T>& a, int rows, hipStream_t stream) {
  if (a.H <= 1024) tanh_stream_vec_kernel<T, 1, USE><<<rows, 256, 0, stream>>>(a);
  else if (a.H <= 2048) tanh_stream_vec_kernel<T, 2, USE><<<rows, 256, 0, stream>>>(a);
  else if (a.H <= 4096) tanh_stream_vec_kernel<T, 4, USE><<<rows, 256, 0, stream>>>(a);
  else tanh_stream_vec_kernel<T, 8, USE><<<rows, 256, 0, stream>>>(a);
}

template <typename T>
int launch(float* x, int64_t x_stride, const void* y, int64_t y_stride, const void* y2, int64_t y2_stride, const void* jw1,
           const void* jw2, float eps, float mult, float post_alpha, const void* post_w, const void* post_b,
           float pre_alpha, const void* pre_w, const void* pre_b, void* out, int64_t out_stride, int rows, int H,
           hipStream_t stream) {
  const TanhArgs<T> a{x, x_stride, (const T*)y, (const T*)y2, y_stride, y2_stride, (const T*)jw1, (const T*)jw2, eps, mult,
                      post_alpha, (const T*)post_w, (const T*)post_b, pre_alpha, (const T*)pre_w, (const T*)pre_b, (T*)out,
                      out_stride, H};
  auto al = [](const void* p, int64_t stride, int e) { return (((uintptr_t)p | (uintptr_t)(stride * e)) & (4 * e - 1)) == 0; };
  constexpr int E = sizeof(T);
  const bool vec = H % 4 == 0 && H <= 8192 && al(x, x_stride, 4) && al(y, y_stride, E) && al(y2, y2_stride, E) && al(jw1, 0, E) &&
                   al(jw2, 0, E) && al(post_w, 0, E) && al(post_b, 0, E) && al(pre_w, 0, E) && al(pre_b, 0, E) &&
                   al(out, out_stride, E);
  if (!vec) tanh_stream_kernel<T><<<rows, 256, 0, stream>>>(a);
  else if (y == nullptr) launch_vec<T, 0>(a, rows, stream);
  else if (y2 == nullptr) launch_vec<T, 1>(a, rows, stream);
  else launch_vec<T, 2>(a, rows, stream);
  OME_CHECK_LAUNCH();
  return 0;
}

}  // namespace

OME_API int ome_tanh_stream(float* x, int64_t x_stride, const void* y, int64_t y_stride, const void* y2, int64_t y2_stride,
                            const void* jw1, const void* jw2, float eps, float mult, float post_alpha, const void* post_w,
                            const void* post_b, float pre_alpha, const void* pre_w, const void* pre_b, void* out,
                            int64_t out_stride, int rows, int H, int f32, hipStream_t stream) {
  if (rows <= 0) return 0;
  if (H <= 0 || x == nullptr || out == nullptr || pre_w == nullptr || pre_b == nullptr) return -2;
  if (y != nullptr && (post_w == nullptr || post_b == nullptr)) return -2;
  if (y2 != nullptr && (y == nullptr || jw1 == nullptr || jw2 == nullptr)) return -2;
  if (f32)
    return launch<float>(x, x_stride, y, y_stride, y2, y2_stride, jw1, jw2, eps, mult, post_alpha, post_w, post_b, pre_alpha,
                         pre_w, pre_b, out, out_stride, rows, H, stream);
  return launch<bf16>(x, x_stride, y, y_stride, y2, y2_stride, jw1, jw2, eps, mult, post_alpha, post_w, post_b, pre_alpha, pre_w,
                      pre_b, out, out_stride, rows, H, stream);
}
