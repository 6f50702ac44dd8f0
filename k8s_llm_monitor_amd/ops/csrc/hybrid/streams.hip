// Several residual streams per token, mixed around every sublayer with learned weights.
//   stream_norm   x_t <- sum_s mix[s][t] x_s + out[t] * y  (the right-hand side reads the streams before the step), then
//                 u = sum_t in[t] x_t  and  h = u / rms(u) * w: what the sublayer just run leaves and what the
//                 next one reads, in one launch
// src: the streams [rows][S][d] fp32 (contiguous per token), or one row per token that stands for all S equal
// streams (src_s == 0, the start of the model).  dst: the new streams [rows][S][d]; may be src itself.  y
// absent: nothing is written, u and h are of the streams as they are.  in absent: u is their plain sum.
// Sums and norm are fp32; a thread owns its columns, so every column is read once and written once.
#include "hy_common.h"

namespace k8sllm {

constexpr int kMaxStreams = 16;

// 4 columns per thread and trip, NV trips; SM bounds S (register arrays, wave-uniform guards)
template <typename T, int SM, int NT, int NV>
__global__ __launch_bounds__(NT) void stream_norm_kernel(T* __restrict__ out, float* dst, const float* src, long src_row,
                                                         long src_s, const void* __restrict__ y, int yt,
                                                         const float* __restrict__ mix, const float* __restrict__ wout,
                                                         const float* __restrict__ win, const float* __restrict__ w,
                                                         int S, int d, float eps) {
  __shared__ float red[NT / 64];
  const long row = blockIdx.x;
  const float* xr = src + row * src_row;
  float* xo = dst + row * S * d;
  float4 x[NV][SM], u[NV];
  float yv[NV][4];
#pragma unroll
  for (int i = 0; i < NV; ++i) {
    const int c = (threadIdx.x + NT * i) * 4;
    u[i] = make_float4(0.f, 0.f, 0.f, 0.f);
    if (c < d) {
#pragma unroll
      for (int s = 0; s < SM; ++s)
        if (s < S) x[i][s] = *reinterpret_cast<const float4*>(xr + s * src_s + c);
      if (yt == 2) {
        const float4 a = *reinterpret_cast<const float4*>(reinterpret_cast<const float*>(y) + row * d + c);
        yv[i][0] = a.x; yv[i][1] = a.y; yv[i][2] = a.z; yv[i][3] = a.w;
      } else if (yt == 1) {
        const uint2 a = *reinterpret_cast<const uint2*>(reinterpret_cast<const bf16_t*>(y) + row * d + c);
        yv[i][0] = lo_bf(a.x); yv[i][1] = hi_bf(a.x); yv[i][2] = lo_bf(a.y); yv[i][3] = hi_bf(a.y);
      }
    }
  }
  float ss = 0.f;
#pragma unroll
  for (int i = 0; i < NV; ++i) {
    const int c = (threadIdx.x + NT * i) * 4;
    if (c < d) {
#pragma unroll
      for (int t = 0; t < SM; ++t)
        if (t < S) {
          float4 v;
          if (yt) {
            const float o = wout[t];
            v = make_float4(o * yv[i][0], o * yv[i][1], o * yv[i][2], o * yv[i][3]);
#pragma unroll
            for (int s = 0; s < SM; ++s)
              if (s < S) {
                const float m = mix[s * S + t];
                v.x += m * x[i][s].x; v.y += m * x[i][s].y; v.z += m * x[i][s].z; v.w += m * x[i][s].w;
              }
            *reinterpret_cast<float4*>(xo + t * d + c) = v;
          } else {
            v = x[i][t];
          }
          const float a = win != nullptr ? win[t] : 1.f;
          u[i].x += a * v.x; u[i].y += a * v.y; u[i].z += a * v.z; u[i].w += a * v.w;
        }
      ss += u[i].x * u[i].x + u[i].y * u[i].y + u[i].z * u[i].z + u[i].w * u[i].w;
    }
  }
  ss = block_sum<NT>(ss, red);
  const float inv = 1.0f / sqrtf(ss / (float)d + eps);
#pragma unroll
  for (int i = 0; i < NV; ++i) {
    const int c = (threadIdx.x + NT * i) * 4;
    if (c < d) {
      const float4 g = *reinterpret_cast<const float4*>(w + c);
      const float h[4] = {u[i].x * inv * g.x, u[i].y * inv * g.y, u[i].z * inv * g.z, u[i].w * inv * g.w};
      T* o = out + row * d + c;
      if constexpr (sizeof(T) == 4) {
        *reinterpret_cast<float4*>(o) = make_float4(h[0], h[1], h[2], h[3]);
      } else {
        *reinterpret_cast<uint2*>(o) = make_uint2(pack2(h[0], h[1]), pack2(h[2], h[3]));
      }
    }
  }
}

// any width: one column per thread and trip; the second pass reads back what the thread itself wrote
template <typename T>
__global__ __launch_bounds__(256) void stream_norm_any_kernel(T* __restrict__ out, float* dst, const float* src,
                                                              long src_row, long src_s, const void* __restrict__ y,
                                                              int yt, const float* __restrict__ mix,
                                                              const float* __restrict__ wout,
                                                              const float* __restrict__ win,
                                                              const float* __restrict__ w, int S, int d, float eps) {
  __shared__ float red[4];
  const long row = blockIdx.x;
  const float* xr = src + row * src_row;
  float* xo = dst + row * S * d;
  float ss = 0.f;
  for (int c = threadIdx.x; c < d; c += 256) {
    float x[kMaxStreams], u = 0.f;
    for (int s = 0; s < S; ++s) x[s] = xr[s * src_s + c];
    const float yv = yt ? ld_any(y, yt, row * d + c) : 0.f;
    for (int t = 0; t < S; ++t) {
      float v = x[t];
      if (yt) {
        v = wout[t] * yv;
        for (int s = 0; s < S; ++s) v += mix[s * S + t] * x[s];
        xo[(long)t * d + c] = v;
      }
      u += (win != nullptr ? win[t] : 1.f) * v;
    }
    ss += u * u;
  }
  ss = block_sum<256>(ss, red);
  const float inv = 1.0f / sqrtf(ss / (float)d + eps);
  const float* xn = yt ? xo : xr;
  const long ns = yt ? d : src_s;
  for (int c = threadIdx.x; c < d; c += 256) {
    float u = 0.f;
    for (int t = 0; t < S; ++t) u += (win != nullptr ? win[t] : 1.f) * xn[t * ns + c];
    stf(out + row * d + c, u * inv * w[c]);
  }
}

}  // namespace k8sllm

using namespace k8sllm;

extern "C" {

// yt: 0 absent, 1 bf16, 2 fp32.  src_row: elements between two rows of src, src_s: between two of its streams
int k8sllm_hy_stream_norm(void* out, float* dst, const float* src, long src_row, long src_s, const void* y, int yt,
                          const float* mix, const float* wout, const float* win, const float* w, long rows, int S, int d,
                          float eps, int f32, hipStream_t s) {
  if (rows <= 0) return 0;
  if (S < 1 || S > kMaxStreams || d < 1) return -1;
#define K8SLLM_SN(T_, SM, NT, NV)                                                                                       \
  hipLaunchKernelGGL((stream_norm_kernel<T_, SM, NT, NV>), dim3((unsigned)rows), dim3(NT), 0, s, (T_*)out, dst, src, src_row, \
                     src_s, y, yt, mix, wout, win, w, S, d, eps)
#define K8SLLM_SNW(T_, SM)                                \
  if (d <= 1024) K8SLLM_SN(T_, SM, 256, 1);               \
  else if (d <= 2048) K8SLLM_SN(T_, SM, 512, 1);          \
  else if (d <= 4096) K8SLLM_SN(T_, SM, 1024, 1);         \
  else K8SLLM_SN(T_, SM, 1024, 2)
#define K8SLLM_SNS(T_)                                                                                                  \
  if (d % 4 || d > 8192 || S > 8)                                                                                       \
    hipLaunchKernelGGL((stream_norm_any_kernel<T_>), dim3((unsigned)rows), dim3(256), 0, s, (T_*)out, dst, src, src_row,   \
                       src_s, y, yt, mix, wout, win, w, S, d, eps);                                                     \
  else if (S <= 2) { K8SLLM_SNW(T_, 2); }                                                                               \
  else if (S <= 4) { K8SLLM_SNW(T_, 4); }                                                                               \
  else { K8SLLM_SNW(T_, 8); }
  if (f32) { K8SLLM_SNS(float) } else { K8SLLM_SNS(bf16_t) }
#undef K8SLLM_SNS
#undef K8SLLM_SNW
#undef K8SLLM_SN
  return (int)hipGetLastError();
}
}
