// The selective state-space recurrence with a decay per channel AND state (any channel count, up to 256
// states; everything from the step sizes on fp32).  Per segment, channel c and state n, token by token:
//     dt = softplus(dt_raw[t][c] + dt_bias[c])
//     S[c][n] <- exp(-exp(a_log[c][n]) dt) S[c][n] + dt x_t[c] B_t[n]
//     y_t[c]  = sum_n S[c][n] C_t[n] + D[c] x_t[c];      out_t[c] = y_t[c] * silu(z_t[c])
// The state slot [C][N] is read at the segment's start (zero for a sequence that starts in this step) and
// written back at its end.  A segment is one sequence's rows of this step: cu[s] .. cu[s+1], ctx[s] tokens
// already in its state, slot[s] its state slot (< 0: padding rows, output zero).
//
// Workgroup = 4 waves = (segment, 256 / LPC channels).  A channel is owned by LPC neighbouring lanes, each
// with NPL of its states (and their exponents' factors) in registers; the read-out's partial sums are DPP adds
// over those lanes.  16 tokens at a time are staged in LDS: step sizes after softplus, dt x, B, C; the raw
// values of the next 16 are fetched into registers while the current ones are processed.  The read-outs of
// a tile meet in LDS (a lane keeps every LPC-th one, so LPC tokens need one LDS write), and the whole
// workgroup adds the skip term, applies the gate and stores rows.  Loads are not predicated: a token past
// the segment reads the segment's last row, a channel past the end the last channel, and what they must
// not contribute is zeroed when it is staged - a branch around a load would wait for it there.
// One exponential per state and token (v_exp_f32 in base 2, log2 e folded into the factor) is what bounds it.
#include "hy_common.h"

namespace k8sllm {

// log(1 + exp(x)) to a few units in the last place without the library's branches: max(x, 0) + log1p(e),
// e = exp(-|x|); log1p by its series below 1/32, by v_log_f32 above
__device__ __forceinline__ float softplus_fast(float x) {
  const float a = -fabsf(x), t = a * 1.44269504088896341f;
  const float lo = fmaf(a, 1.44269504088896341f, -t);  // what rounding the product dropped
  const float e2 = __builtin_amdgcn_exp2f(t), e = fmaf(e2, lo * 0.693147180559945309f, e2);
  const float series = e * fmaf(e, fmaf(e, fmaf(e, -0.25f, 0.333333333f), -0.5f), 1.f);
  const float lg = __builtin_amdgcn_logf(1.f + e) * 0.693147180559945309f;
  return fmaxf(x, 0.f) + (e < 0.03125f ? series : lg);
}

template <typename T, int LPC, int NPL>
__global__ __launch_bounds__(256) void selective_scan_kernel(
    T* __restrict__ out, const T* __restrict__ xc, const T* __restrict__ q, long q_stride, int b_col, int c_col,
    const T* __restrict__ dt, long dt_stride, const float* __restrict__ dt_bias, const float* __restrict__ a_log,
    const float* __restrict__ d_skip, const T* __restrict__ z, long z_stride, float* __restrict__ state,
    const int* __restrict__ cu, const int* __restrict__ ctx, const int* __restrict__ slot, int C, int N) {
  constexpr int TB = 16, PB = 256 / LPC, NS = LPC * NPL;
  constexpr int NV = TB * PB / 256;           // (token, channel) pairs a thread stages and finishes
  constexpr int NB = (TB * NS + 255) / 256;   // B / C elements a thread stages
  __shared__ __attribute__((aligned(16))) float Bs[TB][NS];
  __shared__ __attribute__((aligned(16))) float Cs[TB][NS];
  __shared__ float dts[TB][PB], us[TB][PB];
  __shared__ float ys[TB][PB + 64 / LPC];  // padded: the lanes of a channel write neighbouring rows to different banks
  const int s = blockIdx.x;
  const int sl = slot[s];
  const int t0 = cu[s], t1 = cu[s + 1];
  const int pc = threadIdx.x % PB, tt0 = threadIdx.x / PB;  // staging: channel pc, tokens tt0 + LPC u
  const int cs = blockIdx.y * PB + pc;
  const bool slive = cs < C;
  if (sl < 0) {  // padding rows: defined output, no state
    if (slive)
      for (int t = t0 + tt0; t < t1; t += LPC) stf(out + (long)t * C + cs, 0.f);
    return;
  }
  if (t1 <= t0) return;
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
  const int chunk = lane % LPC, pl = wave * (64 / LPC) + lane / LPC;
  const int c = blockIdx.y * PB + pl, n0 = chunk * NPL;
  const bool live = c < C;
  const bool vec = (N & 3) == 0 && n0 + NPL <= N;
  const bool carried = ctx[s] > 0;
  float S[NPL], A[NPL];
  float* sp = state + ((long)sl * C + c) * N + n0;
  const float* ap = a_log + (long)c * N + n0;
  if (live && vec) {
#pragma unroll
    for (int i = 0; i < NPL; i += 4) {
      const float4 a = *reinterpret_cast<const float4*>(ap + i);
      A[i] = a.x; A[i + 1] = a.y; A[i + 2] = a.z; A[i + 3] = a.w;
      float4 v = make_float4(0.f, 0.f, 0.f, 0.f);
      if (carried) v = *reinterpret_cast<const float4*>(sp + i);
      S[i] = v.x; S[i + 1] = v.y; S[i + 2] = v.z; S[i + 3] = v.w;
    }
#pragma unroll
    for (int i = 0; i < NPL; ++i) A[i] = -expf(A[i]) * 1.44269504088896341f;
  } else {
#pragma unroll
    for (int i = 0; i < NPL; ++i) {
      const bool in = live && n0 + i < N;
      A[i] = in ? -expf(ap[i]) * 1.44269504088896341f : 0.f;
      S[i] = (in && carried) ? sp[i] : 0.f;
    }
  }
  const float bias = slive ? dt_bias[cs] : 0.f, D = slive ? d_skip[cs] : 0.f;
  T rd[NV], rx[NV], rz[NV], rB[NB], rC[NB];
  const int cl = min(cs, C - 1);
  auto fetch = [&](int tb) {
#pragma unroll
    for (int u = 0; u < NV; ++u) {
      const long t = min(tb + tt0 + LPC * u, t1 - 1);
      rd[u] = dt[t * dt_stride + cl];
      rx[u] = xc[t * C + cl];
      rz[u] = z[t * z_stride + cl];
    }
#pragma unroll
    for (int u = 0; u < NB; ++u) {
      const int i = threadIdx.x + 256 * u;
      const T* row = q + (long)min(tb + i / NS, t1 - 1) * q_stride + min(i % NS, N - 1);
      rB[u] = row[b_col];
      rC[u] = row[c_col];
    }
  };
  auto token = [&](int tt) -> float {  // the recurrence for one staged token; the channel's read-out on all its lanes
    const float d = dts[tt][pl], u = us[tt][pl];
    float acc = 0.f;
#pragma unroll
    for (int i = 0; i < NPL; i += 4) {
      const float4 b = *reinterpret_cast<const float4*>(&Bs[tt][n0 + i]);
      const float4 g = *reinterpret_cast<const float4*>(&Cs[tt][n0 + i]);
      S[i] = __builtin_amdgcn_exp2f(d * A[i]) * S[i] + u * b.x;
      S[i + 1] = __builtin_amdgcn_exp2f(d * A[i + 1]) * S[i + 1] + u * b.y;
      S[i + 2] = __builtin_amdgcn_exp2f(d * A[i + 2]) * S[i + 2] + u * b.z;
      S[i + 3] = __builtin_amdgcn_exp2f(d * A[i + 3]) * S[i + 3] + u * b.w;
      acc += S[i] * g.x + S[i + 1] * g.y + S[i + 2] * g.z + S[i + 3] * g.w;
    }
    return lanes_sum<LPC>(acc);
  };
  fetch(t0);
  for (int tb = t0; tb < t1; tb += TB) {
    const int nt = min(TB, t1 - tb);
    float ex[NV], ez[NV];  // this tile's x and gate, for its epilogue
#pragma unroll
    for (int u = 0; u < NV; ++u) {
      const int tt = tt0 + LPC * u;
      const float d = softplus_fast(ldf(&rd[u]) + bias);
      ex[u] = ldf(&rx[u]);
      ez[u] = ldf(&rz[u]);
      dts[tt][pc] = d;
      us[tt][pc] = d * ex[u];
    }
#pragma unroll
    for (int u = 0; u < NB; ++u) {
      const int i = threadIdx.x + 256 * u;
      const bool in = i % NS < N;  // states beyond N stay zero
      if (NB * 256 == TB * NS || i < TB * NS) {
        (&Bs[0][0])[i] = in ? ldf(&rB[u]) : 0.f;
        (&Cs[0][0])[i] = in ? ldf(&rC[u]) : 0.f;
      }
    }
    __syncthreads();
    if (tb + TB < t1) fetch(tb + TB);
    if (nt == TB) {
#pragma unroll
      for (int t4 = 0; t4 < TB; t4 += LPC) {
        float keep = 0.f;
#pragma unroll
        for (int j = 0; j < LPC; ++j) {
          const float acc = token(t4 + j);
          keep = chunk == j ? acc : keep;
        }
        ys[t4 + chunk][pl] = keep;
      }
    } else {
      for (int tt = 0; tt < nt; ++tt) {
        const float acc = token(tt);
        if (chunk == 0) ys[tt][pl] = acc;
      }
    }
    __syncthreads();  // the tile's inputs are consumed and its read-outs complete
#pragma unroll
    for (int u = 0; u < NV; ++u) {
      const int tt = tt0 + LPC * u;
      if (slive && tt < nt) stf(out + (long)(tb + tt) * C + cs, (ys[tt][pc] + D * ex[u]) * silu_f(ez[u]));
    }
  }
  if (live) {
    if (vec) {
#pragma unroll
      for (int i = 0; i < NPL; i += 4) *reinterpret_cast<float4*>(sp + i) = make_float4(S[i], S[i + 1], S[i + 2], S[i + 3]);
    } else {
#pragma unroll
      for (int i = 0; i < NPL; ++i)
        if (n0 + i < N) sp[i] = S[i];
    }
  }
}

}  // namespace k8sllm

using namespace k8sllm;

template <typename T>
static int launch_selective(void* out, const void* xc, const void* q, long q_stride, int b_col, int c_col, const void* dt,
                            long dt_stride, const float* dt_bias, const float* a_log, const float* d_skip, const void* z,
                            long z_stride, float* state, const int* cu, const int* ctx, const int* slot, int S, int C,
                            int N, hipStream_t s) {
#define K8SLLM_SS(LPC, NPL)                                                                                          \
  hipLaunchKernelGGL((selective_scan_kernel<T, LPC, NPL>), dim3((unsigned)S, (unsigned)((C + 256 / LPC - 1) / (256 / LPC))), \
                     dim3(256), 0, s, (T*)out, (const T*)xc, (const T*)q, q_stride, b_col, c_col, (const T*)dt, dt_stride,   \
                     dt_bias, a_log, d_skip, (const T*)z, z_stride, state, cu, ctx, slot, C, N)
  if (N <= 8) K8SLLM_SS(2, 4);
  else if (N <= 16) K8SLLM_SS(4, 4);
  else if (N <= 32) K8SLLM_SS(8, 4);
  else if (N <= 64) K8SLLM_SS(8, 8);
  else if (N <= 128) K8SLLM_SS(16, 8);
  else if (N <= 256) K8SLLM_SS(16, 16);
  else return -1;
#undef K8SLLM_SS
  return (int)hipGetLastError();
}

extern "C" {

// xc, out [T][C] contiguous; q's rows hold B from b_col on and C from c_col on (N each)
int k8sllm_hy_selective_scan(void* out, const void* xc, const void* q, long q_stride, int b_col, int c_col,
                             const void* dt, long dt_stride, const float* dt_bias, const float* a_log, const float* d_skip,
                             const void* z, long z_stride, float* state, const int* cu, const int* ctx, const int* slot,
                             int S, long T, int C, int N, int f32, hipStream_t s) {
  if (S <= 0 || T <= 0) return 0;
  if (C < 1 || N < 1) return -1;
#define K8SLLM_ARGS \
  out, xc, q, q_stride, b_col, c_col, dt, dt_stride, dt_bias, a_log, d_skip, z, z_stride, state, cu, ctx, slot, S, C, N, s
  return f32 ? launch_selective<float>(K8SLLM_ARGS) : launch_selective<bf16_t>(K8SLLM_ARGS);
#undef K8SLLM_ARGS
}
}
