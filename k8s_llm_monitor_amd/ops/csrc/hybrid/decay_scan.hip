// Linear attention with a decay per head and key channel - or one per head -, plain, with the delta rule or
// with a bonus for the current token (any sizes up to 256 key channels; state, decays, unit norms and every
// product fp32).
//   decay_scan   per segment and head, token by token:
//                    S <- diag(g_t) S
//                    u  = beta_t (v_t - S^T k_t)      (delta rule)      |  u = v_t   (plain)
//                    S <- S + k_t u^T;   o_t = S^T q_t
//                or, with a bonus w [H][dk] (the read-out sees the state BEFORE this token's decay and write):
//                    o_t = (S + diag(w) k_t v_t^T)^T q_t;   S <- diag(g_t) S + k_t v_t^T
//                with g_t = exp(-exp(a_log[h]) softplus(z_t + bias)),  sigmoid(z_t + bias)^(1/tau)  or
//                exp(-exp(z_t + bias)), q and k optionally made unit vectors (x / sqrt(sum x^2 + 1e-6)), q times
//                q_scale, beta_t = sigmoid of a projection column.  The state slot [H][dv][dk] (a value row's key channels contiguous) is
//                read at the segment's start (zero for a sequence that starts in this step), written at its end.
// A segment is one sequence's rows of this step: cu[s] .. cu[s+1], ctx[s] tokens already in its state,
// slot[s] its state slot (< 0: a padding row, output zero).
//
// Workgroup = 4 waves = (segment, head, PB value columns).  A value column p is owned by CH neighbouring
// lanes, each holding 8 key channels of S[p][.] in registers; 64 / CH columns per wave.  The read-out is
// taken from the decayed state BEFORE the write: with S' = diag(g) S,
//     o = S'^T q + u (k . q)
// so the two sums over key channels that a token needs (S'^T k and S'^T q) are independent and their
// lane reductions overlap; k . q does not depend on the state and is prepared with the tile.  (Bonus: the
// read-out takes S itself and v (k . diag(w) q) is added, the same shape.)  The inputs
// of 16 tokens at a time are staged in LDS by the whole workgroup (q, k after the unit norm, the decays
// after their exponentials, v, beta, k . q), so the token loop reads only LDS.
//
// Prompts (long segments) run as two launches: decay_prep computes, for every token at once, what does not
// depend on the state - the decays after their exponentials, q and k after the unit norm and the query scale,
// k . q, beta - as fp32 rows in a workspace, and decay_scan_staged runs the recurrence reading those rows:
// a tile's inputs are fetched into registers while the previous tile's tokens are processed, so the
// sequential loop waits neither for global memory nor for exponentials (which the one-launch form
// evaluates once per block of value columns).  Decode steps (one token per segment) keep the one-launch form.
#include "hy_common.h"

namespace k8sllm {

// what a token writes and reads (MODE)
constexpr int kPlain = 0, kDelta = 1, kBonus = 2;
// how a decay comes from its logit x = z + bias (kind); A = exp(a_log[h])
constexpr int kSoftplus = 0, kSigmoidRoot = 1, kExpExp = 2;
__device__ __forceinline__ float decay_f(float x, int kind, float A, float inv_tau) {
  if (kind == kSoftplus) return expf(-A * softplus_f(x));
  if (kind == kSigmoidRoot) return expf(-softplus_f(-x) * inv_tau);
  return expf(-expf(x));
}

// One token of the recurrence for a lane's 8 key channels; returns the column's read-out (all lanes of the
// column hold it).  gv: this token's decays (one number for all channels where HD).
template <int CH, int MODE, bool HD>
__device__ __forceinline__ float scan_token(float (&S)[8], const float* __restrict__ gp, float gh,
                                            const float* __restrict__ kp, const float* __restrict__ qp, float v,
                                            float bt, float kq) {
  float gv[8];
  if (HD) {
#pragma unroll
    for (int i = 0; i < 8; ++i) gv[i] = gh;
  } else {
    const float4 g0 = *reinterpret_cast<const float4*>(gp), g1 = *reinterpret_cast<const float4*>(gp + 4);
    gv[0] = g0.x; gv[1] = g0.y; gv[2] = g0.z; gv[3] = g0.w;
    gv[4] = g1.x; gv[5] = g1.y; gv[6] = g1.z; gv[7] = g1.w;
  }
  const float4 k0 = *reinterpret_cast<const float4*>(kp), k1 = *reinterpret_cast<const float4*>(kp + 4);
  const float4 q0 = *reinterpret_cast<const float4*>(qp), q1 = *reinterpret_cast<const float4*>(qp + 4);
  const float kv[8] = {k0.x, k0.y, k0.z, k0.w, k1.x, k1.y, k1.z, k1.w};
  const float qv[8] = {q0.x, q0.y, q0.z, q0.w, q1.x, q1.y, q1.z, q1.w};
  float pk0 = 0.f, pk1 = 0.f, pq0 = 0.f, pq1 = 0.f;  // two accumulators per sum: half the dependent adds
#pragma unroll
  for (int i = 0; i < 8; i += 2) {
    if (MODE == kBonus) {
      pq0 += S[i] * qv[i];
      pq1 += S[i + 1] * qv[i + 1];
    }
    S[i] *= gv[i];
    S[i + 1] *= gv[i + 1];
    if (MODE == kDelta) {
      pk0 += S[i] * kv[i];
      pk1 += S[i + 1] * kv[i + 1];
    }
    if (MODE != kBonus) {
      pq0 += S[i] * qv[i];
      pq1 += S[i + 1] * qv[i + 1];
    }
  }
  const float pk = MODE == kDelta ? lanes_sum<CH>(pk0 + pk1) : 0.f;
  const float pq = lanes_sum<CH>(pq0 + pq1);
  const float u = MODE == kDelta ? bt * (v - pk) : v;
#pragma unroll
  for (int i = 0; i < 8; ++i) S[i] += kv[i] * u;
  return pq + u * kq;
}

template <typename T, int CH, int MODE, bool HD>
__global__ __launch_bounds__(256) void decay_scan_kernel(float* __restrict__ o, const T* __restrict__ qkv, long stride,
                                                         int q_col, int k_col, int v_col, const T* __restrict__ z,
                                                         long z_stride, const float* __restrict__ z_bias,
                                                         const float* __restrict__ a_log, float inv_tau, int dkind,
                                                         const T* __restrict__ beta, long b_stride,
                                                         const float* __restrict__ bonus,
                                                         float* __restrict__ state, const int* __restrict__ cu,
                                                         const int* __restrict__ ctx, const int* __restrict__ slot,
                                                         int H, int Gk, int dk, int dv, float q_scale, int unit) {
  constexpr int TB = 16, PW = 64 / CH, PB = 4 * PW;
  constexpr int ROW = 8 * CH + (CH / 8) * 4 + 4;  // channel n sits at n + 4 (n / 64): 64-float halves 4 banks apart
  __shared__ __attribute__((aligned(16))) float qs[TB][ROW];
  __shared__ __attribute__((aligned(16))) float ks[TB][ROW];
  __shared__ __attribute__((aligned(16))) float gs[HD ? 1 : TB][HD ? 4 : ROW];  // not used with one decay per head
  __shared__ float vs[TB][PB];
  __shared__ float bts[TB], kqs[TB], ghs[TB];
  const int s = blockIdx.x, h = blockIdx.y;
  const int sl = slot[s];
  const int t0 = cu[s], t1 = cu[s + 1];
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
  const int chunk = lane % CH, pl = wave * PW + lane / CH;
  const int p = blockIdx.z * PB + pl;
  const bool live = p < dv;
  const int inner = H * dv;
  if (sl < 0) {  // padding rows: defined output, no state
    if (live && chunk == 0)
      for (int t = t0; t < t1; ++t) o[(long)t * inner + (long)h * dv + p] = 0.f;
    return;
  }
  if (t1 <= t0) return;
  const int n0 = chunk * 8;
  const int g = h / (H / Gk);
  if (dk != 8 * CH)  // channels beyond dk stay zero (none where the lanes' 8-channel chunks cover dk exactly)
    for (int i = threadIdx.x; i < min(TB, t1 - t0) * ROW; i += 256) {
      (&qs[0][0])[i] = 0.f;
      (&ks[0][0])[i] = 0.f;
      if (!HD) (&gs[0][0])[i] = 0.f;
    }
  float S[8];
  float* sp = state + (((long)sl * H + h) * dv + p) * dk + n0;
  const bool carried = ctx[s] > 0;
  const bool vec = (dk & 7) == 0 && n0 + 8 <= dk;
  if (carried && live && vec) {
    const float4 a = *reinterpret_cast<const float4*>(sp), b = *reinterpret_cast<const float4*>(sp + 4);
    S[0] = a.x; S[1] = a.y; S[2] = a.z; S[3] = a.w;
    S[4] = b.x; S[5] = b.y; S[6] = b.z; S[7] = b.w;
  } else {
#pragma unroll
    for (int i = 0; i < 8; ++i) S[i] = (carried && live && n0 + i < dk) ? sp[i] : 0.f;
  }
  const float A = a_log != nullptr ? expf(a_log[h]) : 0.f;
  const int boff = n0 + (n0 >> 6) * 4;
  float* op = o + (long)t0 * inner + (long)h * dv + p;  // this lane's output column, advanced per tile
  for (int tb = t0; tb < t1; tb += TB) {
    const int nt = min(TB, t1 - tb);
    __syncthreads();  // the previous tile is consumed (and the zero fill is done)
#pragma unroll 4
    for (int i = threadIdx.x; i < nt * dk; i += 256) {  // unrolled: the independent loads go out together
      const int tt = i / dk, n = i - tt * dk;
      const T* row = qkv + (long)(tb + tt) * stride + (long)g * dk + n;
      const int off = n + (n >> 6) * 4;
      qs[tt][off] = ldf(row + q_col);
      ks[tt][off] = ldf(row + k_col);
      if (!HD) {
        const float zz = ldf(z + (long)(tb + tt) * z_stride + (long)h * dk + n) + z_bias[h * dk + n];
        gs[tt][off] = decay_f(zz, dkind, A, inv_tau);
      }
    }
    for (int i = threadIdx.x; i < nt * PB; i += 256) {
      const int tt = i / PB, pp = i % PB;
      const int pg = blockIdx.z * PB + pp;
      vs[tt][pp] = pg < dv ? ldf(qkv + (long)(tb + tt) * stride + v_col + (long)h * dv + pg) : 0.f;
    }
    if (MODE == kDelta && threadIdx.x < nt) bts[threadIdx.x] = sigmoid_f(ldf(beta + (long)(tb + threadIdx.x) * b_stride + h));
    if (HD && threadIdx.x >= 64 && threadIdx.x - 64 < nt)
      ghs[threadIdx.x - 64] = decay_f(ldf(z + (long)(tb + threadIdx.x - 64) * z_stride + h) + z_bias[h], dkind, A, inv_tau);
    __syncthreads();
    {  // 16 threads per token: unit norms, the query scale and k . q
      const int tt = threadIdx.x >> 4, j = threadIdx.x & 15;
      float sq = 0.f, sk = 0.f;
      if (unit) {
        for (int n = j; n < dk; n += 16) {
          const int off = n + (n >> 6) * 4;
          sq += qs[tt][off] * qs[tt][off];
          sk += ks[tt][off] * ks[tt][off];
        }
        sq = lanes_sum<16>(sq);
        sk = lanes_sum<16>(sk);
      }
      const float mq = unit ? q_scale / sqrtf(sq + 1e-6f) : q_scale;
      const float mk = unit ? 1.0f / sqrtf(sk + 1e-6f) : 1.f;
      float kq = 0.f;
      for (int n = j; n < dk; n += 16) {
        const int off = n + (n >> 6) * 4;
        const float qv = qs[tt][off] * mq, kv = ks[tt][off] * mk;
        qs[tt][off] = qv;
        ks[tt][off] = kv;
        kq += MODE == kBonus ? qv * kv * bonus[g * dk + n] : qv * kv;
      }
      kq = lanes_sum<16>(kq);
      if (j == 0) kqs[tt] = kq;
    }
    __syncthreads();
#pragma unroll 2
    for (int tt = 0; tt < nt; ++tt) {
      const float r = scan_token<CH, MODE, HD>(S, &gs[HD ? 0 : tt][HD ? 0 : boff], HD ? ghs[tt] : 0.f, &ks[tt][boff],
                                               &qs[tt][boff], vs[tt][pl], MODE == kDelta ? bts[tt] : 0.f, kqs[tt]);
      if (live && chunk == 0) op[(long)tt * inner] = r;
    }
    op += (long)TB * inner;
  }
  if (live) {
    if (vec) {
      *reinterpret_cast<float4*>(sp) = make_float4(S[0], S[1], S[2], S[3]);
      *reinterpret_cast<float4*>(sp + 4) = make_float4(S[4], S[5], S[6], S[7]);
    } else {
#pragma unroll
      for (int i = 0; i < 8; ++i)
        if (n0 + i < dk) sp[i] = S[i];
    }
  }
}

// ---- the two-launch form for prompts
// workspace rows (fp32): qn, kn [T][Gk][dk], gd [T][H][dk] (one decay per head: [T][H]), kq [T][Gk], bt [T][H]
template <typename T, bool HD>
__global__ __launch_bounds__(256) void decay_prep_kernel(float* __restrict__ qn, float* __restrict__ kn,
                                                         float* __restrict__ gd, float* __restrict__ kq,
                                                         float* __restrict__ bt, const T* __restrict__ qkv, long stride,
                                                         int q_col, int k_col, const T* __restrict__ z, long z_stride,
                                                         const float* __restrict__ z_bias,
                                                         const float* __restrict__ a_log, float inv_tau, int dkind,
                                                         const T* __restrict__ beta, long b_stride,
                                                         const float* __restrict__ bonus, int H, int Gk,
                                                         int dk, float q_scale, int unit) {
  // one workgroup per token: the decays of all heads, beta, then a wave per query / key head
  const long t = blockIdx.x;
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
  const int nd = HD ? H : H * dk;
  const T* zr = z + t * z_stride;
  float* gr = gd + t * nd;
  if (dkind == kSoftplus) {
    for (int e = threadIdx.x; e < nd; e += 256)
      gr[e] = decay_f(ldf(zr + e) + z_bias[e], kSoftplus, expf(a_log[HD ? e : e / dk]), 0.f);
  } else if (dkind == kSigmoidRoot) {
    for (int e = threadIdx.x; e < nd; e += 256) gr[e] = decay_f(ldf(zr + e) + z_bias[e], kSigmoidRoot, 0.f, inv_tau);
  } else {
    for (int e = threadIdx.x; e < nd; e += 256) gr[e] = decay_f(ldf(zr + e) + z_bias[e], kExpExp, 0.f, 0.f);
  }
  if (beta != nullptr)
    for (int h = threadIdx.x; h < H; h += 256) bt[t * H + h] = sigmoid_f(ldf(beta + t * b_stride + h));
  for (int g = wave; g < Gk; g += 4) {
    const T* row = qkv + t * stride + (long)g * dk;
    float sq = 0.f, sk = 0.f;
    if (unit) {
      for (int n = lane; n < dk; n += 64) {
        const float q = ldf(row + q_col + n), k = ldf(row + k_col + n);
        sq += q * q;
        sk += k * k;
      }
      sq = wave_sum(sq);
      sk = wave_sum(sk);
    }
    const float mq = unit ? q_scale / sqrtf(sq + 1e-6f) : q_scale;
    const float mk = unit ? 1.0f / sqrtf(sk + 1e-6f) : 1.f;
    float dot = 0.f;
    for (int n = lane; n < dk; n += 64) {
      const float q = ldf(row + q_col + n) * mq, k = ldf(row + k_col + n) * mk;
      qn[(t * Gk + g) * dk + n] = q;
      kn[(t * Gk + g) * dk + n] = k;
      dot += bonus != nullptr ? q * k * bonus[g * dk + n] : q * k;
    }
    dot = wave_sum(dot);
    if (lane == 0) kq[t * Gk + g] = dot;
  }
}

template <typename T, int CH, int MODE, bool HD>
__global__ __launch_bounds__(256) void decay_scan_staged_kernel(float* __restrict__ o, const T* __restrict__ qkv,
                                                                long stride, int v_col, const float* __restrict__ qn,
                                                                const float* __restrict__ kn,
                                                                const float* __restrict__ gd,
                                                                const float* __restrict__ kq,
                                                                const float* __restrict__ bt, float* __restrict__ state,
                                                                const int* __restrict__ cu, const int* __restrict__ ctx,
                                                                const int* __restrict__ slot, int H, int Gk, int dk,
                                                                int dv) {
  constexpr int TB = 16, PW = 64 / CH, PB = 4 * PW;
  constexpr int ROW = 8 * CH + (CH / 8) * 4 + 4;  // channel n sits at n + 4 (n / 64); a multiple of 4 floats
  constexpr int Q4 = 2 * CH;                      // 4-channel groups of a padded row
  constexpr int NB = (TB * Q4 + 255) / 256;       // ... per thread, of each of q, k, decays
  constexpr int NV = (TB * PB + 255) / 256;       // values per thread
  __shared__ __attribute__((aligned(16))) float qs[TB][ROW];
  __shared__ __attribute__((aligned(16))) float ks[TB][ROW];
  __shared__ __attribute__((aligned(16))) float gs[HD ? 1 : TB][HD ? 4 : ROW];  // not used with one decay per head
  __shared__ float vs[TB][PB];
  __shared__ float bts[TB], kqs[TB], ghs[TB];
  const int s = blockIdx.x, h = blockIdx.y;
  const int sl = slot[s];
  const int t0 = cu[s], t1 = cu[s + 1];
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
  const int chunk = lane % CH, pl = wave * PW + lane / CH;
  const int p = blockIdx.z * PB + pl;
  const bool live = p < dv;
  const int inner = H * dv;
  if (sl < 0) {  // padding rows: defined output, no state
    if (live && chunk == 0)
      for (int t = t0; t < t1; ++t) o[(long)t * inner + (long)h * dv + p] = 0.f;
    return;
  }
  if (t1 <= t0) return;
  const int n0 = chunk * 8;
  const int g = h / (H / Gk);
  float S[8];
  float* sp = state + (((long)sl * H + h) * dv + p) * dk + n0;
  const bool carried = ctx[s] > 0;
  const bool vec = (dk & 7) == 0 && n0 + 8 <= dk;
  if (carried && live && vec) {
    const float4 a = *reinterpret_cast<const float4*>(sp), b = *reinterpret_cast<const float4*>(sp + 4);
    S[0] = a.x; S[1] = a.y; S[2] = a.z; S[3] = a.w;
    S[4] = b.x; S[5] = b.y; S[6] = b.z; S[7] = b.w;
  } else {
#pragma unroll
    for (int i = 0; i < 8; ++i) S[i] = (carried && live && n0 + i < dk) ? sp[i] : 0.f;
  }
  const int boff = n0 + (n0 >> 6) * 4;
  const bool vec4 = (dk & 3) == 0;
  // the next tile's inputs, in registers while this tile's tokens are processed.  Loads are not predicated (a
  // branch around a load would wait for it there): a token past the segment reads its last row, channels
  // past dk the row's last ones, and what they must not contribute is dropped when it is staged
  float4 rq[NB], rk[NB], rg[HD ? 1 : NB];
  T rv[NV];
  float rs;
  const int gp_col = min((int)blockIdx.z * PB + (int)(threadIdx.x % PB), dv - 1);  // 256 % PB == 0: one column per thread
  auto fetch = [&](int tb) {
#pragma unroll
    for (int u = 0; u < NB; ++u) {
      const int i = threadIdx.x + 256 * u;
      const long t = min(tb + i / Q4, t1 - 1);
      const int n = (i % Q4) * 4;
      const float* qp = qn + (t * Gk + g) * dk;
      const float* kp = kn + (t * Gk + g) * dk;
      const float* gp = HD ? nullptr : gd + (t * H + h) * dk;
      if (vec4) {
        const int m = min(n, dk - 4);
        rq[u] = *reinterpret_cast<const float4*>(qp + m);
        rk[u] = *reinterpret_cast<const float4*>(kp + m);
        if (!HD) rg[u] = *reinterpret_cast<const float4*>(gp + m);
      } else {
        const int m0 = min(n, dk - 1), m1 = min(n + 1, dk - 1), m2 = min(n + 2, dk - 1), m3 = min(n + 3, dk - 1);
        rq[u] = make_float4(qp[m0], qp[m1], qp[m2], qp[m3]);
        rk[u] = make_float4(kp[m0], kp[m1], kp[m2], kp[m3]);
        if (!HD) rg[u] = make_float4(gp[m0], gp[m1], gp[m2], gp[m3]);
      }
    }
#pragma unroll
    for (int u = 0; u < NV; ++u) {
      const long t = min(tb + (int)(threadIdx.x + 256 * u) / PB, t1 - 1);
      rv[u] = qkv[t * stride + v_col + (long)h * dv + gp_col];
    }
    {  // threads 0 .. 15: k . q; the next 16: beta; the next 16: the head's decay
      const long t = min(tb + (int)(threadIdx.x % TB), t1 - 1);
      const int w = threadIdx.x / TB;
      const float* src = kq + t * Gk + g;
      if (MODE == kDelta && w == 1) src = bt + t * H + h;
      if (HD && w == 2) src = gd + t * H + h;
      rs = *src;
    }
  };
  fetch(t0);
  float* op = o + (long)t0 * inner + (long)h * dv + p;  // this lane's output column, advanced per tile
  for (int tb = t0; tb < t1; tb += TB) {
    const int nt = min(TB, t1 - tb);
    __syncthreads();  // the previous tile is consumed
#pragma unroll
    for (int u = 0; u < NB; ++u) {
      const int i = threadIdx.x + 256 * u;
      const int tt = i / Q4, n = (i % Q4) * 4;
      if (tt < TB) {
        const int off = tt * ROW + n + (n >> 6) * 4;
        float4 q4 = rq[u], k4 = rk[u];
        if (n + 4 > dk) {  // channels beyond dk: zero keys and queries leave the state and the sums alone
          if (n >= dk) q4.x = k4.x = 0.f;
          if (n + 1 >= dk) q4.y = k4.y = 0.f;
          if (n + 2 >= dk) q4.z = k4.z = 0.f;
          q4.w = k4.w = 0.f;
        }
        *reinterpret_cast<float4*>(&qs[0][0] + off) = q4;
        *reinterpret_cast<float4*>(&ks[0][0] + off) = k4;
        if (!HD) *reinterpret_cast<float4*>(&gs[0][0] + off) = rg[u];
      }
    }
#pragma unroll
    for (int u = 0; u < NV; ++u) {
      const int i = threadIdx.x + 256 * u;
      if (i < TB * PB) (&vs[0][0])[i] = ldf(&rv[u]);
    }
    if (threadIdx.x < TB) kqs[threadIdx.x] = rs;
    else if (MODE == kDelta && threadIdx.x < 2 * TB) bts[threadIdx.x - TB] = rs;
    else if (HD && threadIdx.x >= 2 * TB && threadIdx.x < 3 * TB) ghs[threadIdx.x - 2 * TB] = rs;
    __syncthreads();
    if (tb + TB < t1) fetch(tb + TB);
    auto token = [&](int tt) -> float {
      return scan_token<CH, MODE, HD>(S, &gs[HD ? 0 : tt][HD ? 0 : boff], HD ? ghs[tt] : 0.f, &ks[tt][boff], &qs[tt][boff],
                                      vs[tt][pl], MODE == kDelta ? bts[tt] : 0.f, kqs[tt]);
    };
    if (nt == TB) {  // a lane of the column keeps every KB-th read-out: one store for KB tokens
      constexpr int KB = CH < TB ? CH : TB;
#pragma unroll
      for (int tk = 0; tk < TB; tk += KB) {
        float keep = 0.f;
#pragma unroll
        for (int j = 0; j < KB; ++j) {
          const float r = token(tk + j);
          keep = chunk == j ? r : keep;
        }
        if (live && chunk < KB) op[(long)(tk + chunk) * inner] = keep;
      }
    } else {
      for (int tt = 0; tt < nt; ++tt) {
        const float r = token(tt);
        if (live && chunk == 0) op[(long)tt * inner] = r;
      }
    }
    op += (long)TB * inner;
  }
  if (live) {
    if (vec) {
      *reinterpret_cast<float4*>(sp) = make_float4(S[0], S[1], S[2], S[3]);
      *reinterpret_cast<float4*>(sp + 4) = make_float4(S[4], S[5], S[6], S[7]);
    } else {
#pragma unroll
      for (int i = 0; i < 8; ++i)
        if (n0 + i < dk) sp[i] = S[i];
    }
  }
}

}  // namespace k8sllm

using namespace k8sllm;

// one step's arguments, as k8sllm_hy_decay_scan takes them
struct ScanArgs {
  float* o;
  const void* qkv;
  long stride;
  int q_col, k_col, v_col;
  const void* z;
  long z_stride;
  const float *z_bias, *a_log;
  float inv_tau;
  int dkind;
  const void* beta;
  long b_stride;
  const float* bonus;
  float* state;
  const int *cu, *ctx, *slot;
  int S, H, Gk, dk, dv;
  float q_scale;
  int unit;
  float* ws;
  long rows;
};

template <typename T, int CH, int MODE, bool HD>
static void launch_scan_ch(const ScanArgs& a, hipStream_t s) {
  const dim3 grid((unsigned)a.S, (unsigned)a.H, (unsigned)((a.dv + 256 / CH - 1) / (256 / CH)));
  if (a.ws == nullptr) {
    hipLaunchKernelGGL((decay_scan_kernel<T, CH, MODE, HD>), grid, dim3(256), 0, s, a.o, (const T*)a.qkv, a.stride, a.q_col,
                       a.k_col, a.v_col, (const T*)a.z, a.z_stride, a.z_bias, a.a_log, a.inv_tau, a.dkind,
                       (const T*)a.beta, a.b_stride, a.bonus, a.state, a.cu, a.ctx, a.slot, a.H, a.Gk, a.dk, a.dv,
                       a.q_scale, a.unit);
    return;
  }
  float* qn = a.ws;
  float* kn = qn + a.rows * a.Gk * a.dk;
  float* gd = kn + a.rows * a.Gk * a.dk;
  float* kq = gd + a.rows * a.H * (HD ? 1 : a.dk);
  float* bt = kq + a.rows * a.Gk;
  hipLaunchKernelGGL((decay_prep_kernel<T, HD>), dim3((unsigned)a.rows), dim3(256), 0, s, qn, kn, gd, kq, bt,
                     (const T*)a.qkv, a.stride, a.q_col, a.k_col, (const T*)a.z, a.z_stride, a.z_bias, a.a_log, a.inv_tau,
                     a.dkind, (const T*)a.beta, a.b_stride, a.bonus, a.H, a.Gk, a.dk, a.q_scale, a.unit);
  hipLaunchKernelGGL((decay_scan_staged_kernel<T, CH, MODE, HD>), grid, dim3(256), 0, s, a.o, (const T*)a.qkv, a.stride,
                     a.v_col, qn, kn, gd, kq, bt, a.state, a.cu, a.ctx, a.slot, a.H, a.Gk, a.dk, a.dv);
}

template <typename T, int MODE, bool HD>
static int launch_scan_mode(const ScanArgs& a, hipStream_t s) {
  if (a.dk <= 16) launch_scan_ch<T, 2, MODE, HD>(a, s);
  else if (a.dk <= 32) launch_scan_ch<T, 4, MODE, HD>(a, s);
  else if (a.dk <= 64) launch_scan_ch<T, 8, MODE, HD>(a, s);
  else if (a.dk <= 128) launch_scan_ch<T, 16, MODE, HD>(a, s);
  else if (a.dk <= 256) launch_scan_ch<T, 32, MODE, HD>(a, s);
  else return -1;
  return (int)hipGetLastError();
}

template <typename T>
static int launch_scan_t(const ScanArgs& a, int mode, int per_head, hipStream_t s) {
  if (mode == kDelta) return per_head ? launch_scan_mode<T, kDelta, true>(a, s) : launch_scan_mode<T, kDelta, false>(a, s);
  if (per_head) return -1;  // one decay per head is built for the delta rule
  if (mode == kBonus) return launch_scan_mode<T, kBonus, false>(a, s);
  return launch_scan_mode<T, kPlain, false>(a, s);
}

extern "C" {

// floats of workspace the two-launch form needs for T rows
long k8sllm_hy_decay_scan_ws(long T, int H, int Gk, int dk) { return T * ((long)2 * Gk * dk + (long)H * dk + Gk + H); }

// beta != nullptr: the delta rule; bonus != nullptr ([H][dk], Gk == H): the bonus form; neither: plain.
// dkind: 0 exp(-exp(a_log) softplus(x)), 1 sigmoid(x)^(inv_tau), 2 exp(-exp(x)).  per_head: z and z_bias hold
// one decay logit per head.  ws != nullptr: the two-launch form for prompts, with
// k8sllm_hy_decay_scan_ws(T, ...) floats of workspace (T = rows of the step)
int k8sllm_hy_decay_scan(float* o, const void* qkv, long stride, int q_col, int k_col, int v_col, const void* z,
                         long z_stride, const float* z_bias, const float* a_log, float inv_tau, int dkind, int per_head,
                         const void* beta, long b_stride, const float* bonus, float* state, const int* cu,
                         const int* ctx, const int* slot, int S, int H, int Gk, int dk, int dv, float q_scale, int unit,
                         int f32, float* ws, long T, hipStream_t s) {
  if (S <= 0) return 0;
  if (Gk < 1 || H % Gk || dk < 1 || dv < 1 || dkind < 0 || dkind > 2 || (dkind == 0 && a_log == nullptr)) return -1;
  if (bonus != nullptr && (beta != nullptr || Gk != H)) return -1;
  const ScanArgs a = {o, qkv, stride, q_col, k_col, v_col, z, z_stride, z_bias, a_log, inv_tau, dkind, beta, b_stride, bonus,
                      state, cu, ctx, slot, S, H, Gk, dk, dv, q_scale, unit, ws, T};
  const int mode = beta != nullptr ? kDelta : bonus != nullptr ? kBonus : kPlain;
  return f32 ? launch_scan_t<float>(a, mode, per_head, s) : launch_scan_t<bf16_t>(a, mode, per_head, s);
}
}
