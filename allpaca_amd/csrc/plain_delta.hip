// Plain kernels of two recurrent mixers with 32-bit state per request: the gated delta rule (a matrix a head) and the
// gated linear recurrence (a number a channel).  All arithmetic in 32-bit float with an order of additions that the
// row's own place and the sizes fix (never the batch), any element type in and out.
#include "common.h"
#include <math.h>

namespace {

__device__ __forceinline__ float sigmoid_f(float z) { return 1.0f / (1.0f + expf(-z)); }
__device__ __forceinline__ float softplus_f(float z) { return z > 20.f ? z : log1pf(expf(z)); }
__device__ __forceinline__ float gelu_tanh_f(float z) {
  return 0.5f * z * (1.0f + tanhf(0.7978845608028654f * (z + 0.044715f * z * z * z)));
}

// ---------------------------------------------------------------------------
// Gated delta rule, a segment's rows in order.  Per head, S [dk][dv]:
//   S <- g S;  u = beta (v - S^T k);  S <- S + k u^T;  o = S^T q
// with k and q divided by sqrt(sum of squares + 1e-6), q also times q_scale, beta = sigmoid(b), g = exp(-A softplus(a +
// dt_bias)).  With s = S^T k and r = S^T q of the old S the same is u = beta (v - g s), o = g r + (q . k) u: one pass
// over the state gives both sums, and the next writes it.
// rows [T, ld]: q heads at q_off and k heads at k_off (G of dk), v heads at v_off (H of dv); head h uses q/k head
// h / (H / G).  ba [T, ldba]: the logits a at a_off and b at b_off (H each).
// A block takes one segment x one head x 64 value columns; a thread keeps VEC columns of the rows rg, rg + RG, ... of S.
// Every wave has q and k across its lanes, so that a row costs one barrier.
// ---------------------------------------------------------------------------
template <int VEC, int RPT>   // columns a thread; rows a thread: dk <= 4 * VEC * RPT
__global__ __launch_bounds__(256) void delta_rule_kernel(
    const void* __restrict__ rows, int dtype, int ld, int q_off, int k_off, int v_off, int H, int G, int dk, int dv,
    const void* __restrict__ ba, int ba_dtype, int ldba, int a_off, int b_off, const float* __restrict__ A,
    const float* __restrict__ dt_bias, float q_scale, float* __restrict__ state, const int* __restrict__ seg_row0,
    const int* __restrict__ seg_rows, const int* __restrict__ slots, float* __restrict__ out, int ldo) {
  constexpr int TC = 64 / VEC, RG = 4 * VEC, M = 4;     // threads a row of 64 columns; row groups; 64-element pieces of dk
  __shared__ float red[2][4][64][2];
  const int seg = blockIdx.x, h = blockIdx.y, tid = threadIdx.x, lane = tid % WAVE, wave = tid / WAVE;
  const int cj = (tid % TC) * VEC, col = blockIdx.z * 64 + cj, rg = tid / TC;
  const int r0 = seg_row0[seg], n = seg_rows[seg], hk = h / (H / G);
  float* S = state + ((size_t)slots[seg] * H + h) * dk * dv;
  const float Ah = A[h], bias = dt_bias[h];
  float s[RPT][VEC];
#pragma unroll
  for (int ii = 0; ii < RPT; ++ii) {
    const int i = rg + RG * ii;
    const float* at = S + (size_t)i * dv + col;
    const bool on = i < dk && col < dv;
    if constexpr (VEC == 4) {
      const float4 v = on ? *reinterpret_cast<const float4*>(at) : float4{0.f, 0.f, 0.f, 0.f};
      s[ii][0] = v.x; s[ii][1] = v.y; s[ii][2] = v.z; s[ii][3] = v.w;
    } else {
      s[ii][0] = on ? *at : 0.f;
    }
  }
  for (int t = 0; t < n; ++t) {
    const size_t row = (size_t)(r0 + t) * ld;
    float qv[M], kv[M], v[VEC];
    float qq = 0.f, kk = 0.f, qk = 0.f;
#pragma unroll
    for (int m = 0; m < M; ++m) {
      const int i = lane + 64 * m;
      qv[m] = i < dk ? load_f(rows, dtype, row + q_off + (size_t)hk * dk + i) : 0.f;
      kv[m] = i < dk ? load_f(rows, dtype, row + k_off + (size_t)hk * dk + i) : 0.f;
      qq = fmaf(qv[m], qv[m], qq);
      kk = fmaf(kv[m], kv[m], kk);
      qk = fmaf(qv[m], kv[m], qk);
    }
#pragma unroll
    for (int e = 0; e < VEC; ++e)
      v[e] = col + e < dv ? load_f(rows, dtype, row + v_off + (size_t)h * dv + col + e) : 0.f;
    const float a = load_f(ba, ba_dtype, (size_t)(r0 + t) * ldba + a_off + h) + bias;
    const float beta = sigmoid_f(load_f(ba, ba_dtype, (size_t)(r0 + t) * ldba + b_off + h));
    const float g = expf(-Ah * softplus_f(a));
    const float qi = q_scale / sqrtf(wave_sum(qq) + 1e-6f), ki = 1.0f / sqrtf(wave_sum(kk) + 1e-6f);
    qk = wave_sum(qk) * qi * ki;
    float sk[VEC], sq[VEC], kr[RPT];
#pragma unroll
    for (int e = 0; e < VEC; ++e) sk[e] = sq[e] = 0.f;
#pragma unroll
    for (int ii = 0; ii < RPT; ++ii) {
      const int src = (rg + RG * ii) % 64;
      constexpr int per = 64 / RG;
      kr[ii] = __shfl(kv[ii / per], src, WAVE) * ki;
      const float q = __shfl(qv[ii / per], src, WAVE) * qi;
#pragma unroll
      for (int e = 0; e < VEC; ++e) {
        sk[e] = fmaf(kr[ii], s[ii][e], sk[e]);
        sq[e] = fmaf(q, s[ii][e], sq[e]);
      }
    }
    if (VEC == 4) {                                     // the wave's four row groups
#pragma unroll
      for (int e = 0; e < VEC; ++e) {
        sk[e] += __shfl_xor(sk[e], 16, WAVE);
        sk[e] += __shfl_xor(sk[e], 32, WAVE);
        sq[e] += __shfl_xor(sq[e], 16, WAVE);
        sq[e] += __shfl_xor(sq[e], 32, WAVE);
      }
    }
    float(*rd)[64][2] = red[t & 1];
    if (lane < TC) {
#pragma unroll
      for (int e = 0; e < VEC; ++e) { rd[wave][cj + e][0] = sk[e]; rd[wave][cj + e][1] = sq[e]; }
    }
    __syncthreads();
    float u[VEC];
#pragma unroll
    for (int e = 0; e < VEC; ++e) {
      const float sk_all = ((rd[0][cj + e][0] + rd[1][cj + e][0]) + rd[2][cj + e][0]) + rd[3][cj + e][0];
      const float sq_all = ((rd[0][cj + e][1] + rd[1][cj + e][1]) + rd[2][cj + e][1]) + rd[3][cj + e][1];
      u[e] = beta * (v[e] - g * sk_all);
      if (rg == 0 && col + e < dv) out[(size_t)(r0 + t) * ldo + (size_t)h * dv + col + e] = fmaf(g, sq_all, qk * u[e]);
    }
#pragma unroll
    for (int ii = 0; ii < RPT; ++ii)
#pragma unroll
      for (int e = 0; e < VEC; ++e) s[ii][e] = fmaf(g, s[ii][e], kr[ii] * u[e]);
    // (the next row's sums go to the other half of `red`; the row after that writes this half only behind the next
    // row's barrier, which every thread reaches after it has read here)
  }
#pragma unroll
  for (int ii = 0; ii < RPT; ++ii) {
    const int i = rg + RG * ii;
    if (i >= dk || col >= dv) continue;
    float* at = S + (size_t)i * dv + col;
    if constexpr (VEC == 4) *reinterpret_cast<float4*>(at) = float4{s[ii][0], s[ii][1], s[ii][2], s[ii][3]};
    else *at = s[ii][0];
  }
}

// ---------------------------------------------------------------------------
// Gated linear recurrence, a segment's rows in order, a thread a channel c of `blocks` equal parts of w = C / blocks:
//   r = sigmoid(z_r + b_r), i = sigmoid(z_i + b_i);  log a = rate[c] r;  S <- exp(log a) S + sqrt(1 - a^2) i u
//   out = S * gelu(y + y_b) * out_scale
// z [T, ldz] float32 and zb [2C]: part b's r logits at b * 2w, its i logits w further on.  state [slot][C] float32.
// ---------------------------------------------------------------------------
__global__ __launch_bounds__(256) void gated_recurrence_kernel(
    const void* __restrict__ u, int u_dtype, int ldu, const float* __restrict__ z, int ldz, const float* __restrict__ zb,
    int w, const float* __restrict__ rate, const void* __restrict__ y, int y_dtype, int ldy,
    const float* __restrict__ yb, float out_scale, float* __restrict__ state, int C, const int* __restrict__ seg_row0,
    const int* __restrict__ seg_rows, const int* __restrict__ slots, void* __restrict__ out, int out_dtype, int ldo) {
  const int seg = blockIdx.x, c = blockIdx.y * 256 + threadIdx.x;
  if (c >= C) return;
  const int zr = c / w * 2 * w + c % w, zi = zr + w;
  const float br = zb[zr], bi = zb[zi], k = rate[c], by = yb ? yb[c] : 0.f;
  float* st = state + (size_t)slots[seg] * C + c;
  float S = *st;
  const int r0 = seg_row0[seg], n = seg_rows[seg];
  for (int t = 0; t < n; ++t) {
    const size_t row = r0 + t;
    const float log_a = k * sigmoid_f(z[row * ldz + zr] + br);
    const float in = sigmoid_f(z[row * ldz + zi] + bi) * load_f(u, u_dtype, row * ldu + c);
    S = fmaf(expf(log_a), S, sqrtf(-expm1f(2.0f * log_a)) * in);
    store_f(out, out_dtype, row * ldo + c, S * gelu_tanh_f(load_f(y, y_dtype, row * ldy + c) + by) * out_scale);
  }
  *st = S;
}

}  // namespace

APC_EXPORT int apc_delta_rule(const void* rows, int dtype, int ld, int q_off, int k_off, int v_off, int H, int G, int dk,
                              int dv, const void* ba, int ba_dtype, int ldba, int a_off, int b_off, const float* A,
                              const float* dt_bias, float q_scale, float* state, int n_segs, const int* seg_row0,
                              const int* seg_rows, const int* slots, float* out, int ldo, hipStream_t stream) {
  if (n_segs <= 0) return 0;
  if (H <= 0 || G <= 0 || H % G || dk <= 0 || dv <= 0 || !ba || !A || !dt_bias || !state || !slots || ldo < H * dv ||
      ld < q_off + G * dk || ld < k_off + G * dk || ld < v_off + H * dv || ldba < a_off + H || ldba < b_off + H)
    return APC_ERR_BAD_ARG;
  if (dk > 256 || H > 65535 || ceil_div(dv, 64) > 65535) return APC_ERR_UNSUPPORTED;
  const dim3 grid(n_segs, H, ceil_div(dv, 64));
#define DR_LAUNCH(VEC_, RPT_)                                                                                          \
  hipLaunchKernelGGL((delta_rule_kernel<VEC_, RPT_>), grid, dim3(256), 0, stream, rows, dtype, ld, q_off, k_off, v_off, \
                     H, G, dk, dv, ba, ba_dtype, ldba, a_off, b_off, A, dt_bias, q_scale, state, seg_row0, seg_rows,   \
                     slots, out, ldo)
  // (which kernel runs, and so the order of the additions, is fixed by the sizes alone)
  if (dv % 4 == 0 && !((uintptr_t)state & 15u)) {
    if (dk <= 32) DR_LAUNCH(4, 2);
    else if (dk <= 64) DR_LAUNCH(4, 4);
    else if (dk <= 128) DR_LAUNCH(4, 8);
    else DR_LAUNCH(4, 16);
  } else {
    if (dk <= 32) DR_LAUNCH(1, 8);
    else if (dk <= 64) DR_LAUNCH(1, 16);
    else if (dk <= 128) DR_LAUNCH(1, 32);
    else DR_LAUNCH(1, 64);
  }
#undef DR_LAUNCH
  APC_LAUNCH_CHECK();
  return 0;
}

APC_EXPORT int apc_gated_recurrence(const void* u, int u_dtype, int ldu, const float* z, int ldz, const float* zb,
                                    int blocks, const float* rate, const void* y, int y_dtype, int ldy, const float* yb,
                                    float out_scale, float* state, int C, int n_segs, const int* seg_row0,
                                    const int* seg_rows, const int* slots, void* out, int out_dtype, int ldo,
                                    hipStream_t stream) {
  if (n_segs <= 0) return 0;
  if (C <= 0 || blocks <= 0 || C % blocks || ldu < C || ldz < 2 * C || ldy < C || ldo < C || !zb || !rate || !state || !slots)
    return APC_ERR_BAD_ARG;
  if (ceil_div(C, 256) > 65535) return APC_ERR_UNSUPPORTED;
  hipLaunchKernelGGL(gated_recurrence_kernel, dim3(n_segs, ceil_div(C, 256)), dim3(256), 0, stream, u, u_dtype, ldu, z, ldz,
                     zb, C / blocks, rate, y, y_dtype, ldy, yb, out_scale, state, C, seg_row0, seg_rows, slots, out,
                     out_dtype, ldo);
  APC_LAUNCH_CHECK();
  return 0;
}
