// The gated linear recurrence (see plain_delta.hip for the formulas) over prompt portions, bfloat16 rows, chunks of 64
// rows side by side, each in 4 runs of 16.  S_t = a_t S_(t-1) + b_t is linear in S, so three launches replace the walk
// row by row:
//   summaries  every run for itself, from a state of zero: its end state E and the sum of its log a; a block's 4 runs
//              are put together to the chunk's
//   scan       per segment and channel: the state in front of every chunk, S0_(k+1) = exp(sum_k) S0_k + E_k, starting
//              from the request's state, which is left at the segment's end
//   outputs    every run again from the state in front of it (the chunk's, carried over the runs ahead of it):
//              S_t * gelu(y_t) * out_scale
// A thread has two neighbouring channels of a run and asks for 8 rows of them at a time; a wave is a run.  All arithmetic
// is float32 (exponentials through the hardware's base-2 instruction, 1 - a^2 without cancellation); u, y and the output
// are bfloat16 rows, the gates' logits float32 rows.
#include "mfma.h"
#include <math.h>

namespace {

constexpr int CHUNK = 64;         // rows of a chunk (the step's list of chunks is made for this)
constexpr int RUNS = 4;           // runs of a chunk: the waves of a block
constexpr int RUN = CHUNK / RUNS;
constexpr int RU = 8;             // rows asked for together

__device__ __forceinline__ float sigmoid_fast(float z) { return 1.0f / (1.0f + __expf(-z)); }
// sqrt(1 - exp(x)), x <= 0: near 0 by the series of exp(x) - 1, which loses nothing to cancellation
__device__ __forceinline__ float root_rest(float x) {
  const float series = -x * (1.0f + x * (0.5f + x * (0.16666667f + x * (0.041666667f + x * 0.0083333333f))));
  return sqrtf(x > -0.1f ? series : 1.0f - __expf(x));
}

template <int MODE>   // 1: summaries, 2: outputs
__global__ __launch_bounds__(256) void recurrence_chunk_kernel(
    const bf16_t* __restrict__ u, int ldu, const float* __restrict__ z, int ldz, const float* __restrict__ zb, int w,
    const float* __restrict__ rate, const bf16_t* __restrict__ y, int ldy, const float* __restrict__ yb, float out_scale,
    float* __restrict__ ws, float* __restrict__ logs, float* __restrict__ run_e, float* __restrict__ run_l, int C,
    const int* __restrict__ chunks, const int* __restrict__ seg_row0, const int* __restrict__ seg_rows,
    bf16_t* __restrict__ out, int ldo) {
  __shared__ float4 sums[RUNS][WAVE];
  const int lane = threadIdx.x % WAVE, run = threadIdx.x / WAVE;
  const int c_own = (blockIdx.x * WAVE + lane) * 2, chunk = blockIdx.y;
  const bool on = c_own < C;
  const int c = on ? c_own : 0;                  // (the threads beyond the channels read channel 0 and store nothing)
  const int seg = chunks[2 * chunk], in_seg = chunks[2 * chunk + 1] + run * RUN;
  const int r0 = seg_row0[seg] + in_seg, n = min(RUN, seg_rows[seg] - in_seg);      // (n <= 0: a run without rows)
  const int zr = c / w * 2 * w + c % w, zi = zr + w;
  const float2 br = *reinterpret_cast<const float2*>(zb + zr), bi = *reinterpret_cast<const float2*>(zb + zi);
  const float2 k = *reinterpret_cast<const float2*>(rate + c);
  const float2 by = MODE == 2 && yb ? *reinterpret_cast<const float2*>(yb + c) : float2{0.f, 0.f};
  float2 S = float2{0.f, 0.f};
  if (MODE == 2) {
    S = *reinterpret_cast<const float2*>(ws + (size_t)chunk * C + c);
    for (int x = 0; x < run; ++x) {
      const size_t at = ((size_t)chunk * RUNS + x) * C + c;
      const float2 e = *reinterpret_cast<const float2*>(run_e + at), l = *reinterpret_cast<const float2*>(run_l + at);
      S.x = fmaf(__expf(l.x), S.x, e.x);
      S.y = fmaf(__expf(l.y), S.y, e.y);
    }
  }
  float2 total = float2{0.f, 0.f};
  for (int t0 = 0; t0 < n; t0 += RU) {
    float2 vr[RU], vi[RU];
    uint32_t vu[RU], vy[RU];
#pragma unroll
    for (int x = 0; x < RU; ++x) {
      const size_t row = r0 + min(t0 + x, n - 1);
      vr[x] = *reinterpret_cast<const float2*>(z + row * ldz + zr);
      vi[x] = *reinterpret_cast<const float2*>(z + row * ldz + zi);
      vu[x] = *reinterpret_cast<const uint32_t*>(u + row * ldu + c);
      if (MODE == 2) vy[x] = *reinterpret_cast<const uint32_t*>(y + row * ldy + c);
    }
#pragma unroll
    for (int x = 0; x < RU; ++x) {
      if (t0 + x >= n) break;
      const float l0 = k.x * sigmoid_fast(vr[x].x + br.x), l1 = k.y * sigmoid_fast(vr[x].y + br.y);
      const float i0 = sigmoid_fast(vi[x].x + bi.x) * __uint_as_float(vu[x] << 16);
      const float i1 = sigmoid_fast(vi[x].y + bi.y) * __uint_as_float(vu[x] & 0xffff0000u);
      S.x = fmaf(__expf(l0), S.x, root_rest(2.0f * l0) * i0);
      S.y = fmaf(__expf(l1), S.y, root_rest(2.0f * l1) * i1);
      total.x += l0;
      total.y += l1;
      if (MODE == 2) {
        const float g0 = activation_f(__uint_as_float(vy[x] << 16) + by.x, 3);
        const float g1 = activation_f(__uint_as_float(vy[x] & 0xffff0000u) + by.y, 3);
        if (on)
          *reinterpret_cast<uint32_t*>(out + (size_t)(r0 + t0 + x) * ldo + c) =
              pack_bf16x2(S.x * g0 * out_scale, S.y * g1 * out_scale);
      }
    }
  }
  if (MODE == 1) {
    sums[run][lane] = float4{S.x, S.y, total.x, total.y};
    __syncthreads();
    if (!on) return;
    const size_t at = ((size_t)chunk * RUNS + run) * C + c;
    *reinterpret_cast<float2*>(run_e + at) = S;
    *reinterpret_cast<float2*>(run_l + at) = total;
    if (run == 0) {
      float4 all = sums[0][lane];
#pragma unroll
      for (int x = 1; x < RUNS; ++x) {
        const float4 v = sums[x][lane];
        all = float4{fmaf(__expf(v.z), all.x, v.x), fmaf(__expf(v.w), all.y, v.y), all.z + v.z, all.w + v.w};
      }
      *reinterpret_cast<float2*>(ws + (size_t)chunk * C + c) = float2{all.x, all.y};
      *reinterpret_cast<float2*>(logs + (size_t)chunk * C + c) = float2{all.z, all.w};
    }
  }
}

// ws [chunks][C]: a chunk's end state in, the state in front of it out
__global__ __launch_bounds__(256) void recurrence_states_kernel(float* __restrict__ ws, const float* __restrict__ logs,
                                                                float* __restrict__ state,
                                                                const int* __restrict__ seg_chunks,
                                                                const int* __restrict__ slots, int C) {
  const int seg = blockIdx.y, c = blockIdx.x * 256 + threadIdx.x;
  if (c >= C) return;
  const int k0 = seg_chunks[2 * seg], nk = seg_chunks[2 * seg + 1];
  float* st = state + (size_t)slots[seg] * C + c;
  float s = *st;
  for (int x0 = 0; x0 < nk; x0 += RU) {
    float e[RU], l[RU];
#pragma unroll
    for (int x = 0; x < RU; ++x) {
      const size_t at = (size_t)(k0 + min(x0 + x, nk - 1)) * C + c;
      e[x] = ws[at];
      l[x] = logs[at];
    }
#pragma unroll
    for (int x = 0; x < RU; ++x) {
      if (x0 + x >= nk) break;
      ws[(size_t)(k0 + x0 + x) * C + c] = s;
      s = fmaf(__expf(l[x]), s, e[x]);
    }
  }
  *st = s;
}

}  // namespace

// 1 if the kernels take these sizes, else 0 (the caller then runs the kernel that walks row by row)
APC_EXPORT int apc_gated_recurrence_bf16_takes(int C, int blocks, int ldu, int ldz, int ldy, int ldo) {
  return (C > 0 && blocks > 0 && C % blocks == 0 && (C / blocks) % 2 == 0 && ldu % 2 == 0 && ldz % 2 == 0 && ldy % 2 == 0 &&
          ldo % 2 == 0) ? 1 : 0;
}

// chunks, seg_chunks: as in apc_delta_rule_bf16; work: float32 [10][n_chunks][C]
APC_EXPORT int apc_gated_recurrence_bf16(const void* u, int ldu, const float* z, int ldz, const float* zb, int blocks,
                                         const float* rate, const void* y, int ldy, const float* yb, float out_scale,
                                         float* state, int C, int n_segs, const int* seg_row0, const int* seg_rows,
                                         const int* slots, int n_chunks, const int* chunks, const int* seg_chunks,
                                         float* work, void* out, int ldo, hipStream_t stream) {
  if (n_segs <= 0 || n_chunks <= 0) return 0;
  if (!apc_gated_recurrence_bf16_takes(C, blocks, ldu, ldz, ldy, ldo)) return APC_ERR_UNSUPPORTED;
  if (!u || !z || !zb || !rate || !y || !state || !slots || !chunks || !seg_chunks || !work || !out || ldu < C ||
      ldz < 2 * C || ldy < C || ldo < C || ((uintptr_t)u & 3u) || ((uintptr_t)y & 3u) || ((uintptr_t)out & 3u) ||
      ((uintptr_t)z & 7u) || ((uintptr_t)work & 7u))
    return APC_ERR_BAD_ARG;
  if (n_chunks > 65535 || n_segs > 65535) return APC_ERR_UNSUPPORTED;
  const dim3 grid(ceil_div(C / 2, WAVE), n_chunks);
  const size_t part = (size_t)n_chunks * C;
  float *ws = work, *logs = work + part, *run_e = work + 2 * part, *run_l = run_e + RUNS * part;
#define REC_LAUNCH(MODE_)                                                                                              \
  hipLaunchKernelGGL(recurrence_chunk_kernel<MODE_>, grid, dim3(256), 0, stream, (const bf16_t*)u, ldu, z, ldz, zb,     \
                     C / blocks, rate, (const bf16_t*)y, ldy, yb, out_scale, ws, logs, run_e, run_l, C, chunks,        \
                     seg_row0, seg_rows, (bf16_t*)out, ldo);                                                                               \
  APC_LAUNCH_CHECK()
  REC_LAUNCH(1);
  hipLaunchKernelGGL(recurrence_states_kernel, dim3(ceil_div(C, 256), n_segs), dim3(256), 0, stream, ws, logs, state,
                     seg_chunks, slots, C);
  APC_LAUNCH_CHECK();
  REC_LAUNCH(2);
#undef REC_LAUNCH
  return 0;
}
