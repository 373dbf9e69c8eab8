// Products with a matrix of its own for every head, bfloat16 on MFMA (the up-projections of an attention over cached
// latents, applied to its queries and to its outputs):
//   C[m][h * c_head + n] = sum_k A[m][h * a_head + k] W[h][n][k]
// W: every head's matrix in tiles of 16 rows x 32 columns in the lane order of the MFMA operand (see gemm_bf16.hip).
// Weights are the first operand, so a lane holds four consecutive outputs of one row.  A wave reads both operands
// straight from memory: the matrices of all heads are a few megabytes that the caches hold, and an operand of 16 rows x
// 32 columns is one 16-byte piece a lane either way.
//   few rows (up to 16)  a wave a band of 16 outputs; a block 4 bands of a head
//   more                 a wave 64 rows x 64 outputs; a block 2 x 2 waves
#include "mfma.h"

namespace {

constexpr int TILE = 512;

__device__ __forceinline__ void store4(bf16_t* dst, const floatx4& v, int left) {
  if (left >= 4) {
    uint2 pk;
    pk.x = pack_bf16x2(v[0], v[1]);
    pk.y = pack_bf16x2(v[2], v[3]);
    *reinterpret_cast<uint2*>(dst) = pk;
  } else {
    for (int r = 0; r < left; ++r) dst[r] = float_to_bf16(v[r]);
  }
}

__global__ __launch_bounds__(256) void heads_gemm_few_kernel(const bf16_t* __restrict__ A, int lda, int a_head,
                                                             const bf16_t* __restrict__ W, bf16_t* __restrict__ C,
                                                             int ldc, int c_head, int M, int N, int K) {
  const int lane = threadIdx.x % WAVE, wave = threadIdx.x / WAVE, li = lane % 16, lc = lane / 16;
  const int h = blockIdx.y, bands = (N + 15) / 16, chunks = (K + 31) / 32;
  const int band = blockIdx.x * 4 + wave;
  if (band >= bands) return;
  const bf16_t* w = W + ((size_t)h * bands + band) * chunks * TILE + lane * 8;
  const bf16_t* a = A + (size_t)min(li, M - 1) * lda + (size_t)h * a_head + lc * 8;
  floatx4 acc = floatx4{0.f, 0.f, 0.f, 0.f};
  constexpr int U = 8;
  for (int c0 = 0; c0 < chunks; c0 += U) {
    Frag fw[U], fa[U];
#pragma unroll
    for (int x = 0; x < U; ++x) {
      const int c = min(c0 + x, chunks - 1);
      fw[x] = load_frag(w + (size_t)c * TILE);
      fa[x] = (c0 + x < chunks && c * 32 + lc * 8 < K) ? load_frag(a + c * 32) : zero_frag();
    }
#pragma unroll
    for (int x = 0; x < U; ++x) acc = mfma16(fw[x], fa[x], acc);
  }
  const int n = band * 16 + lc * 4;
  if (li < M && n < N) store4(C + (size_t)li * ldc + (size_t)h * c_head + n, acc, N - n);
}

__global__ __launch_bounds__(256) void heads_gemm_kernel(const bf16_t* __restrict__ A, int lda, int a_head,
                                                         const bf16_t* __restrict__ W, bf16_t* __restrict__ C, int ldc,
                                                         int c_head, int M, int N, int K) {
  const int lane = threadIdx.x % WAVE, wave = threadIdx.x / WAVE, li = lane % 16, lc = lane / 16;
  const int h = blockIdx.z, bands = (N + 15) / 16, chunks = (K + 31) / 32;
  const int m0 = blockIdx.y * 128 + (wave / 2) * 64, band0 = (blockIdx.x * 2 + wave % 2) * 4;
  if (m0 >= M || band0 >= bands) return;
  const bf16_t *w[4], *a[4];
#pragma unroll
  for (int b = 0; b < 4; ++b) w[b] = W + ((size_t)h * bands + min(band0 + b, bands - 1)) * chunks * TILE + lane * 8;
#pragma unroll
  for (int t = 0; t < 4; ++t) a[t] = A + (size_t)min(m0 + t * 16 + li, M - 1) * lda + (size_t)h * a_head + lc * 8;
  floatx4 acc[4][4];
#pragma unroll
  for (int b = 0; b < 4; ++b)
#pragma unroll
    for (int t = 0; t < 4; ++t) acc[b][t] = floatx4{0.f, 0.f, 0.f, 0.f};
  Frag fw[2][4], fa[2][4];
  auto load = [&](int s, int c) {
#pragma unroll
    for (int b = 0; b < 4; ++b) fw[s][b] = load_frag(w[b] + (size_t)c * TILE);
    const bool in = c * 32 + lc * 8 < K;
#pragma unroll
    for (int t = 0; t < 4; ++t) fa[s][t] = in ? load_frag(a[t] + c * 32) : zero_frag();
  };
  auto mul = [&](int s) {
#pragma unroll
    for (int b = 0; b < 4; ++b)
#pragma unroll
      for (int t = 0; t < 4; ++t) acc[b][t] = mfma16(fw[s][b], fa[s][t], acc[b][t]);
  };
  load(0, 0);
  int c = 0;
  for (; c + 2 <= chunks; c += 2) {
    load(1, c + 1);
    mul(0);
    load(0, min(c + 2, chunks - 1));
    mul(1);
  }
  if (c < chunks) mul(0);
#pragma unroll
  for (int t = 0; t < 4; ++t) {
    const int m = m0 + t * 16 + li;
    if (m >= M) continue;
    bf16_t* row = C + (size_t)m * ldc + (size_t)h * c_head;
#pragma unroll
    for (int b = 0; b < 4; ++b) {
      const int n = (band0 + b) * 16 + lc * 4;
      if (n < N) store4(row + n, acc[b][t], N - n);
    }
  }
}

}  // namespace

APC_EXPORT int apc_heads_gemm_bf16(const void* A, int lda, int a_head, const void* W, void* C, int ldc, int c_head, int M,
                                   int H, int N, int K, hipStream_t stream) {
  if (M <= 0 || H <= 0 || N <= 0) return 0;
  if (K <= 0 || a_head < K || c_head < N || lda < (H - 1) * a_head + K || ldc < (H - 1) * c_head + N) return APC_ERR_BAD_ARG;
  if (K % 8 || a_head % 8 || lda % 8 || c_head % 4 || ldc % 4 || ((uintptr_t)A & 15u) || ((uintptr_t)W & 15u) ||
      ((uintptr_t)C & 7u) || H > 65535 || ceil_div(M, 128) > 65535)
    return APC_ERR_UNSUPPORTED;
  const int bands = ceil_div(N, 16);
  if (M <= 16)
    hipLaunchKernelGGL(heads_gemm_few_kernel, dim3(ceil_div(bands, 4), H), dim3(256), 0, stream, (const bf16_t*)A, lda,
                       a_head, (const bf16_t*)W, (bf16_t*)C, ldc, c_head, M, N, K);
  else
    hipLaunchKernelGGL(heads_gemm_kernel, dim3(ceil_div(bands, 8), ceil_div(M, 128), H), dim3(256), 0, stream,
                       (const bf16_t*)A, lda, a_head, (const bf16_t*)W, (bf16_t*)C, ldc, c_head, M, N, K);
  APC_LAUNCH_CHECK();
  return 0;
}
