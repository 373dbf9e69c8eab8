// Plain matrix product  C[M,N] = A[M,K] . W[N,K]^T  in true 32-bit arithmetic.
//
// Every output element is one chain  acc = fma(a[k], w[k], acc)  over k = 0..K-1
// in order, whatever M, N or the tile a row falls into: a row of a batch equals
// that row computed alone bit for bit (the property the reference asks of its
// host product, crates/allpaca-cpu/src/kernels.rs:2506-2525, and enforces on the
// GPU with `ExactRows`, crates/allpaca-core/src/model.rs:10851-10863).
// Operands may be float32 or bfloat16 (widened exactly); no matrix-core mode.
// Reference for the product itself: matmul_nt, crates/allpaca-cpu/src/kernels.rs:97-128.
#include "common.h"

constexpr int TM = 64, TN = 64, TK = 16;

// mode 0: C = acc (C of c_dtype)   mode 1: C += acc (C float32)
// blockIdx.z: one of several products of the same sizes, whose operands lie these many elements apart.
// With `gate` (rows of ldg, read at the output's own place): C = acc * sigmoid(gate).
struct HeadStrides {
  size_t a = 0, w = 0, c = 0;
  const void* gate = nullptr;
  int gate_dtype = APC_F32, ldg = 0;
};
__global__ __launch_bounds__(256) void gemm_plain_kernel(const void* __restrict__ A, int a_dtype, int lda,
                                                         const void* __restrict__ W, int w_dtype, int ldw,
                                                         void* __restrict__ C, int c_dtype, int ldc, int M, int N,
                                                         int K, int mode, HeadStrides hs) {
  __shared__ float As[TK][TM + 4];
  __shared__ float Ws[TK][TN + 4];
  const int tid = threadIdx.x;
  const int tx = tid % 16, ty = tid / 16;
  const int m0 = blockIdx.y * TM, n0 = blockIdx.x * TN;
  float acc[4][4];
#pragma unroll
  for (int i = 0; i < 4; ++i)
#pragma unroll
    for (int j = 0; j < 4; ++j) acc[i][j] = 0.f;

  for (int k0 = 0; k0 < K; k0 += TK) {
    // 64 rows x 16 k = 1024 elements per operand, 4 per thread; consecutive threads read consecutive k
#pragma unroll
    for (int e = 0; e < 4; ++e) {
      const int idx = tid + e * 256;
      const int r = idx / TK, kk = idx % TK;
      const int k = k0 + kk;
      float a = 0.f, w = 0.f;
      if (k < K) {
        if (m0 + r < M) a = load_f(A, a_dtype, blockIdx.z * hs.a + (size_t)(m0 + r) * lda + k);
        if (n0 + r < N) w = load_f(W, w_dtype, blockIdx.z * hs.w + (size_t)(n0 + r) * ldw + k);
      }
      As[kk][r] = a;
      Ws[kk][r] = w;
    }
    __syncthreads();
#pragma unroll
    for (int kk = 0; kk < TK; ++kk) {
      float a[4], w[4];
#pragma unroll
      for (int i = 0; i < 4; ++i) a[i] = As[kk][ty * 4 + i];
#pragma unroll
      for (int j = 0; j < 4; ++j) w[j] = Ws[kk][tx * 4 + j];
#pragma unroll
      for (int i = 0; i < 4; ++i)
#pragma unroll
        for (int j = 0; j < 4; ++j) acc[i][j] = fmaf(a[i], w[j], acc[i][j]);
    }
    __syncthreads();
  }
#pragma unroll
  for (int i = 0; i < 4; ++i) {
    const int m = m0 + ty * 4 + i;
    if (m >= M) continue;
#pragma unroll
    for (int j = 0; j < 4; ++j) {
      const int n = n0 + tx * 4 + j;
      if (n >= N) continue;
      const size_t o = blockIdx.z * hs.c + (size_t)m * ldc + n;
      if (hs.gate) {
        const float z = load_f(hs.gate, hs.gate_dtype, blockIdx.z * hs.c + (size_t)m * hs.ldg + n);
        acc[i][j] *= 1.0f / (1.0f + expf(-z));
      }
      if (mode == 1) ((float*)C)[o] += acc[i][j];
      else store_f(C, c_dtype, o, acc[i][j]);
    }
  }
}

APC_EXPORT int apc_gemm_plain(const void* A, int a_dtype, int lda, const void* W, int w_dtype, int ldw, void* C,
                              int c_dtype, int ldc, int M, int N, int K, int mode, hipStream_t stream) {
  if (M <= 0 || N <= 0) return 0;
  if (K <= 0 || lda < K || ldw < K || ldc < N) return APC_ERR_BAD_ARG;
  if (mode == 1 && c_dtype != APC_F32) return APC_ERR_BAD_ARG;
  const int gy = ceil_div(M, TM);
  if (gy > 65535) return APC_ERR_BAD_ARG;
  hipLaunchKernelGGL(gemm_plain_kernel, dim3(ceil_div(N, TN), gy), dim3(256), 0, stream, A, a_dtype, lda, W, w_dtype,
                     ldw, C, c_dtype, ldc, M, N, K, mode, HeadStrides{});
  APC_LAUNCH_CHECK();
  return 0;
}

// A matrix of its own for every head: C[m][h * c_head + n] = A[m][h * a_head ..] . W[h][n], W [H][N][K] contiguous;
// times sigmoid(gate[m][h * c_head + n]) with a gate.
APC_EXPORT int apc_heads_gemm_plain(const void* A, int a_dtype, int lda, int a_head, const void* W, int w_dtype, void* C,
                                    int c_dtype, int ldc, int c_head, const void* gate, int gate_dtype, int ldg, int M, int H,
                                    int N, int K, hipStream_t stream) {
  if (M <= 0 || H <= 0 || N <= 0) return 0;
  if (K <= 0 || a_head < K || c_head < N || lda < (H - 1) * a_head + K || ldc < (H - 1) * c_head + N ||
      (gate && ldg < (H - 1) * c_head + N))
    return APC_ERR_BAD_ARG;
  const int gy = ceil_div(M, TM);
  if (gy > 65535 || H > 65535) return APC_ERR_BAD_ARG;
  hipLaunchKernelGGL(gemm_plain_kernel, dim3(ceil_div(N, TN), gy, H), dim3(256), 0, stream, A, a_dtype, lda, W, w_dtype, K,
                     C, c_dtype, ldc, M, N, K, 0, HeadStrides{(size_t)a_head, (size_t)N * K, (size_t)c_head, gate, gate_dtype, ldg});
  APC_LAUNCH_CHECK();
  return 0;
}
