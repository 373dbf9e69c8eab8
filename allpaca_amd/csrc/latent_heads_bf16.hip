// What an attention over cached latents does to the projected rows ahead of its products (`latent_rows_bf16_kernel`), and
// products with a matrix of its own for every head, bfloat16 on MFMA (the up-projections of an attention over cached
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

__device__ __forceinline__ void store4(float* dst, const floatx4& v, int left) {
  if (left >= 4) *reinterpret_cast<float4*>(dst) = float4{v[0], v[1], v[2], v[3]};
  else
    for (int r = 0; r < left; ++r) dst[r] = v[r];
}
// times sigmoid of the logits that lie at the outputs' own places
__device__ __forceinline__ void gate4(floatx4& v, const bf16_t* g, int left) {
  if (left >= 4) {
    const uint2 p = *reinterpret_cast<const uint2*>(g);
    const float z[4] = {__uint_as_float(p.x << 16), __uint_as_float(p.x & 0xffff0000u), __uint_as_float(p.y << 16),
                        __uint_as_float(p.y & 0xffff0000u)};
#pragma unroll
    for (int r = 0; r < 4; ++r) v[r] *= 1.0f / (1.0f + __expf(-z[r]));
  } else {
    for (int r = 0; r < left; ++r) v[r] *= 1.0f / (1.0f + __expf(-bf16_to_float(g[r])));
  }
}
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

template <typename Out>
__global__ __launch_bounds__(256) void heads_gemm_few_kernel(const bf16_t* __restrict__ A, int lda, int a_head,
                                                             const bf16_t* __restrict__ W, Out* __restrict__ C,
                                                             int ldc, int c_head, const bf16_t* __restrict__ gate,
                                                             int ldg, int M, int N, int K) {
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
  if (li >= M || n >= N) return;
  if (gate) gate4(acc, gate + (size_t)li * ldg + (size_t)h * c_head + n, N - n);
  store4(C + (size_t)li * ldc + (size_t)h * c_head + n, acc, N - n);
}

template <typename Out>
__global__ __launch_bounds__(256) void heads_gemm_kernel(const bf16_t* __restrict__ A, int lda, int a_head,
                                                         const bf16_t* __restrict__ W, Out* __restrict__ C, int ldc,
                                                         int c_head, const bf16_t* __restrict__ gate, int ldg, int M,
                                                         int N, int K) {
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
    Out* row = C + (size_t)m * ldc + (size_t)h * c_head;
#pragma unroll
    for (int b = 0; b < 4; ++b) {
      const int n = (band0 + b) * 16 + lc * 4;
      if (n >= N) continue;
      if (gate) gate4(acc[b][t], gate + (size_t)m * ldg + (size_t)h * c_head + n, N - n);
      store4(row + n, acc[b][t], N - n);
    }
  }
}

__device__ __forceinline__ void unpack8(const Frag& f, float (&v)[8]) {
#pragma unroll
  for (int k = 0; k < 4; ++k) {
    v[2 * k] = __uint_as_float(f.w[k] << 16);
    v[2 * k + 1] = __uint_as_float(f.w[k] & 0xffff0000u);
  }
}
__device__ __forceinline__ Frag pack8(const float (&v)[8]) {
  Frag f;
#pragma unroll
  for (int k = 0; k < 4; ++k) f.w[k] = pack_bf16x2(v[2 * k], v[2 * k + 1]);
  return f;
}
// 8 pairs (j, j + half) of a rotated part
__device__ __forceinline__ void rotate8(const bf16_t* src, bf16_t* dst, const float* cs, int j, int half) {
  float u[8], v[8], a[8], b[8];
  unpack8(load_frag(src + j), u);
  unpack8(load_frag(src + half + j), v);
#pragma unroll
  for (int e = 0; e < 8; e += 4) {
    const float4 c = *reinterpret_cast<const float4*>(cs + j + e), s = *reinterpret_cast<const float4*>(cs + half + j + e);
    const float cc[4] = {c.x, c.y, c.z, c.w}, ss[4] = {s.x, s.y, s.z, s.w};
#pragma unroll
    for (int k = 0; k < 4; ++k) {
      a[e + k] = u[e + k] * cc[k] - v[e + k] * ss[k];
      b[e + k] = v[e + k] * cc[k] + u[e + k] * ss[k];
    }
  }
  *reinterpret_cast<Frag*>(dst + j) = pack8(a);
  *reinterpret_cast<Frag*>(dst + half + j) = pack8(b);
}

// A block: one row.  The first wave norms the latent and rotates the shared key part into the row's place in its page
// (8 elements a lane); the other waves rotate the queries' parts, 8 pairs a lane.  Sizes and strides are multiples of 8,
// the rotated part of 16.  c_off < 0: queries only.  WAVE_ROW (steps of many rows): a wave does all of a row, a block
// four rows.
template <bool WAVE_ROW>
__global__ __launch_bounds__(256) void latent_rows_bf16_kernel(const bf16_t* __restrict__ proj, int ld, int H, int dn,
                                                               int dr, const bf16_t* __restrict__ kv, int ldkv, int c_off, int R, const float* __restrict__ norm_w,
                                                               float eps, const float* __restrict__ cos_sin,
                                                               const int* __restrict__ positions,
                                                               const int* __restrict__ row_seg,
                                                               const int* __restrict__ block_table, int max_blocks,
                                                               bf16_t* __restrict__ pages, int P, bf16_t* __restrict__ q,
                                                               int ldq, int n_rows) {
  const int r = WAVE_ROW ? blockIdx.x * 4 + threadIdx.x / WAVE : blockIdx.x;
  if (r >= n_rows) return;
  const int wave = WAVE_ROW ? 0 : threadIdx.x / WAVE, lane = threadIdx.x % WAVE, half = dr / 2, L = R + dr;
  const int pos = positions[r];
  const float* cs = cos_sin + (size_t)pos * dr;
  const bf16_t* row = proj + (size_t)r * ld;
  int first = WAVE_ROW ? lane : threadIdx.x, step = WAVE_ROW ? WAVE : 256;
  if (c_off >= 0) {
    if (wave == 0) {
      const bf16_t* src = kv + (size_t)r * ldkv + c_off;
      const int page = block_table[(size_t)row_seg[r] * max_blocks + pos / P];
      bf16_t* dst = pages + ((size_t)page * P + pos % P) * L;
      float ss = 0.f;
      for (int i = lane * 8; i < R; i += WAVE * 8) {
        float v[8];
        unpack8(load_frag(src + i), v);
#pragma unroll
        for (int e = 0; e < 8; ++e) ss = fmaf(v[e], v[e], ss);
      }
      const float inv = 1.0f / sqrtf(wave_sum(ss) / (float)R + eps);
      for (int i = lane * 8; i < R; i += WAVE * 8) {
        float v[8];
        unpack8(load_frag(src + i), v);
#pragma unroll
        for (int e = 0; e < 8; ++e) v[e] = v[e] * inv * norm_w[i + e];
        *reinterpret_cast<Frag*>(dst + i) = pack8(v);
      }
      if (lane * 8 < half) rotate8(src + R, dst + R, cs, lane * 8, half);
      if (!WAVE_ROW) return;
    }
    if (!WAVE_ROW) {
      first -= WAVE;
      step -= WAVE;
    }
  }
  const int per_head = half / 8;
  for (int i = first; i < H * per_head; i += step) {
    const int h = i / per_head, j = i % per_head * 8;
    rotate8(row + (size_t)h * (dn + dr) + dn, q + (size_t)r * ldq + (size_t)h * L + R, cs, j, half);
  }
}

}  // namespace

APC_EXPORT int apc_latent_rows_bf16_takes(int ld, int dn, int dr, int ldkv, int c_off, int R, int ldq) {
  return (ld % 8 == 0 && ldkv % 8 == 0 && dn % 8 == 0 && dr > 0 && dr % 16 == 0 && dr <= 1024 && R % 8 == 0 && ldq % 8 == 0 &&
          (c_off < 0 || c_off % 8 == 0)) ? 1 : 0;
}

APC_EXPORT int apc_latent_rows_bf16(const void* proj, int ld, int H, int dn, int dr, const void* kv, int ldkv, int c_off,
                                    int R,
                                    const float* norm_w, float eps, const float* cos_sin, const int* positions,
                                    const int* row_seg, const int* block_table, int max_blocks, void* pages, int P,
                                    void* q, int ldq, int n_rows, hipStream_t stream) {
  if (n_rows <= 0) return 0;
  if (!apc_latent_rows_bf16_takes(ld, dn, dr, ldkv, c_off, R, ldq)) return APC_ERR_UNSUPPORTED;
  if (H <= 0 || dn <= 0 || R <= 0 || P <= 0 || max_blocks <= 0 || ldq < H * (R + dr) || ld < H * (dn + dr) || !cos_sin ||
      (c_off >= 0 && (!kv || ldkv < c_off + R + dr || !norm_w || !pages)) || ((uintptr_t)kv & 15u) || ((uintptr_t)proj & 15u) || ((uintptr_t)q & 15u) ||
      ((uintptr_t)pages & 15u) || ((uintptr_t)cos_sin & 15u))
    return APC_ERR_BAD_ARG;
#define ROWS_LAUNCH(WAVE_ROW_, BLOCKS_)                                                                                 \
  hipLaunchKernelGGL((latent_rows_bf16_kernel<WAVE_ROW_>), dim3(BLOCKS_), dim3(256), 0, stream, (const bf16_t*)proj, ld, \
                     H, dn, dr, (const bf16_t*)kv, ldkv, c_off, R, norm_w, eps, cos_sin, positions, row_seg, block_table, max_blocks,            \
                     (bf16_t*)pages, P, (bf16_t*)q, ldq, n_rows)
  if (n_rows >= 1024) ROWS_LAUNCH(true, ceil_div(n_rows, 4));
  else ROWS_LAUNCH(false, n_rows);
#undef ROWS_LAUNCH
  APC_LAUNCH_CHECK();
  return 0;
}

// C bfloat16, or float32 with c_f32; gate (bfloat16 logits at the outputs' own places, may be null)
APC_EXPORT int apc_heads_gemm_bf16(const void* A, int lda, int a_head, const void* W, void* C, int ldc, int c_head,
                                   int c_f32, const void* gate, int ldg, int M, int H, int N, int K,
                                   hipStream_t stream) {
  if (M <= 0 || H <= 0 || N <= 0) return 0;
  if (K <= 0 || a_head < K || c_head < N || lda < (H - 1) * a_head + K || ldc < (H - 1) * c_head + N ||
      (gate && ldg < (H - 1) * c_head + N))
    return APC_ERR_BAD_ARG;
  if (K % 8 || a_head % 8 || lda % 8 || c_head % 4 || ldc % 4 || ((uintptr_t)A & 15u) || ((uintptr_t)W & 15u) ||
      ((uintptr_t)C & (c_f32 ? 15u : 7u)) || (gate && (ldg % 4 || ((uintptr_t)gate & 7u))) || H > 65535 || ceil_div(M, 128) > 65535)
    return APC_ERR_UNSUPPORTED;
  const int bands = ceil_div(N, 16);
#define HEADS_LAUNCH(Out_)                                                                                             \
  do {                                                                                                                 \
    if (M <= 16)                                                                                                       \
      hipLaunchKernelGGL(heads_gemm_few_kernel<Out_>, dim3(ceil_div(bands, 4), H), dim3(256), 0, stream,               \
                         (const bf16_t*)A, lda, a_head, (const bf16_t*)W, (Out_*)C, ldc, c_head, (const bf16_t*)gate,  \
                         ldg, M, N, K);                                                                                \
    else                                                                                                               \
      hipLaunchKernelGGL(heads_gemm_kernel<Out_>, dim3(ceil_div(bands, 8), ceil_div(M, 128), H), dim3(256), 0, stream, \
                         (const bf16_t*)A, lda, a_head, (const bf16_t*)W, (Out_*)C, ldc, c_head, (const bf16_t*)gate,  \
                         ldg, M, N, K);                                                                                \
  } while (0)
  if (c_f32) HEADS_LAUNCH(float);
  else HEADS_LAUNCH(bf16_t);
#undef HEADS_LAUNCH
  APC_LAUNCH_CHECK();
  return 0;
}
