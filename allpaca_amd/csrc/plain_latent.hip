// Plain kernels of an attention over cached latents (see parts/latent_attention.py) and of the element-wise tanh norm.
// All arithmetic in 32-bit float with an order of additions that the row's own place fixes (never the batch), any
// element type in and out.
//
//   rows        c = rms_norm(c') * w and the rotated key part kr into the row's slot of its page; the rotated part of
//               every query head to the end of the head's query in latent space
//   heads       out[:, h] = a[:, h] . W_h^T with a matrix of its own for every head
//   attention   every head's query [R + dr] against the rows [c | kr] of the positions up to the row's own; the values
//               are the rows' first R elements
// Pages: [slot][R + dr].
#include "common.h"
#include <math.h>

namespace {

__global__ __launch_bounds__(256) void latent_rows_kernel(const void* __restrict__ proj, int dtype, int ld, int H, int dn,
                                                          int dr, const void* __restrict__ kv, int ldkv, int c_off, int R, const float* __restrict__ norm_w,
                                                          float eps, const float* __restrict__ cos_sin,
                                                          const int* __restrict__ positions,
                                                          const int* __restrict__ row_seg,
                                                          const int* __restrict__ block_table, int max_blocks,
                                                          void* __restrict__ pages, int page_dtype, int P,
                                                          void* __restrict__ q, int q_dtype, int ldq) {
  __shared__ float red[256 / WAVE];
  const int r = blockIdx.x, tid = threadIdx.x, half = dr / 2;
  const int pos = positions[r];
  const float* cs = cos_sin + (size_t)pos * dr;
  const size_t base = (size_t)r * ld, kv_base = (size_t)r * ldkv + c_off;
  for (int i = tid; i < H * half; i += 256) {
    const int h = i / half, j = i % half;
    const size_t src = base + (size_t)h * (dn + dr) + dn + j, dst = (size_t)r * ldq + (size_t)h * (R + dr) + R + j;
    const float u = load_f(proj, dtype, src), v = load_f(proj, dtype, src + half), c = cs[j], s = cs[half + j];
    store_f(q, q_dtype, dst, u * c - v * s);
    store_f(q, q_dtype, dst + half, v * c + u * s);
  }
  if (!norm_w) return;
  float ss = 0.f;
  for (int i = tid; i < R; i += 256) {
    const float v = load_f(kv, dtype, kv_base + i);
    ss = fmaf(v, v, ss);
  }
  ss = block_sum<256>(ss, red);
  const float inv = 1.0f / sqrtf(ss / (float)R + eps);
  const int page = block_table[(size_t)row_seg[r] * max_blocks + pos / P];
  const size_t out = ((size_t)page * P + pos % P) * (R + dr);
  for (int i = tid; i < R; i += 256)
    store_f(pages, page_dtype, out + i, load_f(kv, dtype, kv_base + i) * inv * norm_w[i]);
  for (int j = tid; j < half; j += 256) {
    const float u = load_f(kv, dtype, kv_base + R + j), v = load_f(kv, dtype, kv_base + R + half + j);
    const float c = cs[j], s = cs[half + j];
    store_f(pages, page_dtype, out + R + j, u * c - v * s);
    store_f(pages, page_dtype, out + R + half + j, v * c + u * s);
  }
}

// A block: one row and one head.  Keys in tiles of 256 from position 0 on: a score a thread, the tile's maximum and sum
// over the block, then a value element (or several) a thread over the tile's keys in order.
constexpr int LK = 256;
constexpr int L_PER = 8;      // value elements a thread keeps: R up to 2,048

__global__ __launch_bounds__(256) void latent_attention_plain_kernel(
    const void* __restrict__ q, int q_dtype, int ldq, void* __restrict__ out, int out_dtype, int ldo, int H, int R, int dr,
    const void* __restrict__ pages, int page_dtype, int P, const int* __restrict__ block_table, int max_blocks,
    const int* __restrict__ positions, const int* __restrict__ row_seg, float scale) {
  extern __shared__ float qs[];          // [R + dr]
  __shared__ float ps[LK];
  __shared__ float red[256 / WAVE];
  const int r = blockIdx.x, h = blockIdx.y, tid = threadIdx.x, L = R + dr;
  const int pos = positions[r];
  const int* bt = block_table + (size_t)row_seg[r] * max_blocks;
  for (int i = tid; i < L; i += 256) qs[i] = load_f(q, q_dtype, (size_t)r * ldq + (size_t)h * L + i);
  __syncthreads();
  float acc[L_PER];
#pragma unroll
  for (int e = 0; e < L_PER; ++e) acc[e] = 0.f;
  float m = -INFINITY, l = 0.f;
  for (int k0 = 0; k0 <= pos; k0 += LK) {
    const int t = k0 + tid;
    float s = -INFINITY;
    if (t <= pos) {
      const size_t row = ((size_t)bt[t / P] * P + t % P) * L;
      float d = 0.f;
      for (int i = 0; i < L; ++i) d = fmaf(qs[i], load_f(pages, page_dtype, row + i), d);
      s = d * scale;
    }
    const float m_new = fmaxf(m, block_max<256>(s, red));
    const float p = t <= pos ? expf(s - m_new) : 0.f;
    const float f = expf(m - m_new);
    __syncthreads();
    ps[tid] = p;
    l = l * f + block_sum<256>(p, red);
    m = m_new;
    __syncthreads();
    const int n = min(LK, pos + 1 - k0);
#pragma unroll
    for (int e = 0; e < L_PER; ++e) {
      const int i = tid + e * 256;
      if (i >= R) break;
      float a = acc[e] * f;
      for (int k = 0; k < n; ++k) {
        const int tk = k0 + k;
        a = fmaf(ps[k], load_f(pages, page_dtype, ((size_t)bt[tk / P] * P + tk % P) * L + i), a);
      }
      acc[e] = a;
    }
    __syncthreads();
  }
#pragma unroll
  for (int e = 0; e < L_PER; ++e) {
    const int i = tid + e * 256;
    if (i < R) store_f(out, out_dtype, (size_t)r * ldo + (size_t)h * R + i, acc[e] / l);
  }
}

// ---------------------------------------------------------------------------
// tanh(alpha x) w + b.  With y: x += tanh(pa y) pw + pb first (x float32, in place), then, with h: h = tanh(alpha x) w + b.
// Without y: h[r] from x[rows[r]].  EXACT: the library's tanh; else 1 - 2 e / (1 + e) with e = exp(-2 |v|), off by about
// 1e-7 of 1.
// ---------------------------------------------------------------------------
template <bool EXACT>
__device__ __forceinline__ float squash(float v) {
  if (EXACT) return tanhf(v);
  const float e = __expf(-2.0f * fabsf(v));
  return copysignf(__fdividef(1.0f - e, 1.0f + e), v);
}

struct TanhNorm {
  float alpha;
  const float* w;
  const float* b;
};

template <bool EXACT>
__global__ __launch_bounds__(256) void tanh_norm_kernel(const void* __restrict__ x, int x_dtype, int ldx,
                                                        const int* __restrict__ rows, TanhNorm n, void* __restrict__ h,
                                                        int h_dtype, int ldh, int dim) {
  const int r = blockIdx.x, i = blockIdx.y * 256 + threadIdx.x;
  if (i >= dim) return;
  const size_t src = rows ? rows[r] : r;
  store_f(h, h_dtype, (size_t)r * ldh + i, fmaf(squash<EXACT>(n.alpha * load_f(x, x_dtype, src * ldx + i)), n.w[i], n.b[i]));
}

template <bool EXACT>
__global__ __launch_bounds__(256) void tanh_norm_add_kernel(float* __restrict__ x, int ldx, const void* __restrict__ y,
                                                            int y_dtype, int ldy, TanhNorm post, TanhNorm n,
                                                            void* __restrict__ h, int h_dtype, int ldh, int dim) {
  const int r = blockIdx.x, i = blockIdx.y * 256 + threadIdx.x;
  if (i >= dim) return;
  const float v = x[(size_t)r * ldx + i] +
                  fmaf(squash<EXACT>(post.alpha * load_f(y, y_dtype, (size_t)r * ldy + i)), post.w[i], post.b[i]);
  x[(size_t)r * ldx + i] = v;
  if (h) store_f(h, h_dtype, (size_t)r * ldh + i, fmaf(squash<EXACT>(n.alpha * v), n.w[i], n.b[i]));
}

// The same for float32 x and y, 4 elements of ROWS rows a thread on 16-byte accesses: weights and biases are read once for
// the rows, and all loads of x and y go out ahead of the first store.
template <bool EXACT, int ROWS>
__global__ __launch_bounds__(256) void tanh_norm_add_f4_kernel(float* __restrict__ x, int ldx, const float* __restrict__ y,
                                                               int ldy, TanhNorm post, TanhNorm n, void* __restrict__ h,
                                                               int h_dtype, int ldh, int n_rows, int dim) {
  const int r0 = blockIdx.x * ROWS, i = (blockIdx.y * 256 + threadIdx.x) * 4;
  if (i >= dim) return;
  const int rows = min(ROWS, n_rows - r0);
  float4 xv[ROWS], yv[ROWS];
#pragma unroll
  for (int k = 0; k < ROWS; ++k) {
    const size_t r = r0 + min(k, rows - 1);
    xv[k] = *reinterpret_cast<const float4*>(x + r * ldx + i);
    yv[k] = *reinterpret_cast<const float4*>(y + r * ldy + i);
  }
  const float4 pw = *reinterpret_cast<const float4*>(post.w + i), pb = *reinterpret_cast<const float4*>(post.b + i);
  float4 w = float4{0.f, 0.f, 0.f, 0.f}, b = w;
  if (h) {
    w = *reinterpret_cast<const float4*>(n.w + i);
    b = *reinterpret_cast<const float4*>(n.b + i);
  }
#pragma unroll
  for (int k = 0; k < ROWS; ++k) {
    if (k >= rows) return;
    float4 v;
    v.x = xv[k].x + fmaf(squash<EXACT>(post.alpha * yv[k].x), pw.x, pb.x);
    v.y = xv[k].y + fmaf(squash<EXACT>(post.alpha * yv[k].y), pw.y, pb.y);
    v.z = xv[k].z + fmaf(squash<EXACT>(post.alpha * yv[k].z), pw.z, pb.z);
    v.w = xv[k].w + fmaf(squash<EXACT>(post.alpha * yv[k].w), pw.w, pb.w);
    *reinterpret_cast<float4*>(x + (size_t)(r0 + k) * ldx + i) = v;
    if (!h) continue;
    float4 o;
    o.x = fmaf(squash<EXACT>(n.alpha * v.x), w.x, b.x);
    o.y = fmaf(squash<EXACT>(n.alpha * v.y), w.y, b.y);
    o.z = fmaf(squash<EXACT>(n.alpha * v.z), w.z, b.z);
    o.w = fmaf(squash<EXACT>(n.alpha * v.w), w.w, b.w);
    const size_t at = (size_t)(r0 + k) * ldh + i;
    if (h_dtype == APC_F32) {
      *reinterpret_cast<float4*>((float*)h + at) = o;
    } else {
      uint2 pk;
      pk.x = pack_bf16x2(o.x, o.y);
      pk.y = pack_bf16x2(o.z, o.w);
      *reinterpret_cast<uint2*>((bf16_t*)h + at) = pk;
    }
  }
}

}  // namespace

// kv [rows][ldkv]: the rows of the latents (which may be those of the queries), read from column c_off on; c_off < 0:
// queries only (nothing goes into the pages)
APC_EXPORT int apc_latent_rows(const void* proj, int dtype, int ld, int H, int dn, int dr, const void* kv,
                               int ldkv, int c_off, int R, const float* norm_w, float eps, const float* cos_sin, const int* positions,
                               const int* row_seg, const int* block_table, int max_blocks, void* pages, int page_dtype,
                               int P, void* q, int q_dtype, int ldq, int n_rows, hipStream_t stream) {
  if (n_rows <= 0) return 0;
  if (H <= 0 || dn <= 0 || dr < 0 || dr % 2 || R <= 0 || P <= 0 || max_blocks <= 0 || ldq < H * (R + dr) ||
      ld < H * (dn + dr) || (c_off >= 0 && (!kv || ldkv < c_off + R + dr || !norm_w || !pages)) || (dr && !cos_sin))
    return APC_ERR_BAD_ARG;
  hipLaunchKernelGGL(latent_rows_kernel, dim3(n_rows), dim3(256), 0, stream, proj, dtype, ld, H, dn, dr, kv, ldkv, c_off, R,
                     c_off >= 0 ? norm_w : nullptr, eps, cos_sin, positions, row_seg, block_table, max_blocks, pages,
                     page_dtype, P, q, q_dtype, ldq);
  APC_LAUNCH_CHECK();
  return 0;
}

APC_EXPORT int apc_latent_attention_plain(const void* q, int q_dtype, int ldq, void* out, int out_dtype, int ldo,
                                          int n_rows, int H, int R, int dr, const void* pages, int page_dtype, int P,
                                          const int* block_table, int max_blocks, const int* positions,
                                          const int* row_seg, float scale, hipStream_t stream) {
  if (n_rows <= 0) return 0;
  if (H <= 0 || R <= 0 || dr < 0 || P <= 0 || max_blocks <= 0 || ldq < H * (R + dr) || ldo < H * R) return APC_ERR_BAD_ARG;
  if (R > L_PER * 256 || H > 65535 || (size_t)(R + dr) * sizeof(float) > 48 * 1024) return APC_ERR_UNSUPPORTED;
  hipLaunchKernelGGL(latent_attention_plain_kernel, dim3(n_rows, H), dim3(256), (size_t)(R + dr) * sizeof(float), stream,
                     q, q_dtype, ldq, out, out_dtype, ldo, H, R, dr, pages, page_dtype, P, block_table, max_blocks,
                     positions, row_seg, scale);
  APC_LAUNCH_CHECK();
  return 0;
}

APC_EXPORT int apc_tanh_norm(const void* x, int x_dtype, int ldx, const int* rows, float alpha, const float* w,
                             const float* b, void* h, int h_dtype, int ldh, int n_rows, int dim, int exact,
                             hipStream_t stream) {
  if (n_rows <= 0) return 0;
  if (dim <= 0 || ldx < dim || ldh < dim || !w || !b) return APC_ERR_BAD_ARG;
  const dim3 grid(n_rows, ceil_div(dim, 256));
  if (grid.y > 65535) return APC_ERR_UNSUPPORTED;
  const TanhNorm n{alpha, w, b};
  if (exact)
    hipLaunchKernelGGL(tanh_norm_kernel<true>, grid, dim3(256), 0, stream, x, x_dtype, ldx, rows, n, h, h_dtype, ldh, dim);
  else
    hipLaunchKernelGGL(tanh_norm_kernel<false>, grid, dim3(256), 0, stream, x, x_dtype, ldx, rows, n, h, h_dtype, ldh, dim);
  APC_LAUNCH_CHECK();
  return 0;
}

// h may be null: only the sum
APC_EXPORT int apc_tanh_norm_add(float* x, int ldx, const void* y, int y_dtype, int ldy, float p_alpha, const float* pw,
                                 const float* pb, float alpha, const float* w, const float* b, void* h, int h_dtype,
                                 int ldh, int n_rows, int dim, int exact, hipStream_t stream) {
  if (n_rows <= 0) return 0;
  if (dim <= 0 || ldx < dim || ldy < dim || !pw || !pb || (h && (ldh < dim || !w || !b))) return APC_ERR_BAD_ARG;
  const TanhNorm post{p_alpha, pw, pb}, n{alpha, w, b};
  auto a16 = [](const void* p) { return ((uintptr_t)p & 15u) == 0; };
  if (y_dtype == APC_F32 && dim % 4 == 0 && ldx % 4 == 0 && ldy % 4 == 0 && a16(x) && a16(y) && a16(pw) && a16(pb) &&
      (!h || (ldh % 4 == 0 && a16(h) && a16(w) && a16(b)))) {
    const int rows = n_rows >= 1024 ? 4 : 1;                  // (a step of few rows wants its blocks)
    const dim3 grid(ceil_div(n_rows, rows), ceil_div(dim, 1024));
    if (grid.y > 65535) return APC_ERR_UNSUPPORTED;
#define TANH_ADD(EXACT_, ROWS_)                                                                                         \
  hipLaunchKernelGGL((tanh_norm_add_f4_kernel<EXACT_, ROWS_>), grid, dim3(256), 0, stream, x, ldx, (const float*)y, ldy, \
                     post, n, h, h_dtype, ldh, n_rows, dim)
    if (exact && rows == 4) TANH_ADD(true, 4);
    else if (exact) TANH_ADD(true, 1);
    else if (rows == 4) TANH_ADD(false, 4);
    else TANH_ADD(false, 1);
#undef TANH_ADD
  } else {
    const dim3 grid(n_rows, ceil_div(dim, 256));
    if (grid.y > 65535) return APC_ERR_UNSUPPORTED;
    if (exact)
      hipLaunchKernelGGL(tanh_norm_add_kernel<true>, grid, dim3(256), 0, stream, x, ldx, y, y_dtype, ldy, post, n, h,
                         h_dtype, ldh, dim);
    else
      hipLaunchKernelGGL(tanh_norm_add_kernel<false>, grid, dim3(256), 0, stream, x, ldx, y, y_dtype, ldy, post, n, h,
                         h_dtype, ldh, dim);
  }
  APC_LAUNCH_CHECK();
  return 0;
}
