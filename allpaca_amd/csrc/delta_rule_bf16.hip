// The gated delta rule (see plain_delta.hip for the formulas) over prompt portions, bfloat16 rows on MFMA, a segment's
// rows in chunks of 64.  With S0 the state in front of a chunk, c_t the product of the decays of its rows 0 .. t, n_t the
// inverse norm of the raw key k_t (q_t's, with its scale: m_t), the writes u_t of a chunk solve a triangular system:
//   u_t + sum_{s<t} A[t][s] u_s = beta_t v_t - beta_t c_t n_t S0^T k_t,   A[t][s] = beta_t (c_t / c_s) n_t n_s (k_t . k_s)
//   o_t = c_t m_t S0^T q_t + sum_{s<=t} P[t][s] u_s,                      P[t][s] = (c_t / c_s) m_t n_s (q_t . k_s)
//   S   = c_end S0 + sum_s k_s ((c_end / c_s) n_s u_s)^T
// (the chunked form of the delta rule, Yang et al. 2024, with the inverse kept apart from values and keys).
//
//   factors   every chunk and head for itself: A, the inverse of I + A (16 x 16 blocks of its diagonal by substitution,
//             the blocks below by products in 32-bit), P, the rows' coefficients, and the chunk's keys across (key
//             element by row), which the state's sum reads
//   walk      a block a segment, head and 16 value columns: the chunks in order with the state in registers
//
// Raw keys and queries are exact operands; their norms and every decay are factors of 32-bit rows.  Everything else that
// is 32-bit in the formulas and has to be an MFMA operand (S0, the right-hand side, the inverse, P, the writes) goes in
// as two bfloat16 pieces, value = hi + lo, so that a product keeps 16 bits of it and not 8.
#include "mfma.h"
#include <math.h>

namespace {

constexpr int C = 64;          // rows of a chunk (the step's list of chunks is made for this)
constexpr int NV = 16;         // value columns of a block of the walk
constexpr int NCOEF = 4;       // beta, beta c n, c m, (c_end / c) n
constexpr int COEF = NCOEF * C + 8;   // floats of a chunk's and head's coefficients; behind the rows': c_end
constexpr int FACT = 4 * C * C;       // bfloat16 of a chunk's and head's factors: inverse (hi, lo), P (hi, lo), each [C][C]
constexpr int AR = C + 4;      // row of A and of the inverse in LDS (floats)

__device__ __forceinline__ float softplus_f(float z) { return z > 20.f ? z : log1pf(__expf(z)); }
__device__ __forceinline__ void unpack8f(const Frag& f, float* v) {
#pragma unroll
  for (int w = 0; w < 4; ++w) {
    v[2 * w] = __uint_as_float(f.w[w] << 16);
    v[2 * w + 1] = __uint_as_float(f.w[w] & 0xffff0000u);
  }
}
// four consecutive float32 as two bfloat16 pieces each: hi to `ph`, lo to `pl`
__device__ __forceinline__ void store_split4(bf16_t* ph, bf16_t* pl, float a, float b, float c, float d) {
  uint2 hi, lo;
  hi.x = pack_bf16x2(a, b);
  hi.y = pack_bf16x2(c, d);
  lo.x = pack_bf16x2(a - __uint_as_float(hi.x << 16), b - __uint_as_float(hi.x & 0xffff0000u));
  lo.y = pack_bf16x2(c - __uint_as_float(hi.y << 16), d - __uint_as_float(hi.y & 0xffff0000u));
  *reinterpret_cast<uint2*>(ph) = hi;
  *reinterpret_cast<uint2*>(pl) = lo;
}
__device__ __forceinline__ floatx4 mfma16_f32(float a, float b, floatx4 c) {
  // v_mfma_f32_16x16x4_f32: lane l gives A[l % 16][l / 16] and B[l / 16][l % 16]; the result as in mfma16
  return __builtin_amdgcn_mfma_f32_16x16x4f32(a, b, c, 0, 0, 0);
}

// ------------------------------------------------------------------------------------------------ factors
template <int DKP>   // key size rounded up to 64, 128 or 256
__global__ __launch_bounds__(256) void delta_factors_kernel(
    const bf16_t* __restrict__ rows, int ld, int q_off, int k_off, int H, int G, int dk, const bf16_t* __restrict__ ba,
    int ldba, int a_off, int b_off, const float* __restrict__ A_rate, const float* __restrict__ dt_bias, float q_scale,
    const int* __restrict__ chunks, const int* __restrict__ seg_row0, const int* __restrict__ seg_rows,
    bf16_t* __restrict__ fact, float* __restrict__ coef, bf16_t* __restrict__ kt) {
  constexpr int KS = DKP / 32;
  __shared__ __attribute__((aligned(16))) float As[C * AR];
  __shared__ __attribute__((aligned(16))) float Ts[C * AR];
  __shared__ float Ms[4][16 * 17];
  __shared__ float lg[C], be[C], kn[C], qn[C];
  const int chunk = blockIdx.x, h = blockIdx.y, hk = h / (H / G);
  const int tid = threadIdx.x, lane = tid % WAVE, wave = tid / WAVE, li = lane % 16, lc = lane / 16;
  const int seg = chunks[2 * chunk], c0 = chunks[2 * chunk + 1];
  const int r0 = seg_row0[seg] + c0, nc = min(C, seg_rows[seg] - c0);

  // ---- the wave's 16 rows t as columns of the tiles, and all 64 rows s as their rows
  const int t = wave * 16 + li;
  Frag kf[KS], qf[KS];
  {
    const bf16_t* kr = rows + (size_t)(r0 + min(t, nc - 1)) * ld + k_off + (size_t)hk * dk;
    const bf16_t* qr = kr - k_off + q_off;
    float kk = 0.f, qq = 0.f;
#pragma unroll
    for (int ks = 0; ks < KS; ++ks) {
      const int e = ks * 32 + lc * 8;
      const bool on = t < nc && e < dk;
      kf[ks] = on ? load_frag(kr + e) : zero_frag();
      qf[ks] = on ? load_frag(qr + e) : zero_frag();
      float a[8], b[8];
      unpack8f(kf[ks], a);
      unpack8f(qf[ks], b);
#pragma unroll
      for (int x = 0; x < 8; ++x) {
        kk = fmaf(a[x], a[x], kk);
        qq = fmaf(b[x], b[x], qq);
      }
    }
    kk += __shfl_xor(kk, 16, WAVE);
    kk += __shfl_xor(kk, 32, WAVE);
    qq += __shfl_xor(qq, 16, WAVE);
    qq += __shfl_xor(qq, 32, WAVE);
    if (lc == 0) {
      kn[t] = 1.0f / sqrtf(kk + 1e-6f);
      qn[t] = q_scale / sqrtf(qq + 1e-6f);
    }
  }
  if (wave == 0) {             // the rows' decays, summed up in the exponent, and step sizes; rows beyond the chunk: none
    float g = 0.f, b = 0.f;
    if (lane < nc) {
      const bf16_t* r = ba + (size_t)(r0 + lane) * ldba;
      g = -A_rate[h] * softplus_f(bf16_to_float(r[a_off + h]) + dt_bias[h]);
      b = 1.0f / (1.0f + __expf(-bf16_to_float(r[b_off + h])));
    }
#pragma unroll
    for (int o = 1; o < WAVE; o <<= 1) {
      const float v = __shfl_up(g, o, WAVE);
      if (lane >= o) g += v;
    }
    lg[lane] = g;
    be[lane] = b;
  }
  __syncthreads();
  bf16_t* F = fact + ((size_t)chunk * H + h) * FACT;
  if (wave == 0) {
    float* co = coef + ((size_t)chunk * H + h) * COEF;
    const float c = __expf(lg[lane]);
    const bool on = lane < nc;
    co[lane] = be[lane];
    co[C + lane] = be[lane] * c * kn[lane];
    co[2 * C + lane] = c * qn[lane];
    co[3 * C + lane] = on ? __expf(lg[C - 1] - lg[lane]) * kn[lane] : 0.f;
    if (lane == 0) co[NCOEF * C] = __expf(lg[C - 1]);
  }
  {
    const float lt = lg[t], bt = be[t] * kn[t], qt = qn[t];
#pragma unroll
    for (int st = 0; st < 4; ++st) {
      floatx4 a = floatx4{0.f, 0.f, 0.f, 0.f}, p = floatx4{0.f, 0.f, 0.f, 0.f};
      if (st <= wave) {
        const int s = st * 16 + li;
        const bf16_t* kr = rows + (size_t)(r0 + min(s, nc - 1)) * ld + k_off + (size_t)hk * dk;
#pragma unroll
        for (int ks = 0; ks < KS; ++ks) {
          const int e = ks * 32 + lc * 8;
          const Frag f = (s < nc && e < dk) ? load_frag(kr + e) : zero_frag();
          a = mfma16(f, kf[ks], a);
          p = mfma16(f, qf[ks], p);
        }
#pragma unroll
        for (int r = 0; r < 4; ++r) {
          const int s_ = st * 16 + lc * 4 + r;
          const float w = s_ <= t ? __expf(lt - lg[s_]) * kn[s_] : 0.f;
          a[r] = s_ < t ? a[r] * (w * bt) : 0.f;
          p[r] *= w * qt;
        }
      }
      const int at = t * C + st * 16 + lc * 4;
      *reinterpret_cast<float4*>(As + t * AR + st * 16 + lc * 4) = float4{a[0], a[1], a[2], a[3]};
      store_split4(F + 2 * C * C + at, F + 3 * C * C + at, p[0], p[1], p[2], p[3]);
    }
  }
  // ---- the keys across, once for the heads that share them
  if (h % (H / G) == 0) {
    bf16_t* K = kt + ((size_t)chunk * G + hk) * dk * C;
    for (int idx = tid; idx < dk * (C / 8); idx += 256) {
      const int i = idx % dk, s0 = idx / dk * 8;
      const bf16_t* src = rows + (size_t)r0 * ld + k_off + (size_t)hk * dk + i;
      uint32_t v[8];
#pragma unroll
      for (int x = 0; x < 8; ++x) v[x] = src[(size_t)min(s0 + x, nc - 1) * ld];
      Frag f;
#pragma unroll
      for (int x = 0; x < 4; ++x)
        f.w[x] = (s0 + 2 * x < nc ? v[2 * x] : 0u) | (s0 + 2 * x + 1 < nc ? v[2 * x + 1] << 16 : 0u);
      *reinterpret_cast<Frag*>(K + (size_t)i * C + s0) = f;
    }
  }
  __syncthreads();

  // ---- the inverse T of I + A.  Diagonal blocks: lane j's column by substitution, x_i = [i = j] - sum_{m<i} A[i][m] x_m
  {
    const float* a = As + (wave * 16) * AR + wave * 16;
    float x[16];
#pragma unroll
    for (int i = 0; i < 16; ++i) {
      float v = i == li ? 1.f : 0.f;
#pragma unroll
      for (int m = 0; m < i; ++m) v = fmaf(-a[i * AR + m], x[m], v);
      x[i] = v;
    }
    if (lc == 0) {
#pragma unroll
      for (int i = 0; i < 16; ++i) Ts[(wave * 16 + i) * AR + wave * 16 + li] = x[i];
    }
  }
  __syncthreads();
  // blocks below it, a diagonal at a time: T_ij = -T_ii sum_{j <= m < i} A_im T_mj
#pragma unroll
  for (int d = 1; d < 4; ++d) {
    const int i = wave, j = wave - d;
    if (j >= 0) {
      floatx4 acc = floatx4{0.f, 0.f, 0.f, 0.f};
      for (int m = j; m < i; ++m)
#pragma unroll
        for (int k = 0; k < 4; ++k)
          acc = mfma16_f32(As[(i * 16 + li) * AR + m * 16 + k * 4 + lc], Ts[(m * 16 + k * 4 + lc) * AR + j * 16 + li], acc);
      float* M = Ms[wave];
#pragma unroll
      for (int r = 0; r < 4; ++r) M[(lc * 4 + r) * 17 + li] = acc[r];
      wave_lds_order();
      floatx4 tt = floatx4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int k = 0; k < 4; ++k)
        tt = mfma16_f32(Ts[(i * 16 + li) * AR + i * 16 + k * 4 + lc], M[(k * 4 + lc) * 17 + li], tt);
#pragma unroll
      for (int r = 0; r < 4; ++r) Ts[(i * 16 + lc * 4 + r) * AR + j * 16 + li] = -tt[r];
    }
    __syncthreads();
  }
  for (int idx = tid; idx < C * (C / 4); idx += 256) {
    const int i = idx / (C / 4), j = idx % (C / 4) * 4;
    const bool low = j / 16 <= i / 16;
    const float4 v = low ? *reinterpret_cast<const float4*>(Ts + i * AR + j) : float4{0.f, 0.f, 0.f, 0.f};
    store_split4(F + i * C + j, F + C * C + i * C + j, v.x, v.y, v.z, v.w);
  }
}

// ------------------------------------------------------------------------------------------------ walk
// Wave w: rows 16 w .. of the chunk in the products over rows, key elements [w DKP/4, (w+1) DKP/4) of the state.
template <int DKP>
__global__ __launch_bounds__(256) void delta_walk_kernel(
    const bf16_t* __restrict__ rows, int ld, int q_off, int k_off, int v_off, int H, int G, int dk, int dv,
    const bf16_t* __restrict__ fact, const float* __restrict__ coef, const bf16_t* __restrict__ kt,
    float* __restrict__ state, const int* __restrict__ seg_chunks, const int* __restrict__ seg_row0,
    const int* __restrict__ seg_rows, const int* __restrict__ slots, float* __restrict__ out, int ldo, int n_tiles) {
  constexpr int KS = DKP / 32, ST = DKP / 64;     // steps over a key; tiles of 16 state rows a wave
  constexpr int SR = DKP + 8, UR = C + 8;
  __shared__ __attribute__((aligned(16))) bf16_t Sh[NV * SR], Sl[NV * SR];          // the state, [column][key element]
  __shared__ __attribute__((aligned(16))) bf16_t Rh[NV * UR], Rl[NV * UR];          // the right-hand side, [column][row]
  __shared__ __attribute__((aligned(16))) bf16_t Uh[NV * UR], Ul[NV * UR];          // the writes
  __shared__ __attribute__((aligned(16))) bf16_t Eh[NV * UR], El[NV * UR];          // the writes as the state takes them
  const int tid = threadIdx.x, lane = tid % WAVE, wave = tid / WAVE, li = lane % 16, lc = lane / 16;
  // the blocks of a head (they read the same factors and keys) on one XCD
  int h, tile;
  {
    const int id = blockIdx.x;
    if (H % 8 == 0) { const int xcd = id % 8, slot = id / 8; h = xcd + 8 * (slot / n_tiles); tile = slot % n_tiles; }
    else { h = id / n_tiles; tile = id % n_tiles; }
  }
  const int seg = blockIdx.y, hk = h / (H / G), j = tile * NV + li;
  const bool col = j < dv;
  const int jc = min(j, dv - 1);
  const int first = seg_chunks[2 * seg], n = seg_chunks[2 * seg + 1], rows_all = seg_rows[seg], base = seg_row0[seg];
  float* S = state + ((size_t)slots[seg] * H + h) * dk * dv;
  floatx4 s[ST];
#pragma unroll
  for (int it = 0; it < ST; ++it)
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int i = (wave * ST + it) * 16 + lc * 4 + r;
      s[it][r] = (i < dk && col) ? S[(size_t)i * dv + j] : 0.f;
    }

  // What a chunk reads from memory; the next chunk's is asked for when a chunk begins, so that a whole chunk's work lies
  // between the asking and the use: without a condition (behind the last chunk it is that chunk's again) and without a
  // step of arithmetic on the way, either of which would make the wave wait.  Elements beyond the key size are read
  // from its first ones: the state's image has zeros there.
  struct Chunk {
    Frag kf[KS], qf[KS];                          // the wave's rows of keys and queries
    Frag ktf[ST][2];                              // the wave's key elements across
    Frag th[2], tl[2], ph[2], pl[2];              // the wave's rows of the inverse and of P
    bf16_t vr[4];
    float4 cb, ck, cq, ce;
    float c_end;
  };
  auto load = [&](Chunk& x, int c) {
    const int r0 = base + c * C, nc = min(C, rows_all - c * C);
    const bf16_t* kr = rows + (size_t)(r0 + min(wave * 16 + li, nc - 1)) * ld + k_off + (size_t)hk * dk;
    const bf16_t* qr = kr - k_off + q_off;
#pragma unroll
    for (int ks = 0; ks < KS; ++ks) {
      const int e = ks * 32 + lc * 8, at = e < dk ? e : 0;
      x.kf[ks] = load_frag(kr + at);
      x.qf[ks] = load_frag(qr + at);
    }
    const float* co = coef + ((size_t)(first + c) * H + h) * COEF + wave * 16 + lc * 4;
    x.cb = *reinterpret_cast<const float4*>(co);
    x.ck = *reinterpret_cast<const float4*>(co + C);
    x.cq = *reinterpret_cast<const float4*>(co + 2 * C);
    x.ce = *reinterpret_cast<const float4*>(co + 3 * C);
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int t = min(wave * 16 + lc * 4 + r, nc - 1);
      x.vr[r] = rows[(size_t)(r0 + t) * ld + v_off + (size_t)h * dv + jc];
    }
    x.c_end = coef[((size_t)(first + c) * H + h) * COEF + NCOEF * C];
    const bf16_t* F = fact + ((size_t)(first + c) * H + h) * FACT + (wave * 16 + li) * C + lc * 8;
#pragma unroll
    for (int kk = 0; kk < 2; ++kk) {
      x.th[kk] = load_frag(F + kk * 32);
      x.tl[kk] = load_frag(F + C * C + kk * 32);
      x.ph[kk] = load_frag(F + 2 * C * C + kk * 32);
      x.pl[kk] = load_frag(F + 3 * C * C + kk * 32);
    }
    const bf16_t* K = kt + ((size_t)(first + c) * G + hk) * dk * C;
#pragma unroll
    for (int it = 0; it < ST; ++it) {
      const int i = (wave * ST + it) * 16 + li, at = i < dk ? i : 0;
#pragma unroll
      for (int kk = 0; kk < 2; ++kk) x.ktf[it][kk] = load_frag(K + (size_t)at * C + kk * 32 + lc * 8);
    }
  };
  auto walk = [&](const Chunk& x, Chunk& next, int c) {
    const int nc = min(C, rows_all - c * C);
    load(next, min(c + 1, n - 1));
#pragma unroll
    for (int it = 0; it < ST; ++it) {
      const int i = (wave * ST + it) * 16 + lc * 4, at = li * SR + i;
      const bool in = i < dk;                     // (the key size is a multiple of 8)
      store_split4(Sh + at, Sl + at, in ? s[it][0] : 0.f, in ? s[it][1] : 0.f, in ? s[it][2] : 0.f, in ? s[it][3] : 0.f);
    }
    __syncthreads();
    // ---- S0^T k and S0^T q of the wave's rows: tile rows t, columns j
    floatx4 sk = floatx4{0.f, 0.f, 0.f, 0.f}, o = floatx4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int ks = 0; ks < KS; ++ks) {
      const Frag fh = *reinterpret_cast<const Frag*>(Sh + li * SR + ks * 32 + lc * 8);
      const Frag fl = *reinterpret_cast<const Frag*>(Sl + li * SR + ks * 32 + lc * 8);
      sk = mfma16(x.kf[ks], fh, sk);
      o = mfma16(x.qf[ks], fh, o);
      sk = mfma16(x.kf[ks], fl, sk);
      o = mfma16(x.qf[ks], fl, o);
    }
    {
      const float ck[4] = {x.ck.x, x.ck.y, x.ck.z, x.ck.w}, cb[4] = {x.cb.x, x.cb.y, x.cb.z, x.cb.w};
      const float cq[4] = {x.cq.x, x.cq.y, x.cq.z, x.cq.w};
      float y[4];
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        y[r] = fmaf(-ck[r], sk[r], cb[r] * bf16_to_float(x.vr[r]));
        o[r] *= cq[r];
      }
      const int at = li * UR + wave * 16 + lc * 4;
      store_split4(Rh + at, Rl + at, y[0], y[1], y[2], y[3]);
    }
    __syncthreads();
    // ---- the writes of the wave's rows
    {
      floatx4 u = floatx4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int kk = 0; kk < 2; ++kk) {
        if (kk * 32 > wave * 16 + 15) continue;    // (later rows do not enter)
        const Frag fh = *reinterpret_cast<const Frag*>(Rh + li * UR + kk * 32 + lc * 8);
        const Frag fl = *reinterpret_cast<const Frag*>(Rl + li * UR + kk * 32 + lc * 8);
        u = mfma16(x.th[kk], fh, u);
        u = mfma16(x.th[kk], fl, u);
        u = mfma16(x.tl[kk], fh, u);
      }
      const int at = li * UR + wave * 16 + lc * 4;
      store_split4(Uh + at, Ul + at, u[0], u[1], u[2], u[3]);
      store_split4(Eh + at, El + at, u[0] * x.ce.x, u[1] * x.ce.y, u[2] * x.ce.z, u[3] * x.ce.w);
    }
    __syncthreads();
    // ---- the state behind the chunk, then the outputs
#pragma unroll
    for (int it = 0; it < ST; ++it) {
#pragma unroll
      for (int r = 0; r < 4; ++r) s[it][r] *= x.c_end;
#pragma unroll
      for (int kk = 0; kk < 2; ++kk) {
        s[it] = mfma16(x.ktf[it][kk], *reinterpret_cast<const Frag*>(Eh + li * UR + kk * 32 + lc * 8), s[it]);
        s[it] = mfma16(x.ktf[it][kk], *reinterpret_cast<const Frag*>(El + li * UR + kk * 32 + lc * 8), s[it]);
      }
    }
#pragma unroll
    for (int kk = 0; kk < 2; ++kk) {
      if (kk * 32 > wave * 16 + 15) continue;
      const Frag fh = *reinterpret_cast<const Frag*>(Uh + li * UR + kk * 32 + lc * 8);
      const Frag fl = *reinterpret_cast<const Frag*>(Ul + li * UR + kk * 32 + lc * 8);
      o = mfma16(x.ph[kk], fh, o);
      o = mfma16(x.ph[kk], fl, o);
      o = mfma16(x.pl[kk], fh, o);
    }
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int t = wave * 16 + lc * 4 + r;
      if (t < nc && col) out[(size_t)(base + c * C + t) * ldo + (size_t)h * dv + j] = o[r];
    }
    // (the state's image is written next: all reads of it lie ahead of the second barrier above; the right-hand side and
    // the writes are next stored behind the next chunk's first and second barriers)
  };
  Chunk a, b;
  load(a, 0);
  for (int c = 0; c < n; c += 2) {
    walk(a, b, c);
    if (c + 1 < n) walk(b, a, c + 1);
  }
#pragma unroll
  for (int it = 0; it < ST; ++it)
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int i = (wave * ST + it) * 16 + lc * 4 + r;
      if (i < dk && col) S[(size_t)i * dv + j] = s[it][r];
    }
}

}  // namespace

// 1 if the kernels take these sizes, else 0 (the caller then runs the kernel that walks row by row)
APC_EXPORT int apc_delta_rule_bf16_takes(int ld, int q_off, int k_off, int H, int G, int dk, int dv) {
  return (H > 0 && G > 0 && H % G == 0 && dk > 0 && dv > 0 && dk <= 256 && dk % 8 == 0 && ld % 8 == 0 && q_off % 8 == 0 &&
          k_off % 8 == 0) ? 1 : 0;
}
// elements of the working memory of a chunk: bfloat16 of the factors, float32 of the coefficients, of all heads
APC_EXPORT int apc_delta_rule_fact_size(int H) { return H * FACT; }
APC_EXPORT int apc_delta_rule_coef_size(int H) { return H * COEF; }

// chunks: int32 [n_chunks][2] (segment, first row of the chunk in it), all segments' chunks of 64 rows in order;
// seg_chunks: int32 [n_segs][2] (a segment's first chunk, its chunks); fact, coef: see above, times n_chunks; kt bfloat16
// [n_chunks][G][dk][64].
APC_EXPORT int apc_delta_rule_bf16(const void* rows, int ld, int q_off, int k_off, int v_off, int H, int G, int dk, int dv,
                                   const void* ba, int ldba, int a_off, int b_off, const float* A, const float* dt_bias,
                                   float q_scale, float* state, int n_segs, const int* seg_row0, const int* seg_rows,
                                   const int* slots, int n_chunks, const int* chunks, const int* seg_chunks, void* fact,
                                   float* coef, void* kt, float* out, int ldo, hipStream_t stream) {
  if (n_segs <= 0 || n_chunks <= 0) return 0;
  if (!apc_delta_rule_bf16_takes(ld, q_off, k_off, H, G, dk, dv)) return APC_ERR_UNSUPPORTED;
  if (!rows || !ba || !A || !dt_bias || !state || !seg_row0 || !seg_rows || !slots || !chunks || !seg_chunks || !fact ||
      !coef || !kt || !out || ldo < H * dv || ld < q_off + G * dk || ld < k_off + G * dk || ld < v_off + H * dv ||
      ldba < a_off + H || ldba < b_off + H || ((uintptr_t)rows & 15u) || ((uintptr_t)fact & 15u) || ((uintptr_t)kt & 15u))
    return APC_ERR_BAD_ARG;
  const int n_tiles = ceil_div(dv, NV);
  if (H > 65535 || n_segs > 65535 || (long)H * n_tiles > 0x7fffffffL) return APC_ERR_UNSUPPORTED;
#define DELTA_LAUNCH(DKP_)                                                                                              \
  do {                                                                                                                  \
    hipLaunchKernelGGL(delta_factors_kernel<DKP_>, dim3(n_chunks, H), dim3(256), 0, stream, (const bf16_t*)rows, ld,     \
                       q_off, k_off, H, G, dk, (const bf16_t*)ba, ldba, a_off, b_off, A, dt_bias, q_scale, chunks,       \
                       seg_row0, seg_rows, (bf16_t*)fact, coef, (bf16_t*)kt);                                           \
    APC_LAUNCH_CHECK();                                                                                                 \
    hipLaunchKernelGGL(delta_walk_kernel<DKP_>, dim3(H * n_tiles, n_segs), dim3(256), 0, stream, (const bf16_t*)rows, ld, \
                       q_off, k_off, v_off, H, G, dk, dv, (const bf16_t*)fact, coef, (const bf16_t*)kt, state, seg_chunks, \
                       seg_row0, seg_rows, slots, out, ldo, n_tiles);                                                   \
    APC_LAUNCH_CHECK();                                                                                                 \
  } while (0)
  if (dk <= 64) DELTA_LAUNCH(64);
  else if (dk <= 128) DELTA_LAUNCH(128);
  else DELTA_LAUNCH(256);
#undef DELTA_LAUNCH
  return 0;
}
