// Attention of all heads over cached latents, bfloat16 on MFMA with float32 softmax.
//
//   A position's cached row is [c | kr]: R + dr elements, one row for all heads.  Head h of a row of the step has a query
//   of the same size;  s = (q . row) * scale over the positions up to the row's own;  out = sum softmax(s) * row[:R].
//   Pages: [slot][R + dr], a page is P * (R + dr) elements.
//
// (row of the step, head) pairs are one axis: pair = row * H + head, and the queries are a [pairs][R + dr] matrix as they
// lie.  Since every head reads the same keys, a block takes any PT * 32 consecutive pairs of one request (two rows of 32
// heads, 8 rows of 8, 32 of the heads of one decoded row), and keys are shared by all of them.  The values are the keys'
// first R elements: a tile of keys is brought into LDS once and read twice, along the row for the scores and across the
// rows, by the LDS's transposing read, for the values.
//
// A tile of 64 keys lies in LDS as blocks of 32 elements: [block][key][64 bytes], the 16-byte piece p of key t at place
// p ^ ((t / 4) % 4).  Direct loads fill it 1 KiB an instruction (16 keys x 64 bytes; a lane keeps the address of its key's
// row for the whole tile), operand reads of 16 keys and transposing reads of 4 keys x 32 elements are free of bank
// conflicts, and nothing is padded.  Two such buffers take turns: the loads of a tile run during the pass before.
// The direct loads are written as instructions: left to the compiler, every LDS read behind one waits until all of them
// have landed (it cannot tell that they fill the other buffer).  What keeps reads and loads apart are the barriers of a
// pass: a buffer is filled behind the barrier that all its readers have passed, and read behind one that stands behind
// `vmcnt(0)` of every wave.  The queries come through the second buffer in the same way before the first pass, and O goes
// out through LDS in whole rows.
//
// A pass over a tile, 8 waves (two a SIMD, so that one's vector instructions and waits stand beside the other's products):
//   scores   S^T = K Q^T on 16 x 16 x 32: a wave 16 keys x PT * 16 pairs; its queries stay in registers
//   maxima   of the tile through LDS (four waves have a pair's keys between them); the reference that a pair's scores
//            are taken against moves only when a maximum exceeds it by more than 2^8, and only then are sums rescaled
//   weights  exp to LDS in bfloat16, [pair][key]
//   values   O^T += V^T P^T on 32 x 32 x 16: a wave every eighth block of 32 value elements, all pairs
// The keys of an item may be cut into ranges of whole tiles, a block each (decoded rows; few prompt rows over many keys):
// a block then leaves O, its reference and its sum in 32 bits, and `latent_merge_kernel` adds the ranges.
#include "mfma.h"
#include <math.h>

namespace {

constexpr int KT = 64;                 // keys a tile
constexpr int NW = 8, NT = NW * WAVE;  // waves, threads a block
constexpr int PROW = KT + 8;           // bfloat16 elements of a pair's row of weights in LDS
constexpr float RISE = 8.f;            // by how much (in powers of 2) a score may exceed its pair's reference
constexpr float LOG2E = 1.4426950408889634f;
constexpr float NO_KEY = -1e30f;

typedef short s16x4 __attribute__((ext_vector_type(4)));
typedef __attribute__((address_space(3))) s16x4* lds_s16x4;

struct LatentItems {
  const int* row0;      // first row of every item (null: item i is row i)
  const int* rows;      // its rows (null: 1)
  int n;                // items
  int blocks;           // blocks an item (for the item with the most rows)
};

// everything of this wave in LDS, then the block; `asm volatile` with a memory clobber keeps the compiler's accesses on
// their side
__device__ __forceinline__ void lds_barrier() { asm volatile("s_waitcnt lgkmcnt(0)\n\ts_barrier" ::: "memory"); }
// the same behind this wave's direct loads
__device__ __forceinline__ void loads_barrier() { asm volatile("s_waitcnt vmcnt(0) lgkmcnt(0)\n\ts_barrier" ::: "memory"); }

// 16 bytes a lane from `src` (a lane's own address) + OFFSET bytes to LDS at `lds` + 16 * lane (the same `lds` for the
// wave; the instruction adds its offset to both addresses).  m0 is a register the compiler sets right ahead of an
// instruction of its own that reads it and never keeps anything in.
template <int OFFSET>
__device__ __forceinline__ void load_to_lds(const bf16_t* src, int lds) {
  static_assert(OFFSET >= 0 && OFFSET < 4096, "the instruction's offset has 12 bits");
  asm volatile("s_mov_b32 m0, %1\n\ts_nop 0\n\tglobal_load_lds_dwordx4 %0, off offset:%2" ::"v"(src),
               "s"(lds - OFFSET), "n"(OFFSET));
}
__device__ __forceinline__ int lds_address(const void* p) {
  return (int)(uintptr_t)(const __attribute__((address_space(3))) void*)p;
}

// c = a . q and c += a . q with q, the queries of the wave's pairs, which only these read, in accumulation registers (ACC;
// what does not fit there in vector registers), beside O in the vector registers, where a rescaling wants it.  Written as instructions, because
// left to itself the compiler copies them there in every pass; it does not know the instruction, so what waits for the
// results is `scores_done`.
typedef uint32_t u32x4 __attribute__((ext_vector_type(4)));
template <bool ACC>
__device__ __forceinline__ void mfma16_set(floatx4& c, const Frag& a, const u32x4& q) {
  if constexpr (ACC)
    asm volatile("v_mfma_f32_16x16x32_bf16 %0, %1, %2, 0" : "=&v"(c) : "v"(__builtin_bit_cast(u32x4, a)), "a"(q));
  else
    asm volatile("v_mfma_f32_16x16x32_bf16 %0, %1, %2, 0" : "=&v"(c) : "v"(__builtin_bit_cast(u32x4, a)), "v"(q));
}
template <bool ACC>
__device__ __forceinline__ void mfma16_add(floatx4& c, const Frag& a, const u32x4& q) {
  if constexpr (ACC)
    asm volatile("v_mfma_f32_16x16x32_bf16 %0, %1, %2, %0" : "+v"(c) : "v"(__builtin_bit_cast(u32x4, a)), "a"(q));
  else
    asm volatile("v_mfma_f32_16x16x32_bf16 %0, %1, %2, %0" : "+v"(c) : "v"(__builtin_bit_cast(u32x4, a)), "v"(q));
}
__device__ __forceinline__ void scores_done(floatx4& s0, floatx4& s1) {
  asm volatile("s_nop 15\n\ts_nop 3" : "+v"(s0), "+v"(s1));
}
// f over the lanes whose numbers differ by 16 and 32, without LDS: a swap of rows (halves) between two copies of x leaves
// the lane's own and the other's
template <class F>
__device__ __forceinline__ float over_row_groups(float x, F f) {
  auto a = __builtin_amdgcn_permlane16_swap(__float_as_uint(x), __float_as_uint(x), false, false);
  x = f(__uint_as_float(a[0]), __uint_as_float(a[1]));
  auto b = __builtin_amdgcn_permlane32_swap(__float_as_uint(x), __float_as_uint(x), false, false);
  return f(__uint_as_float(b[0]), __uint_as_float(b[1]));
}
// nothing moves across: LDS reads stay as far ahead of what takes them as they are written
__device__ __forceinline__ void in_order() { __builtin_amdgcn_sched_barrier(0); }

// every other block of 32 elements of a key's row from `src` (this lane's piece of the first of them) to LDS; of `left` and
// more elements from there on nothing is in the row, and `none`, its first piece, comes instead
template <int B, int NB, bool EVEN>
__device__ __forceinline__ void fill_blocks(const bf16_t* src, const bf16_t* none, int left, int lds) {
  if constexpr (B < NB) {
    load_to_lds<B * 64>(EVEN || B * 32 < left ? src : none - B * 32, lds + B * (KT * 64));
    fill_blocks<B + 2, NB, EVEN>(src, none, left, lds);
  }
}

// RT: blocks of 32 value elements, NB: blocks of 32 elements of a row (EVEN: a row fills them), PT: 32-pair groups a block
// of threads takes
template <int RT, int NB, int PT, bool EVEN>
__global__ __launch_bounds__(NT, 2) void latent_attention_kernel(
    const bf16_t* __restrict__ q, bf16_t* __restrict__ out, int H, int R, int L, const bf16_t* __restrict__ pages,
    int pshift, const int* __restrict__ block_table, int max_blocks, const int* __restrict__ positions,
    const int* __restrict__ row_seg, LatentItems items, int n_splits, float scale2, float* __restrict__ parts,
    float* __restrict__ ml) {
  static_assert(NB % 2 == 0, "the waves bring a tile's blocks in two halves");
  constexpr int NP = PT * 32, NG = KT / 16;     // pairs of a block; waves that share a pair's keys
  constexpr int NV = (RT + NW - 1) / NW;        // value blocks a wave
  // a wave's queries: QA blocks in accumulation registers, one more in vector registers, what is left in LDS
  constexpr int QA = PT == 2 && NB > 16 ? 16 : NB, QR = NB < QA + 1 ? NB : QA + 1, QL = NB - QR;
  constexpr int BUF = NB * KT * 32;             // elements of a tile's buffer
  __shared__ __attribute__((aligned(1024))) bf16_t bufs[2 * BUF];
  __shared__ __attribute__((aligned(16))) bf16_t ps[NP * PROW];
  __shared__ float mx[NG * NP];
  __shared__ __attribute__((aligned(16))) bf16_t qs[QL ? QL * NP * 32 : 8];
  const int lane = threadIdx.x % WAVE, wave = __builtin_amdgcn_readfirstlane(threadIdx.x / WAVE);
  const int li = lane % 16, lc = lane / 16, l32 = lane % 32, hh = lane / 32;

  const int split = blockIdx.x % n_splits, rest = blockIdx.x / n_splits;
  const int item = items.n - 1 - rest / items.blocks;            // (later rows of a prompt see more keys: they go first)
  const int row0 = items.row0 ? items.row0[item] : item;
  const int n_pairs = (items.rows ? items.rows[item] : 1) * H;
  const int pair0 = (rest % items.blocks) * NP;
  if (pair0 >= n_pairs) return;
  const int pos0 = positions[row0];
  const int* bt = block_table + (size_t)row_seg[row0] * max_blocks;
  const int last = pos0 + (min(pair0 + NP, n_pairs) - 1) / H;     // the last key any pair of the block sees
  const int first_last = pos0 + pair0 / H;                        // ... and the last one that all of them see
  const int n_tiles = last / KT + 1, per = (n_tiles + n_splits - 1) / n_splits;
  const int j0 = split * per, j1 = min(j0 + per, n_tiles);

  const int group = wave % NG, second = wave / NG;               // the wave's 16 keys, and which half of pairs and blocks
  const int kb = group * 16, pb = second * (PT * 16);
  // direct loads: this wave brings keys kb .. kb + 15 of every other block of a tile; a lane the piece (lane % 4) ^
  // (lane / 16) of key kb + lane / 4.  Pieces behind the row's end bring the row's first one, whose products meet zeros.
  const int key_of_lane = kb + lane / 4, piece = (lane % 4) ^ lc;
  auto row_of = [&](int j, int page) {
    const int t = min(j * KT + key_of_lane, last);
    return pages + (((size_t)page << pshift) + (t & ((1 << pshift) - 1))) * L;
  };
  auto page_of = [&](int j) { return bt[min(j * KT + key_of_lane, last) >> pshift]; };
  auto fill = [&](const bf16_t* dst, const bf16_t* row) {
    const int at = __builtin_amdgcn_readfirstlane(lds_address(dst) + group * 1024 + second * (KT * 64));
    const int e = second * 32 + piece * 8;
    fill_blocks<0, NB, EVEN>(row + e, row, L - e, at);
  };
  // the queries come as a tile does, into the second buffer, and go on into registers; the first tile comes with them
  fill(bufs + BUF, q + ((size_t)row0 * H + min(pair0 + min(key_of_lane, NP - 1), n_pairs - 1)) * L);
  int next_page = 0;
  if (j0 < j1) {
    fill(bufs, row_of(j0, page_of(j0)));
    if (j0 + 1 < j1) next_page = page_of(j0 + 1);
  }
  loads_barrier();
  // this lane's pairs of the scores: pb + p * 16 + li
  auto q_at = [&](int p) { return (pb + p * 16 + li) * 32 + (lc ^ (li / 4)) * 8; };
  u32x4 qf[PT][QR];
  int posq[PT];
#pragma unroll
  for (int p = 0; p < PT; ++p) {
    posq[p] = pos0 + min(pair0 + pb + p * 16 + li, n_pairs - 1) / H;
#pragma unroll
    for (int b = 0; b < NB; ++b) {
      Frag f = *reinterpret_cast<const Frag*>(bufs + BUF + b * (KT * 32) + q_at(p));
      if constexpr (!EVEN) {
        uint32_t keep = b * 32 + lc * 8 < L ? ~0u : 0u;
        asm("" : "+v"(keep));                     // (a select would become a branch around every read)
#pragma unroll
        for (int k = 0; k < 4; ++k) f.w[k] &= keep;
      }
      if (b < QR) qf[p][b < QR ? b : 0] = __builtin_bit_cast(u32x4, f);
      else *reinterpret_cast<Frag*>(qs + (b - QR) * (NP * 32) + q_at(p)) = f;     // (this lane reads it again)
    }
  }
#pragma unroll
  for (int p = 0; p < PT; ++p)
#pragma unroll
    for (int b = 0; b < QR; ++b)
      if (b < QA) asm volatile("" : "+a"(qf[p][b]));
  lds_barrier();

  floatx16 o[NV][PT];
#pragma unroll
  for (int v = 0; v < NV; ++v)
#pragma unroll
    for (int t = 0; t < PT; ++t)
#pragma unroll
      for (int r = 0; r < 16; ++r) o[v][t][r] = 0.f;
  float m[PT], l[PT], mo[PT];      // reference and sum of the pairs of the scores; reference of the pairs t * 32 + l32 of O
#pragma unroll
  for (int t = 0; t < PT; ++t) m[t] = mo[t] = NO_KEY, l[t] = 0.f;

  const int k_at = (kb + li) * 32 + (lc ^ (li / 4)) * 8;                // element in a block of 32 x 64 keys
  const int v_col = ((lane / 16) % 2) * 2 + (lane % 4) / 2;             // the 16-byte piece of this lane's 4 elements
  const int v_key = 8 * hh + (lane % 16) / 4;
  const int v_at0 = v_key * 32 + (v_col ^ (2 * hh)) * 8 + (lane % 2) * 4;
  const int v_at1 = (v_key + 4) * 32 + (v_col ^ (2 * hh + 1)) * 8 + (lane % 2) * 4;

  for (int j = j0; j < j1; ++j) {
    const bf16_t* cur = bufs + ((j - j0) & 1) * BUF;
    if (j + 1 < j1) {
      fill(bufs + ((j - j0 + 1) & 1) * BUF, row_of(j + 1, next_page));
      if (j + 2 < j1) next_page = page_of(j + 2);
    }
    // scores; with one group of pairs even and odd blocks of a row go into sums of their own, so that no product waits for
    // the one before it
    floatx4 s[2];
    {
      constexpr int AHEAD = NB > 10 && PT == 2 ? 3 : 4;
      static_assert(QL <= 1, "one block of queries is read from LDS");
      Frag kf[AHEAD], ql[PT];
      auto key = [&](int b) { return *reinterpret_cast<const Frag*>(cur + b * (KT * 32) + k_at); };
#pragma unroll
      for (int b = 0; b < AHEAD; ++b) kf[b] = key(b);
      in_order();
#pragma unroll
      for (int b = 0; b < NB; ++b) {
#pragma unroll
        for (int p = 0; p < PT; ++p) {
          floatx4& c = s[PT == 1 ? b % 2 : p];
          if (b < 3 - PT) mfma16_set<true>(c, kf[b % AHEAD], qf[p][b]);
          else if (b < QA) mfma16_add<true>(c, kf[b % AHEAD], qf[p][b < QR ? b : 0]);
          else if (b < QR) mfma16_add<false>(c, kf[b % AHEAD], qf[p][b < QR ? b : 0]);
          else mfma16_add<false>(c, kf[b % AHEAD], __builtin_bit_cast(u32x4, ql[p]));
        }
        if (b + AHEAD < NB) kf[b % AHEAD] = key(b + AHEAD);
        if (b + 2 >= QR && b + 2 < NB)
#pragma unroll
          for (int p = 0; p < PT; ++p) ql[p] = *reinterpret_cast<const Frag*>(qs + (b + 2 - QR) * (NP * 32) + q_at(p));
        in_order();
      }
    }
    scores_done(s[0], s[1]);
    if constexpr (PT == 1) s[0] += s[1];
    const bool masked = j * KT + KT - 1 > first_last;
#pragma unroll
    for (int p = 0; p < PT; ++p) {
      s[p] *= scale2;
      if (masked) {
        asm volatile("" : "+v"(s[p]));                  // (a branch, not selects in every tile)
        const int after = posq[p] - (j * KT + kb + lc * 4);
#pragma unroll
        for (int r = 0; r < 4; ++r) s[p][r] = r > after ? -INFINITY : s[p][r];
      }
      float top = fmaxf(fmaxf(s[p][0], s[p][1]), fmaxf(s[p][2], s[p][3]));
      top = over_row_groups(top, [](float a, float b) { return fmaxf(a, b); });
      if (lc == 0) mx[group * NP + pb + p * 16 + li] = top;
    }
    lds_barrier();
    // a pair's reference moves by the same rule, from the same maxima, wherever it is kept
    auto top_of = [&](int pair) {
      float t = mx[pair];
#pragma unroll
      for (int g = 1; g < NG; ++g) t = fmaxf(t, mx[g * NP + pair]);
      return t;
    };
#pragma unroll
    for (int p = 0; p < PT; ++p) {
      const float t = top_of(pb + p * 16 + li), mn = t > m[p] + RISE ? t : m[p];
      l[p] *= __builtin_amdgcn_exp2f(m[p] - mn);
      m[p] = mn;
    }
#pragma unroll
    for (int t = 0; t < PT; ++t) {
      const float top = top_of(t * 32 + l32);
      const bool rise = top > mo[t] + RISE;
      if (__any(rise)) {
        const float mn = rise ? top : mo[t], f = __builtin_amdgcn_exp2f(mo[t] - mn);
        mo[t] = mn;
#pragma unroll
        for (int v = 0; v < NV; ++v)
#pragma unroll
          for (int r = 0; r < 16; ++r) o[v][t][r] *= f;
      }
    }
    // weights
#pragma unroll
    for (int p = 0; p < PT; ++p) {
      float w[4];
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        w[r] = __builtin_amdgcn_exp2f(s[p][r] - m[p]);
        l[p] += w[r];
      }
      uint2 pk;
      pk.x = pack_bf16x2(w[0], w[1]);
      pk.y = pack_bf16x2(w[2], w[3]);
      *reinterpret_cast<uint2*>(ps + (pb + p * 16 + li) * PROW + kb + lc * 4) = pk;
    }
    lds_barrier();
    // values: steps of one block of value elements over 16 keys, the weights of 16 keys shared by the blocks
    if (RT >= NW || wave < RT) {
      constexpr int K = KT / 16, N = K * NV, AHEAD = NB > 10 && PT == 2 ? 2 : 4;
      Frag vf[AHEAD], pf[2][PT];
      auto weights = [&](int k) {
#pragma unroll
        for (int t = 0; t < PT; ++t)
          pf[k % 2][t] = *reinterpret_cast<const Frag*>(ps + (t * 32 + l32) * PROW + k * 16 + hh * 8);
      };
      auto value = [&](int i) {
        const bf16_t* base = cur + (wave + NW * (i % NV)) * (KT * 32) + (i / NV) * (16 * 32);
        const uint2 a = __builtin_bit_cast(uint2, __builtin_amdgcn_ds_read_tr16_b64_v4i16((lds_s16x4)(base + v_at0)));
        const uint2 b = __builtin_bit_cast(uint2, __builtin_amdgcn_ds_read_tr16_b64_v4i16((lds_s16x4)(base + v_at1)));
        Frag f;
        f.w[0] = a.x; f.w[1] = a.y; f.w[2] = b.x; f.w[3] = b.y;
        return f;
      };
      weights(0);
#pragma unroll
      for (int i = 0; i < AHEAD; ++i) vf[i] = value(i);
      in_order();
#pragma unroll
      for (int i = 0; i < N; ++i) {
        const int k = i / NV, v = i % NV;
        if (v == 0 && k + 1 < K) weights(k + 1);
#pragma unroll
        for (int t = 0; t < PT; ++t) o[v][t] = mfma32(vf[i % AHEAD], pf[k % 2][t], o[v][t]);
        if (i + AHEAD < N) vf[i % AHEAD] = value(i + AHEAD);
        in_order();
      }
    }
    loads_barrier();
  }
  // sums of the pairs' weights over all their keys
#pragma unroll
  for (int p = 0; p < PT; ++p) {
    l[p] = over_row_groups(l[p], [](float a, float b) { return a + b; });
    if (lc == 0) mx[group * NP + pb + p * 16 + li] = l[p];
  }
  lds_barrier();
#pragma unroll
  for (int t = 0; t < PT; ++t) {
    const int pair = pair0 + t * 32 + l32;
    float sum = mx[t * 32 + l32];
#pragma unroll
    for (int g = 1; g < NG; ++g) sum += mx[g * NP + t * 32 + l32];
    if (pair >= n_pairs) continue;
    const size_t gp = (size_t)row0 * H + pair;
    if (n_splits > 1) {
      if (wave == 0 && hh == 0) {
        ml[(gp * n_splits + split) * 2] = mo[t];
        ml[(gp * n_splits + split) * 2 + 1] = sum;
      }
      if (j0 >= j1) continue;
      float* dst = parts + (gp * n_splits + split) * R;
#pragma unroll
      for (int v = 0; v < NV; ++v)
#pragma unroll
        for (int k = 0; k < 4; ++k) {
          const int r = (wave + NW * v) * 32 + k * 8 + hh * 4;
          if (r < R) *reinterpret_cast<floatx4*>(dst + r) =
              floatx4{o[v][t][k * 4], o[v][t][k * 4 + 1], o[v][t][k * 4 + 2], o[v][t][k * 4 + 3]};
        }
    } else {
      // through LDS, so that a wave writes whole rows
      const float inv = 1.0f / sum;
      bf16_t* dst = bufs + (t * 32 + l32) * (R + 8);
#pragma unroll
      for (int v = 0; v < NV; ++v)
#pragma unroll
        for (int k = 0; k < 4; ++k) {
          const int r = (wave + NW * v) * 32 + k * 8 + hh * 4;
          if (r >= R) continue;
          uint2 pk;
          pk.x = pack_bf16x2(o[v][t][k * 4] * inv, o[v][t][k * 4 + 1] * inv);
          pk.y = pack_bf16x2(o[v][t][k * 4 + 2] * inv, o[v][t][k * 4 + 3] * inv);
          *reinterpret_cast<uint2*>(dst + r) = pk;
        }
    }
  }
  if (n_splits > 1) return;
  lds_barrier();
  for (int pair = wave; pair < min(NP, n_pairs - pair0); pair += NW)
    for (int r = lane * 8; r < R; r += WAVE * 8)
      *reinterpret_cast<Frag*>(out + ((size_t)row0 * H + pair0 + pair) * R + r) =
          *reinterpret_cast<const Frag*>(bufs + pair * (R + 8) + r);
}

// a block: one pair of an item; 4 value elements a thread.  The ranges' factors are made once, by the first wave.
constexpr int SPLITS_MAX = 256, SPLITS_LANE = SPLITS_MAX / WAVE;
__global__ __launch_bounds__(128) void latent_merge_kernel(const float* __restrict__ parts, const float* __restrict__ ml,
                                                           int n_splits, int H, int R, LatentItems items,
                                                           bf16_t* __restrict__ out) {
  __shared__ float factor[SPLITS_MAX];
  const int item = blockIdx.x / items.blocks, pair = blockIdx.x % items.blocks;
  if (pair >= (items.rows ? items.rows[item] : 1) * H) return;
  const size_t gp = (size_t)(items.row0 ? items.row0[item] : item) * H + pair;
  if (threadIdx.x < WAVE) {
    float m[SPLITS_LANE], l[SPLITS_LANE], top = NO_KEY, sum = 0.f;
#pragma unroll
    for (int k = 0; k < SPLITS_LANE; ++k) {
      const int s = threadIdx.x + k * WAVE;
      m[k] = s < n_splits ? ml[(gp * n_splits + s) * 2] : NO_KEY;
      l[k] = s < n_splits ? ml[(gp * n_splits + s) * 2 + 1] : 0.f;
      if (l[k] > 0.f) top = fmaxf(top, m[k]);
    }
    top = wave_max(top);
#pragma unroll
    for (int k = 0; k < SPLITS_LANE; ++k) {
      m[k] = l[k] > 0.f ? __builtin_amdgcn_exp2f(m[k] - top) : 0.f;        // a range without a key of this pair: 0
      sum = fmaf(l[k], m[k], sum);
    }
    sum = wave_sum(sum);
#pragma unroll
    for (int k = 0; k < SPLITS_LANE; ++k) factor[threadIdx.x + k * WAVE] = m[k] / sum;
  }
  __syncthreads();
  const float* src = parts + gp * n_splits * R;
  for (int r = threadIdx.x * 4; r < R; r += 512) {
    floatx4 acc = floatx4{0.f, 0.f, 0.f, 0.f};
    for (int s0 = 0; s0 < n_splits; s0 += 8) {
      floatx4 v[8];
#pragma unroll
      for (int k = 0; k < 8; ++k) v[k] = *reinterpret_cast<const floatx4*>(src + (size_t)min(s0 + k, n_splits - 1) * R + r);
#pragma unroll
      for (int k = 0; k < 8; ++k) {
        const float f = s0 + k < n_splits ? factor[s0 + k] : 0.f;
#pragma unroll
        for (int e = 0; e < 4; ++e) acc[e] = f != 0.f ? fmaf(f, v[k][e], acc[e]) : acc[e];    // (0: nothing was left)
      }
    }
    uint2 pk;
    pk.x = pack_bf16x2(acc[0], acc[1]);
    pk.y = pack_bf16x2(acc[2], acc[3]);
    *reinterpret_cast<uint2*>(out + gp * R + r) = pk;
  }
}

// the smallest kernel whose value blocks hold R elements and whose row blocks hold R + dr; 0: none
int value_blocks(int R, int L) {
  for (int rt = 2; rt <= 16; rt *= 2)
    if (R <= rt * 32 && L <= (rt + 2) * 32) return rt;
  return 0;
}

}  // namespace

APC_EXPORT int apc_latent_attention_takes(int H, int R, int dr, int page_tokens) {
  return (H > 0 && R > 0 && dr >= 0 && R % 8 == 0 && dr % 8 == 0 && value_blocks(R, R + dr) && page_tokens > 0 &&
          (page_tokens & (page_tokens - 1)) == 0) ? 1 : 0;
}

// Items (row0 [n_items], rows [n_items] or null for single rows; max_rows: the most rows of one) of consecutive rows of
// one request.  q [T][H * (R + dr)] and out [T][H * R] contiguous.  n_splits > 1: parts float32 [T * H][n_splits][R] and
// ml float32 [T * H][n_splits][2].
APC_EXPORT int apc_latent_attention_bf16(const void* q, void* out, int H, int R, int dr, const void* pages,
                                         int page_tokens, const int* block_table, int max_blocks, const int* positions,
                                         const int* row_seg, const int* row0, const int* rows, int n_items, int max_rows,
                                         int n_splits, float* parts, float* ml, float scale, hipStream_t stream) {
  if (n_items <= 0) return 0;
  if (!apc_latent_attention_takes(H, R, dr, page_tokens)) return APC_ERR_UNSUPPORTED;
  if (max_blocks <= 0 || max_rows <= 0 || n_splits < 1 || n_splits > SPLITS_MAX ||
      (n_splits > 1 && (!parts || !ml)) || (max_rows > 1 && !rows) || ((uintptr_t)q & 15u) || ((uintptr_t)out & 15u) ||
      ((uintptr_t)pages & 15u) || ((uintptr_t)parts & 15u))
    return APC_ERR_BAD_ARG;
  const int L = R + dr, rt = value_blocks(R, L), pairs = max_rows * H;
  const int two = pairs > 32 ? 1 : 0;
  const int blocks = ceil_div(pairs, two ? 64 : 32);
  if ((long)blocks * n_items * n_splits > 0x7fffffffL || (long)pairs * n_items > 0x7fffffffL) return APC_ERR_UNSUPPORTED;
  const LatentItems items{row0, rows, n_items, blocks};
  const int pshift = __builtin_ctz(page_tokens);
#define LATENT_LAUNCH(RT_, PT_, EVEN_)                                                                                \
  hipLaunchKernelGGL((latent_attention_kernel<RT_, RT_ + 2, PT_, EVEN_>), dim3(blocks * n_items * n_splits), dim3(NT), \
                     0, stream, (const bf16_t*)q, (bf16_t*)out, H, R, L, (const bf16_t*)pages, pshift, block_table,    \
                     max_blocks, positions, row_seg, items, n_splits, scale * LOG2E, parts, ml)
#define LATENT_BY(RT_)                                           \
  do {                                                           \
    if (two && L == (RT_ + 2) * 32) LATENT_LAUNCH(RT_, 2, true); \
    else if (two) LATENT_LAUNCH(RT_, 2, false);                  \
    else if (L == (RT_ + 2) * 32) LATENT_LAUNCH(RT_, 1, true);   \
    else LATENT_LAUNCH(RT_, 1, false);                           \
  } while (0)
  if (rt == 2) LATENT_BY(2);
  else if (rt == 4) LATENT_BY(4);
  else if (rt == 8) LATENT_BY(8);
  else LATENT_BY(16);
#undef LATENT_BY
#undef LATENT_LAUNCH
  APC_LAUNCH_CHECK();
  if (n_splits > 1) {
    const LatentItems per_pair{row0, rows, n_items, pairs};
    hipLaunchKernelGGL(latent_merge_kernel, dim3(pairs * n_items), dim3(128), 0, stream, parts, ml, n_splits, H, R,
                       per_pair, (bf16_t*)out);
    APC_LAUNCH_CHECK();
  }
  return 0;
}
