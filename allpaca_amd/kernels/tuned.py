"""Checked wrappers of the bfloat16 MFMA kernels (library `tuned`).  Each checks what the kernel
assumes.  Matrix products take weights in the tiled layout (`packing.PackedWeight`), which only
matrices of a width that is a multiple of 8 get (`ops.prepare_matrix`): other widths stay row-major
and run on the plain kernel.  Attention returns False for sizes it does not take (a page size that is
no multiple of 8, a head size that is no multiple of 16 or above 256) and the caller runs the plain
kernel: never a wrong result."""
from __future__ import annotations

import math
from typing import Optional

import torch

from . import lib as _lib
from . import ops as _ops
from .packing import PackedWeight

MANY_ROWS_SPLIT_MAX = 1024   # up to here the tiled kernel may cut K into slices to get enough blocks
SKINNY_MAX_ROWS = 16     # the streaming kernel: up to one 16-row tile of activations
SPLITK_MAX_ROWS = 128    # the tiled kernel with K cut into slices: 17..128 rows


def _k_split(M: int, N: int, K: int) -> int:
    """Slices of K for the split kernel with 17..128 rows: about 240 blocks in all (measured best at the shapes of 3B
    and 8B models: 32 column tiles in 6-8 slices, 48 in 4-5, 224 whole), at least 4 K-steps of 64 each."""
    blocks = -(-N // 128) * -(-M // 128)
    s = max(1, min(12, round(240 / blocks)))
    return max(1, min(s, K // 256))


def _k_split_many_rows(M: int, N: int, K: int) -> int:
    """Slices of K for 129..1024 rows: a matrix with few output columns gives the 128 x 128 tiles too few blocks
    for 256 compute units (o_proj and down of an 8B model at 512 rows: 128), and slicing K, at the price of writing
    and adding float32 partial sums, was measured faster up to about 200 blocks (down, 4096 x 14336, 256 rows: 150
    us whole, 52 us in 4 slices); with more outputs than K and 150 blocks or more it was not."""
    blocks = -(-N // 128) * -(-M // 128)
    if blocks <= 56:
        s = 5
    elif blocks <= 68:
        s = 4
    elif blocks <= 88:
        s = 3
    elif blocks <= 208 and not (blocks >= 150 and N > K):
        s = 2
    else:
        s = 1
    return max(1, min(s, K // 256))


def _tiled_k_split(M: int, N: int, K: int) -> int:
    """Slices of K on the tiled kernel for M rows (1: K in one piece)."""
    if M <= SPLITK_MAX_ROWS:
        return _k_split(M, N, K)
    return _k_split_many_rows(M, N, K) if M <= MANY_ROWS_SPLIT_MAX else 1


# The chip these rules and the kernels' launch plans were measured on (`csrc/host/rules.h`, `gemm_direct_bf16.hip`:
# rounds of 256 blocks over 8 XCDs; `attention_wide_bf16.hip`: 160 KiB of LDS a compute unit).
CHIP_UNITS = 256
CHIP_LDS_BYTES = 160 * 1024
_chips_checked: set = set()


def check_chip(device: torch.device) -> None:
    """Says so, once per device, if the GPU is not the one the dispatch rules were measured on: the results stay
    right (no kernel assumes the counts for correctness), the cuts may be badly chosen."""
    import warnings
    key = (device.type, device.index)
    if device.type != "cuda" or key in _chips_checked:
        return
    _chips_checked.add(key)
    prop = torch.cuda.get_device_properties(device)
    units = getattr(prop, "multi_processor_count", CHIP_UNITS)
    lds = getattr(prop, "shared_memory_per_block_optin", 0) or getattr(prop, "shared_memory_per_block", 0)
    if units != CHIP_UNITS or (lds and lds < CHIP_LDS_BYTES):
        warnings.warn(f"{prop.name}: {units} compute units and {lds} bytes of LDS a block; the bfloat16 kernels' dispatch "
                      f"rules were measured on {CHIP_UNITS} units with {CHIP_LDS_BYTES} bytes and may be badly tuned here")


def _aligned(*ts: torch.Tensor) -> bool:
    return all(t.data_ptr() % 16 == 0 for t in ts)


def _act_ok(a: torch.Tensor) -> bool:
    return (a.dtype == torch.bfloat16 and a.shape[1] % 8 == 0 and _ops._rows(a, "a") % 8 == 0 and _aligned(a))


MODE_ACT = 16     # the products' modes from here on: an activation (MODE_ACT + its code) on the sums, bfloat16 out


def gemm_bf16(a: torch.Tensor, w: PackedWeight, out: torch.Tensor, accumulate: bool = False, activation: int = 0) -> None:
    """out = a . w^T (bfloat16 or float32 out), or out += a . w^T (float32 out); w in the tiled layout.  `activation`
    (a code of `ops.ACTIVATIONS`): out = act(a . w^T), applied to the float32 sums, bfloat16 out."""
    _ops._gpu(a, w.data, out)
    M, K = a.shape
    N = w.N
    if not (w.K == K):
        raise ValueError(f"gemm: a is [*, {K}] but w is {w.shape}")
    if not (out.shape == (M, N)):
        raise ValueError(f"gemm: out must be [{M}, {N}], got {tuple(out.shape)}")
    _ops._need(not accumulate or out.dtype == torch.float32, "gemm: accumulation needs a float32 destination")
    _ops._need(out.dtype in (torch.bfloat16, torch.float32), "gemm: out must be bfloat16 or float32")
    _ops._need(not activation or (not accumulate and out.dtype == torch.bfloat16), "gemm: an activation stores bfloat16")
    _ops._need(w.data.is_contiguous() and w.data.shape[0] * 16 >= N and w.data.shape[1] * 32 >= K,
               "gemm: the tiled weight does not cover [N, K]")
    if not _act_ok(a):
        raise ValueError("gemm_bf16: activations must be bfloat16 rows of a width and stride that are multiples "
                         "of 8, 16-byte aligned")
    lda, ldc = _ops._rows(a, "a"), _ops._rows(out, "out")
    mode = MODE_ACT + activation if activation else 2 if accumulate else (0 if out.dtype == torch.bfloat16 else 1)
    L = _lib.load("tuned")
    if M > SKINNY_MAX_ROWS:
        # more than 1,024 rows: the product of many rows says itself whether it wants K in two slices
        ks = _tiled_k_split(M, N, K) if M <= MANY_ROWS_SPLIT_MAX else L.apc_gemm_direct_k_split(M, N, K)
        if ks > 1:
            ws = torch.empty(ks * M * N, dtype=torch.float32, device=a.device)
            _lib.check(L.apc_gemm_splitk_bf16(a.data_ptr(), lda, w.data.data_ptr(), 0, out.data_ptr(), ldc, M, N, K,
                                              mode, ks, ws.data_ptr(), _ops._stream()), "gemm_splitk_bf16")
            return
    fn = L.apc_skinny_gemm_bf16 if M <= SKINNY_MAX_ROWS else L.apc_gemm_bf16
    _lib.check(fn(a.data_ptr(), lda, w.data.data_ptr(), out.data_ptr(), ldc, M, N, K, mode, _ops._stream()),
               "gemm_bf16")


def swiglu_bf16(h: torch.Tensor, wg: PackedWeight, wu: PackedWeight, out: torch.Tensor) -> None:
    """out[t, f] = silu(h . Wg[f]) * (h . Wu[f]); Wg, Wu in the tiled layout."""
    _ops._gpu(h, wg.data, wu.data, out)
    M, K = h.shape
    F = out.shape[1]
    if not (wg.shape == (F, K) and wu.shape == (F, K)):
        raise ValueError(f"swiglu: weights must both be [{F}, {K}]")
    _ops._need(out.shape[0] == M and out.dtype == torch.bfloat16, "swiglu: out must be bfloat16 [rows, F]")
    if not _act_ok(h):
        raise ValueError("swiglu_bf16: activations must be bfloat16 rows of a width and stride that are multiples "
                         "of 8, 16-byte aligned")
    lda, ldc = _ops._rows(h, "h"), _ops._rows(out, "out")
    L = _lib.load("tuned")
    ks = _tiled_k_split(M, 2 * F, K) if M > SKINNY_MAX_ROWS else 1
    if ks > 1:
        ws = torch.empty(2 * ks * M * F, dtype=torch.float32, device=h.device)
        _lib.check(L.apc_gemm_splitk_bf16(h.data_ptr(), lda, wg.data.data_ptr(), wu.data.data_ptr(), out.data_ptr(), ldc,
                                          M, F, K, 3, ks, ws.data_ptr(), _ops._stream()), "gemm_splitk_bf16")
        return
    fn = L.apc_skinny_swiglu_bf16 if M <= SKINNY_MAX_ROWS else L.apc_gemm_swiglu_bf16
    _lib.check(fn(h.data_ptr(), lda, wg.data.data_ptr(), wu.data.data_ptr(), out.data_ptr(), ldc, M, F, K,
                  _ops._stream()), "swiglu_bf16")


def gemm_emit_bf16(a: torch.Tensor, w: PackedWeight, residual: torch.Tensor, g: torch.Tensor):
    """residual += a . w^T, and for the RMS norm with weight g that reads the residual next: the row
    bfloat16(residual * g) and sums of residual^2 per row and group of columns.  Returns (raw [M, N], ss) or None,
    with nothing done, for sizes no kernel takes.  ss is [16, ceil(N/16) rounded up to 4] from the streaming kernel
    (up to 16 rows) and [M, ceil(N/256)] from the tiled kernel with K in slices; the products below take what the
    same number of rows gives."""
    _ops._gpu(a, w.data, residual, g)
    M, K = a.shape
    N = w.N
    if (not _act_ok(a) or residual.dtype != torch.float32 or g.dtype != torch.float32 or g.numel() != N
            or not g.is_contiguous()):
        return None
    if not (w.K == K and residual.shape == (M, N)):
        raise ValueError(f"gemm: a [{M}, {K}], w {w.shape}, residual {tuple(residual.shape)}")
    L = _lib.load("tuned")
    lda, ldc = _ops._rows(a, "a"), _ops._rows(residual, "residual")
    if M > MANY_ROWS_SPLIT_MAX:
        # the product of many rows: its own epilogue leaves the row, or with K in two slices the kernel that adds them
        # (sums of squares per tile of columns, or per 1,024 columns)
        parts = L.apc_gemm_direct_emit_parts(a.data_ptr(), lda, residual.data_ptr(), ldc, M, N, K)
        if not parts:
            return None
        raw = torch.empty((M, N), dtype=torch.bfloat16, device=a.device)
        ss = torch.empty((M, parts), dtype=torch.float32, device=a.device)
        ks = L.apc_gemm_direct_k_split(M, N, K)
        ws = torch.empty(ks * M * N, dtype=torch.float32, device=a.device) if ks > 1 else None
        _lib.check(L.apc_gemm_direct_emit_bf16(a.data_ptr(), lda, w.data.data_ptr(), residual.data_ptr(), ldc, M, N, K,
                                               g.data_ptr(), raw.data_ptr(), N, ss.data_ptr(), parts,
                                               ws.data_ptr() if ws is not None else 0, _ops._stream()),
                   "gemm_direct_emit_bf16")
        return raw, ss
    if M > SKINNY_MAX_ROWS:   # the tiled kernel: only where K is cut into slices (the finishing kernel leaves the row)
        ks = _tiled_k_split(M, N, K)
        if ks == 1:
            # With K in one piece the product's own epilogue would have to do it; measured at 2,048 rows that costs
            # 20-27 us a product, more than the norm's kernel (10 us) that it would save.
            return None
        raw = torch.empty((M, N), dtype=torch.bfloat16, device=a.device)
        ss = torch.empty((M, -(-N // 256)), dtype=torch.float32, device=a.device)
        ws = torch.empty(ks * M * N, dtype=torch.float32, device=a.device)
        _lib.check(L.apc_gemm_splitk_emit_bf16(a.data_ptr(), lda, w.data.data_ptr(), residual.data_ptr(), ldc, M, N, K,
                                               ks, ws.data_ptr(), g.data_ptr(), raw.data_ptr(), N, ss.data_ptr(),
                                               _ops._stream()), "gemm_splitk_emit_bf16")
        return raw, ss
    raw = torch.empty((M, N), dtype=torch.bfloat16, device=a.device)
    ss = torch.empty((16, -(-(-(-N // 16)) // 4) * 4), dtype=torch.float32, device=a.device)
    _lib.check(L.apc_skinny_gemm_emit_bf16(a.data_ptr(), lda, w.data.data_ptr(), residual.data_ptr(), ldc, M, N, K,
                                           g.data_ptr(), raw.data_ptr(), N, ss.data_ptr(), _ops._stream()),
               "skinny_gemm_emit_bf16")
    return raw, ss


def _pre_ok(raw: torch.Tensor, ss: torch.Tensor, K: int) -> bool:
    return (raw.shape[0] <= SKINNY_MAX_ROWS and _act_ok(raw) and ss.dtype == torch.float32 and ss.is_contiguous()
            and tuple(ss.shape) == (16, -(-(-(-K // 16)) // 4) * 4))


def _pre_tiled(raw: torch.Tensor, ss: torch.Tensor, eps: float, w, wu, out: torch.Tensor, n_cols: int, mode: int) -> bool:
    """The same on the tiled kernel (more than 16 rows), K in slices or in one piece: ss is [M, parts] with up to
    256 sums of squares a row (what the tiled kernels leave: a part per 256 or per 128 columns)."""
    M, K = raw.shape
    if not (M > SKINNY_MAX_ROWS and _act_ok(raw) and ss.dtype == torch.float32 and ss.is_contiguous()
            and ss.dim() == 2 and ss.shape[0] == M and 1 <= ss.shape[1] <= 256):
        return False
    n_mats = 2 if wu is not None else 1
    ks = _tiled_k_split(M, n_cols * n_mats, K)
    L = _lib.load("tuned")
    wu_ptr = wu.data.data_ptr() if wu is not None else 0
    if ks == 1:
        _lib.check(L.apc_gemm_pre_bf16(raw.data_ptr(), _ops._rows(raw, "raw"), ss.data_ptr(), ss.shape[1], float(eps),
                                       w.data.data_ptr(), wu_ptr, out.data_ptr(), _ops._rows(out, "out"), M, n_cols, K,
                                       mode, _ops._stream()), "gemm_pre_bf16")
        return True
    ws = torch.empty(n_mats * ks * M * n_cols, dtype=torch.float32, device=raw.device)
    _lib.check(L.apc_gemm_splitk_pre_bf16(raw.data_ptr(), _ops._rows(raw, "raw"), ss.data_ptr(), ss.shape[1], float(eps),
                                          w.data.data_ptr(), wu_ptr, out.data_ptr(), _ops._rows(out, "out"), M, n_cols,
                                          K, mode, ks, ws.data_ptr(), _ops._stream()), "gemm_splitk_pre_bf16")
    return True


def gemm_pre_bf16(raw: torch.Tensor, ss: torch.Tensor, eps: float, w: PackedWeight, out: torch.Tensor) -> bool:
    """out = (raw . w^T) / sqrt(sum(ss) / K + eps) for a row that `gemm_emit_bf16` left: the product of the
    normalised row.  False, with nothing done, for sizes the kernel does not take."""
    _ops._gpu(raw, ss, w.data, out)
    M, K = raw.shape
    if out.dtype not in (torch.bfloat16, torch.float32):
        return False
    if not (w.K == K and out.shape == (M, w.N)):
        raise ValueError(f"gemm: raw [{M}, {K}], w {w.shape}, out {tuple(out.shape)}")
    if M > SKINNY_MAX_ROWS:
        return _pre_tiled(raw, ss, eps, w, None, out, w.N, 0 if out.dtype == torch.bfloat16 else 1)
    if not _pre_ok(raw, ss, K):
        return False
    L = _lib.load("tuned")
    _lib.check(L.apc_skinny_gemm_pre_bf16(raw.data_ptr(), _ops._rows(raw, "raw"), ss.data_ptr(), -(-K // 16), float(eps),
                                          w.data.data_ptr(), out.data_ptr(), _ops._rows(out, "out"), M, w.N, K,
                                          0 if out.dtype == torch.bfloat16 else 1, _ops._stream()),
               "skinny_gemm_pre_bf16")
    return True


def qkv_rope_bf16(a: torch.Tensor, pre, w: PackedWeight, q_out: torch.Tensor, n_heads: int, n_kv_heads: int,
                  head_dim: int, cos_sin: torch.Tensor, positions: torch.Tensor, row_seg: torch.Tensor,
                  block_table: torch.Tensor, cache: torch.Tensor, page_tokens: int) -> bool:
    """q, k, v in one product that also rotates q and k (whole heads) and writes k and v into the pages; rotated q
    goes to the first n_heads * head_dim columns of q_out.  Up to 16 rows: the streaming kernel (head size a
    multiple of 32); more rows: the tiled kernel where it cuts K into slices, in its finishing kernel (256 a
    multiple of the head size).  `a`: the normalised rows, or with `pre` = (ss, eps) the row that
    `gemm_emit_bf16` left.  False, with nothing done, for sizes neither takes."""
    _ops._gpu(a, w.data, q_out, cos_sin, positions, row_seg, block_table, cache)
    M, K = a.shape
    H, Hk, d = n_heads, n_kv_heads, head_dim
    N = (H + 2 * Hk) * d
    few = M <= SKINNY_MAX_ROWS
    if not (_act_ok(a) and q_out.dtype == torch.bfloat16 and cache.dtype == torch.bfloat16):
        return False
    if few and not (d % 32 == 0 and q_out.stride(0) % 4 == 0 and q_out.data_ptr() % 8 == 0):
        return False
    ks = 1 if few else _tiled_k_split(M, N, K)
    if not few and (ks == 1 or 256 % d or d % 2):
        return False
    ss, eps = None, 0.0
    if pre is not None:
        ss, eps = pre
        if few and not _pre_ok(a, ss, K):
            return False
        if not few and not (ss.dtype == torch.float32 and ss.is_contiguous() and ss.dim() == 2 and ss.shape[0] == M
                            and 1 <= ss.shape[1] <= 256):
            return False
    if not (w.K == K and w.N == N and q_out.shape[0] == M and q_out.shape[1] >= H * d):
        raise ValueError(f"qkv: a [{M}, {K}], w {w.shape}, {H}+2*{Hk} heads of {d}, q_out {tuple(q_out.shape)}")
    _ops._need(cos_sin.dtype == torch.float32 and cos_sin.is_contiguous() and tuple(cos_sin.shape[1:]) == (2, d // 2),
               "cos/sin table must be float32 [positions, 2, head_dim/2]")
    if not (cache.dim() == 5 and cache.is_contiguous() and tuple(cache.shape[1:]) == (2, Hk, page_tokens, d)):
        raise ValueError(f"cache must be [pages, 2, {Hk}, {page_tokens}, {d}], got {tuple(cache.shape)}")
    _ops._need(block_table.dim() == 2 and block_table.dtype == torch.int32 and block_table.is_contiguous(),
               "block table must be contiguous int32 [segments, blocks]")
    L = _lib.load("tuned")
    ss_ptr = ss.data_ptr() if ss is not None else 0
    if few:
        _lib.check(L.apc_skinny_qkv_rope_bf16(
            a.data_ptr(), _ops._rows(a, "a"), ss_ptr, -(-K // 16) if ss is not None else 0, float(eps), w.data.data_ptr(),
            q_out.data_ptr(), _ops._rows(q_out, "q_out"), M, K, H, Hk, d, cos_sin.data_ptr(),
            _ops._i32(positions, M, "positions"), _ops._i32(row_seg, M, "row_seg"), block_table.data_ptr(),
            block_table.shape[1], cache.data_ptr(), page_tokens, _ops._stream()), "skinny_qkv_rope_bf16")
        return True
    ws = torch.empty(ks * M * N, dtype=torch.float32, device=a.device)
    _lib.check(L.apc_gemm_splitk_qkv_rope_bf16(
        a.data_ptr(), _ops._rows(a, "a"), ss_ptr, ss.shape[1] if ss is not None else 0, float(eps), w.data.data_ptr(),
        q_out.data_ptr(), _ops._rows(q_out, "q_out"), M, K, H, Hk, d, cos_sin.data_ptr(),
        _ops._i32(positions, M, "positions"), _ops._i32(row_seg, M, "row_seg"), block_table.data_ptr(),
        block_table.shape[1], cache.data_ptr(), page_tokens, ks, ws.data_ptr(), _ops._stream()),
        "gemm_splitk_qkv_rope_bf16")
    return True


def swiglu_pre_bf16(raw: torch.Tensor, ss: torch.Tensor, eps: float, wg: PackedWeight, wu: PackedWeight,
                    out: torch.Tensor) -> bool:
    """SwiGLU of the normalised row, from what `gemm_emit_bf16` left (see `gemm_pre_bf16`)."""
    _ops._gpu(raw, ss, wg.data, wu.data, out)
    M, K = raw.shape
    F = out.shape[1]
    if out.dtype != torch.bfloat16:
        return False
    if not (wg.shape == (F, K) and wu.shape == (F, K) and out.shape[0] == M):
        raise ValueError(f"swiglu: weights must both be [{F}, {K}]")
    if M > SKINNY_MAX_ROWS:
        return _pre_tiled(raw, ss, eps, wg, wu, out, F, 3)
    if not _pre_ok(raw, ss, K):
        return False
    L = _lib.load("tuned")
    _lib.check(L.apc_skinny_swiglu_pre_bf16(raw.data_ptr(), _ops._rows(raw, "raw"), ss.data_ptr(), -(-K // 16),
                                            float(eps), wg.data.data_ptr(), wu.data.data_ptr(), out.data_ptr(),
                                            _ops._rows(out, "out"), M, F, K, _ops._stream()), "skinny_swiglu_pre_bf16")
    return True


def _decode_parts(pairs: int, span: int) -> int:
    """Ranges that the decode kernel cuts the keys of every row into (four to a block, one per wave): as many blocks
    a (row, kv head) pair as keep the launch at one block a compute unit or under, and no range under 64 keys.  The
    kernel sizes a row's ranges from the row's own length, so the count depends on the step's shape alone.  Measured at
    8B shapes (32 heads over 8, heads of 128), 1 to 16 rows over 512 to 8,192 keys, ranges of 64 to 512 keys: the
    fastest choice was in every case the shortest range whose launch fits the chip once (8 rows over 2,063 keys: 256
    blocks 18.9 us, 320 blocks 21.4 us, 192 blocks 20.6 us; over 8,192 keys: 256 blocks 53.3 us, 512 blocks 54.6 us,
    1,024 blocks 56.5 us)."""
    per_pair = max(1, CHIP_UNITS // max(1, pairs))
    return max(1, min(WHOLE_WAVES * per_pair, -(-span // 64)))


# Keys of a range of the decode kernel, the same for every row and counted from position 0, instead of the rule above
# (0: the rule): for measurements and tests.
KEYS_PER_PART = 0


# From how many (row, kv head) pairs on a decode step's attention runs as one block per pair that finishes its heads
# itself (no partial results through memory, no second kernel): the pairs alone then give every compute unit work
# (measured at the shapes of an 8B model: 7-15 % faster from 32 rows on, slower with 16).
WHOLE_MIN_PAIRS = 256
WHOLE_WAVES = 4   # waves of such a block (NW in attention_bf16.hip)


# With fewer pairs: the blocks of a pair leave one partial result each and the one that finishes last adds them (no
# second kernel), where the sizes allow; False: partial results per wave and a kernel that merges them.
LAST_BLOCK_MERGES = True
# Portions whose tiles of 128 rows are mostly whole (heads of 128 or 64, pages of a power of two from 16 on) run on the kernel
# that takes such a tile a block (attention_wide_bf16.hip); False sends every portion to the kernels of 64-row blocks.
WIDE_TILES = True
_counters: dict = {}
# Ranges that the keys of a tile of prompt rows are cut into: never more (0 sends a tile's keys to one block always),
# and the keys a range must keep
KEY_SPLITS_MAX = 8
KEY_RANGE_MIN = 2048


def _key_splits(step, n_heads: int, window: int) -> int:
    """Into how many ranges of keys the 128-row attention kernel cuts every tile of this step: a block per (tile, head)
    leaves compute units idle when a step has few tiles (a chunk of 512 prompt tokens at 32 heads: 128 blocks for 256
    units), so the keys are shared out until the chip has a block a unit, as long as a range keeps KEY_RANGE_MIN keys
    (measured at 8B shapes, 512 rows: 1.2 times as fast at 4,096 keys, 1.56 at 32,768, a loss at 2,048: a block's
    start and the kernel that adds the ranges cost a few tiles of 64 keys), or half as many while the chip stays at
    most half full (a block alone on its compute unit and its neighbours' runs at the pace of its own chain of loads:
    128 rows over 2,048 keys in 2 ranges 1.27 times as fast, over 4,096 keys in 4 ranges 1.9 times).  1: no cutting."""
    blocks = step.n_tiles * n_heads
    pos0 = getattr(step, "host_pos0", None)
    rows = getattr(step, "host_rows", None)
    if not KEY_SPLITS_MAX or blocks <= 0 or not pos0 or not rows:
        return 1
    keys = max([p + n for p, n in zip(pos0, rows) if n > 1] or [0])     # of the longest prompt in the step
    if window:
        keys = min(keys, window + 128)
    few = min(keys // max(1, KEY_RANGE_MIN // 2), 128 // blocks)
    return max(1, min(KEY_SPLITS_MAX, 256 // blocks, max(keys // KEY_RANGE_MIN, few)))


def _pair_counters(device: torch.device, pairs: int) -> torch.Tensor:
    """Zeroed int32 counters, one per (row, kv head tile), that live as long as the process: a call leaves them zero
    again, and a replayed graph keeps pointing at them.  Grown by allocating anew; the old ones stay (graphs)."""
    key = (device.type, device.index if device.index is not None else torch.cuda.current_device())
    have = _counters.setdefault(key, [])
    if not have or have[-1].numel() < pairs:
        have.append(torch.zeros(max(1024, pairs), dtype=torch.int32, device=device))
    return have[-1]


def attention_bf16(q: torch.Tensor, q_off: int, out: torch.Tensor, n_heads: int, n_kv_heads: int, head_dim: int,
                   cache: torch.Tensor, page_tokens: int, block_table: torch.Tensor, step, window: int = 0,
                   scale: Optional[float] = None) -> bool:
    """Attention of a whole step: single-row segments on the split-key decode kernel, longer segments on the
    tiled prefill kernel.  Returns False (nothing done) if the sizes are not ones these kernels take."""
    _ops._gpu(q, out, cache, block_table)
    ldq, ldo = _ops._rows(q, "attention q"), _ops._rows(out, "attention out")
    T = q.shape[0]
    if scale is not None and not scale > 0:
        return False
    if (head_dim % 16 or head_dim > 256 or page_tokens % 8 or ldq % 8 or q_off % 8 or not _aligned(q, cache)
            or q.dtype != torch.bfloat16 or cache.dtype != torch.bfloat16 or out.dtype != torch.bfloat16):
        return False
    _ops._need(q_off + n_heads * head_dim <= q.shape[1], "attention: q heads exceed the row")
    _ops._need(out.shape == (T, n_heads * head_dim), "attention out must be [rows, heads*head_dim]")
    _ops._need(n_heads % n_kv_heads == 0, "heads must be a multiple of kv heads")
    if not (cache.dim() == 5 and cache.is_contiguous()
            and tuple(cache.shape[1:]) == (2, n_kv_heads, page_tokens, head_dim)):
        raise ValueError(f"cache must be [pages, 2, {n_kv_heads}, {page_tokens}, {head_dim}], got {tuple(cache.shape)}")
    _ops._need(block_table.dim() == 2 and block_table.dtype == torch.int32 and block_table.is_contiguous(),
               "block table must be contiguous int32 [segments, blocks]")
    _ops._need(step.positions.numel() >= T and step.row_seg.numel() >= T, "step rows differ from q rows")
    sc = (1.0 / math.sqrt(head_dim)) if scale is None else float(scale)
    L = _lib.load("tuned")
    stream = _ops._stream()
    if step.n_tiles:
        # (only the kernel of 128-row blocks cuts keys into ranges: no room is taken for the others)
        wide = WIDE_TILES and L.apc_attention_prefill_wide_takes(head_dim, page_tokens, step.n_tiles, T - step.n_decode_rows)
        splits = _key_splits(step, n_heads, window) if wide else 1
        parts = (torch.empty(splits * T * n_heads * (head_dim + 2), dtype=torch.float32, device=q.device)
                 if splits > 1 else None)
        _lib.check(L.apc_attention_prefill_bf16(
            q.data_ptr(), ldq, q_off, out.data_ptr(), ldo, n_heads, n_kv_heads, head_dim, cache.data_ptr(),
            page_tokens, block_table.data_ptr(), block_table.shape[1], step.positions.data_ptr(),
            step.row_seg.data_ptr(), step.tile_row0.data_ptr(), step.tile_rows.data_ptr(), step.n_tiles,
            (T - step.n_decode_rows) if WIDE_TILES else 0, int(window), sc, splits, T,
            parts.data_ptr() if parts is not None else 0, stream), "attention_prefill_bf16")
    if step.n_decode_rows:
        n = step.n_decode_rows
        span = min(step.max_decode_context, window) if window else step.max_decode_context
        rows = step.decode_rows.data_ptr() if step.decode_rows is not None else 0
        pairs = n * n_kv_heads * -(-(n_heads // n_kv_heads) // 16)
        n_parts = -(-step.max_decode_context // KEYS_PER_PART) if KEYS_PER_PART else _decode_parts(pairs, span)
        # (rows so short that one block's waves take a pair's ranges need no partial results either)
        if ((pairs >= WHOLE_MIN_PAIRS or n_parts <= WHOLE_WAVES)
                and L.apc_attention_decode_whole_fits(n_heads, n_kv_heads, head_dim)):
            _lib.check(L.apc_attention_decode_bf16(
                q.data_ptr(), ldq, q_off, out.data_ptr(), ldo, n, n_heads, n_kv_heads, head_dim, cache.data_ptr(),
                page_tokens, block_table.data_ptr(), block_table.shape[1], step.positions.data_ptr(),
                step.row_seg.data_ptr(), rows, int(window), sc, 0, 0, 0, 0, stream), "attention_decode_bf16 (whole)")
            return True
        kw = KEYS_PER_PART
        if LAST_BLOCK_MERGES and L.apc_attention_decode_last_fits(n_heads, n_kv_heads, head_dim, n_parts):
            # one partial result a block; the block of a (row, kv head) that finishes last adds them: one launch
            nz = -(-n_parts // WHOLE_WAVES)
            ws = torch.empty(n * n_heads * nz * (head_dim + 2), dtype=torch.float32, device=q.device)
            _lib.check(L.apc_attention_decode_bf16(
                q.data_ptr(), ldq, q_off, out.data_ptr(), ldo, n, n_heads, n_kv_heads, head_dim, cache.data_ptr(),
                page_tokens, block_table.data_ptr(), block_table.shape[1], step.positions.data_ptr(),
                step.row_seg.data_ptr(), rows, int(window), sc, kw, n_parts, ws.data_ptr(),
                _pair_counters(q.device, pairs).data_ptr(), stream), "attention_decode_bf16 (last block merges)")
            return True
        ws = torch.empty(n * n_heads * n_parts * (head_dim + 2), dtype=torch.float32, device=q.device)
        _lib.check(L.apc_attention_decode_bf16(
            q.data_ptr(), ldq, q_off, out.data_ptr(), ldo, n, n_heads, n_kv_heads, head_dim, cache.data_ptr(),
            page_tokens, block_table.data_ptr(), block_table.shape[1], step.positions.data_ptr(),
            step.row_seg.data_ptr(), rows, int(window), sc, kw, n_parts, ws.data_ptr(), 0, stream),
            "attention_decode_bf16")
    return True


MASKED_DECODE_BLOCKS = 768    # blocks the decoded rows' key ranges are cut for (3 a compute unit are resident)
MASKED_DECODE_SPLITS = 64     # at most: the adding kernel takes 64 parts


def masked_attention_bf16(q, out, n_heads, n_kv_heads, key_dim, value_dim, cache, page_tokens, block_table, step,
                          mask: str, mask_size: int, sink: bool, scale: float, key_parts: int = 1, sinks=None,
                          gate=None, softcap: float = 0.0, distance_bias=None, keep_first: int = 0,
                          out_scale: float = 1.0) -> bool:
    """Attention with a chunked or sliding mask and an optional sink on the MFMA kernels: segments of several rows on
    the tiled kernel, single rows on the kernel that cuts a row's keys into ranges.  False (nothing done) for sizes
    they do not take; the caller then runs the plain kernel."""
    _ops._gpu(q, out, cache, block_table)
    ldq, ldo = _ops._rows(q, "attention q"), _ops._rows(out, "attention out")
    T = q.shape[0]
    L = _lib.load("tuned")
    f32 = out.dtype == torch.float32
    if gate is not None and gate.dtype != torch.float32:
        return False
    r1, r2 = distance_bias if distance_bias is not None else (None, None)
    r1_p, r2_p = _ops._f32(r1, n_heads, "distance bias r1"), _ops._f32(r2, n_heads, "distance bias r2")
    _ops._check_sinks_gate(sink, sinks, gate, T, n_heads)
    sinks_p = _ops._f32(sinks, n_heads, "sinks")
    gate_p, ldg = (gate.data_ptr(), _ops._rows(gate, "head gate")) if gate is not None else (0, 0)
    if (not scale > 0 or ldq % 8 or ldo % 4 or not _aligned(q, cache) or out.data_ptr() % (16 if f32 else 8)
            or q.dtype != torch.bfloat16 or cache.dtype != torch.bfloat16
            or out.dtype not in (torch.bfloat16, torch.float32)
            or not L.apc_attention_masked_takes(n_heads, n_kv_heads, key_dim, value_dim, page_tokens, key_parts)):
        return False
    _ops._check_key_parts(n_heads, n_kv_heads, key_dim, key_parts)
    _ops._need(q.shape[1] == n_heads * (key_dim // key_parts), "attention: q must be [rows, heads * key_dim / key_parts]")
    _ops._need(out.shape == (T, n_heads * value_dim), "attention out must be [rows, heads * value_dim]")
    _ops._split_pages(cache, n_kv_heads, key_dim, value_dim, page_tokens)
    _ops._need(block_table.dim() == 2 and block_table.dtype == torch.int32 and block_table.is_contiguous(),
               "block table must be contiguous int32 [segments, blocks]")
    _ops._need(step.positions.numel() >= T and step.row_seg.numel() >= T, "step rows differ from q rows")
    code, stream = _ops.MASKS[mask], _ops._stream()
    keep = int(keep_first)
    _ops._need(keep >= 0 and (not keep or mask == "window"), "attention: kept first tokens go with a window")
    if step.n_tiles:
        _lib.check(L.apc_attention_masked_prefill_bf16(
            q.data_ptr(), ldq, out.data_ptr(), ldo, n_heads, n_kv_heads, key_dim, value_dim, cache.data_ptr(),
            page_tokens, block_table.data_ptr(), block_table.shape[1], step.positions.data_ptr(),
            step.row_seg.data_ptr(), step.tile_row0.data_ptr(), step.tile_rows.data_ptr(), step.n_tiles, code,
            int(mask_size), keep, 1 if sink else 0, sinks_p, gate_p, ldg, float(scale), int(key_parts),
            1 if f32 else 0, float(softcap), r1_p, r2_p, float(out_scale), stream), "attention_masked_prefill_bf16")
    if step.n_decode_rows:
        n = step.n_decode_rows
        keys = min(step.max_decode_context, mask_size) if code else step.max_decode_context
        # a row's first pass starts at a multiple of 256 at or below its first key; kept first keys are passes of their own
        passes = -(-(keys + 255) // 256) + -(-min(keep, step.max_decode_context) // 256)
        splits = max(1, min(passes, MASKED_DECODE_SPLITS, MASKED_DECODE_BLOCKS // max(1, n * n_kv_heads)))
        parts = torch.empty(n * n_heads * splits * (value_dim + 2), dtype=torch.float32, device=q.device)
        _lib.check(L.apc_attention_masked_decode_bf16(
            q.data_ptr(), ldq, out.data_ptr(), ldo, n, n_heads, n_kv_heads, key_dim, value_dim, cache.data_ptr(),
            page_tokens, block_table.data_ptr(), block_table.shape[1], step.positions.data_ptr(),
            step.row_seg.data_ptr(), step.decode_rows.data_ptr() if step.decode_rows is not None else 0, code,
            int(mask_size), keep, 1 if sink else 0, sinks_p, gate_p, ldg, float(scale), splits, parts.data_ptr(),
            int(key_parts), 1 if f32 else 0, float(softcap), r1_p, r2_p, float(out_scale), stream),
            "attention_masked_decode_bf16")
    return True


LINEAR_CHUNK_MIN_ROWS = 5    # segments of at least this many rows make a step run on the kernel of 64-row chunks


def linear_attention_bf16(proj, q_off, k_off, v_off, H, dk, dv, silu, decay, state, step, slots, out,
                          powers=None, rot: int = 0, cos_sin=None, k_scale: float = 1.0) -> bool:
    """Linear attention with a decay on the MFMA kernel that walks a segment in chunks of 64 rows.  False (nothing
    done) for sizes it does not take and for steps whose segments are all short (decoded rows): the caller then runs
    the kernel that walks row by row.  With a rotation or a key scale, q and k of `proj` are first rotated (and k
    scaled) where they lie, in bfloat16: the chunk kernels' operands are 16 bits anyway."""
    ld, ldo = _ops._rows(proj, "projected rows"), _ops._rows(out, "linear attention out")
    L = _lib.load("tuned")
    if (step.max_rows < LINEAR_CHUNK_MIN_ROWS or proj.dtype != torch.bfloat16 or ldo % 4 or not _aligned(proj, out)
            or not L.apc_linear_attention_bf16_takes(ld, q_off, k_off, v_off, H, dk, dv)):
        return False
    if rot or float(k_scale) != 1.0:
        if silu or rot % 16 or (rot and not _aligned(cos_sin)):
            return False
        T = proj.shape[0]
        _lib.check(L.apc_linear_rotate_bf16(proj.data_ptr(), ld, q_off, k_off, H, dk, int(rot),
                                            cos_sin.data_ptr() if rot else 0,
                                            _ops._i32(step.positions, T, "positions") if rot else 0, float(k_scale), T,
                                            _ops._stream()), "linear_rotate_bf16")
    S = step.n_segs
    if powers is None:         # (a caller that keeps the table, as the mixer does, saves this read-back)
        powers = decay_powers(decay.tolist(), proj.device)
    n_chunks, chunks, seg_chunks = _row_chunks(step, proj.device)
    ws = torch.empty((n_chunks, H, dk, dv), dtype=torch.float32, device=proj.device)
    _lib.check(L.apc_linear_attention_bf16(
        proj.data_ptr(), ld, q_off, k_off, v_off, H, dk, dv, 1 if silu else 0,
        _ops._f32(powers, H * (LINEAR_CHUNK_ROWS + 1), "powers of the decay"),
        state.data_ptr(), S, _ops._i32(step.seg_row0, S, "seg_row0"), _ops._i32(step.seg_rows, S, "seg_rows"),
        _ops._i32(slots, S, "slots"), n_chunks, chunks.data_ptr(), seg_chunks.data_ptr(), ws.data_ptr(),
        out.data_ptr(), ldo, _ops._stream()), "linear_attention_bf16")
    return True


SCAN_CHUNK_MIN_ROWS = 5      # as above, for the selective scan


def selective_scan_bf16(x, dt, dt_bias, A, bc, D, z, state, step, slots, out) -> bool:
    """The selective scan over prompt portions, chunks of 64 rows side by side (summaries, a scan over the chunks, the
    outputs).  False (nothing done) for sizes the kernels do not take and for steps whose segments are all short
    (decoded rows): the caller then runs the kernel that walks row by row."""
    L = _lib.load("tuned")
    T, C = out.shape
    N = int(A.shape[1])
    if step.max_rows < SCAN_CHUNK_MIN_ROWS or not L.apc_selective_scan_bf16_takes(C, N):
        return False
    S = step.n_segs
    n_chunks, chunks, seg_chunks = _row_chunks(step, x.device)
    ws = torch.empty((n_chunks, C, N), dtype=torch.float32, device=x.device)
    sums = torch.empty((n_chunks, C), dtype=torch.float32, device=x.device)
    _lib.check(L.apc_selective_scan_bf16(
        x.data_ptr(), _ops._rows(x, "x"), dt.data_ptr(), _ops._rows(dt, "dt"), _ops._f32(dt_bias, C, "dt bias"),
        A.data_ptr(), bc.data_ptr(), _ops._rows(bc, "B and C"), _ops._f32(D, C, "D"), z.data_ptr(), _ops._rows(z, "z"),
        state.data_ptr(), C, N, S, _ops._i32(step.seg_row0, S, "seg_row0"), _ops._i32(step.seg_rows, S, "seg_rows"),
        _ops._i32(slots, S, "slots"), n_chunks, chunks.data_ptr(), seg_chunks.data_ptr(), ws.data_ptr(),
        sums.data_ptr(), out.data_ptr(), _ops._rows(out, "out"), _ops._stream()), "selective_scan_bf16")
    return True


DELTA_CHUNK_MIN_ROWS = 5     # as above, for the gated delta rule and the gated recurrence


def delta_rule_bf16(rows, ld, q_off, k_off, v_off, H, G, dk, dv, ba, ldba, a_off, b_off, A, dt_bias, state, step, slots,
                    out, ldo) -> bool:
    """The gated delta rule over prompt portions in chunks of 64 rows on MFMA: every chunk's factors side by side, then a
    walk over the chunks.  False (nothing done) for sizes the kernels do not take and for steps whose segments are all
    short (decoded rows): the caller then runs the kernel that walks row by row."""
    L = _lib.load("tuned")
    if (step.max_rows < DELTA_CHUNK_MIN_ROWS or not _aligned(rows)
            or not L.apc_delta_rule_bf16_takes(ld, q_off, k_off, H, G, dk, dv)):
        return False
    S = step.n_segs
    n_chunks, chunks, seg_chunks = _row_chunks(step, rows.device)
    fact = torch.empty(n_chunks * L.apc_delta_rule_fact_size(H), dtype=torch.bfloat16, device=rows.device)
    coef = torch.empty(n_chunks * L.apc_delta_rule_coef_size(H), dtype=torch.float32, device=rows.device)
    kt = torch.empty(n_chunks * G * dk * LINEAR_CHUNK_ROWS, dtype=torch.bfloat16, device=rows.device)
    _lib.check(L.apc_delta_rule_bf16(
        rows.data_ptr(), ld, q_off, k_off, v_off, H, G, dk, dv, ba.data_ptr(), ldba, a_off, b_off, _ops._f32(A, H, "A"),
        _ops._f32(dt_bias, H, "dt bias"), float(dk) ** -0.5, state.data_ptr(), S, _ops._i32(step.seg_row0, S, "seg_row0"),
        _ops._i32(step.seg_rows, S, "seg_rows"), _ops._i32(slots, S, "slots"), n_chunks, chunks.data_ptr(),
        seg_chunks.data_ptr(), fact.data_ptr(), coef.data_ptr(), kt.data_ptr(), out.data_ptr(), ldo, _ops._stream()),
        "delta_rule_bf16")
    return True


def gated_recurrence_bf16(u, z, z_bias, blocks: int, rate, y, y_bias, state, step, slots, out, out_scale: float) -> bool:
    """The gated linear recurrence over prompt portions, chunks of 64 rows side by side (summaries, a scan over the
    chunks, the outputs).  False (nothing done) as above."""
    L = _lib.load("tuned")
    T, C = out.shape
    ldu, ldz, ldy, ldo = _ops._rows(u, "u"), _ops._rows(z, "gate logits"), _ops._rows(y, "y"), _ops._rows(out, "out")
    if (step.max_rows < DELTA_CHUNK_MIN_ROWS or not L.apc_gated_recurrence_bf16_takes(C, blocks, ldu, ldz, ldy, ldo)
            or any(t.data_ptr() % 4 for t in (u, y, out)) or z.data_ptr() % 8):
        return False
    S = step.n_segs
    n_chunks, chunks, seg_chunks = _row_chunks(step, u.device)
    ws = torch.empty((10, n_chunks, C), dtype=torch.float32, device=u.device)
    _lib.check(L.apc_gated_recurrence_bf16(
        u.data_ptr(), ldu, z.data_ptr(), ldz, _ops._f32(z_bias, 2 * C, "gate biases"), blocks, _ops._f32(rate, C, "rate"),
        y.data_ptr(), ldy, _ops._f32(y_bias, C, "y bias"), float(out_scale), state.data_ptr(), C, S,
        _ops._i32(step.seg_row0, S, "seg_row0"), _ops._i32(step.seg_rows, S, "seg_rows"), _ops._i32(slots, S, "slots"),
        n_chunks, chunks.data_ptr(), seg_chunks.data_ptr(), ws.data_ptr(), out.data_ptr(), ldo,
        _ops._stream()), "gated_recurrence_bf16")
    return True


LINEAR_CHUNK_ROWS = 64


def decay_powers(decay, device) -> torch.Tensor:
    """float32 [heads, 65]: decay^0 .. decay^64 of every head (`decay`: the heads' numbers), formed in double precision
    on the host and rounded once: what the chunk kernels multiply scores, outputs and states with."""
    rows = [[float(d) ** n for n in range(LINEAR_CHUNK_ROWS + 1)] for d in decay]
    return torch.tensor(rows, dtype=torch.float64).to(torch.float32).to(device).contiguous()


def _row_chunks(step, device):
    """(chunks in all, int32 [chunks][2] (segment, first row in it), int32 [segments][2] (a segment's first chunk, its
    chunks)) of a step's segments cut into chunks of 64 rows: made on the host from the step's own lists, once a step
    (every layer of the step asks for the same)."""
    made = getattr(step, "_row_chunks", None)
    if made is None:
        import numpy as np
        chunks, per_seg = [], []
        for s, n in enumerate(step.host_rows):
            per_seg.append((len(chunks), -(-n // LINEAR_CHUNK_ROWS)))
            chunks += [(s, c0) for c0 in range(0, n, LINEAR_CHUNK_ROWS)]
        flat = np.asarray(chunks + per_seg, dtype=np.int32).reshape(-1)
        dev = torch.from_numpy(flat).to(device)
        made = (len(chunks), dev[:2 * len(chunks)], dev[2 * len(chunks):])
        step._row_chunks = made
    return made


class PackedExperts:
    """The matrices of a layer's experts in the tiled layout of the MFMA kernels: `data` holds, for every expert, the
    tiles of its matrices (`per_expert` of them: gate and up, or down alone), each packed like a `PackedWeight`."""

    def __init__(self, data: torch.Tensor, n_experts: int, N: int, K: int, per_expert: int = 1):
        self.data, self.E, self.N, self.K, self.per_expert = data, n_experts, N, K, per_expert


# pairs an expert on average from which a row tile holds 64 and 128 rows instead of 16 (and the products run on the
# tiled kernel through LDS instead of streaming an expert's matrices once a tile)
ROUTED_TILE_64_MIN, ROUTED_TILE_128_MIN = 24, 96


def pack_experts(gate_up: torch.Tensor, down: torch.Tensor):
    """[E, 2 F, D] (gate rows, then up rows; [E, F, D] for experts without a gate) and [E, D, F] bfloat16 ->
    (PackedExperts, PackedExperts), or None for sizes the kernels do not take."""
    from .packing import pack_mfma
    E, D, F = down.shape
    gated = gate_up.shape[1] == 2 * F
    if not _lib.load("tuned").apc_routed_bf16_takes(E, F, D):
        return None
    firsts = (slice(0, F), slice(F, 2 * F)) if gated else (slice(0, F),)
    gu = torch.stack([torch.stack([pack_mfma(gate_up[e, s].contiguous()).data for s in firsts])
                      for e in range(E)]).contiguous()
    dn = torch.stack([pack_mfma(down[e].contiguous()).data for e in range(E)]).contiguous()
    return PackedExperts(gu, E, F, D, len(firsts)), PackedExperts(dn, E, D, F)


def routed_experts_bf16(h, w_gate_up: PackedExperts, w_down: PackedExperts, E: int, F: int, ids, weights, K: int,
                        y, kind: int = 0, alpha: float = 1.0, limit: float = 0.0, weight_input: bool = False) -> None:
    """The chosen experts of every row on the MFMA kernels (pairs sorted by expert on the GPU, nothing read back).
    `weight_input`: a pair's weight multiplies the expert's input instead of its output."""
    T, D = h.shape
    _ops._gpu(h, w_gate_up.data, w_down.data, ids, weights, y)
    _ops._need(h.dtype == torch.bfloat16 and (w_gate_up.E, w_gate_up.N, w_gate_up.K) == (E, F, D)
               and (w_down.E, w_down.N, w_down.K) == (E, D, F) and w_gate_up.per_expert == (1 if kind == 2 else 2), "routed experts: matrices do not fit the sizes")
    L = _lib.load("tuned")
    n_pairs = T * K
    tile_rows = 128 if n_pairs >= ROUTED_TILE_128_MIN * E else 64 if n_pairs >= ROUTED_TILE_64_MIN * E else 16
    max_tiles = L.apc_routed_max_tiles(n_pairs, E, tile_rows)
    dev = h.device
    work = torch.empty(2 * n_pairs + 3 * max_tiles + 1, dtype=torch.int32, device=dev)
    act = torch.empty((n_pairs, F), dtype=torch.bfloat16, device=dev)
    ys = torch.empty((n_pairs, D), dtype=torch.float32, device=dev)
    hs = torch.empty((n_pairs, D), dtype=torch.bfloat16, device=dev) if tile_rows != 16 else None
    _lib.check(L.apc_routed_experts_bf16(
        h.data_ptr(), _ops._rows(h, "h"), w_gate_up.data.data_ptr(), w_down.data.data_ptr(), E, F, D,
        _ops._i32(ids, n_pairs, "ids"), _ops._f32(weights, n_pairs, "weights"), K, T, tile_rows, work.data_ptr(),
        act.data_ptr(), ys.data_ptr(), hs.data_ptr() if hs is not None else 0, y.data_ptr(), _ops._rows(y, "y"),
        int(kind), float(alpha), float(limit), 1 if weight_input else 0, _ops._stream()),
        "routed_experts_bf16")


def rotary_pages_bf16(q, ldq, q_off, H, dq, q_rot0, q_out, ldqo, ka, ldka, ka_off, da, kb, ldkb, kb_off, db, kb_shared,
                      k_rot0, v, ldv, v_off, dv, G, rot, cos_sin, step, block_table, cache, page_tokens, q_norm_w=None,
                      k_norm_w=None, norm_eps: float = 0.0) -> bool:
    """Heads put together, rotated and written into the pages on 16-byte accesses (bfloat16 rows and pages; the second
    key part may be float32 rows); False (nothing done) for sizes the kernel does not take."""
    L = _lib.load("tuned")
    T = q.shape[0]
    if H <= 0 or G <= 0 or (kb is not None and kb.dtype not in (torch.bfloat16, torch.float32)):
        return False
    if not L.apc_rotary_pages_bf16_takes(ldq, q_off, dq, q_rot0, ldqo, ldka, ka_off, da, ldkb, kb_off, db, k_rot0, ldv,
                                         v_off, dv, rot):
        return False
    if not _aligned(q, q_out, ka, v, cache) or (kb is not None and not _aligned(kb)) or (rot and not _aligned(cos_sin)):
        return False
    if q_norm_w is not None or k_norm_w is not None:
        # a wave a head: no second key part, heads of up to 512 elements
        if kb is not None or db or max(dq, da, dv) > 512 or not all(w is None or _aligned(w) for w in (q_norm_w, k_norm_w)):
            return False
    _lib.check(L.apc_rotary_pages_bf16(
        q.data_ptr(), ldq, q_off, H, dq, q_rot0, q_out.data_ptr(), ldqo, ka.data_ptr(), ldka, ka_off, da,
        kb.data_ptr() if kb is not None else 0, 1 if kb is not None and kb.dtype == torch.float32 else 0, ldkb, kb_off,
        db, 1 if kb_shared else 0, k_rot0, v.data_ptr(), ldv, v_off, dv, G, rot, cos_sin.data_ptr() if rot else 0,
        _ops._i32(step.positions, T, "positions"), _ops._i32(step.row_seg, T, "row_seg"), block_table.data_ptr(),
        block_table.shape[1], cache.data_ptr(), page_tokens, T, _ops._f32(q_norm_w, dq, "q norm weight"),
        _ops._f32(k_norm_w, da + db, "k norm weight"), float(norm_eps), _ops._stream()), "rotary_pages_bf16")
    return True


# --------------------------------------------------------------------------- a matrix of its own for every head
class PackedHeads:
    """[heads, N, K] matrices in the tiled layout: `data` [heads, bands, chunks, 64, 8]."""

    def __init__(self, data: torch.Tensor, H: int, N: int, K: int):
        self.data, self.H, self.N, self.K = data, H, N, K


def pack_heads(w: torch.Tensor, a_head: int, out_head: int):
    """[H, N, K] bfloat16 -> PackedHeads, or None where the kernel does not take the heads' places in the rows (`a_head`
    elements apart in the product's input, `out_head` in its output)."""
    from .packing import can_pack, pack_mfma
    if not can_pack(w[0]) or a_head % 8 or out_head % 4:
        return None
    H, N, K = w.shape
    return PackedHeads(torch.stack([pack_mfma(w[h].contiguous()).data for h in range(H)]).contiguous(), H, N, K)


def heads_linear_bf16(a: torch.Tensor, a_head: int, w: PackedHeads, out: torch.Tensor, out_head: int, gate=None) -> None:
    _ops._gpu(a, w.data, out)
    lda, ldo = _ops._rows(a, "heads_linear a"), _ops._rows(out, "heads_linear out")
    T = a.shape[0]
    f32 = out.dtype == torch.float32
    _ops._need(a.dtype == torch.bfloat16 and (f32 or out.dtype == torch.bfloat16) and out.shape[0] == T
               and (w.H - 1) * a_head + w.K <= a.shape[1] and (w.H - 1) * out_head + w.N <= out.shape[1],
               "heads_linear: bfloat16 rows that hold the heads' ranges")
    ldg = _ops._rows(gate, "gate") if gate is not None else 0
    _ops._need(gate is None or (gate.dtype == torch.bfloat16 and ldg % 4 == 0 and gate.data_ptr() % 8 == 0),
               "heads_linear_bf16: the gate's logits are bfloat16 rows of a stride that is a multiple of 4")
    _ops._need(lda % 8 == 0 and ldo % 4 == 0 and _aligned(a) and out.data_ptr() % (16 if f32 else 8) == 0,
               "heads_linear_bf16: rows of a stride that is a multiple of 8 (out: 4), aligned")
    L = _lib.load("tuned")
    _lib.check(L.apc_heads_gemm_bf16(a.data_ptr(), lda, int(a_head), w.data.data_ptr(), out.data_ptr(), ldo, int(out_head),
                                     1 if f32 else 0, gate.data_ptr() if gate is not None else 0, ldg, T, w.H, w.N, w.K,
                                     _ops._stream()), "heads_gemm_bf16")


def latent_rows_bf16(proj, ld, H, dn, dr, kv, ldkv, c_off, R, norm_w, eps, cos_sin, step, block_table, pages,
                     page_tokens, q_out, ldq) -> bool:
    """The same on 16-byte accesses; False (nothing done) for sizes the kernel does not take."""
    L = _lib.load("tuned")
    T = proj.shape[0]
    if not L.apc_latent_rows_bf16_takes(ld, dn, dr, ldkv, c_off, R, ldq) or not _aligned(proj, kv, pages, q_out, cos_sin):
        return False
    _lib.check(L.apc_latent_rows_bf16(
        proj.data_ptr(), ld, H, dn, dr, kv.data_ptr(), ldkv, c_off, R, _ops._f32(norm_w, R, "norm weight"), float(eps), cos_sin.data_ptr(),
        _ops._i32(step.positions, T, "positions"), _ops._i32(step.row_seg, T, "row_seg"), block_table.data_ptr(),
        block_table.shape[1], pages.data_ptr(), page_tokens, q_out.data_ptr(), ldq, T, _ops._stream()), "latent_rows_bf16")
    return True


LATENT_BLOCKS = 256          # blocks that the keys of few rows are cut for (a block a compute unit at a latent of 512)
LATENT_SPLITS_MAX = 128      # (the adding kernel takes up to 256; 128 was the fastest for one row over 32,768 keys)
LATENT_DECODE_TILES = 2      # key tiles that a range of a decoded row's keys must keep
LATENT_RANGE_TILES = 8       # key tiles (of 64) that a range of a prompt tile's keys must keep


def latent_attention_bf16(q, out, n_heads: int, rank: int, rot_dim: int, pages, page_tokens: int, block_table, step,
                          scale: float) -> bool:
    """Attention of all heads over cached latents on MFMA: tiles of prompt rows, then single rows.  False (nothing done)
    for sizes the kernel does not take."""
    _ops._gpu(q, out, pages, block_table)
    T, H, R, dr = q.shape[0], int(n_heads), int(rank), int(rot_dim)
    L = _lib.load("tuned")
    if (q.dtype != torch.bfloat16 or pages.dtype != torch.bfloat16 or out.dtype != torch.bfloat16
            or not q.is_contiguous() or not out.is_contiguous() or not _aligned(q, out, pages)
            or not L.apc_latent_attention_takes(H, R, dr, page_tokens)):
        return False
    _ops._need(tuple(q.shape) == (T, H * (R + dr)) and tuple(out.shape) == (T, H * R), "latent attention: q [rows, heads * "
               "(rank + rot_dim)], out [rows, heads * rank]")
    _ops._latent_pages(pages, R + dr, page_tokens, block_table)
    _ops._need(step.positions.numel() >= T and step.row_seg.numel() >= T, "step rows differ from q rows")

    def run(row0, rows, n: int, max_rows: int, splits: int, what: str) -> None:
        parts = ml = None
        if splits > 1:
            parts = torch.empty((T * H, splits, R), dtype=torch.float32, device=q.device)
            ml = torch.empty((T * H, splits, 2), dtype=torch.float32, device=q.device)
        _lib.check(L.apc_latent_attention_bf16(
            q.data_ptr(), out.data_ptr(), H, R, dr, pages.data_ptr(), page_tokens, block_table.data_ptr(),
            block_table.shape[1], step.positions.data_ptr(), step.row_seg.data_ptr(),
            row0.data_ptr() if row0 is not None else 0, rows.data_ptr() if rows is not None else 0, n, max_rows, splits,
            parts.data_ptr() if parts is not None else 0, ml.data_ptr() if ml is not None else 0, float(scale),
            _ops._stream()), what)

    if step.n_tiles:
        most = min(step.max_rows, _ops.attention_tile_rows(torch.bfloat16))
        blocks = step.n_tiles * -(-most * H // 64)
        keys = max([p + n for p, n in zip(step.host_pos0, step.host_rows) if n > 1] or [step.max_context])
        splits = max(1, min(LATENT_BLOCKS // blocks, -(-keys // 64) // LATENT_RANGE_TILES, LATENT_SPLITS_MAX))
        run(step.tile_row0, step.tile_rows, step.n_tiles, most, splits, "latent_attention_bf16 (prompt rows)")
    if step.n_decode_rows:
        n = step.n_decode_rows
        blocks = n * -(-H // (64 if H > 32 else 32))
        splits = max(1, min(LATENT_BLOCKS // blocks, -(-step.max_decode_context // (64 * LATENT_DECODE_TILES)), LATENT_SPLITS_MAX))
        run(step.decode_rows, None, n, 1, splits, "latent_attention_bf16 (decoded rows)")
    return True
