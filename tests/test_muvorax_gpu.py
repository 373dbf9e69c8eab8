"""The Muvorax decoder on the GPU against the plain implementation (tests/plain_muvorax.py): every new kernel alone,
then whole models of several shapes through the step function, the cache manager and the engine."""
import json
import os
import subprocess
import sys

import numpy as np
import pytest
import torch

import plain_muvorax as P
from helpers import tmp_root
from muvorax_helpers import (CONFIGS, _dense, _lat, _layer, _lig, _model, _moe, _scan, model_folder, oracle,
                             oracle_logits, oracle_noise, planted, tokens_for, write_folder)
from test_seredra_gpu import DEV, DTYPES, bf, close, dev, make_step, run_cut, scattered_tables

pytestmark = pytest.mark.gpu


def rows_of(segs):
    return sum(n for _, n in segs)


# =========================================================================================== kernels alone
def latent_pages(tables, n_pages, P_, cs, dtype, hole=float("nan")):
    """pages [n + 1, P, L] with every request's rows at its places; what no request has written holds `hole`."""
    L = cs[0].shape[1]
    pages = np.full((n_pages + 1, P_, L), hole, dtype=np.float32)
    for tb, c in zip(tables, cs):
        for pos in range(c.shape[0]):
            pages[tb[pos // P_], pos % P_] = c[pos]
    return dev(pages, dtype)


def check_latent_attention(H, R, dr, P_, segs, dtype, seed, scale=0.8, plant=(), splits=None, monkeypatch=None):
    """`plant`: (segment, row in it, head, position): that head's query of that row asks, with a large query, for the key
    at that position."""
    from allpaca_amd.kernels import ops, tuned
    rng = np.random.default_rng(seed)
    tdt = DTYPES[dtype]
    L = R + dr
    lens = [p + n for p, n in segs]
    n_pages, tables = scattered_tables(rng, lens, P_)
    cs = [bf(rng.normal(size=(n, L))) * 0.5 for n in lens]
    T = rows_of(segs)
    row0 = np.cumsum([0] + [n for _, n in segs])
    q = bf(rng.normal(size=(T, H, L)) / L ** 0.5 * 3)
    for s, r, h, pos in plant:
        cs[s][pos] *= 2.0
    for s, r, h, pos in plant:
        q[row0[s] + r, h] = bf(cs[s][pos] / np.linalg.norm(cs[s][pos]) * 14.0)
    cache = latent_pages(tables, n_pages, P_, cs, tdt)
    step = make_step(segs, tables)
    out = torch.full((T, H * R), float("nan"), dtype=tdt, device=DEV)
    if splits is not None:
        monkeypatch.setattr(tuned, "LATENT_BLOCKS", splits)
        monkeypatch.setattr(tuned, "LATENT_RANGE_TILES", 1)
        monkeypatch.setattr(tuned, "LATENT_DECODE_TILES", 1)
    ops.latent_attention(dev(q.reshape(T, -1), tdt), out, H, R, dr, cache, P_, step.block_tables[0], step, scale)
    got = out.float().cpu().numpy().reshape(T, H, R)
    for i, ((p0, n), c) in enumerate(zip(segs, cs)):
        keys = np.broadcast_to(c[:, None], (lens[i], H, L))
        want = P.softmax_attention(q[row0[i]:row0[i] + n], keys, keys[..., :R], scale, q_pos0=p0)
        what = f"segment {i} of {segs} H {H} R {R} dr {dr} page {P_}"
        close(got[row0[i]:row0[i] + n].reshape(n, -1), want.reshape(n, -1), dtype, what, rel=0.012)
        for s, r, h, pos in plant:
            if s == i:      # the planted key carries its row: its values are what comes out
                near = np.linalg.norm(got[row0[i] + r, h] - c[pos, :R]) / np.linalg.norm(c[pos, :R])
                assert near < 0.7, (what, r, h, pos, near)


@pytest.mark.parametrize("H, R, dr, P_", [(5, 14, 4, 3), (1, 8, 2, 1), (12, 96, 16, 16), (8, 64, 32, 16), (3, 40, 24, 8),
                                          (16, 128, 64, 32), (40, 72, 8, 16), (7, 256, 64, 16), (32, 512, 64, 16),
                                          (20, 448, 32, 64), (70, 64, 0, 16), (2, 64, 120, 4)])
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_attention_over_cached_latents_with_keys_that_stand_out(H, R, dr, P_, dtype):
    """A portion of 70 rows from position 200 beside decoded rows at positions 300, 64, 63 and 0 and a portion of two
    rows across a tile's edge, on scattered pages whose unwritten places hold NaN.  Some heads ask for one key: the
    first, one far back, either side of a page's border and of a key tile's, the row itself."""
    segs = [(200, 70), (300, 1), (64, 1), (63, 1), (0, 1), (127, 2)]
    plant = [(0, 69, 0, 1), (0, 5, H - 1, 63), (0, 64, H // 2, 64), (0, 3, 0, 203), (0, 30, H - 1, 200 // P_ * P_ - 1),
             (1, 0, 0, 0), (1, 0, H - 1, 300), (2, 0, 0, 63), (5, 0, H - 1, 127), (5, 1, 0, 128)]
    if len({(s, r, h) for s, r, h, _ in plant}) < len(plant):      # one head: a row asks for one key
        plant = list({(s, r, h): (s, r, h, p) for s, r, h, p in plant}.values())
    check_latent_attention(H, R, dr, P_, segs, dtype, H + R + dr, plant=plant)


@pytest.mark.parametrize("H, R, dr, blocks", [(32, 512, 64, 256), (8, 64, 32, 64), (40, 96, 16, 32), (3, 40, 24, 1024)])
def test_ranges_of_keys_are_added(H, R, dr, blocks, monkeypatch):
    """Keys cut into ranges, a block each: more ranges than key tiles for the short rows (a range without a key), ranges
    that end on either side of what a row of a prompt tile sees."""
    segs = [(1000, 1), (5, 1), (640, 66), (0, 3), (700, 1)]
    plant = [(0, 0, 0, 3), (0, 0, H - 1, 999), (1, 0, 0, 5), (2, 0, 0, 639), (2, 65, H - 1, 705), (2, 64, 0, 64), (4, 0, 0, 448)]
    check_latent_attention(H, R, dr, 16, segs, "bfloat16", 5, plant=plant, splits=blocks, monkeypatch=monkeypatch)


def test_a_reference_that_moves_late(monkeypatch):
    """Scores that rise from tile to tile by more than the kernel's references may lag behind, and others that rise by
    less: the sums are rescaled in some tiles and not in others."""
    from allpaca_amd.kernels import ops
    rng = np.random.default_rng(11)
    H, R, dr, P_, n = 4, 64, 32, 16, 400
    L = R + dr
    c = bf(rng.normal(size=(n, L)))
    q = bf(rng.normal(size=(n, H, L)))
    u = rng.normal(size=L)
    u /= np.linalg.norm(u)
    for h, rise in enumerate((0.2, 2.0, 14.0, -3.0)):             # natural units a key tile
        q[:, h] = bf(u * 8.0 + 0.02 * q[:, h])
        if h == 0:
            c = bf(c - np.outer(c @ u, u) + np.outer(np.arange(n) / 64.0, u))
        q[:, h] = bf(q[:, h] * rise / 8.0)
    n_pages, tables = scattered_tables(rng, [n], P_)
    for segs in ([(0, n)], [(n - 1, 1)]):
        step = make_step(segs, tables)
        T = segs[0][1]
        out = torch.empty((T, H * R), dtype=torch.bfloat16, device=DEV)
        cache = latent_pages(tables, n_pages, P_, [c], torch.bfloat16)
        ops.latent_attention(dev(q[n - T:].reshape(T, -1), torch.bfloat16), out, H, R, dr, cache, P_, step.block_tables[0],
                             step, 1.0)
        keys = np.broadcast_to(c[:, None], (n, H, L))
        want = P.softmax_attention(q[n - T:], keys, keys[..., :R], 1.0, q_pos0=n - T)
        got = out.float().cpu().numpy().reshape(T, H, R)
        for h in range(H):
            close(got[:, h], want[:, h], "bfloat16", f"head {h}", rel=0.015)
