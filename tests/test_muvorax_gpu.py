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


@pytest.mark.parametrize("H, R, dr, P_", [(5, 14, 4, 3), (1, 8, 2, 1), (12, 96, 16, 16), (9, 64, 16, 16), (3, 40, 24, 8),
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


@pytest.mark.parametrize("H, R, dr, blocks", [(32, 512, 64, 256), (10, 64, 16, 64), (40, 96, 16, 32), (3, 40, 24, 1024)])
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
    H, R, dr, P_, n = 4, 64, 48, 16, 400
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


@pytest.mark.parametrize("H, dn, dr, R, P_, own, scaling", [(5, 6, 4, 14, 3, True, (3.0, 16, 8.0, 1.0)),
                                                            (12, 32, 16, 96, 16, True, (4.0, 64, 16.0, 2.0)),
                                                            (3, 40, 24, 40, 8, True, None), (4, 64, 32, 96, 16, False, None),
                                                            (1, 8, 2, 8, 1, True, None), (2, 16, 64, 640, 16, True, (2.0, 32, 4.0, 0.5)),
                                                            (3, 8, 0, 24, 4, True, None)])
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_latents_and_rotated_parts_into_pages_and_queries(H, dn, dr, R, P_, own, scaling, dtype):
    """The latent's norm and the shared rotated key part into the row's place of its page, nothing else of the pages
    touched, and the queries' rotated parts behind their place for the latent part; a portion that starts inside a page
    beside single rows."""
    from allpaca_amd.kernels import ops
    from allpaca_amd.parts.base import Runtime
    from allpaca_amd.parts.rope import rotary_table
    rng = np.random.default_rng(H + R + dr)
    tdt = DTYPES[dtype]
    segs, lens = [(P_ + 1, 2 * P_ + 3), (0, 1), (5 * P_ - 1, 1)], [3 * P_ + 4, 1, 5 * P_]
    n_pages, tables = scattered_tables(rng, lens, P_)
    T, width = rows_of(segs), H * (dn + dr) + (R + dr if own else 0)
    x = bf(rng.normal(size=(T, width)))
    norm_w = np.float32(1 + 0.3 * rng.normal(size=R))
    rule = dict(zip(("factor", "original", "fast", "slow"), scaling)) if scaling else None
    table = None
    if dr:
        table = rotary_table(dr, 700.0, Runtime(torch.device(DEV), tdt, 8 * P_), dict(rule, rope_type="yarn") if rule else None)
    # the kernels' pairs are (i, i + dr/2); the plain rotation's are neighbours: the same numbers in another order
    order = np.concatenate([np.arange(0, dr, 2), np.arange(1, dr, 2)]).astype(int)

    def halves(v):
        return v[..., order]

    rows = x.copy()
    for h in range(H):
        a = h * (dn + dr) + dn
        rows[:, a:a + dr] = halves(x[:, a:a + dr])
    if own:
        rows[:, width - dr:] = halves(x[:, width - dr:]) if dr else rows[:, width - dr:]
    cache = torch.full((n_pages + 1, P_, R + dr), 7.0, dtype=tdt, device=DEV)
    q = torch.full((T, H * (R + dr)), 5.0, dtype=tdt, device=DEV)
    step = make_step(segs, tables)
    stride = -(-width // 8) * 8
    proj = torch.zeros((T, stride), dtype=tdt, device=DEV)[:, :width]
    proj.copy_(dev(rows, tdt))
    ops.latent_rows(proj, H, dn, dr, H * (dn + dr) if own else None, R, dev(norm_w) if own else None, 1e-5, table, step,
                    step.block_tables[0], cache, P_, q)
    pos = np.concatenate([np.arange(p0, p0 + n) for p0, n in segs])
    spec = dict(base=700.0, dims=dr, scaling=rule)
    got = q.float().cpu().numpy().reshape(T, H, R + dr)
    assert (got[..., :R] == 5.0).all()
    want = P.rotate_pairs(x[:, :H * (dn + dr)].reshape(T, H, dn + dr)[..., dn:], pos, spec)
    close(got[..., R:].reshape(T, -1), halves(want).reshape(T, -1), dtype, "q", rel=0.006) if dr else None
    pages = cache.float().cpu().numpy()
    written = np.zeros(pages.shape[:2], dtype=bool)
    r = 0
    for (p0, n), tb in zip(segs, tables):
        for a in range(n if own else 0):
            page, slot = tb[(p0 + a) // P_], (p0 + a) % P_
            written[page, slot] = True
            c = P.unit_rms(x[r + a:r + a + 1, H * (dn + dr):H * (dn + dr) + R], 1e-5) * norm_w
            close(pages[page, slot, :R], c[0], dtype, "latent", rel=0.006)
            if dr:
                kr = halves(P.rotate_pairs(x[r + a:r + a + 1, width - dr:], pos[r + a:r + a + 1], spec))
                close(pages[page, slot, R:], kr[0], dtype, "rotated key part", rel=0.006)
        r += n
    assert (pages[~written] == 7.0).all()


@pytest.mark.parametrize("T, H, N, K, a_head, out_head", [(3, 5, 14, 6, 10, 18), (16, 12, 96, 32, 48, 112), (1, 1, 8, 8, 8, 8),
                                                          (17, 4, 40, 24, 24, 44), (300, 3, 72, 40, 64, 80),
                                                          (130, 2, 512, 128, 192, 576), (9, 32, 128, 512, 512, 128),
                                                          (5, 3, 20, 264, 264, 20), (70, 2, 66, 16, 16, 68)])
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_a_matrix_of_its_own_for_every_head(T, H, N, K, a_head, out_head, dtype):
    from allpaca_amd.kernels import ops
    rng = np.random.default_rng(T + N)
    tdt = DTYPES[dtype]
    a = bf(rng.normal(size=(T, H * a_head)))
    w = bf(rng.normal(size=(H, N, K)) / K ** 0.5)
    out = torch.full((T, H * out_head), 3.0, dtype=tdt, device=DEV)
    ops.heads_linear(dev(a, tdt), a_head, ops.prepare_heads(dev(w, tdt), tdt, a_head, out_head), out, out_head)
    got = out.float().cpu().numpy().reshape(T, H, out_head)
    assert (got[..., N:] == 3.0).all()                          # what lies between the heads' outputs stays
    want = np.einsum("thk,hnk->thn", a.reshape(T, H, a_head)[..., :K], w)
    close(got[..., :N].reshape(T, -1), want.reshape(T, -1), dtype, "heads", rel=0.006)


@pytest.mark.parametrize("T, D", [(7, 36), (3, 1030), (300, 2048), (5, 4096), (1031, 1028), (1026, 30)])
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_tanh_norm_and_its_sum(T, D, dtype):
    """The norm of chosen rows; the sum of a normed output into the residual with and without the next norm; large and
    tiny arguments."""
    from allpaca_amd.kernels import ops
    rng = np.random.default_rng(D)
    tdt, exact = DTYPES[dtype], dtype == "float32"
    x, y = np.float32(rng.normal(size=(T, D)) * 3), np.float32(rng.normal(size=(T, D)) * 2)
    x[0, :4], y[0, :4] = [0.0, 1e-6, 60.0, -1000.0], [-60.0, 0.0, 1e-5, 500.0]
    one = (0.7, np.float32(rng.normal(size=D)), np.float32(rng.normal(size=D)))
    two = (1.3, np.float32(rng.normal(size=D)), np.float32(rng.normal(size=D)))
    on_gpu = [(a, dev(w), dev(b)) for a, w, b in (one, two)]
    rows = [T - 1, 0, T // 2]
    h = torch.empty((3, D), dtype=tdt, device=DEV)
    ops.tanh_norm(dev(x), on_gpu[0], h, torch.tensor(rows, dtype=torch.int32, device=DEV), exact=exact)
    close(h.float().cpu().numpy(), P.squash(x[rows].astype(np.float64), *one), dtype, "rows", rel=0.004)
    want = x.astype(np.float64) + P.squash(y.astype(np.float64), *one)
    for y_dtype in (torch.float32, tdt):
        yd = dev(y, y_dtype)
        w = x.astype(np.float64) + P.squash(yd.double().cpu().numpy(), *one)
        for nxt in (True, False):
            xd = dev(x)
            h = torch.empty((T, D), dtype=tdt, device=DEV) if nxt else None
            ops.tanh_norm_add(xd, yd, on_gpu[0], on_gpu[1] if nxt else None, h, exact=exact)
            close(xd.cpu().numpy(), w, "float32", "sum")
            if nxt:
                close(h.float().cpu().numpy(), P.squash(w, *two), dtype, "next", rel=0.004)
    assert np.isfinite(want).all()


@pytest.mark.parametrize("N, K, groups, keep, scale", [(9, 2, 3, 2, 1.7), (8, 3, 4, 2, 2.5), (12, 3, 2, 2, 0.6), (4, 2, 4, 3, 3.0),
                                                       (1, 1, 1, 1, 1.0), (256, 8, 8, 4, 2.5), (70, 5, 7, 1, 1.0),
                                                       (6, 1, 2, 1, 0.5), (640, 4, 64, 3, 1.0), (5, 5, 1, 1, 1.0)])
def test_router_with_groups(N, K, groups, keep, scale):
    """Choice by score + correction inside the groups whose two largest such scores add up to most, with corrections
    that make choice scores negative (an excluded expert must lose against them); weights by the score alone."""
    from allpaca_amd.kernels import ops
    rng = np.random.default_rng(N + K)
    T = 65
    z = np.float32(rng.normal(size=(T, N)) * 2)
    corr = np.float32(rng.normal(size=N) * 0.4 - 0.6)
    z[3, :] = z[3, 0]
    ids = torch.empty((T, K), dtype=torch.int32, device=DEV)
    w = torch.empty((T, K), dtype=torch.float32, device=DEV)
    ops.route_topk(dev(z), dev(corr), K, ids, w, True, score="sigmoid", groups=groups, keep_groups=keep, weight_scale=scale)
    negative = 0
    for t in range(T):
        want_ids, want_w = P.route(z[t].astype(np.float64), corr.astype(np.float64), K, scale, groups, keep)
        assert ids[t].cpu().tolist() == list(want_ids), (t, ids[t].cpu().tolist(), list(want_ids))
        assert np.allclose(w[t].cpu().numpy(), want_w, rtol=2e-6)
        negative += int((P.sigmoid(z[t].astype(np.float64)) + corr)[want_ids].min() < 0)
    assert negative or N > 64 or K < 2        # the case the exclusion must not be a zero for does come up


@pytest.mark.parametrize("D, F, E, K, T", [(36, 20, 5, 2, 19), (128, 64, 8, 2, 150), (64, 32, 3, 3, 40), (128, 32, 2, 1, 300),
                                           (96, 72, 10, 4, 7), (256, 128, 4, 2, 700), (64, 24, 6, 5, 1)])
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_experts_without_a_gate(D, F, E, K, T, dtype):
    """Few and many rows an expert (tiles of 16, 64 and 128 rows on the matrix cores), more choices than four, an expert
    nobody chose."""
    from allpaca_amd.kernels import ops
    rng = np.random.default_rng(D + F + E + T)
    tdt = DTYPES[dtype]
    h = bf(rng.normal(size=(T, D)))
    up, down = bf(rng.normal(size=(E, F, D)) / D ** 0.5), bf(rng.normal(size=(E, D, F)) / F ** 0.5)
    ids = np.stack([rng.permutation(E - 1 if E - 1 >= K else E)[:K] for _ in range(T)]).astype(np.int32)
    weights = np.float32(0.2 + 0.8 * rng.random(size=(T, K)))
    wu, wd = ops.prepare_experts(dev(up, tdt), dev(down, tdt), tdt)
    for weight_input in (False, True):
        y = torch.empty((T, D), dtype=torch.float32, device=DEV)
        ops.routed_experts(dev(h, tdt), wu, wd, E, F, dev(ids, torch.int32), dev(weights), K, y, activation="relu2",
                           weight_input=weight_input)
        want = np.zeros((T, D))
        for t in range(T):
            for e, we in zip(ids[t], weights[t].astype(np.float64)):
                want[t] += (we * we if weight_input else we) * (P.relu2(up[e] @ h[t]) @ down[e].T)
        close(y.cpu().numpy(), want, dtype, f"experts {weight_input}", rel=0.012)


@pytest.mark.parametrize("T, D, F", [(3, 96, 200), (16, 512, 1024), (40, 1024, 384), (100, 64, 30), (300, 2048, 256),
                                     (1100, 256, 512), (1030, 96, 130), (2050, 4096, 256)])
def test_activations_in_the_product_s_epilogue(T, D, F):
    """The bfloat16 products with an activation on their sums: the streaming kernel, the tiled one whole and with K in
    slices, the one for many rows."""
    from allpaca_amd.kernels import ops
    g = torch.Generator(device=DEV).manual_seed(T)
    h = torch.randn(T, D, generator=g, device=DEV).bfloat16()
    w = (torch.randn(F, D, generator=g, device=DEV) / D ** 0.5).bfloat16()
    z = (h.double() @ w.double().T).cpu().numpy()
    packed = ops.prepare_matrix(w, torch.bfloat16)
    for name, fn in (("gelu_tanh", P.gelu_tanh), ("relu2", P.relu2), ("silu", P.silu)):
        out = torch.full((T, F), float("nan"), dtype=torch.bfloat16, device=DEV)
        ops.linear_act(h, packed, out, name)
        close(out.float().cpu().numpy(), fn(z), "bfloat16", name, rel=0.006)


# =========================================================================================== whole models
# a mixer or a feed-forward alone: one layer
ALONE = {
    "latent": (_model(40, 24, 1e-5, [_layer(_lat(3, 4, 6, 8, 10, 0.5, 25.0, (2.0, 8, 4.0, 1.0)), None)]), 91),
    "scan": (_model(40, 24, 1e-5, [_layer(_scan(12, 3, 2, 3), None)]), 92),
    "lightning": (_model(40, 24, 1e-5, [_layer(_lig(2, 6, 10, (0.8, 0.97)), None)]), 93),
    "borrower": (_model(40, 24, 1e-5, [_layer(_lat(2, 4, 6, 8, 10, 0.5, 25.0), None), _layer(_lig(1, 4, 4, (0.7,)), _dense(12)),
                                       _layer(_lat(5, 8, 6, 2, 10, 0.4, 25.0, kv_from=0), _moe(8, 4, 2, 1.5, (2, 1)))]), 94),
}


def folder_of(name, dtype="float32"):
    """The model's folder; with "bfloat16" the one whose matrices are stored in 16 bits (the same values: the planted
    weights are numbers that bfloat16 holds), which a bfloat16 run keeps in the matrix-core kernels' layout."""
    if name in ALONE:
        path = os.path.join(tmp_root(), "muvorax_" + name)
        if not os.path.isdir(path):
            write_folder(path, *ALONE[name])
        return path
    return model_folder(name, dtype)


def make_runner(name, dtype, page_tokens=4, num_pages=160, max_requests=3, poison=False, use_graphs=False):
    from allpaca_amd.engine.runner import ModelRunner
    from allpaca_amd.models import load_model
    _, model = load_model(folder_of(name, dtype), DTYPES[dtype], DEV)
    return ModelRunner(model, page_tokens, num_pages, max_requests=max_requests, poison_free_pages=poison,
                       use_graphs=use_graphs)


def check(got, name, toks, dtype, what=""):
    """Logits of a whole model against the plain implementation's.  bfloat16: at most one and a half times what rounding
    the stored activations to bfloat16 costs the plain implementation itself (and 1% of the logits' size)."""
    folder = folder_of(name)
    want = oracle_logits(folder, toks)
    if dtype == "float32":
        close(got, want, "float32", what)
    else:
        rms, rows = oracle_noise(folder, toks)
        close(got, want, "bfloat16", what, rel=max(0.01, 1.5 * rms), rel_rows=max(0.01, 1.5 * rows))


@pytest.mark.parametrize("name", sorted(ALONE))
def test_a_mixer_alone(name):
    cfg, _ = ALONE[name]
    toks = np.random.default_rng(3).integers(0, cfg["vocab"], size=23).tolist()
    want = P.forward(*oracle(folder_of(name)), toks)
    for P_ in (1, 4):
        runner = make_runner(name, "float32", page_tokens=P_, num_pages=64)
        close(run_cut(runner, toks, [23]), want, "float32", "whole")
        close(run_cut(runner, toks, [1]), want, "float32", "token by token")
        close(run_cut(runner, toks, [2, 5, 3]), want, "float32", "portions")


def test_a_folder_whose_config_leaves_sizes_to_the_tensors_shapes():
    import shutil
    from test_muvorax_plain import bare
    from allpaca_amd.engine.runner import ModelRunner
    from allpaca_amd.models import load_model
    src = model_folder("MA")
    path = os.path.join(tmp_root(), "muvorax_MA_bare")
    shutil.copytree(src, path, dirs_exist_ok=True)
    with open(os.path.join(path, "config.json"), "w") as f:
        json.dump(bare(CONFIGS["MA"][0]), f)
    cfg, model = load_model(path, torch.float32, DEV)
    assert cfg.vocab == 83 and cfg.layers[1].mixer.kv_rank == 14 and cfg.layers[3].mlp.ff == 12
    toks = tokens_for("MA", 19, 4)
    close(run_cut(ModelRunner(model, 4, 64, max_requests=2), toks, [19]), oracle_logits(src, toks), "float32", "bare")


def test_layers_one_by_one_in_32_bit():
    """The residual stream after every layer, for a prompt and for its last token alone."""
    for name in CONFIGS:
        toks = tokens_for(name, 37, 3)
        want = []
        P.forward(*oracle(model_folder(name)), toks, taps=want)
        runner = make_runner(name, "float32")
        got = []
        runner.model.layer_tap = lambda i, x: got.append(x.detach().cpu().numpy().copy())
        run_cut(runner, toks, [36, 1])
        n = len(want)
        assert len(got) == 2 * n
        for i in range(n):
            close(np.concatenate([got[i], got[n + i]]), want[i], "float32", f"{name} layer {i}")


@pytest.mark.parametrize("name", sorted(CONFIGS))
@pytest.mark.parametrize("dtype, page_tokens", [("float32", 4), ("bfloat16", 4), ("bfloat16", 16), ("bfloat16", 3)])
def test_whole_prompts_decoding_and_portions(name, dtype, page_tokens):
    """101 tokens: more than a tile of keys and a chunk of the recurrent kernels; portions start and end inside pages,
    tiles, chunks and the convolutions' reach.  (Pages of 3 positions: the attention on its plain kernel.)"""
    toks = tokens_for(name, 101, 1)
    runner = make_runner(name, dtype, page_tokens=page_tokens)
    check(run_cut(runner, toks, [101]), name, toks, dtype, "whole")
    check(run_cut(runner, toks, [1]), name, toks, dtype, "token by token")
    check(run_cut(runner, toks, [40, 1]), name, toks, dtype, "prompt, then decoding")
    for cuts in ([2], [3, 2, 7, 1, 5], [6, 13, 2, 2, 66], [65, 1, 1, 2, 19, 3]):
        check(run_cut(runner, toks, cuts), name, toks, dtype, f"portions {cuts}")
    runner.cache.check()


def test_a_bfloat16_run_is_on_the_matrix_core_kernels():
    """A prompt portion and a decoded row of a model whose sizes the bfloat16 kernels take: the new mechanisms run on
    them and not on the plain kernels they would otherwise fall back to."""
    from allpaca_amd.engine.batch import Entry
    from allpaca_amd.kernels import lib as klib
    toks = tokens_for("MB", 70, 5)
    runner = make_runner("MB", "bfloat16", page_tokens=16)
    runner.admit("s")
    with klib.timing() as t:
        runner.step([Entry("s", toks[:69], [68])])
        runner.step([Entry("s", toks[69:], [0])])
    used = set(t.totals())
    runner.release("s")
    for name in ("apc_latent_rows_bf16", "apc_heads_gemm_bf16", "apc_latent_attention_bf16", "apc_linear_attention_bf16",
                 "apc_selective_scan_bf16", "apc_routed_experts_bf16", "apc_gemm_bf16"):
        assert name in used, (name, sorted(used))
    for name in ("apc_latent_rows", "apc_heads_gemm_plain", "apc_latent_attention_plain", "apc_routed_glu", "apc_gemm_plain",
                 "apc_act_rows"):
        assert name not in used, (name, sorted(used))


def test_cuttings_agree_to_the_bit_in_32_bit():
    for name in ("MA", "MC"):
        toks = tokens_for(name, 50, 8)
        runner = make_runner(name, "float32")
        whole = run_cut(runner, toks, [50])
        for cuts in ([1], [2], [7, 3, 1]):
            assert np.array_equal(whole, run_cut(runner, toks, cuts)), (name, cuts)


@pytest.mark.parametrize("name", ["MA", "MB"])
def test_first_tokens_and_page_sizes(name):
    for P_ in (1, 3, 16):
        runner = make_runner(name, "float32", page_tokens=P_, num_pages=200 if P_ == 1 else 80)
        for n in (1, 2, 3, 5, 7):
            toks = tokens_for(name, n, 40 + n)
            close(run_cut(runner, toks, [n]), oracle_logits(model_folder(name), toks), "float32", f"{n} tokens")
            close(run_cut(runner, toks, [1]), oracle_logits(model_folder(name), toks), "float32", f"{n} tokens, singly")


@pytest.mark.parametrize("name, dtype, page_tokens", [("MA", "float32", 4), ("MB", "float32", 4), ("MB", "bfloat16", 16),
                                                     ("MB", "bfloat16", 8), ("MC", "float32", 4), ("MD", "float32", 16),
                                                     ("MD", "bfloat16", 16)])
def test_mixed_batches_with_pages_and_slots_used_again(name, dtype, page_tokens):
    """Five requests of unequal lengths through three places and a pool that cannot hold them all at once: portions of
    some beside single tokens of others, free pages filled with a huge number, some requests left out of some steps.
    A request that comes later takes the pages and the state slot of one that has ended: a state that was not cleared,
    or a latent read from a page's unwritten places, would show."""
    from allpaca_amd.engine.batch import Entry
    rng = np.random.default_rng(9)
    lens = [37, 5, 90, 21, 70]
    reqs = {f"r{i}": tokens_for(name, n, 70 + i) for i, n in enumerate(lens)}
    P_ = page_tokens
    total = 50 * 4 // P_
    runner = make_runner(name, dtype, page_tokens=P_, num_pages=total, max_requests=3, poison=True)
    groups = range(len(runner.cache.paged_groups))

    def room(s, n, taken):
        need = runner.cache.pages_needed(s, n)
        return all(need[g] <= runner.cache.free_pages(g) - 2 * taken for g in groups)

    waiting, live, at, got = list(reqs), [], {}, {k: [] for k in reqs}
    while waiting or live:
        while waiting and len(live) < 3 and all(runner.cache.free_pages(g) >= -(-len(reqs[waiting[0]]) // P_) + 2
                                                for g in groups):
            s = waiting.pop(0)
            runner.admit(s)
            live.append(s)
            at[s] = 0
        entries = []
        for s in live:
            if rng.random() < 0.2 and len(live) > 1:
                continue                                   # left out of this step
            left = len(reqs[s]) - at[s]
            n = min(left, int(rng.choice([1, 1, 2, 3, 9, 16, 40])))
            if not room(s, n, len(entries)):
                n = 1
            entries.append(Entry(s, reqs[s][at[s]:at[s] + n], list(range(n))))
        if not entries:
            continue
        logits = runner.step(entries).cpu().numpy()
        r = 0
        for e in entries:
            n = len(e.tokens)
            got[e.seq].append(logits[r:r + n])
            r += n
            at[e.seq] += n
            if at[e.seq] == len(reqs[e.seq]):
                runner.release(e.seq)
                live.remove(e.seq)
    assert any(g.pool.allocations > total for g in runner.cache.paged_groups)      # pages came back and went out again
    for s, toks in reqs.items():
        check(np.concatenate(got[s]), name, toks, dtype, s)
    runner.cache.check()


def test_free_pages_full_of_nan_change_no_bit():
    """What lies in places of pages that a request has not written never enters a product, in either element type."""
    for name, dtype, P_ in (("MA", "float32", 4), ("MB", "bfloat16", 16)):
        toks = tokens_for(name, 75, 12)
        outs = []
        for poison in (False, float("nan")):
            runner = make_runner(name, dtype, page_tokens=P_, poison=poison)
            outs.append(run_cut(runner, toks, [33, 2, 30, 1]))
        assert np.array_equal(outs[0], outs[1]), name


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_long_decoding(dtype):
    """A short prompt, then 280 tokens one by one: many key tiles and pages go by, the states run through hundreds of
    single steps, the keys begin to be cut into ranges."""
    toks = tokens_for("MB", 300, 2)
    check(run_cut(make_runner("MB", dtype, page_tokens=16, num_pages=160), toks, [20, 1]), "MB", toks, dtype,
          "long decoding")


def test_a_key_far_back_in_a_whole_model():
    """An owner of latents and a borrower; the embedding of one token is made large, so that its key, hundreds of
    positions back, stands out for the rows that follow: in a prompt, in portions, in decoded rows."""
    from allpaca_amd.engine.runner import ModelRunner
    from allpaca_amd.models import load_model
    cfg = _model(60, 32, 1e-6, [_layer(_lat(4, 8, 8, 8, 16, 0.6, 100.0, (2.0, 64, 8.0, 1.0)), _dense(40)),
                                _layer(_lat(2, 8, 8, 16, 16, 0.6, 100.0, (2.0, 64, 8.0, 1.0), kv_from=0), None)])
    w = planted(cfg, 77)
    w["embed"][7] *= 6.0
    path = os.path.join(tmp_root(), "muvorax_far_key")
    if not os.path.isdir(path):
        write_folder(path, cfg, 77, weights=w)
    rng = np.random.default_rng(4)
    toks = [int(t) if t != 7 else 8 for t in rng.integers(0, 60, size=420)]
    toks[5] = 7
    want = P.forward(*P.read_model_folder(path), toks)
    plain = list(toks)
    plain[5] = 8
    moved = np.abs(P.forward(*P.read_model_folder(path), plain)[400:] - want[400:]).max()
    assert moved > 1e-2, moved                     # the far token does reach the last rows
    _, model = load_model(path, torch.float32, DEV)
    runner = ModelRunner(model, 16, 64, max_requests=2, poison_free_pages=True)
    close(run_cut(runner, toks, [420]), want, "float32", "whole")
    close(run_cut(runner, toks, [390, 1]), want, "float32", "decoded")
    close(run_cut(runner, toks, [100, 3, 100, 43, 2]), want, "float32", "portions")


def test_greedy_generation_through_the_engine():
    """Requests of unequal lengths through the engine's scheduler, sampler and decode graphs, in float32: the tokens
    are the plain implementation's."""
    from allpaca_amd.engine import Engine
    from allpaca_amd.sampling import GenerationParams
    for name in ("MA", "MB"):
        folder = model_folder(name)
        prompts = [tokens_for(name, n, 90 + n) for n in (1, 9, 30, 4, 17)]
        want = [P.greedy(*oracle(folder), p, 10) for p in prompts]
        for graphs in (True, False):
            engine = Engine(folder, dtype="float32", max_tokens=512, page_tokens=4, max_active_requests=3,
                            chunk_tokens=8, max_batch_tokens=16, use_graphs=graphs)
            assert engine.runner.use_graphs == graphs
            outs = engine.generate(prompts, GenerationParams(max_tokens=10, temperature=0.0))
            assert [o.token_ids for o in outs] == want, (name, graphs)


def test_graphs_replay_decode_steps_in_bfloat16():
    """Decode steps recorded as graphs and replayed give the tokens of the same engine without graphs."""
    from allpaca_amd.engine import Engine
    from allpaca_amd.sampling import GenerationParams
    folder = model_folder("MB", "bfloat16")
    prompts = [tokens_for("MB", n, 50 + n) for n in (3, 40, 11)]
    outs = []
    for graphs in (True, False):
        engine = Engine(folder, dtype="bfloat16", max_tokens=1024, page_tokens=16, max_active_requests=3,
                        use_graphs=graphs)
        assert engine.runner.use_graphs == graphs
        outs.append([o.token_ids for o in engine.generate(prompts, GenerationParams(max_tokens=20, temperature=0.0))])
    assert outs[0] == outs[1]


def test_command_line_and_replay_program(tmp_path):
    """The command line on a model folder of the design (float32, greedy: the plain implementation's tokens), and the
    replay program: three requests through a pool that holds two of them."""
    root = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
    folder = model_folder("MA")
    prompts = [tokens_for("MA", 7, 5), tokens_for("MA", 19, 6)]
    spec = ";".join(",".join(str(t) for t in p) for p in prompts)
    cmd = [sys.executable, os.path.join(root, "bin", "allpaca-amd"), "generate", "--model", folder, "--dtype", "fp32",
           "--prompt-tokens", spec, "--max-tokens", "6", "--temperature", "0", "--json"]
    r = subprocess.run(cmd, capture_output=True, text=True, timeout=300)
    assert r.returncode == 0, r.stderr[-2000:]
    outs = [json.loads(ln) for ln in r.stdout.strip().splitlines() if ln.startswith("{")]
    assert [o["token_ids"] for o in outs] == [P.greedy(*oracle(folder), p, 6) for p in prompts]
    # the design's preset with random weights, sampled with temperature, top-k and top-p in bfloat16
    cmd = [sys.executable, os.path.join(root, "bin", "allpaca-amd"), "generate", "--synthetic", "muvorax-tiny",
           "--prompt-tokens", "1,2,3;4,5", "--max-tokens", "5", "--temperature", "0.8", "--top-k", "20", "--top-p",
           "0.9", "--json"]
    r = subprocess.run(cmd, capture_output=True, text=True, timeout=300)
    assert r.returncode == 0, r.stderr[-2000:]
    outs = [json.loads(ln) for ln in r.stdout.strip().splitlines() if ln.startswith("{")]
    assert len(outs) == 2 and all(len(o["token_ids"]) == 5 for o in outs)

    name = "MB"
    folder = model_folder(name)
    a, b, c = tokens_for(name, 70, 31), tokens_for(name, 9, 32), tokens_for(name, 50, 33)
    steps = [
        dict(step=0, entries=[dict(id="a", tokens=a[:33], want=list(range(33))), dict(id="b", tokens=b[:1], want=[0])], end=[]),
        dict(step=1, entries=[dict(id="b", tokens=b[1:3], want=[0, 1])], end=[]),
        dict(step=2, entries=[dict(id="a", tokens=a[33:69], want=list(range(36))), dict(id="b", tokens=b[3:], want=list(range(6)))],
             end=["b"]),
        dict(step=3, entries=[dict(id="a", tokens=a[69:], want=[0]), dict(id="c", tokens=c[:2], want=[0, 1])], end=["a"]),
        dict(step=4, entries=[dict(id="c", tokens=c[2:], want=list(range(48)))], end=["c"]),
    ]
    for dtype in ("float32", "bfloat16"):
        out = str(tmp_path / f"replay_{dtype}")
        cmd = [sys.executable, os.path.join(root, "bin", "trace_run"), "--model", folder, "--dtype", dtype, "--out", out,
               "--max-tokens", "192", "--max-live", "2", "--poison-free-pages"]
        r = subprocess.run(cmd, input="".join(json.dumps(s) + "\n" for s in steps), capture_output=True, text=True,
                           timeout=280)
        assert r.returncode == 0, r.stderr[-3000:]
        assert [ln for ln in r.stdout.split("\n") if ln.startswith("done")] == [f"done {i}" for i in range(5)]
        V = CONFIGS[name][0]["vocab"]
        got = {k: [] for k in "abc"}
        for s in steps:
            rows = np.fromfile(os.path.join(out, f"{s['step']}.f32"), dtype="<f4").reshape(-1, V)
            at = 0
            for e in s["entries"]:
                got[e["id"]].append(rows[at:at + len(e["want"])])
                at += len(e["want"])
            assert at == rows.shape[0]
        for k, toks in zip("abc", (a, b, c)):
            check(np.concatenate(got[k]), name, toks, dtype, f"replay {k}")


def test_a_model_without_pages_generates():
    """Recurrent layers alone: no pool of pages, only state slots, through the engine with and without graphs."""
    from allpaca_amd.engine import Engine
    from allpaca_amd.sampling import GenerationParams
    for name in ("scan", "lightning"):
        folder = folder_of(name)
        cfg, W = oracle(folder)
        prompts = [np.random.default_rng(n).integers(0, cfg["vocab"], size=n).tolist() for n in (1, 9, 14)]
        want = [P.greedy(cfg, W, p, 8) for p in prompts]
        for graphs in (True, False):
            engine = Engine(folder, dtype="float32", max_tokens=256, page_tokens=4, max_active_requests=2, chunk_tokens=8,
                            max_batch_tokens=16, use_graphs=graphs)
            outs = engine.generate(prompts, GenerationParams(max_tokens=8, temperature=0.0))
            assert [o.token_ids for o in outs] == want, (name, graphs)
