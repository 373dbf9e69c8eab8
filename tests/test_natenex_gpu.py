"""The Natenex decoder on the GPU against the plain implementation (tests/plain_natenex.py): every new kernel alone,
then whole models of several shapes through the step function, the cache manager and the engine."""
import json
import os
import subprocess
import sys

import numpy as np
import pytest
import torch

import plain_natenex as P
from helpers import tmp_root
from natenex_helpers import (CONFIGS, _del, _lat, _layer, _model, _par, model_folder, oracle, oracle_logits, oracle_noise,
                             planted, tokens_for, write_folder)
from test_seredra_gpu import DEV, DTYPES, bf, close, dev, fill_pages, make_step, run_cut, scattered_tables

pytestmark = pytest.mark.gpu


def rows_of(segs):
    return sum(n for _, n in segs)


# =========================================================================================== kernels alone
@pytest.mark.parametrize("H, G, dk, dv, P_, W, keep", [(4, 2, 12, 10, 4, 11, 5), (3, 3, 16, 14, 3, 40, 0), (6, 1, 7, 5, 1, 1, 1),
                                                       (8, 2, 64, 64, 16, 40, 24), (12, 4, 96, 96, 16, 64, 64),
                                                       (4, 1, 128, 128, 16, 100, 130), (6, 2, 40, 24, 8, 17, 33),
                                                       (8, 8, 32, 64, 16, 1, 7), (16, 1, 64, 128, 32, 65, 257),
                                                       (2, 2, 256, 32, 64, 30, 63)])
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_a_window_with_kept_first_tokens_over_pages_with_keys_that_stand_out(H, G, dk, dv, P_, W, keep, dtype):
    """Portions that start inside and behind the kept tokens beside decoded rows, on scattered pages; the pages that
    window and kept tokens no longer reach hold NaN, as do all unwritten places.  Some rows ask, with a large query,
    for one key: the last kept one, the first that is not kept, just inside and just outside the window, themselves."""
    from allpaca_amd.kernels import ops
    rng = np.random.default_rng(H + dk + W + keep)
    tdt = DTYPES[dtype]
    segs = [(200, 70), (300, 1), (64, 1), (63, 1), (0, 1), (127, 2), (0, 90), (keep, 1), (max(keep - 1, 0), 3), (W, 2),
            (keep + W, 1), (700, 3), (777, 1)]
    lens = [p + n for p, n in segs]
    n_pages, tables = scattered_tables(rng, lens, P_)
    keys = [bf(rng.normal(size=(n, G, dk))) for n in lens]
    vals = [bf(rng.normal(size=(n, G, dv))) for n in lens]
    T = rows_of(segs)
    row0 = np.cumsum([0] + [n for _, n in segs])
    q = bf(rng.normal(size=(T, H, dk)))
    wanted = [("kept", keep - 1), ("not kept", keep), ("inside", None), ("outside", None), ("own", None)]
    for s, (p0, n) in enumerate(segs):
        for i in {0, n // 2, n - 1}:
            pos = p0 + i
            for h, (what, j) in zip(range(H), wanted[(s + i) % 5:] + wanted[:(s + i) % 5]):
                j = {"inside": pos - W + 1, "outside": pos - W, "own": pos}.get(what, j)
                if 0 <= j <= pos:
                    q[row0[s] + i, h] = bf(keys[s][j, h // (H // G)] * (25.0 / np.sqrt(dk)))
    cache = np.full((n_pages + 1, G, P_ * (dk + dv)), np.nan, dtype=np.float32)
    fill_pages(cache, tables, keys, vals, P_)
    scale = 0.9 / np.sqrt(dk)
    want = []
    for s, (p0, n) in enumerate(segs):
        want.append(P.softmax_attention(q[row0[s]:row0[s] + n], keys[s], vals[s], scale, p0, dict(size=W, keep_first=keep)))
        # pages that no row of the step (nor a later one) reaches are given back: the spare page stands for them
        for page in range(len(tables[s])):
            if page * P_ >= keep and (page + 1) * P_ - 1 < p0 - W + 1:
                tables[s][page] = n_pages
    step = make_step(segs, tables)
    out = torch.full((T, H * dv), float("nan"), dtype=tdt, device=DEV)
    ops.masked_attention(dev(q.reshape(T, -1), tdt), out, H, G, dk, dv, dev(cache, tdt), P_, step.block_tables[0], step,
                         "window", W, False, scale, keep_first=keep, out_scale=1.7)
    got = out.float().cpu().numpy().reshape(T, H, dv)
    for s, (p0, n) in enumerate(segs):
        close(got[row0[s]:row0[s] + n].reshape(n, -1), 1.7 * want[s].reshape(n, -1), dtype,
              f"segment {segs[s]} window {W} keep {keep}", rel=0.012)


def delta_case(rng, segs, H, G, dk, dv, tdt, fast):
    T = rows_of(segs)
    width = -(-(2 * G * dk + H * dv) // 8) * 8
    rows = bf(rng.normal(size=(T, width)))
    rows[rng.integers(0, T, size=3), :2 * G * dk] *= 2.0 ** -13      # keys and queries near zero: eps under the root matters
    ba = bf(rng.normal(size=(T, -(-2 * H // 8) * 8 + 8)) * (2.0 if fast else 1.0))
    A = np.float32(np.exp(rng.normal(size=H) * (1.5 if fast else 0.7) - (0.0 if fast else 2.0)))
    bias = np.float32(rng.normal(size=H) - 1.0)
    return rows, ba, A, bias


@pytest.mark.parametrize("H, G, dk, dv", [(3, 1, 6, 5), (4, 2, 64, 32), (4, 4, 128, 128), (6, 2, 72, 40), (2, 1, 136, 24), (1, 1, 8, 16),
                                          (8, 4, 32, 65), (16, 8, 96, 64), (2, 2, 256, 20), (5, 5, 40, 18)])
@pytest.mark.parametrize("dtype, fast", [("float32", False), ("bfloat16", False), ("bfloat16", True), ("float32", True)])
def test_the_gated_delta_rule_over_portions_and_single_rows(H, G, dk, dv, dtype, fast):
    """Three steps of four requests from a random state: portions of several chunks and of parts of one, of 63, 64 and 65
    rows, single rows; decays from nearly one to nearly nothing (`fast`), keys that repeat (the system a chunk solves is
    then far from the identity)."""
    from allpaca_amd.kernels import ops
    rng = np.random.default_rng(H * 10 + dk + dv)
    tdt = DTYPES[dtype]
    cuts = [[150, 64, 1, 7], [63, 65, 2, 1], [1, 1, 1, 1], [5, 128, 40, 3]]
    state = np.float32(rng.normal(size=(5, H, dk, dv)))
    slots = [2, 0, 3, 1]
    gpu_state = dev(state)
    S = {i: state[slots[i]].astype(np.float64) for i in range(4)}
    at = [0] * 4
    for lens in cuts:
        segs = [(a, n) for a, n in zip(at, lens)]
        step = make_step(segs, [[1]] * 4, slots)
        rows, ba, A, bias = delta_case(rng, segs, H, G, dk, dv, tdt, fast)
        if lens[0] > 100:
            rows[20:90, G * dk:2 * G * dk] = rows[20, G * dk:2 * G * dk]
        T = rows.shape[0]
        out = torch.full((T, H * dv), float("nan"), dtype=torch.float32, device=DEV)
        a_off, b_off = 3, 3 + H
        ops.delta_rule(dev(rows, tdt), 0, G * dk, 2 * G * dk, H, G, dk, dv, dev(ba, tdt), a_off, b_off, dev(A), dev(bias),
                       gpu_state, step, step.state_slots, out)
        got, r = out.cpu().numpy(), 0
        for i, n in enumerate(lens):
            x, y = rows[r:r + n], ba[r:r + n]
            q = np.repeat(P.unit(x[:, :G * dk].reshape(n, G, dk)) * dk ** -0.5, H // G, axis=1)
            k = np.repeat(P.unit(x[:, G * dk:2 * G * dk].reshape(n, G, dk)), H // G, axis=1)
            beta, g = P.sigmoid(y[:, b_off:b_off + H]), np.exp(-A * P.softplus(y[:, a_off:a_off + H] + bias))
            v = x[:, 2 * G * dk:2 * G * dk + H * dv].reshape(n, H, dv)
            want, S[i] = P.delta_rule(q, k, v, beta, g, S[i])
            what = f"{n} rows of request {i} of {lens}"
            close(got[r:r + n], want.reshape(n, -1), dtype, what, rel=0.001)
            close(gpu_state[slots[i]].cpu().numpy().reshape(dk * H, dv), S[i].reshape(dk * H, dv), dtype, what + ", state",
                  rel=0.001)
            r += n
            at[i] += n
    assert np.array_equal(gpu_state[4].cpu().numpy(), state[4])          # another slot is left alone


@pytest.mark.parametrize("C, blocks", [(15, 5), (128, 4), (8, 1), (130, 13), (1, 1), (2048, 16), (576, 2), (64, 32)])
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_the_gated_recurrence_over_portions_and_single_rows(C, blocks, dtype):
    """Steps of four requests from a random state: portions of several chunks, of whole and of broken runs, single rows;
    decays from one (to rounding: the root of 1 - a^2 without cancellation) to nothing; a factor on what leaves."""
    from allpaca_amd.kernels import ops
    rng = np.random.default_rng(C)
    tdt = DTYPES[dtype]
    w = C // blocks
    lam = rng.normal(size=C) * 3.0 - 4.0
    lam[:max(1, C // 8)] = -14.0
    rate = np.float32(-8.0 * P.softplus(lam))
    br, bi, yb = (np.float32(rng.normal(size=C) * 0.5) for _ in range(3))

    def laid(r, i):           # a part's r logits, then its i logits
        return np.concatenate([r.reshape(*r.shape[:-1], blocks, w), i.reshape(*i.shape[:-1], blocks, w)],
                              axis=-1).reshape(*r.shape[:-1], 2 * C)

    state = np.float32(rng.normal(size=(5, C)))
    slots = [3, 1, 0, 4]
    gpu_state = dev(state)
    S = {i: state[slots[i]].astype(np.float64) for i in range(4)}
    for lens in ([150, 64, 1, 17], [63, 66, 16, 2], [1, 1, 1, 1], [300, 33, 15, 48]):
        T = sum(lens)
        segs = [(0, n) for n in lens]
        step = make_step(segs, [[1]] * 4, slots)
        u, y = bf(rng.normal(size=(T, C))), bf(rng.normal(size=(T, C)))
        zr, zi = np.float32(rng.normal(size=(T, C)) * 2), np.float32(rng.normal(size=(T, C)) * 2)
        out = torch.full((T, C + C % 2 + 2), 9.0, dtype=tdt, device=DEV)
        ops.gated_recurrence(dev(u, tdt), dev(laid(zr, zi)), dev(laid(br, bi)), blocks, dev(rate), dev(y, tdt), dev(yb),
                             gpu_state, step, step.state_slots, out[:, :C], out_scale=0.6)
        assert (out[:, C:] == 9.0).all()
        got, r = out[:, :C].float().cpu().numpy(), 0
        for i, n in enumerate(lens):
            a = slice(r, r + n)
            s, S[i] = P.gated_recurrence(u[a], P.sigmoid(zr[a] + br.astype(float)), P.sigmoid(zi[a] + bi.astype(float)), lam, S[i])
            close(got[a], 0.6 * s * P.gelu_tanh(y[a] + yb), dtype, f"{n} rows of request {i} of {lens}", rel=0.004)
            close(gpu_state[slots[i]].cpu().numpy()[None], S[i][None], "float32", "state")
            r += n
    assert np.array_equal(gpu_state[2].cpu().numpy(), state[2])


@pytest.mark.parametrize("C, taps, act", [(15, 3, "none"), (704, 4, "silu"), (72, 2, "none"), (40, 1, "silu"), (16, 8, "silu"),
                                          (24, 4, "none")])
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_convolution_with_an_input_bias_whose_state_moves_on_with_single_rows(C, taps, act, dtype):
    """What the convolution keeps are its inputs with their bias; ahead of the sequence there are zeros, not biases.
    Steps of portions, then steps of single rows alone (the state is moved on in the same launch), then portions."""
    from allpaca_amd.kernels import ops
    rng = np.random.default_rng(C + taps)
    tdt = DTYPES[dtype]
    cuts = [[5, 1, 2], [1, 1, 1], [1, 1, 1], [3, 1, 9], [1, 1, 1]]
    total = [sum(c[i] for c in cuts) for i in range(3)]
    rows = [bf(rng.normal(size=(n, C + 8))) for n in total]
    w, b, ib = (np.float32(rng.normal(size=s)) for s in ((C, taps), C, C))
    state = torch.zeros((4, taps - 1, C), dtype=torch.float32, device=DEV) if taps > 1 else None
    got, at = [[], [], []], [0, 0, 0]
    for lens in cuts:
        step = make_step([(a, n) for a, n in zip(at, lens)], [[1]] * 3, [2, 0, 1])
        x = np.concatenate([r[a:a + n] for r, a, n in zip(rows, at, lens)])
        out = torch.full((x.shape[0], C), float("nan"), dtype=tdt, device=DEV)
        ops.conv_channels(dev(x, tdt), C, dev(w), dev(b), state, step, step.state_slots if taps > 1 else None, act, out,
                          in_bias=dev(ib))
        r = 0
        for i, n in enumerate(lens):
            got[i].append(out[r:r + n].float().cpu().numpy())
            r, at[i] = r + n, at[i] + n
    for i in range(3):
        y = P.short_conv(rows[i][:, :C] + ib, w.astype(float)) + b
        close(np.concatenate(got[i]), P.silu(y) if act == "silu" else y, dtype, f"request {i}", rel=0.006)


@pytest.mark.parametrize("T, H, N, K", [(3, 5, 14, 6), (16, 12, 96, 32), (17, 4, 40, 24), (130, 2, 512, 128), (9, 32, 128, 512),
                                        (70, 2, 66, 16), (1, 1, 8, 8)])
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_head_products_with_a_gate_and_with_32_bit_outputs(T, H, N, K, dtype):
    from allpaca_amd.kernels import ops
    rng = np.random.default_rng(T + N)
    tdt = DTYPES[dtype]
    a, w = bf(rng.normal(size=(T, H * K))), bf(rng.normal(size=(H, N, K)) / K ** 0.5)
    gate = bf(rng.normal(size=(T, H * N)) * 2)
    wide = torch.zeros((T, -(-(H * N) // 8) * 8 + 8), dtype=tdt, device=DEV)
    wide[:, 8:8 + H * N] = dev(gate, tdt)
    packed = ops.prepare_heads(dev(w, tdt), tdt, K, N)
    want = np.einsum("thk,hnk->thn", a.reshape(T, H, K), w).reshape(T, -1)
    out = torch.full((T, H * N), float("nan"), dtype=tdt, device=DEV)
    ops.heads_linear(dev(a, tdt), K, packed, out, N, gate=wide[:, 8:8 + H * N])
    close(out.float().cpu().numpy(), want * P.sigmoid(gate), dtype, "gated", rel=0.006)
    out = torch.full((T, H * N), float("nan"), dtype=torch.float32, device=DEV)
    ops.heads_linear(dev(a, tdt), K, packed, out, N)
    close(out.cpu().numpy(), want, "float32", "32-bit outputs")


def test_head_norm_over_every_head_with_one_weight_and_a_silu_gate():
    from allpaca_amd.kernels import ops
    rng = np.random.default_rng(0)
    for T, H, dv in ((3, 5, 7), (40, 8, 128), (9, 3, 65)):
        o, g, w = np.float32(rng.normal(size=(T, H * dv))), np.float32(rng.normal(size=(T, H * dv))), np.float32(rng.normal(size=dv))
        out = torch.empty((T, H * dv), dtype=torch.float32, device=DEV)
        ops.gated_rmsnorm(dev(o), dev(np.tile(w, H)), 1e-3, dev(g), out, group=dv, gate_act="silu")
        want = P.rms_norm(o.reshape(T, H, dv).astype(float), w, 1e-3).reshape(T, -1) * P.silu(g.astype(float))
        close(out.cpu().numpy(), want, "float32", "norm")


# =========================================================================================== whole models
# a mixer alone: one layer
ALONE = {
    "window": (_model(40, 24, 1e-5, 2.0, [_layer(_par(4, 2, 6, 8, 0.5, (30.0, 4), (7, 3), 6, 2, 3, (1.0, 0.0)))]), 71),
    "recurrence": (_model(40, 24, 1e-5, 2.0, [_layer(_par(1, 1, 2, 2, 0.5, (30.0, 0), (2, 0), 12, 3, 4, (0.0, 1.0)))]), 72),
    "latents": (_model(40, 24, 1e-5, 2.0, [_layer(_lat(3, 4, 6, 8, 14, 10, 0.5, 25.0, (2.0, 1.0, 4.0, 12)))]), 73),
    "delta": (_model(40, 24, 1e-5, 2.0, [_layer(_del(6, 3, 5, 7, 3))]), 74),
    "shared": (_model(40, 24, 1e-5, 2.0, [_layer(_del(2, 1, 4, 6, 2), 12), _layer(_del(2, 1, 4, 6, 2), 12, of=0)]), 75),
}


def folder_of(name, dtype="float32"):
    """The model's folder; with "bfloat16" the one whose matrices are stored in 16 bits (the same values: the planted
    weights are numbers that bfloat16 holds), which a bfloat16 run keeps in the matrix-core kernels' layout."""
    if name in ALONE:
        path = os.path.join(tmp_root(), "natenex_" + name)
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
    from test_natenex_plain import bare
    from allpaca_amd.engine.runner import ModelRunner
    from allpaca_amd.models import load_model
    src = model_folder("NA")
    path = os.path.join(tmp_root(), "natenex_NA_bare")
    shutil.copytree(src, path, dirs_exist_ok=True)
    with open(os.path.join(path, "config.json"), "w") as f:
        json.dump(bare(CONFIGS["NA"][0]), f)
    cfg, model = load_model(path, torch.float32, DEV)
    assert cfg.vocab == 71 and cfg.layers[2].mixer.q_rank == 13 and cfg.layers[3].ff == 22
    toks = tokens_for("NA", 19, 4)
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
    """101 tokens: more than every window, a tile of keys and a chunk of the recurrent kernels; portions start and end
    inside pages, windows, tiles, chunks and the convolutions' reach.  (Pages of 3 positions: attention on its plain
    kernel.)"""
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
    toks = tokens_for("NB", 70, 5)
    runner = make_runner("NB", "bfloat16", page_tokens=16)
    runner.admit("s")
    with klib.timing() as t:
        runner.step([Entry("s", toks[:69], [68])])
        runner.step([Entry("s", toks[69:], [0])])
    used = set(t.totals())
    runner.release("s")
    for name in ("apc_latent_rows_bf16", "apc_heads_gemm_bf16", "apc_latent_attention_bf16", "apc_delta_rule_bf16",
                 "apc_gated_recurrence_bf16", "apc_attention_masked_prefill_bf16", "apc_attention_masked_decode_bf16",
                 "apc_rotary_pages_bf16", "apc_gemm_bf16"):
        assert name in used, (name, sorted(used))
    for name in ("apc_latent_rows", "apc_heads_gemm_plain", "apc_latent_attention_plain", "apc_masked_attention_plain",
                 "apc_gemm_plain", "apc_act_rows", "apc_weighted_pair", "apc_rotary_pages"):
        assert name not in used, (name, sorted(used))


def test_cuttings_agree_to_the_bit_in_32_bit():
    for name in ("NA", "NC"):
        toks = tokens_for(name, 50, 8)
        runner = make_runner(name, "float32")
        whole = run_cut(runner, toks, [50])
        for cuts in ([1], [2], [7, 3, 1]):
            assert np.array_equal(whole, run_cut(runner, toks, cuts)), (name, cuts)


@pytest.mark.parametrize("name", ["NA", "NB", "NC"])
def test_first_tokens_and_page_sizes(name):
    for P_ in (1, 3, 16):
        runner = make_runner(name, "float32", page_tokens=P_, num_pages=200 if P_ == 1 else 80)
        for n in (1, 2, 3, 5, 7):
            toks = tokens_for(name, n, 40 + n)
            close(run_cut(runner, toks, [n]), oracle_logits(model_folder(name), toks), "float32", f"{n} tokens")
            close(run_cut(runner, toks, [1]), oracle_logits(model_folder(name), toks), "float32", f"{n} tokens, singly")


@pytest.mark.parametrize("name, dtype, page_tokens", [("NA", "float32", 4), ("NB", "float32", 4), ("NB", "bfloat16", 16),
                                                     ("NB", "bfloat16", 8), ("NC", "float32", 4), ("ND", "float32", 16),
                                                     ("ND", "bfloat16", 16)])
def test_mixed_batches_with_pages_and_slots_used_again(name, dtype, page_tokens):
    """Five requests of unequal lengths through three places and a pool that cannot hold them all at once: portions of
    some beside single tokens of others, free pages filled with a huge number, some requests left out of some steps.
    A request that comes later takes the pages and the state slot of one that has ended: a state that was not cleared,
    a key read from a page that was given back, or a kept page that was given back would show."""
    from allpaca_amd.engine.batch import Entry
    rng = np.random.default_rng(9)
    lens = [37, 5, 90, 21, 70]
    reqs = {f"r{i}": tokens_for(name, n, 70 + i) for i, n in enumerate(lens)}
    P_ = page_tokens
    total = 60 * 4 // P_
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
    assert all(g.pool.allocations > 0 for g in runner.cache.paged_groups)
    for s, toks in reqs.items():
        check(np.concatenate(got[s]), name, toks, dtype, s)
    runner.cache.check()


@pytest.mark.parametrize("dtype, P_", [("float32", 4), ("bfloat16", 8), ("bfloat16", 16)])
def test_a_pool_that_only_holds_windows_and_kept_tokens(dtype, P_):
    """One request after the other, each longer than the pool: pages that the window has passed go round many times
    beside the kept ones, in portions and in single tokens, free pages full of NaN."""
    from allpaca_amd.engine.runner import ModelRunner
    from allpaca_amd.models import load_model
    cfg = _model(60, 32, 1e-6, 2.0, [_layer(_par(4, 2, 16, 16, 0.4, (100.0, 8), (20, 9), 16, 2, 3, (1.0, 0.5)), 40),
                                     _layer(_par(4, 2, 16, 16, 0.4, (100.0, 8), (20, 9), 16, 2, 3, (1.0, 0.5)), 40, of=0)])
    path = os.path.join(tmp_root(), "natenex_small_pool")
    if not os.path.isdir(path):
        write_folder(path, cfg, 78)
    _, model = load_model(path, DTYPES[dtype], DEV)
    runner = ModelRunner(model, P_, -(-9 // P_) + -(-20 // P_) + 1 + -(-10 // P_), max_requests=1, poison_free_pages=float("nan"))
    for seed, cuts in ((1, [10]), (2, [1]), (3, [7, 1, 1, 10, 2])):
        toks = np.random.default_rng(seed).integers(0, 60, size=150).tolist()
        want = P.forward(*P.read_model_folder(path), toks)
        close(run_cut(runner, toks, cuts), want, dtype, f"{cuts}", rel=0.03)
    assert runner.cache.paged_groups[0].pool.allocations > 2 * runner.cache.paged_groups[0].pool.num_pages


def test_free_pages_full_of_nan_change_no_bit():
    """What lies in places of pages that a request has not written never enters a product, in either element type."""
    for name, dtype, P_ in (("NA", "float32", 4), ("NB", "bfloat16", 16)):
        toks = tokens_for(name, 75, 12)
        outs = []
        for poison in (False, float("nan")):
            runner = make_runner(name, dtype, page_tokens=P_, poison=poison)
            outs.append(run_cut(runner, toks, [33, 2, 30, 1]))
        assert np.array_equal(outs[0], outs[1]), name


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_long_decoding(dtype):
    """A short prompt, then 280 tokens one by one: windows, key tiles and pages go by, the states run through hundreds of
    single steps, the keys begin to be cut into ranges."""
    toks = tokens_for("NB", 300, 2)
    check(run_cut(make_runner("NB", dtype, page_tokens=16, num_pages=160), toks, [20, 1]), "NB", toks, dtype,
          "long decoding")


@pytest.mark.parametrize("kept", [True, False])
def test_a_key_far_back_in_a_whole_model(kept):
    """The embedding of one token is made large, so that its key stands out for the rows that follow: the latents see it
    hundreds of positions back; the window sees it as the last kept token and not as the next one."""
    from allpaca_amd.engine.runner import ModelRunner
    from allpaca_amd.models import load_model
    window = _layer(_par(4, 2, 8, 8, 0.5, (100.0, 4), (30, 6), 8, 1, 1, (1.0, 0.0)), 40)
    cfg = _model(60, 32, 1e-6, 1.0, [window] if not kept else [window, _layer(_lat(4, 8, 8, 8, 24, 16, 0.6, 100.0), 40)])
    w = planted(cfg, 79)
    w["embed"][7] *= 6.0
    path = os.path.join(tmp_root(), f"natenex_far_key_{kept}")
    if not os.path.isdir(path):
        write_folder(path, cfg, 79, weights=w)
    rng = np.random.default_rng(4)
    toks = [int(t) if t != 7 else 8 for t in rng.integers(0, 60, size=420)]
    toks[5 if kept else 6] = 7
    want = P.forward(*P.read_model_folder(path), toks)
    plain = [8 if t == 7 else t for t in toks]
    moved = np.abs(P.forward(*P.read_model_folder(path), plain)[400:] - want[400:]).max()
    assert (moved > 1e-2) == kept, moved
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
    for name in ("NA", "NB"):
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
    folder = model_folder("NB", "bfloat16")
    prompts = [tokens_for("NB", n, 50 + n) for n in (3, 40, 11)]
    outs = []
    for graphs in (True, False):
        engine = Engine(folder, dtype="bfloat16", max_tokens=1024, page_tokens=16, max_active_requests=3,
                        use_graphs=graphs)
        assert engine.runner.use_graphs == graphs
        outs.append([o.token_ids for o in engine.generate(prompts, GenerationParams(max_tokens=60, temperature=0.0))])
    assert outs[0] == outs[1]


def test_a_model_without_pages_generates():
    """Recurrent layers alone: no pool of pages, only state slots, through the engine with and without graphs."""
    from allpaca_amd.engine import Engine
    from allpaca_amd.sampling import GenerationParams
    for name in ("delta", "shared"):
        folder = folder_of(name)
        cfg, W = oracle(folder)
        prompts = [np.random.default_rng(n).integers(0, cfg["vocab"], size=n).tolist() for n in (1, 9, 14)]
        want = [P.greedy(cfg, W, p, 8) for p in prompts]
        for graphs in (True, False):
            engine = Engine(folder, dtype="float32", max_tokens=256, page_tokens=4, max_active_requests=2, chunk_tokens=8,
                            max_batch_tokens=16, use_graphs=graphs)
            outs = engine.generate(prompts, GenerationParams(max_tokens=8, temperature=0.0))
            assert [o.token_ids for o in outs] == want, (name, graphs)


def test_command_line_and_replay_program(tmp_path):
    """The command line on a model folder of the design (float32, greedy: the plain implementation's tokens), and the
    replay program: three requests through a pool that holds two of them."""
    root = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
    folder = model_folder("NA")
    prompts = [tokens_for("NA", 7, 5), tokens_for("NA", 19, 6)]
    spec = ";".join(",".join(str(t) for t in p) for p in prompts)
    cmd = [sys.executable, os.path.join(root, "bin", "allpaca-amd"), "generate", "--model", folder, "--dtype", "fp32",
           "--prompt-tokens", spec, "--max-tokens", "6", "--temperature", "0", "--json"]
    r = subprocess.run(cmd, capture_output=True, text=True, timeout=300)
    assert r.returncode == 0, r.stderr[-2000:]
    outs = [json.loads(ln) for ln in r.stdout.strip().splitlines() if ln.startswith("{")]
    assert [o["token_ids"] for o in outs] == [P.greedy(*oracle(folder), p, 6) for p in prompts]
    # the design's preset with random weights, sampled with temperature, top-k and top-p in bfloat16
    cmd = [sys.executable, os.path.join(root, "bin", "allpaca-amd"), "generate", "--synthetic", "natenex-tiny",
           "--prompt-tokens", "1,2,3;4,5", "--max-tokens", "5", "--temperature", "0.8", "--top-k", "20", "--top-p",
           "0.9", "--json"]
    r = subprocess.run(cmd, capture_output=True, text=True, timeout=300)
    assert r.returncode == 0, r.stderr[-2000:]
    outs = [json.loads(ln) for ln in r.stdout.strip().splitlines() if ln.startswith("{")]
    assert len(outs) == 2 and all(len(o["token_ids"]) == 5 for o in outs)

    name = "NB"
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
