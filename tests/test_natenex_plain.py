"""The plain implementation of the Natenex decoder (tests/plain_natenex.py) pinned by hand, its two forms held against
each other, and the parts of the engine that need no GPU: configuration, tensor names, sizes from shapes, cache needs,
kept pages."""
import copy
import math

import numpy as np
import pytest

import plain_natenex as P
from natenex_helpers import CONFIGS, planted


def weights(cfg, seed):
    return {k: v.double().numpy() for k, v in planted(cfg, seed).items()}


def test_norms_by_hand():
    x = np.array([3.0, 4.0])
    assert np.allclose(P.rms_norm(x, np.array([2.0, 1.0]), 0.5), np.array([6.0, 4.0]) / math.sqrt(13.0))
    assert np.allclose(P.unit(x), x / math.sqrt(25.0 + 1e-6)) and np.allclose(P.unit(np.zeros(3)), 0.0)


def test_rotation_of_halves_by_hand_and_the_frequency_rule():
    rot = dict(base=100.0, dims=4)
    out = P.rotate_halves(np.array([[[1.0, 2.0, 3.0, 4.0, 9.0]]]), [3], rot)[0, 0]
    a, b = 3.0, 3.0 * 100.0 ** -0.5
    assert np.allclose(out, [math.cos(a) - 3 * math.sin(a), 2 * math.cos(b) - 4 * math.sin(b),
                             3 * math.cos(a) + math.sin(a), 4 * math.cos(b) + 2 * math.sin(b), 9.0])
    # three bands: short waves stay, long ones are slowed, those between are blended
    rot = dict(base=10000.0, dims=32, scaling=dict(factor=4.0, low=1.0, high=4.0, original=64))
    plain = 10000.0 ** (-2.0 * np.arange(16) / 32)
    f = P.frequencies(rot)
    waves = 2 * math.pi / plain
    assert np.allclose(f[waves < 16], plain[waves < 16]) and np.allclose(f[waves > 64], plain[waves > 64] / 4)
    mid = np.flatnonzero((waves >= 16) & (waves <= 64))
    assert len(mid) and all(plain[i] / 4 < f[i] < plain[i] for i in mid)
    s = (64 / waves[mid[0]] - 1.0) / 3.0
    assert np.isclose(f[mid[0]], (1 - s) * plain[mid[0]] / 4 + s * plain[mid[0]])


def test_the_window_and_the_kept_tokens_by_hand():
    mask = dict(size=3, keep_first=2)
    seen = {i: [j for j in range(10) if P.visible(i, j, mask)] for i in (0, 1, 4, 5, 9)}
    assert seen == {0: [0], 1: [0, 1], 4: [0, 1, 2, 3, 4], 5: [0, 1, 3, 4, 5], 9: [0, 1, 7, 8, 9]}
    assert [j for j in range(10) if P.visible(4, j, None)] == [0, 1, 2, 3, 4]
    # one key that all rows look for is the output of those that see it
    q, k = np.zeros((10, 1, 2)), np.zeros((10, 1, 2))
    q[:, 0, 0], k[4, 0, 0] = 60.0, 1.0
    v = np.arange(10.0).reshape(10, 1, 1)
    o = P.softmax_attention(q, k, v, 1.0, 0, mask)[:, 0, 0]
    assert np.allclose(o[[4, 5, 6]], 4.0) and np.isclose(o[7], np.mean([0, 1, 5, 6, 7]))


def test_recurrences_by_hand():
    lam = np.array([0.3])
    sp = math.log(1 + math.exp(0.3))
    s, last = P.gated_recurrence(np.array([[2.0], [3.0]]), np.array([[0.5], [0.1]]), np.array([[1.0], [0.25]]), lam)
    a0, a1 = math.exp(-4.0 * sp), math.exp(-0.8 * sp)
    first = math.sqrt(1 - a0 ** 2) * 2.0
    assert np.allclose(s[:, 0], [first, a1 * first + math.sqrt(1 - a1 ** 2) * 0.75]) and last[0] == s[1, 0]
    # delta rule: a key written twice with a step of one keeps the second value alone
    k = np.array([[[1.0, 0.0]], [[1.0, 0.0]]])
    v = np.array([[[5.0]], [[7.0]]])
    one = np.ones((2, 1))
    o, S = P.delta_rule(k, k, v, one, one)
    assert np.allclose(o[:, 0, 0], [5.0, 7.0]) and np.allclose(S[0], [[7.0], [0.0]])
    o, S = P.delta_rule(k, k, v, 0.5 * one, np.array([[1.0], [0.8]]))
    s1 = 2.5
    s2 = 0.8 * s1 + 0.5 * (7.0 - 0.8 * s1)
    assert np.allclose(o[:, 0, 0], [s1, s2]) and np.isclose(S[0, 0, 0], s2)


def test_a_chunk_s_writes_solve_a_triangular_system():
    """The identity the engine's chunk kernels rest on: with c_t the product of the decays up to row t, the writes u of a
    chunk are (I + A)^-1 (beta v - beta c S0^T k), and state and outputs are sums over them."""
    rng = np.random.default_rng(3)
    T, d, e = 9, 5, 4
    q, k, v = P.unit(rng.normal(size=(T, d))), P.unit(rng.normal(size=(T, d))), rng.normal(size=(T, e))
    beta, g, S0 = rng.random(T), 0.7 + 0.3 * rng.random(T), rng.normal(size=(d, e))
    o, S = P.delta_rule(q[:, None], k[:, None], v[:, None], beta[:, None], g[:, None], S0[None])
    c = np.cumprod(g)
    ratio = np.tril(c[:, None] / c[None, :])
    A = np.tril(beta[:, None] * ratio * (k @ k.T), -1)
    u = np.linalg.solve(np.eye(T) + A, beta[:, None] * (v - c[:, None] * (k @ S0)))
    assert np.allclose(o[:, 0], c[:, None] * (q @ S0) + (ratio * (q @ k.T)) @ u)
    assert np.allclose(S[0], c[-1] * S0 + (k * (c[-1] / c)[:, None]).T @ u)


@pytest.mark.parametrize("name", sorted(CONFIGS))
def test_portions_and_single_tokens_give_the_whole_sequence_s_logits(name):
    cfg, seed = CONFIGS[name]
    W = weights(cfg, seed)
    toks = np.random.default_rng(seed).integers(0, cfg["vocab"], size=23).tolist()
    want = P.forward(cfg, W, toks)
    for cuts in ([1], [2], [5, 1, 9, 3]):
        st, got, at, i = P.Stepper(cfg, W), [], 0, 0
        while at < len(toks):
            n = min(cuts[min(i, len(cuts) - 1)], len(toks) - at)
            got.append(st.feed(toks[at:at + n]))
            at, i = at + n, i + 1
        assert np.allclose(np.concatenate(got), want, atol=1e-9), (name, cuts)


def test_every_mechanism_moves_the_logits():
    """What the tests' weights would hide could be wrong unseen: every constant of the design, changed a little, moves
    the logits by far more than any tolerance."""
    cfg, seed = CONFIGS["NA"]
    W = weights(cfg, seed)
    toks = np.random.default_rng(1).integers(0, cfg["vocab"], size=34).tolist()
    want = P.forward(cfg, W, toks)
    size = float(np.sqrt(np.mean(want ** 2)))

    def moved(change, weights_change=None):
        c, w = copy.deepcopy(cfg), dict(W)
        change(c)
        if weights_change:
            weights_change(w)
        return float(np.sqrt(np.mean((P.forward(c, w, toks) - want) ** 2))) / size

    def left(**kw):
        return lambda c: [c["layers"][i]["mixer"]["left"].update(**kw) for i in (0, 3)]

    def w_moved(name, f):
        assert name in W
        return moved(lambda c: None, lambda w: w.update({name: f(w[name])}))

    rot = cfg["layers"][0]["mixer"]["left"]["rot"]
    assert moved(left(mask=dict(size=12, keep_first=5))) > 1e-3
    assert moved(left(mask=dict(size=10, keep_first=5))) > 1e-3
    assert moved(left(mask=dict(size=11, keep_first=6))) > 1e-3
    assert moved(left(mask=dict(size=11, keep_first=4))) > 1e-3
    assert moved(left(scale=0.55)) > 1e-3
    assert moved(left(rot=dict(base=40.0, dims=6))) > 1e-3
    for k, v in (("factor", 3.5), ("low", 1.3), ("high", 3.0), ("original", 40)):
        assert moved(left(rot=dict(rot, scaling=dict(rot["scaling"], **{k: v})))) > 1e-3, k
    assert moved(lambda c: [c["layers"][i]["mixer"].update(left_scale=0.7) for i in (0, 3)]) > 1e-3
    assert moved(lambda c: [c["layers"][i]["mixer"].update(right_scale=1.2) for i in (0, 3)]) > 1e-3
    assert moved(lambda c: c["layers"][2]["mixer"].update(scale=0.5)) > 1e-3
    assert moved(lambda c: c["layers"][2]["mixer"]["rot"].update(base=30.0)) > 1e-3
    assert moved(lambda c: c["embedding"].update(scale=2.7)) > 1e-3
    for name in W:
        if name.endswith((".dq", ".dkv")):
            assert w_moved(name, lambda v: v + 0.05 * np.random.default_rng(0).normal(size=v.shape)) > 1e-4, name
        elif name.split(".")[-1] in ("norm", "norm1", "norm2", "b", "lam", "A_log", "dt_bias", "a", "conv", "ra", "ri", "g"):
            assert w_moved(name, lambda v: v * 1.1 + 0.05) > 1e-4, name


# ---------------------------------------------------------------------------------------------- the engine's side, no GPU
def test_tensor_names_and_shapes_are_the_plain_implementation_s():
    from allpaca_amd.models import DecoderModel, describe_model
    for name, (cfg, _) in CONFIGS.items():
        _, typed, spec = describe_model(cfg)
        got = {n: tuple(ps.shape) for n, ps in DecoderModel(spec).param_specs().items()}
        assert got == P.tensor_shapes(cfg), name


def bare(cfg):
    """The configuration without the sizes that the tensors' shapes give (a delta rule names one of its two)."""
    c = copy.deepcopy(cfg)
    c.pop("vocab"), c.pop("width")
    for layer in c["layers"]:
        m = layer["mixer"]
        for part in (m, m.get("left", {}), m.get("right", {})):
            for k in ("heads", "rot_dim", "vdim", "q_rank", "kv_rank", "conv", "width", "blocks"):
                part.pop(k, None)
            if layer["type"] != "delta":
                part.pop("dim", None)
            part.pop("kv_heads", None)
        if layer.get("mlp"):
            layer["mlp"].pop("ff")
    return c


def test_sizes_that_the_file_leaves_out_come_from_the_shapes():
    from allpaca_amd.models import describe_model
    for name, (cfg, _) in CONFIGS.items():
        _, full, _ = describe_model(cfg)
        _, filled, _ = describe_model(bare(cfg), P.tensor_shapes(cfg))
        assert filled == full, name


def test_configuration_errors_name_the_key():
    from allpaca_amd.config import ConfigError
    from allpaca_amd.models import describe_model
    cfg = CONFIGS["NA"][0]

    def broken(change, word):
        c = copy.deepcopy(cfg)
        change(c["layers"])
        with pytest.raises(ConfigError) as e:
            describe_model(c)
        assert word in str(e.value), str(e.value)

    broken(lambda L: L[3].update(weights_of=3), "weights_of")
    broken(lambda L: L[3].update(weights_of=9), "weights_of")
    broken(lambda L: L[3].update(weights_of=1), "layer 1")
    broken(lambda L: L[3]["mixer"].update(left_scale=0.1), "layer 0")
    broken(lambda L: L[3].update(mlp=None), "layer 0")
    broken(lambda L: L[0]["mixer"]["left"].update(kv_heads=4), "kv_heads")
    broken(lambda L: L[0]["mixer"]["left"]["rot"].update(dims=12), "dims")
    broken(lambda L: L[0]["mixer"]["left"]["mask"].update(size=0), "size")
    broken(lambda L: L[0]["mixer"]["left"]["mask"].update(keep_first=-1), "keep_first")
    broken(lambda L: L[0]["mixer"]["left"]["rot"]["scaling"].update(high=1.0), "high")
    broken(lambda L: L[0]["mixer"]["right"].update(blocks=4), "blocks")
    broken(lambda L: L[0]["mixer"].pop("right_scale"), "right_scale")
    broken(lambda L: L[2]["mixer"]["rot"].update(dims=2), "rot_dim")
    broken(lambda L: L[2]["mixer"].pop("q_rank"), "q_rank")
    broken(lambda L: L[1]["mixer"].update(conv=0), "conv")
    broken(lambda L: L[1].update(type="mamba"), "type")
    broken(lambda L: L[0]["mlp"].update(kind="moe"), "kind")


def test_a_layer_with_another_s_weights_has_a_cache_of_its_own():
    from allpaca_amd.cache import CacheManager
    from allpaca_amd.models import DecoderModel, describe_model
    from allpaca_amd.parts import FixedState, PagedKeysValues, PagedLatents
    _, cfg, spec = describe_model(CONFIGS["NB"][0])
    assert [l.weights_of for l in cfg.layers] == [None, None, None, 0, 1, 0]        # (a borrower of a borrower)
    assert [e.block for e in spec.plan] == [0, 1, 2, 0, 1, 0] and all(e.cache_of is None for e in spec.plan)
    needs = DecoderModel(spec).cache_needs()
    assert needs[1] == needs[4] == {"mixer.left": PagedKeysValues(2, 64, 32, 40, 24), "mixer.right": FixedState((128,)),
                                    "mixer.right.state": FixedState((3, 128))}
    assert needs[0] == needs[3] == {"mixer": FixedState((4, 64, 48)), "mixer.state": FixedState((3, 704))}
    assert needs[2] == PagedLatents(64, 16)
    cm = CacheManager(needs, 16, 16, 2)
    assert len(cm.paged_groups) == 2
    # six stored places, not four: every layer of the list has its own
    assert sum(len(g.entries) for g in cm.paged_groups) == 3 and sum(len(g.entries) for g in cm.state_groups) == 3 * 2 + 2 * 2
    # a convolution of one tap keeps no rows; a later layer may lend its weights
    _, _, spec = describe_model(CONFIGS["NC"][0])
    assert DecoderModel(spec).cache_needs()[1] == FixedState((1, 16, 16))
    late = copy.deepcopy(CONFIGS["NA"][0])
    late["layers"] = [dict(late["layers"][3], weights_of=1), dict(late["layers"][0])]
    _, _, spec = describe_model(late)
    assert [e.block for e in spec.plan] == [0, 0] and spec.blocks[0].weight_prefix == "l1."


def test_pages_of_kept_first_tokens_stay_beside_the_window():
    from allpaca_amd.cache import CacheManager
    from allpaca_amd.cache.estimate import CacheEstimate
    from allpaca_amd.cache.pages import FREED
    from allpaca_amd.parts import PagedKeysValues
    for P_, W, keep in ((4, 10, 6), (4, 3, 1), (2, 5, 0), (1, 2, 3), (16, 17, 33), (4, 8, 40)):
        need = PagedKeysValues(2, 8, 8, W, keep)
        cm = CacheManager([need], P_, 64, 2)
        est = CacheEstimate.of([need], P_, 2)
        cm.admit("a")
        rng = np.random.default_rng(P_ + W)
        while cm.length("a") < 60:
            n = int(rng.integers(1, 4))
            cm.reserve("a", n)
            cm.commit("a", n)
            cm.check()
            L, table = cm.length("a"), cm.block_table("a", 0)
            for page, held in enumerate(table):
                # a page is needed if the next row (or a later one) sees one of its positions
                wanted = page * P_ < keep or (page + 1) * P_ - 1 >= L - W + 1
                assert (held != FREED) == wanted, (P_, W, keep, L, page)
            assert sum(p != FREED for p in table) <= est.pages_of_a_request(L, 0)
        cm.release("a")
        cm.check()
        assert cm.free_pages() == 64


def test_a_preset_of_the_design():
    from allpaca_amd.config import preset
    from allpaca_amd.models import describe_model
    arch, cfg, spec = describe_model(preset("natenex-tiny"))
    assert arch.name == "natenex" and len(spec.plan) == len(cfg.layers) == len(spec.blocks) + 1
