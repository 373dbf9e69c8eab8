"""The plain implementation of the Muvorax decoder (tests/plain_muvorax.py) pinned by hand, its two forms held against
each other, and the parts of the engine that need no GPU: configuration, tensor names, sizes from shapes, cache needs."""
import copy
import math

import numpy as np
import pytest

import plain_muvorax as P
from muvorax_helpers import CONFIGS, planted


def weights(cfg, seed):
    return {k: v.double().numpy() for k, v in planted(cfg, seed).items()}


def test_the_norm_by_hand():
    out = P.squash(np.array([0.0, 1.0, -50.0]), 0.5, np.array([2.0, 3.0, 4.0]), np.array([0.1, 0.2, 0.3]))
    assert np.allclose(out, [0.1, 3.0 * math.tanh(0.5) + 0.2, -4.0 + 0.3])


def test_rotation_of_neighbours_by_hand_and_the_frequency_rule():
    rot = dict(base=100.0, dims=4)
    v = np.array([[[1.0, 2.0, 3.0, 4.0]]])
    out = P.rotate_pairs(v, [3], rot)[0, 0]
    a0, a1 = 3.0, 3.0 * 100.0 ** -0.5
    assert np.allclose(out, [math.cos(a0) - 2 * math.sin(a0), 2 * math.cos(a0) + math.sin(a0),
                             3 * math.cos(a1) - 4 * math.sin(a1), 4 * math.cos(a1) + 3 * math.sin(a1)])
    rot = dict(base=10000.0, dims=32, scaling=dict(factor=4.0, original=64, fast=16.0, slow=2.0))
    f, mag = P.frequencies(rot)
    plain = 10000.0 ** (-2.0 * np.arange(16) / 32)
    assert np.isclose(mag, 0.1 * math.log(4.0) + 1.0)
    assert np.allclose(f[0], plain[0]) and np.allclose(f[-1], plain[-1] / 4.0)
    assert (np.diff(f / plain) <= 1e-12).all() and 0.25 < (f / plain)[1] < 1.0
    # a score depends on the distance alone, and magnitudes enter it twice
    q, k = np.random.default_rng(0).normal(size=(2, 32))
    s = [P.rotate_pairs(q[None], [p + 7], rot)[0] @ P.rotate_pairs(k[None], [p], rot)[0] for p in (0, 5, 40)]
    assert np.allclose(s, s[0]) and np.isclose(P.rotate_pairs(q[None], [9], rot)[0] @ P.rotate_pairs(q[None], [9], rot)[0],
                                               mag * mag * (q @ q))


def test_recurrences_by_hand():
    q = np.ones((2, 1, 1)); k = np.array([[[1.0]], [[2.0]]]); v = np.array([[[3.0]], [[5.0]]])
    o, S = P.decayed_sums(q, k, v, [0.5])
    assert np.allclose(o[:, 0, 0], [3.0, 0.5 * 3.0 + 10.0]) and np.allclose(S, [[[11.5]]])
    x = np.array([[1.0], [2.0]]); dt = np.array([[0.5], [1.0]])
    y, S = P.selective_scan(x, dt, np.array([[-1.0]]), np.array([[1.0], [1.0]]), np.array([[2.0], [3.0]]), np.array([10.0]))
    s1 = math.exp(-1.0) * 0.5 + 2.0
    assert np.allclose(y[:, 0], [1.0 + 10.0, 3.0 * s1 + 20.0]) and np.allclose(S, [[s1]])


def test_the_router_by_hand():
    logit = lambda s: math.log(s / (1 - s))
    z = np.array([logit(v) for v in (0.9, 0.1, 0.6, 0.5, 0.3, 0.2)])
    none = np.zeros(6)
    ids, w = P.route(z, none, 2)
    assert list(ids) == [0, 2] and np.allclose(w, [0.6, 0.4])
    # three groups of two: 1.0, 1.1 and 0.5; the second one alone is kept although expert 0 scores most
    ids, w = P.route(z, none, 2, 2.0, 3, 1)
    assert list(ids) == [2, 3] and np.allclose(w, [2.0 * 6 / 11, 2.0 * 5 / 11])
    # the correction enters the choice (also of the groups) and not the weights; choice scores may be negative, and an
    # expert of a group that is not kept is still worse
    ids, w = P.route(z, np.array([-2.0, -2.0, -3.0, -3.0, -1.0, -1.5]), 2, 1.0, 3, 1)
    assert list(ids) == [4, 5] and np.allclose(w, [0.6, 0.4])
    # groups of one expert: its own score
    ids, _ = P.route(z, none, 2, 1.0, 6, 2)
    assert list(ids) == [0, 2]


def test_applying_the_up_projections_to_queries_and_outputs_is_the_same_attention():
    """The identity the engine rests on: scores of queries mapped into the latent space against cached rows, outputs
    mapped out of it."""
    rng = np.random.default_rng(2)
    T, H, dn, dr, dv, R = 9, 3, 4, 2, 5, 7
    q, c, kr = rng.normal(size=(T, H, dn + dr)), rng.normal(size=(T, R)), rng.normal(size=(T, dr))
    uk, uv = rng.normal(size=(H, dn, R)), rng.normal(size=(H, dv, R))
    k = np.concatenate([np.einsum("tr,hdr->thd", c, uk), np.broadcast_to(kr[:, None], (T, H, dr))], axis=-1)
    want = P.softmax_attention(q, k, np.einsum("tr,hdr->thd", c, uv), 0.6)
    ql = np.concatenate([np.einsum("thd,hdr->thr", q[..., :dn], uk), q[..., dn:]], axis=-1)
    rows = np.broadcast_to(np.concatenate([c, kr], axis=1)[:, None], (T, H, R + dr))
    o = P.softmax_attention(ql, rows, rows[..., :R], 0.6)
    assert np.allclose(np.einsum("thr,hdr->thd", o, uv), want)


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
    cfg, seed = CONFIGS["MA"]
    W = weights(cfg, seed)
    toks = np.random.default_rng(1).integers(0, cfg["vocab"], size=30).tolist()
    want = P.forward(cfg, W, toks)
    size = float(np.sqrt(np.mean(want ** 2)))

    def moved(change, weights_change=None):
        c, w = copy.deepcopy(cfg), dict(W)
        change(c["layers"])
        if weights_change:
            weights_change(w)
        return float(np.sqrt(np.mean((P.forward(c, w, toks) - want) ** 2))) / size

    def w_moved(name, f):
        assert name in W
        return moved(lambda L: None, lambda w: w.update({name: f(w[name])}))

    assert moved(lambda L: L[1]["mixer"]["rot"].pop("scaling")) > 1e-3
    assert moved(lambda L: L[1]["mixer"]["rot"].update(base=60.0)) > 1e-3
    assert moved(lambda L: L[1]["mixer"].update(scale=0.45)) > 1e-3
    assert moved(lambda L: L[3]["mixer"].update(scale=0.6)) > 1e-3
    assert moved(lambda L: L[0]["mixer"].update(decay=[0.9, 0.99, 0.6])) > 1e-3
    assert moved(lambda L: L[0]["mlp"]["router"].update(scale=1.6)) > 1e-3
    assert moved(lambda L: L[0]["mlp"]["router"].update(top=3)) > 1e-3
    assert moved(lambda L: L[0]["mlp"]["router"]["groups"].update(keep=1)) > 1e-3
    assert w_moved("l0.mlp.correction", lambda v: v * 0) > 1e-3
    for name in ("l0.norm1", "l1.norm1b", "l3.norm2", "l0.norm2b", "final.norm"):
        assert w_moved(name + ".alpha", lambda v: v * 1.1) > 1e-3, name
        assert w_moved(name + ".b", lambda v: v + 0.05) > 1e-3, name
    assert w_moved("l1.mix.dkv.norm", lambda v: v * 1.1) > 1e-3
    assert w_moved("l0.mix.norm", lambda v: v * 1.1) > 1e-3
    assert w_moved("l2.mix.conv.b", lambda v: v + 0.2) > 1e-3
    assert w_moved("l2.mix.D", lambda v: v * 1.2) > 1e-3


# ---------------------------------------------------------------------------------------------- the engine's side, no GPU
def test_tensor_names_and_shapes_are_the_plain_implementation_s():
    from allpaca_amd.models import DecoderModel, describe_model
    for name, (cfg, _) in CONFIGS.items():
        _, typed, spec = describe_model(cfg)
        got = {n: tuple(ps.shape) for n, ps in DecoderModel(spec).param_specs().items()}
        assert got == P.tensor_shapes(cfg), name


def bare(cfg):
    """The configuration without the sizes that the tensors' shapes give."""
    c = copy.deepcopy(cfg)
    c.pop("vocab"), c.pop("width")
    for layer in c["layers"]:
        m = layer["mixer"]
        for k in ("heads", "dim", "rot_dim", "vdim", "kv_rank", "inner", "state", "dt_rank", "conv"):
            m.pop(k, None)
        f = layer.get("mlp")
        if f and f["kind"] == "dense":
            f.pop("ff")
        elif f:
            f["expert"].pop("ff"), f["router"].pop("experts")
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
    cfg = CONFIGS["MA"][0]

    def broken(change, word):
        c = copy.deepcopy(cfg)
        change(c)
        with pytest.raises(ConfigError) as e:
            describe_model(c)
        assert word in str(e.value), str(e.value)

    broken(lambda c: c["layers"][3]["mixer"].update(kv_from=3), "kv_from")
    broken(lambda c: c["layers"][3]["mixer"].update(kv_from=0), "kv_from")
    broken(lambda c: c["layers"][3]["mixer"].update(kv_rank=8), "kv_rank")
    broken(lambda c: c["layers"][3]["mixer"]["rot"].update(base=51.0), "rot")
    broken(lambda c: c["layers"][3]["mixer"]["rot"].pop("scaling"), "rot")
    broken(lambda c: c["layers"][1]["mixer"]["rot"].update(dims=6), "rot_dim")
    broken(lambda c: c["layers"][1]["mixer"].pop("scale"), "scale")
    broken(lambda c: c["layers"][0]["mixer"].update(decay=[0.5]), "decay")
    broken(lambda c: c["layers"][2].update(type="mamba2"), "type")
    broken(lambda c: c["layers"][2]["mixer"].update(conv=0), "conv")
    broken(lambda c: c["layers"][0]["mlp"]["router"]["groups"].update(count=2), "groups")
    broken(lambda c: c["layers"][0]["mlp"]["router"]["groups"].update(keep=4), "groups")
    broken(lambda c: c["layers"][0]["mlp"]["router"].update(top=7), "top")
    broken(lambda c: c["layers"][1]["mlp"].update(kind="swiglu"), "kind")
    broken(lambda c: c.pop("norm"), "norm")


def test_cache_needs_of_owners_borrowers_and_recurrent_layers():
    from allpaca_amd.cache import CacheManager
    from allpaca_amd.cache.estimate import CacheEstimate
    from allpaca_amd.models import DecoderModel, describe_model
    from allpaca_amd.parts import FixedState, PagedLatents
    _, _, spec = describe_model(CONFIGS["MA"][0])
    needs = DecoderModel(spec).cache_needs()
    assert needs[0] == FixedState((3, 10, 6), "float32")
    assert needs[1] == PagedLatents(14, 4) and needs[1].page_shape(8) == (8, 18)
    assert needs[2] == {"mixer": FixedState((18, 5), "float32"), "mixer.state": FixedState((3, 18), "float32")}
    assert needs[3] is None and spec.plan[3].cache_of == 1
    cm = CacheManager(needs, 4, 16, 2)
    assert len(cm.paged_groups) == 1 and len(cm.state_groups) == 3
    # a position costs one row whatever the number of heads
    assert CacheEstimate.of(needs, 4, 2).groups[0].page_bytes == 4 * 18 * 2
    # two owners of other latents are two groups; a convolution of one tap keeps no rows
    _, _, spec = describe_model(CONFIGS["MD"][0])
    assert len(CacheManager(DecoderModel(spec).cache_needs(), 4, 16, 2).paged_groups) == 2
    _, _, spec = describe_model(CONFIGS["MC"][0])
    assert DecoderModel(spec).cache_needs()[1] == FixedState((8, 1), "float32")


def test_rows_of_neighbouring_pairs_are_put_in_halves_on_both_sides():
    """Binding reorders the rows that make rotated elements; a score of rotated halves is that of rotated neighbours."""
    import torch
    from allpaca_amd.parts.latent_attention import AbsorbedLatentAttention
    part = AbsorbedLatentAttention(8, 2, 3, 6, 4, 5, 0.5, rope_interleaved=True)
    w = torch.arange(12.0).reshape(2, 6, 1).expand(2, 6, 8)
    assert part._halves(w)[0, :, 0].tolist() == [0, 2, 4, 1, 3, 5] and part._halves(w)[1, :, 0].tolist() == [6, 8, 10, 7, 9, 11]
    same = AbsorbedLatentAttention(8, 2, 3, 6, 4, 5, 0.5, rope_interleaved=False)
    assert same._halves(w) is w
    with pytest.raises(ValueError):
        AbsorbedLatentAttention(8, 2, 3, 5, 4, 5, 0.5)


def test_a_preset_of_the_design():
    from allpaca_amd.config import preset
    from allpaca_amd.models import describe_model
    arch, cfg, spec = describe_model(preset("muvorax-tiny"))
    assert arch.name == "muvorax" and len(spec.plan) == len(cfg.layers) and any(e.cache_of is not None for e in spec.plan)
