"""Small Natenex configurations that differ in every size and option, model folders with planted weights for them, and
the plain implementation's logits."""
from __future__ import annotations

import copy
import functools
import os
from typing import Dict, List, Sequence

import numpy as np
import torch

import plain_natenex as P
from helpers import tmp_root


def _rot(base, dims, scaling=None):
    out = dict(base=base, dims=dims)
    if scaling is not None:
        out["scaling"] = dict(zip(("factor", "low", "high", "original"), scaling))
    return out


def _par(heads, kv_heads, dim, vdim, scale, rot, mask, width, blocks, conv, scales=(1.0, 1.0)):
    left = dict(heads=heads, kv_heads=kv_heads, dim=dim, vdim=vdim, scale=scale, rot=_rot(*rot))
    if mask is not None:
        left["mask"] = dict(size=mask[0], keep_first=mask[1])
    return dict(type="parallel", mixer=dict(left=left, right=dict(width=width, blocks=blocks, conv=conv),
                                            left_scale=scales[0], right_scale=scales[1]))


def _lat(heads, dim, rot_dim, vdim, q_rank, kv_rank, scale, base, scaling=None):
    return dict(type="latent_attention", mixer=dict(heads=heads, dim=dim, rot_dim=rot_dim, vdim=vdim, q_rank=q_rank,
                                                    kv_rank=kv_rank, scale=scale, rot=_rot(base, rot_dim, scaling)))


def _del(heads, kv_heads, dim, vdim, conv):
    return dict(type="delta", mixer=dict(heads=heads, kv_heads=kv_heads, dim=dim, vdim=vdim, conv=conv))


def _layer(mixer, ff=None, of=None):
    out = dict(copy.deepcopy(mixer), mlp=None if ff is None else dict(kind="dense", ff=ff))
    if of is not None:
        out["weights_of"] = of
    return out


def _model(vocab, width, eps, scale, layers):
    return dict(architecture="Natenex", vocab=vocab, width=width, embedding=dict(scale=scale), norm=dict(eps=eps),
                layers=layers)


# A: odd sizes everywhere (nothing a matrix-core kernel takes): a window of 11 with 5 kept tokens, values wider than keys,
#    5 blocks of 3 channels; a delta rule of 3 heads a key head; latents of 13 and 9; the last layer is the first again
_PA = _par(6, 2, 10, 7, 0.5, (40.0, 6, (3.0, 1.0, 4.0, 30)), (11, 5), 15, 5, 3, (0.8, 1.3))
TINY_NA = _model(71, 27, 1e-5, 3.0, [
    _layer(_PA, 22), _layer(_del(6, 2, 6, 5, 4)), _layer(_lat(5, 7, 4, 6, 13, 9, 0.45, 25.0), 30), _layer(_PA, 22, of=0)])
# B: sizes the matrix-core kernels take: a window of 40 with 24 kept tokens, 8 query heads a pair of kv heads, a recurrence
#    of 128 channels in 4 blocks; keys of 64 with values of 48; 9 heads over latents of 96 and 64; the delta layer thrice
_PB = _par(8, 2, 64, 32, 0.2, (3000.0, 32, (4.0, 1.0, 4.0, 128)), (40, 24), 128, 4, 4, (1.1, 0.6))
_DB = _del(4, 4, 64, 48, 4)
TINY_NB = _model(256, 128, 1e-6, 6.0, [
    _layer(_DB, 160), _layer(_PB, 256), _layer(_lat(9, 32, 16, 48, 96, 64, 0.15, 900.0), 192), _layer(_DB, 160, of=0),
    _layer(_PB, 256, of=1), _layer(_DB, 160, of=3)])
# C: the values that make terms vanish or coincide: one head, one block, one tap, a window of one token without kept
#    ones, no rotation, scales of 1, more kept tokens than the window has, every earlier token
TINY_NC = _model(50, 32, 1e-6, 1.0, [
    _layer(_par(1, 1, 8, 8, 0.35, (10000.0, 0), (1, 0), 8, 1, 1)),
    _layer(_del(1, 1, 16, 16, 1), 24),
    _layer(_par(2, 2, 8, 8, 0.3, (10000.0, 8), (4, 20), 16, 16, 2, (1.0, 2.0)), 16),
    _layer(_lat(1, 8, 2, 8, 8, 8, 0.3, 10000.0)),
    _layer(_par(3, 1, 8, 16, 0.3, (77.0, 2), None, 12, 2, 4, (0.5, 1.0)), 8),
    _layer(_del(2, 1, 4, 8, 2), 8)])
# D: multiples of 8 that are no multiples of 16 or 32, keys of 72 and 136 in the delta rule (padded to 128 and 256), a
#    window of 17 with 33 kept tokens (pages that hold both), a frequency rule on the latents' rotation
TINY_ND = _model(300, 96, 1e-6, 2.0, [
    _layer(_del(4, 2, 72, 40, 3), 104),
    _layer(_par(6, 3, 40, 24, 0.25, (500.0, 16), (17, 33), 144, 6, 3, (0.7, 0.9)), 72),
    _layer(_lat(3, 24, 16, 40, 56, 72, 0.17, 300.0, (2.0, 1.0, 3.0, 64)), 200),
    _layer(_del(3, 3, 136, 24, 4)),
    _layer(_lat(6, 40, 32, 24, 40, 40, 0.13, 5000.0))])

CONFIGS = {"NA": (TINY_NA, 61), "NB": (TINY_NB, 62), "NC": (TINY_NC, 63), "ND": (TINY_ND, 64)}


def planted(cfg: dict, seed: int) -> Dict[str, torch.Tensor]:
    """Weights of a size at which every mechanism shows in the logits: matrices N(0, 1/sqrt(fan-in)), those that make
    queries and keys larger (so that the softmax is not flat and one key more or less moves the logits), decays from
    slow to fast, biases of a size that matters."""
    from allpaca_amd.models import DecoderModel, describe_model
    _, _, spec = describe_model(cfg)
    g = torch.Generator().manual_seed(seed)
    out = {}
    for name, ps in DecoderModel(spec).param_specs().items():
        shape = tuple(ps.shape)
        rnd = torch.randn(shape, generator=g)
        parts = name.split(".")
        last = parts[-1]
        if last == "conv":
            t = rnd / shape[1] ** 0.5 + (torch.arange(shape[1]) == shape[1] - 1).float()
        elif last == "b" and len(shape) == 1 or last == "b" and parts[-2] in ("ra", "ri"):
            t = 0.3 * rnd
        elif last == "A_log":
            t = 0.8 * rnd - 1.5
        elif last == "dt_bias":
            t = 0.5 * rnd - 1.0
        elif last == "lam":
            t = 1.2 * rnd - 3.5
        elif last == "norm" and parts[-2] in ("q", "k"):
            t = 1.6 + 0.3 * rnd
        elif len(shape) == 1:
            t = 1.0 + 0.2 * rnd
        elif name == "embed":
            t = 0.5 * rnd
        elif last in ("ra", "ri"):
            t = 1.5 * rnd / shape[2] ** 0.5
        elif last in ("uq", "uk"):
            t = 1.7 * rnd / shape[1] ** 0.5
        else:
            t = rnd / shape[1] ** 0.5
        out[name] = t.to(torch.bfloat16).float()     # values that bfloat16 holds, so both runs load the same numbers
    return out


def write_folder(path: str, cfg: dict, seed: int, dtype: str = "float32", weights=None) -> str:
    from allpaca_amd.weights import write_model_folder
    write_model_folder(path, cfg, seed, torch.float32 if dtype == "float32" else torch.bfloat16,
                       overrides=planted(cfg, seed) if weights is None else weights)
    return path


@functools.lru_cache(maxsize=None)
def model_folder(name: str, dtype: str = "float32") -> str:
    cfg, seed = CONFIGS[name]
    return write_folder(os.path.join(tmp_root(), f"natenex_{name}_{dtype}"), cfg, seed, dtype)


@functools.lru_cache(maxsize=None)
def oracle(folder: str):
    return P.read_model_folder(folder)


_LOGITS: Dict = {}


def oracle_logits(folder: str, tokens: Sequence[int]) -> np.ndarray:
    key = (folder, tuple(tokens))
    if key not in _LOGITS:
        _LOGITS[key] = P.forward(*oracle(folder), list(tokens))
    return _LOGITS[key]


def oracle_noise(folder: str, tokens: Sequence[int]):
    """What rounding every stored activation to bfloat16 costs the plain implementation itself (exact arithmetic
    otherwise), relative to the size of the logits: (root mean square over all rows, the row that 9 in 10 stay under)."""
    key = (folder, tuple(tokens), "bf16")
    if key not in _LOGITS:
        want = oracle_logits(folder, tokens)
        err = P.forward(*oracle(folder), list(tokens), rnd=P.to_bf16) - want
        size = float(np.sqrt(np.mean(want ** 2)))
        _LOGITS[key] = (float(np.sqrt(np.mean(err ** 2))) / size,
                        float(np.quantile(np.sqrt(np.mean(err ** 2, axis=1)), 0.9)) / size)
    return _LOGITS[key]


def tokens_for(name: str, n: int, seed: int) -> List[int]:
    return np.random.default_rng(seed).integers(0, CONFIGS[name][0]["vocab"], size=n).tolist()
