"""Small Muvorax configurations that differ in every size and option, model folders with planted weights for them, and
the plain implementation's logits."""
from __future__ import annotations

import functools
import os
from typing import Dict, List, Sequence

import numpy as np
import torch

import plain_muvorax as P
from helpers import tmp_root


def _lat(heads, dim, rot_dim, vdim, kv_rank, scale, base, scaling=None, kv_from=None):
    m = dict(heads=heads, dim=dim, rot_dim=rot_dim, vdim=vdim, kv_rank=kv_rank, scale=scale,
             rot=dict(base=base, dims=rot_dim))
    if scaling is not None:
        m["rot"]["scaling"] = dict(zip(("factor", "original", "fast", "slow"), scaling))
    if kv_from is not None:
        m["kv_from"] = kv_from
    return dict(type="latent_attention", mixer=m)


def _scan(inner, state, dt_rank, conv):
    return dict(type="mamba1", mixer=dict(inner=inner, state=state, dt_rank=dt_rank, conv=conv))


def _lig(heads, dim, vdim, decay):
    return dict(type="lightning", mixer=dict(heads=heads, dim=dim, vdim=vdim, decay=list(decay)))


def _dense(ff):
    return dict(kind="dense", ff=ff)


def _moe(ff, experts, top, scale=None, groups=None):
    r = dict(experts=experts, top=top)
    if scale is not None:
        r["scale"] = scale
    if groups is not None:
        r["groups"] = dict(zip(("count", "keep"), groups))
    return dict(kind="moe", expert=dict(ff=ff), router=r)


def _layer(mixer, mlp):
    return dict(mixer, mlp=mlp)


def _model(vocab, width, eps, layers):
    return dict(architecture="Muvorax", vocab=vocab, width=width, norm=dict(eps=eps), layers=layers)


# A: odd sizes everywhere (nothing a matrix-core kernel takes): lightning first, 5 heads of latent attention with 6 + 4
#    elements over a latent of 14, values of 10, a frequency rule; scan of 18 channels, 5 states, 4 taps; a borrower of
#    other head count and sizes; groups 3 of which 2 are kept; a layer without feed-forward
TINY_MA = _model(83, 36, 1e-5, [
    _layer(_lig(3, 10, 6, (0.9, 0.99, 0.5)), _moe(20, 9, 2, 1.7, (3, 2))),
    _layer(_lat(5, 6, 4, 10, 14, 0.4, 50.0, (3.0, 16, 8.0, 1.0)), _dense(28)),
    _layer(_scan(18, 5, 3, 4), None),
    _layer(_lat(3, 10, 4, 6, 14, 0.5, 50.0, (3.0, 16, 8.0, 1.0), kv_from=1), _moe(12, 4, 3, 0.6, (2, 2)))])
# B: sizes the matrix-core kernels take: 12 heads of 32 + 16 over a latent of 96 (pairs of rows and heads that do not
#    fill a block's tile), two borrowers with other heads, groups of 2 experts; scan of 256 channels
TINY_MB = _model(256, 128, 1e-6, [
    _layer(_scan(256, 16, 8, 4), _moe(64, 8, 3, 2.5, (4, 2))),
    _layer(_lat(12, 32, 16, 32, 96, 0.15, 20000.0, (4.0, 64, 16.0, 2.0)), _moe(32, 12, 4, 1.3, (4, 3))),
    _layer(_lig(4, 64, 32, (0.97, 0.99, 0.999, 0.9)), _dense(256)),
    _layer(_lat(4, 64, 16, 64, 96, 0.12, 20000.0, (4.0, 64, 16.0, 2.0), kv_from=1), _dense(128)),
    _layer(_lat(40, 16, 16, 16, 96, 0.2, 20000.0, (4.0, 64, 16.0, 2.0), kv_from=1), None)])
# C: the values that make terms vanish or coincide: one head, one state, a step size of rank 1, one tap, a decay of 1,
#    every expert chosen, one expert alone, one group, groups of one expert, a scale of 1, no frequency rule, one pair
TINY_MC = _model(50, 32, 1e-6, [
    _layer(_lat(1, 8, 2, 16, 8, 0.35, 10000.0), _moe(16, 3, 3)),
    _layer(_scan(8, 1, 1, 1), _moe(24, 1, 1, 1.0, (1, 1))),
    _layer(_lig(1, 16, 16, (1.0,)), None),
    _layer(_lat(2, 8, 2, 8, 8, 0.3, 10000.0, kv_from=0), _moe(8, 4, 2, 3.0, (4, 3))),
    _layer(_lat(3, 4, 8, 4, 16, 0.3, 7.0), _dense(8)),
    _layer(_scan(16, 3, 2, 2), _dense(16))])
# D: multiples of 8 that are no multiples of 16 or 32 (a latent of 40 with 24 rotated elements, values of 24 and 40, 72
#    channels), two owners with different latents and a borrower of each
TINY_MD = _model(300, 96, 1e-6, [
    _layer(_lat(6, 40, 24, 24, 40, 0.13, 5000.0, (2.0, 32, 4.0, 0.5)), _moe(72, 10, 4, 1.0, (5, 3))),
    _layer(_lat(3, 24, 8, 40, 72, 0.17, 300.0), _dense(200)),
    _layer(_scan(72, 8, 6, 3), _dense(104)),
    _layer(_lat(5, 24, 24, 16, 40, 0.15, 5000.0, (2.0, 32, 4.0, 0.5), kv_from=0), None),
    _layer(_lat(8, 8, 8, 8, 72, 0.25, 300.0, kv_from=1), _moe(24, 6, 1, 0.5, (2, 1))),
    _layer(_lig(3, 40, 24, (0.97, 0.9, 0.99)), _dense(56))])

CONFIGS = {"MA": (TINY_MA, 81), "MB": (TINY_MB, 82), "MC": (TINY_MC, 83), "MD": (TINY_MD, 84)}


def planted(cfg: dict, seed: int) -> Dict[str, torch.Tensor]:
    """Weights of a size at which every mechanism shows in the logits: matrices N(0, 1/sqrt(fan-in)), those that make
    queries and keys larger (so that the softmax is not flat and one key more or less moves the logits), norms that
    neither saturate nor stay linear, biases and corrections of a size that matters, routers that separate the experts."""
    from allpaca_amd.models import DecoderModel, describe_model
    _, _, spec = describe_model(cfg)
    types = [layer["type"] for layer in cfg["layers"]]
    g = torch.Generator().manual_seed(seed)
    out = {}
    for name, ps in DecoderModel(spec).param_specs().items():
        shape = tuple(ps.shape)
        rnd = torch.randn(shape, generator=g)
        parts = name.split(".")
        last = parts[-1]
        kind = types[int(parts[0][1:])] if parts[0][1:].isdigit() else ""
        if last == "alpha":
            t = 0.6 + 0.2 * rnd.abs()
        elif last == "conv":
            t = rnd / shape[1] ** 0.5 + (torch.arange(shape[1]) == shape[1] - 1).float()
        elif last == "b":
            t = (rnd - 1.0) if parts[-2] == "dt" else 0.2 * rnd
        elif last == "A_log":
            t = 0.7 * rnd - 1.0
        elif last == "correction":
            t = 0.3 * rnd
        elif len(shape) == 1:
            t = 1.0 + 0.2 * rnd
        elif name == "embed":
            t = rnd
        elif last == "router":
            t = 2.0 * rnd / shape[1] ** 0.5
        elif kind == "latent_attention" and last in ("q", "uk", "dkv"):
            t = 2.0 * rnd / shape[1] ** 0.5
        elif last == "up":
            t = 1.5 * rnd / shape[1] ** 0.5
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
    return write_folder(os.path.join(tmp_root(), f"muvorax_{name}_{dtype}"), cfg, seed, dtype)


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
