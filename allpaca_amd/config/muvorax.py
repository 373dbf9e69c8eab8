"""Typed configuration of the Muvorax decoder, read from config.json.

Keys: `vocab`, `width`, `norm.eps` (of the root mean squares inside the mixers), `max_positions` (optional) and
`layers`, a list of {"type", "mixer", "mlp"}.
  type "latent_attention": `heads`, `dim` (unrotated elements of a head's query and key), `rot_dim` (rotated ones),
      `vdim`, `kv_rank` (size of the latent of keys and values), `scale`, `rot` ({"base", "dims" = rot_dim, "scaling":
      {"factor", "original", "fast", "slow"} or absent}), `kv_from` (the layer whose latents it reads instead of its
      own; absent: its own).
  type "mamba1": `inner`, `state`, `dt_rank`, `conv` (a selective scan).
  type "lightning": `heads`, `dim`, `vdim`, `decay` (one number a head).
  `mlp`: null, {"kind": "dense", "ff"}, or {"kind": "moe", "expert": {"ff"}, "router": {"experts", "top", "scale"
      (absent: 1), "groups": {"count", "keep"} (absent: one group)}}.
A size that the file leaves out is taken from the shape of the tensor that has it (`sizes_from_tensors`); constants
come from the file alone."""
from __future__ import annotations

from dataclasses import dataclass
from typing import Any, List, Mapping, Optional, Tuple, Union

from .lesarax import DEFAULT_MAX_POSITIONS, _obj, _rot
from .llama import ConfigError
from .risizen import _int, _num
from .seredra import SeredraYarn


@dataclass(frozen=True)
class MuvoraxLatent:
    heads: int
    dim: int
    rot_dim: int
    vdim: int
    kv_rank: int
    scale: float
    rot_base: float
    scaling: Optional[SeredraYarn] = None
    kv_from: Optional[int] = None


@dataclass(frozen=True)
class MuvoraxScan:
    inner: int
    state: int
    dt_rank: int
    conv: int


@dataclass(frozen=True)
class MuvoraxLightning:
    heads: int
    dim: int
    vdim: int
    decay: Tuple[float, ...]


@dataclass(frozen=True)
class MuvoraxDense:
    ff: int


@dataclass(frozen=True)
class MuvoraxExperts:
    ff: int
    experts: int
    top: int
    scale: float = 1.0
    groups: int = 1
    keep: int = 1


@dataclass(frozen=True)
class MuvoraxLayer:
    mixer: Union[MuvoraxLatent, MuvoraxScan, MuvoraxLightning]
    mlp: Union[None, MuvoraxDense, MuvoraxExperts]


TYPES = ("latent_attention", "mamba1", "lightning")


def sizes_from_tensors(d: Mapping[str, Any], shapes: Mapping[str, Tuple[int, ...]]) -> Mapping[str, Any]:
    """config.json with the sizes it leaves out filled in from the shapes of the stored tensors (`embed`,
    `l<i>.mix.*`, `l<i>.mlp.*`).  A size the file names is left as it is: a disagreement shows when the weights load."""
    def dim_of(name: str, axis: int = 0) -> Optional[int]:
        shape = shapes.get(name)
        return int(shape[axis]) if shape is not None and len(shape) > axis else None

    def fill(m: dict, key: str, value) -> None:
        if m.get(key) is None and value is not None:
            m[key] = value

    def over(a: Optional[int], b) -> Optional[int]:
        return a // b if a and isinstance(b, int) and not isinstance(b, bool) and b > 0 and a % b == 0 else None

    out = dict(d)
    if len(shapes.get("embed", ())) == 2:
        fill(out, "vocab", int(shapes["embed"][0]))
        fill(out, "width", int(shapes["embed"][1]))
    layers = d.get("layers")
    if not isinstance(layers, list):
        return out
    out["layers"] = new_layers = []
    for i, entry in enumerate(layers):
        if not isinstance(entry, Mapping) or not isinstance(entry.get("mixer"), Mapping):
            new_layers.append(entry)
            continue
        p, kind = f"l{i}.mix.", entry.get("type")
        m = dict(entry["mixer"])
        if kind == "latent_attention":
            rot = m.get("rot") if isinstance(m.get("rot"), Mapping) else {}
            fill(m, "kv_rank", dim_of(p + "uk", 1))
            down, rank = dim_of(p + "dkv"), m.get("kv_rank")
            if down is not None and isinstance(rank, int) and down > rank:
                fill(m, "rot_dim", down - rank)
            fill(m, "rot_dim", rot.get("dims"))
            if rot and rot.get("dims") is None and m.get("rot_dim") is not None:
                m["rot"] = dict(rot, dims=m["rot_dim"])
            q_rows, k_rows, r = dim_of(p + "q"), dim_of(p + "uk"), m.get("rot_dim")
            if isinstance(r, int) and r > 0 and q_rows and k_rows:
                fill(m, "heads", over(q_rows - k_rows, r))      # (a head's query has the rotated part, its key matrix not)
            fill(m, "dim", over(k_rows, m.get("heads")))
            fill(m, "heads", over(k_rows, m.get("dim")))
            fill(m, "vdim", over(dim_of(p + "uv"), m.get("heads")))
        elif kind == "mamba1":
            fill(m, "inner", dim_of(p + "conv"))
            fill(m, "conv", dim_of(p + "conv", 1))
            fill(m, "dt_rank", dim_of(p + "dt", 1))
            fill(m, "state", dim_of(p + "A_log", 1))
        elif kind == "lightning":
            if isinstance(m.get("decay"), list):
                fill(m, "heads", len(m["decay"]))
            fill(m, "dim", over(dim_of(p + "q"), m.get("heads")))
            fill(m, "vdim", over(dim_of(p + "v"), m.get("heads")))
        e = dict(entry, mixer=m)
        f = entry.get("mlp")
        if isinstance(f, Mapping):
            f = dict(f)
            if f.get("kind") == "dense":
                fill(f, "ff", dim_of(f"l{i}.mlp.up"))
            elif f.get("kind") == "moe":
                expert = dict(f["expert"]) if isinstance(f.get("expert"), Mapping) else {}
                router = dict(f["router"]) if isinstance(f.get("router"), Mapping) else {}
                fill(expert, "ff", dim_of(f"l{i}.mlp.e0.up"))
                fill(router, "experts", dim_of(f"l{i}.mlp.router"))
                f["expert"], f["router"] = expert, router
            e["mlp"] = f
        new_layers.append(e)
    return out


def _latent(m: Mapping[str, Any], mw: str, i: int, layers: List[MuvoraxLayer]) -> MuvoraxLatent:
    rot_dim = _int(m, "rot_dim", mw, least=0)
    dims, base = _rot(m, mw)
    if dims != rot_dim:
        raise ConfigError(f"config.json: {mw}rot.dims {dims} must equal rot_dim {rot_dim}")
    sc = m["rot"].get("scaling")
    if sc is not None:
        s, sw = _obj(m["rot"], "scaling", mw + "rot."), mw + "rot.scaling."
        sc = SeredraYarn(_num(s, "factor", sw), _num(s, "original", sw), _num(s, "fast", sw), _num(s, "slow", sw))
        if not (sc.factor > 0 and sc.original > 0 and sc.fast > 0 and sc.slow > 0):
            raise ConfigError(f"config.json: {sw}factor, original, fast and slow must be positive")
    mixer = MuvoraxLatent(heads=_int(m, "heads", mw), dim=_int(m, "dim", mw), rot_dim=rot_dim, vdim=_int(m, "vdim", mw),
                          kv_rank=_int(m, "kv_rank", mw), scale=_num(m, "scale", mw), rot_base=base, scaling=sc,
                          kv_from=None if m.get("kv_from") is None else _int(m, "kv_from", mw, least=0))
    if mixer.kv_from is not None:
        if mixer.kv_from >= i:
            raise ConfigError(f"config.json: {mw}kv_from {mixer.kv_from} must name an earlier layer")
        src = layers[mixer.kv_from].mixer
        if not isinstance(src, MuvoraxLatent) or src.kv_from is not None:
            raise ConfigError(f"config.json: {mw}kv_from names layer {mixer.kv_from}, which has no latents of its own")
        if (src.kv_rank, src.rot_dim, src.rot_base, src.scaling) != (mixer.kv_rank, mixer.rot_dim, mixer.rot_base,
                                                                     mixer.scaling):
            raise ConfigError(f"config.json: {mw}kv_rank, rot_dim and rot must equal those of layer {mixer.kv_from}")
    return mixer


def _lightning(m: Mapping[str, Any], mw: str) -> MuvoraxLightning:
    heads = _int(m, "heads", mw)
    decay = m.get("decay")
    if (not isinstance(decay, list) or len(decay) != heads
            or any(isinstance(v, bool) or not isinstance(v, (int, float)) for v in decay)):
        raise ConfigError(f"config.json: {mw}decay must be a list of {heads} numbers, one a head")
    return MuvoraxLightning(heads=heads, dim=_int(m, "dim", mw), vdim=_int(m, "vdim", mw),
                            decay=tuple(float(v) for v in decay))


def _experts(mlp: Mapping[str, Any], fw: str) -> MuvoraxExperts:
    r, rw = _obj(mlp, "router", fw), fw + "router."
    groups, keep = 1, 1
    if r.get("groups") is not None:
        g, gw = _obj(r, "groups", rw), rw + "groups."
        groups, keep = _int(g, "count", gw), _int(g, "keep", gw)
    out = MuvoraxExperts(ff=_int(_obj(mlp, "expert", fw), "ff", fw + "expert."), experts=_int(r, "experts", rw),
                         top=_int(r, "top", rw), scale=1.0 if r.get("scale") is None else _num(r, "scale", rw),
                         groups=groups, keep=keep)
    if out.experts % groups or keep > groups:
        raise ConfigError(f"config.json: {rw}groups: {groups} groups of which {keep} are kept do not divide "
                          f"{out.experts} experts")
    if out.top > keep * (out.experts // groups):
        raise ConfigError(f"config.json: {rw}top {out.top} exceeds the {keep * (out.experts // groups)} experts that "
                          f"can be chosen from")
    return out


@dataclass(frozen=True)
class MuvoraxConfig:
    vocab: int
    width: int
    eps: float
    layers: Tuple[MuvoraxLayer, ...]
    max_positions: int = DEFAULT_MAX_POSITIONS

    @classmethod
    def from_dict(cls, d: Mapping[str, Any]) -> "MuvoraxConfig":
        vocab, width = _int(d, "vocab", ""), _int(d, "width", "")
        eps = _num(_obj(d, "norm", ""), "eps", "norm.")
        raw = d.get("layers")
        if not isinstance(raw, list) or not raw:
            raise ConfigError("config.json: 'layers' must be a non-empty list")
        layers: List[MuvoraxLayer] = []
        for i, entry in enumerate(raw):
            where = f"layers[{i}]."
            kind = entry.get("type") if isinstance(entry, Mapping) else entry
            if kind not in TYPES:
                raise ConfigError(f"config.json: {where}type {kind!r} is not a mixer of this design (known: "
                                  + ", ".join(repr(t) for t in TYPES) + ")")
            m, mw = _obj(entry, "mixer", where), where + "mixer."
            if kind == "latent_attention":
                mixer = _latent(m, mw, i, layers)
            elif kind == "mamba1":
                mixer = MuvoraxScan(inner=_int(m, "inner", mw), state=_int(m, "state", mw),
                                    dt_rank=_int(m, "dt_rank", mw), conv=_int(m, "conv", mw))
            else:
                mixer = _lightning(m, mw)
            mlp = entry.get("mlp")
            if mlp is not None:
                fw = where + "mlp."
                fk = mlp.get("kind") if isinstance(mlp, Mapping) else mlp
                if fk == "dense":
                    mlp = MuvoraxDense(_int(mlp, "ff", fw))
                elif fk == "moe":
                    mlp = _experts(mlp, fw)
                else:
                    raise ConfigError(f"config.json: {fw}kind {fk!r} is not known (known: 'dense', 'moe')")
            layers.append(MuvoraxLayer(mixer, mlp))
        mp = d.get("max_positions")
        return cls(vocab=vocab, width=width, eps=eps, layers=tuple(layers),
                   max_positions=DEFAULT_MAX_POSITIONS if mp is None else _int(d, "max_positions", ""))
