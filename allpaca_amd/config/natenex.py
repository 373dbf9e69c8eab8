"""Typed configuration of the Natenex decoder, read from config.json.

Keys: `vocab`, `width`, `embedding.scale`, `norm.eps`, `max_positions` (optional) and `layers`, a list of
{"type", "mixer", "mlp", "weights_of"}.
  type "parallel": `left` (an attention: `heads`, `kv_heads`, `dim`, `vdim`, `scale`, `rot` {"base", "dims", "scaling":
      {"factor", "low", "high", "original"} or absent}, `mask` {"size", "keep_first"} or absent: every earlier token),
      `right` (a gated recurrence: `width`, `blocks`, `conv`), `left_scale`, `right_scale`.
  type "latent_attention": `heads`, `dim` (unrotated elements of a head's query and key), `rot_dim` (rotated ones),
      `vdim`, `q_rank`, `kv_rank` (sizes of the latents), `scale`, `rot` {"base", "dims" = rot_dim, "scaling" as above}.
  type "delta": `heads`, `kv_heads`, `dim`, `vdim`, `conv`.
  `mlp`: null or {"kind": "dense", "ff"}.
  `weights_of` j: the layer has no tensors of its own, it uses those of layer j with a cache of its own.
A size that the file leaves out is taken from the shape of the tensor that has it (`sizes_from_tensors`); constants
come from the file alone."""
from __future__ import annotations

from dataclasses import dataclass
from typing import Any, List, Mapping, Optional, Tuple, Union

from .lesarax import DEFAULT_MAX_POSITIONS, _obj, _rot
from .llama import ConfigError
from .risizen import _int, _num


@dataclass(frozen=True)
class NatenexScaling:
    factor: float
    low: float
    high: float
    original: float


@dataclass(frozen=True)
class NatenexWindow:
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    scale: float
    rot_dims: int
    rot_base: float
    scaling: Optional[NatenexScaling] = None
    window: int = 0                                 # 0: every earlier token
    keep_first: int = 0


@dataclass(frozen=True)
class NatenexRecurrence:
    width: int
    blocks: int
    conv: int


@dataclass(frozen=True)
class NatenexParallel:
    left: NatenexWindow
    right: NatenexRecurrence
    left_scale: float
    right_scale: float


@dataclass(frozen=True)
class NatenexLatent:
    heads: int
    dim: int
    rot_dim: int
    vdim: int
    q_rank: int
    kv_rank: int
    scale: float
    rot_base: float
    scaling: Optional[NatenexScaling] = None


@dataclass(frozen=True)
class NatenexDelta:
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    conv: int


@dataclass(frozen=True)
class NatenexLayer:
    mixer: Union[NatenexParallel, NatenexLatent, NatenexDelta]
    ff: int = 0                                     # 0: no feed-forward
    weights_of: Optional[int] = None                # the layer whose tensors it uses (never one that borrows itself)


TYPES = ("parallel", "latent_attention", "delta")


def _is_int(v) -> bool:
    return isinstance(v, int) and not isinstance(v, bool)


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
        return a // b if a and _is_int(b) and b > 0 and a % b == 0 else None

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
        src = entry.get("weights_of")
        for _ in range(len(layers)):                # (a borrower of a borrower)
            if not _is_int(src) or not 0 <= src < len(layers) or not isinstance(layers[src], Mapping) \
                    or layers[src].get("weights_of") is None:
                break
            src = layers[src]["weights_of"]
        owner = src if _is_int(src) else i
        p, kind = f"l{owner}.mix.", entry.get("type")
        m = dict(entry["mixer"])
        if kind == "parallel":
            left = dict(m["left"]) if isinstance(m.get("left"), Mapping) else {}
            right = dict(m["right"]) if isinstance(m.get("right"), Mapping) else {}
            fill(left, "dim", dim_of(p + "left.q.norm"))
            fill(left, "heads", over(dim_of(p + "left.q"), left.get("dim")))
            fill(left, "kv_heads", over(dim_of(p + "left.k"), left.get("dim")))
            fill(left, "vdim", over(dim_of(p + "left.v"), left.get("kv_heads")))
            fill(right, "width", dim_of(p + "right.lam"))
            fill(right, "conv", dim_of(p + "right.conv", 1))
            fill(right, "blocks", dim_of(p + "right.ra"))
            m["left"], m["right"] = left, right
        elif kind == "latent_attention":
            rot = m.get("rot") if isinstance(m.get("rot"), Mapping) else {}
            fill(m, "q_rank", dim_of(p + "dq"))
            fill(m, "kv_rank", dim_of(p + "uk", 1))
            down, rank = dim_of(p + "dkv"), m.get("kv_rank")
            if down is not None and _is_int(rank) and down > rank:
                fill(m, "rot_dim", down - rank)
            fill(m, "rot_dim", rot.get("dims"))
            if rot and rot.get("dims") is None and m.get("rot_dim") is not None:
                m["rot"] = dict(rot, dims=m["rot_dim"])
            q_rows, k_rows, r = dim_of(p + "uq"), dim_of(p + "uk"), m.get("rot_dim")
            if _is_int(r) and r > 0 and q_rows and k_rows:
                fill(m, "heads", over(q_rows - k_rows, r))      # (a head's query has the rotated part, its key matrix not)
            fill(m, "dim", over(k_rows, m.get("heads")))
            fill(m, "heads", over(k_rows, m.get("dim")))
            fill(m, "vdim", over(dim_of(p + "uv"), m.get("heads")))
        elif kind == "delta":
            fill(m, "heads", dim_of(p + "A_log"))
            fill(m, "vdim", dim_of(p + "norm"))
            fill(m, "conv", dim_of(p + "q.conv", 1))
            fill(m, "kv_heads", over(dim_of(p + "q"), m.get("dim")))
            fill(m, "dim", over(dim_of(p + "q"), m.get("kv_heads")))
        e = dict(entry, mixer=m)
        f = entry.get("mlp")
        if isinstance(f, Mapping) and f.get("kind") == "dense":
            e["mlp"] = f = dict(f)
            fill(f, "ff", dim_of(f"l{owner}.mlp.up"))
        new_layers.append(e)
    return out


def _scaling(m: Mapping[str, Any], mw: str) -> Optional[NatenexScaling]:
    if m["rot"].get("scaling") is None:
        return None
    s, sw = _obj(m["rot"], "scaling", mw + "rot."), mw + "rot.scaling."
    sc = NatenexScaling(*(_num(s, k, sw) for k in ("factor", "low", "high", "original")))
    if not (sc.factor > 0 and sc.original > 0 and sc.low > 0 and sc.high > sc.low):
        raise ConfigError(f"config.json: {sw}factor, low and original must be positive, high larger than low")
    return sc


def _heads(m: Mapping[str, Any], where: str) -> Tuple[int, int]:
    heads, kv = _int(m, "heads", where), _int(m, "kv_heads", where)
    if heads % kv:
        raise ConfigError(f"config.json: {where}heads {heads} is no multiple of kv_heads {kv}")
    return heads, kv


def _parallel(m: Mapping[str, Any], mw: str) -> NatenexParallel:
    l, lw = _obj(m, "left", mw), mw + "left."
    heads, kv = _heads(l, lw)
    dims, base = _rot(l, lw)
    window = keep = 0
    if l.get("mask") is not None:
        k, kw = _obj(l, "mask", lw), lw + "mask."
        window = _int(k, "size", kw)
        keep = 0 if k.get("keep_first") is None else _int(k, "keep_first", kw, least=0)
    left = NatenexWindow(heads=heads, kv_heads=kv, dim=_int(l, "dim", lw), vdim=_int(l, "vdim", lw),
                         scale=_num(l, "scale", lw), rot_dims=dims, rot_base=base, scaling=_scaling(l, lw),
                         window=window, keep_first=keep)
    if dims > left.dim:
        raise ConfigError(f"config.json: {lw}rot.dims {dims} exceeds dim {left.dim}")
    r, rw = _obj(m, "right", mw), mw + "right."
    right = NatenexRecurrence(width=_int(r, "width", rw), blocks=_int(r, "blocks", rw), conv=_int(r, "conv", rw))
    if right.width % right.blocks:
        raise ConfigError(f"config.json: {rw}blocks {right.blocks} does not divide width {right.width}")
    return NatenexParallel(left, right, _num(m, "left_scale", mw), _num(m, "right_scale", mw))


def _latent(m: Mapping[str, Any], mw: str) -> NatenexLatent:
    rot_dim = _int(m, "rot_dim", mw, least=0)
    dims, base = _rot(m, mw)
    if dims != rot_dim:
        raise ConfigError(f"config.json: {mw}rot.dims {dims} must equal rot_dim {rot_dim}")
    return NatenexLatent(heads=_int(m, "heads", mw), dim=_int(m, "dim", mw), rot_dim=rot_dim, vdim=_int(m, "vdim", mw),
                         q_rank=_int(m, "q_rank", mw), kv_rank=_int(m, "kv_rank", mw), scale=_num(m, "scale", mw),
                         rot_base=base, scaling=_scaling(m, mw))


def _delta(m: Mapping[str, Any], mw: str) -> NatenexDelta:
    heads, kv = _heads(m, mw)
    return NatenexDelta(heads=heads, kv_heads=kv, dim=_int(m, "dim", mw), vdim=_int(m, "vdim", mw),
                        conv=_int(m, "conv", mw))


@dataclass(frozen=True)
class NatenexConfig:
    vocab: int
    width: int
    embedding_scale: float
    eps: float
    layers: Tuple[NatenexLayer, ...]
    max_positions: int = DEFAULT_MAX_POSITIONS

    @classmethod
    def from_dict(cls, d: Mapping[str, Any]) -> "NatenexConfig":
        vocab, width = _int(d, "vocab", ""), _int(d, "width", "")
        eps = _num(_obj(d, "norm", ""), "eps", "norm.")
        raw = d.get("layers")
        if not isinstance(raw, list) or not raw:
            raise ConfigError("config.json: 'layers' must be a non-empty list")
        layers: List[NatenexLayer] = []
        for i, entry in enumerate(raw):
            where = f"layers[{i}]."
            kind = entry.get("type") if isinstance(entry, Mapping) else entry
            if kind not in TYPES:
                raise ConfigError(f"config.json: {where}type {kind!r} is not a mixer of this design (known: "
                                  + ", ".join(repr(t) for t in TYPES) + ")")
            m, mw = _obj(entry, "mixer", where), where + "mixer."
            mixer = {"parallel": _parallel, "latent_attention": _latent, "delta": _delta}[kind](m, mw)
            mlp, ff = entry.get("mlp"), 0
            if mlp is not None:
                fk = mlp.get("kind") if isinstance(mlp, Mapping) else mlp
                if fk != "dense":
                    raise ConfigError(f"config.json: {where}mlp.kind {fk!r} is not known (known: 'dense')")
                ff = _int(mlp, "ff", where + "mlp.")
            layers.append(NatenexLayer(mixer, ff, None if entry.get("weights_of") is None
                                       else _int(entry, "weights_of", where, least=0)))
        for i, layer in enumerate(layers):
            j, hops = layer.weights_of, 0
            if j is None:
                continue
            while j < len(layers) and layers[j].weights_of is not None and hops <= len(layers):
                j, hops = layers[j].weights_of, hops + 1
            if j >= len(layers) or hops > len(layers):
                raise ConfigError(f"config.json: layers[{i}].weights_of {layer.weights_of} names no layer with tensors")
            if (layers[j].mixer, layers[j].ff) != (layer.mixer, layer.ff):
                raise ConfigError(f"config.json: layers[{i}] uses the weights of layer {j} and must equal it")
            layers[i] = NatenexLayer(layer.mixer, layer.ff, j)
        mp = d.get("max_positions")
        return cls(vocab=vocab, width=width, embedding_scale=_num(_obj(d, "embedding", ""), "scale", "embedding."),
                   eps=eps, layers=tuple(layers),
                   max_positions=DEFAULT_MAX_POSITIONS if mp is None else _int(d, "max_positions", ""))
