"""Mixers side by side: every member reads the same input, and the result is the weighted sum of their outputs,
  out = sum_m scale_m * member_m(h).
The members are mixers of any kind (an attention beside a recurrent mixer, say), built from their own descriptions; a
member's tensors stand under "<member's name>." and what it keeps per request under "<role>.<member's name>" (pages or
state that a later layer may read) and "<role>.<member's name>.state" (what it keeps for itself alone).

Members that come in pieces (`in_matrices`, `core`, `out_matrix`: all of them, or this is not done) share their first
and their last product: one product of h gives every member's columns, every member leaves what its output matrix
multiplies, times its scale, in its own columns of one row, and one product over that row adds the members up."""
from __future__ import annotations

from typing import Dict, Mapping, Sequence

import torch

from ..kernels import ops
from .base import MIXERS, Mixer, Runtime, as_normed, build_part, to_device
from .spec import ParamSpec, PartSpec


def _up8(n: int) -> int:
    return -(-n // 8) * 8


def _stacked(pieces, rows: int, cols: int, axis: int, rt: Runtime) -> torch.Tensor:
    """[rows, cols] on the run's device: the matrices of `pieces` ((place along `axis`, matrix)), zeros elsewhere."""
    dt = pieces[0][1].dtype if all(m.dtype == pieces[0][1].dtype for _, m in pieces) else torch.float32
    w = torch.zeros((rows, cols), dtype=dt, device=rt.device)
    for at, m in pieces:
        w.narrow(axis, at, m.shape[axis]).copy_(to_device(m, rt, dt))
    return w


def _member_views(views: Mapping, name: str) -> dict:
    own = {"mixer": views.get(f"mixer.{name}"), "mixer.state": views.get(f"mixer.{name}.state")}
    return {k: v for k, v in own.items() if v is not None}


@MIXERS.register("parallel")
class ParallelMixers(Mixer):
    def __init__(self, members: Sequence[Mapping]):
        """`members`: dicts {"name", "kind", "params", "scale"} in the order in which the outputs are added."""
        if len(members) < 2:
            raise ValueError("mixers side by side: at least two members")
        self.names = [str(m["name"]) for m in members]
        if len(set(self.names)) != len(self.names):
            raise ValueError(f"mixers side by side: member names must differ, got {self.names}")
        self.scales = [float(m.get("scale", 1.0)) for m in members]
        self.members = [build_part(MIXERS, PartSpec(m["kind"], dict(m.get("params", {})))) for m in members]

    @property
    def graph_safe(self) -> bool:
        return all(getattr(m, "graph_safe", False) for m in self.members)

    def param_specs(self) -> Dict[str, ParamSpec]:
        return {f"{name}.{n}": ps for name, m in zip(self.names, self.members) for n, ps in m.param_specs().items()}

    def cache_need(self):
        needs = {name: m.cache_need() for name, m in zip(self.names, self.members)}
        return needs if any(n is not None for n in needs.values()) else None

    def state_need(self):
        needs = {name: m.state_need() for name, m in zip(self.names, self.members)}
        return needs if any(n is not None for n in needs.values()) else None

    def bind(self, tensors: Mapping[str, torch.Tensor], rt: Runtime) -> None:
        self.rt = rt
        own = [{n[len(name) + 1:]: t for n, t in tensors.items() if n.startswith(name + ".")} for name in self.names]
        self.joint = all(hasattr(m, "core") for m in self.members)
        if not self.joint:
            for m, t in zip(self.members, own):
                m.bind(t, rt)
            return
        # columns of the shared rows, every member's from a multiple of 8 on
        self.in_at, self.out_at, a, b = [], [], 0, 0
        for m in self.members:
            self.in_at.append(a)
            self.out_at.append(b)
            a, b = _up8(a + m.in_width), _up8(b + m.out_width)
        self.in_width, self.out_width = a, b
        self.D = self.members[0].D
        mats = [(at, m.in_matrices(t)) for at, m, t in zip(self.in_at, self.members, own)]
        outs = [(at, m.out_matrix(t)) for at, m, t in zip(self.out_at, self.members, own)]
        self.w_in = ops.prepare_matrix(_stacked([(at, torch.cat(list(ms), dim=0)) for at, ms in mats], self.in_width,
                                                self.D, 0, rt), rt.dtype)
        self.w_o = ops.prepare_matrix(_stacked(outs, self.D, self.out_width, 1, rt), rt.dtype)
        # (gaps between the members' columns meet zeros of the matrix, and must be finite themselves)
        self.gaps = sum(m.out_width for m in self.members) != self.out_width
        for m, t in zip(self.members, own):
            m.bind_core(t, rt)

    def _forward_joint(self, h, step, views) -> torch.Tensor:
        h = as_normed(h).tensor()
        T, dev, dt = h.shape[0], h.device, self.rt.dtype
        proj = torch.empty((T, self.in_width), dtype=dt, device=dev)
        ops.linear(h, self.w_in, proj)
        mixed = (torch.zeros if self.gaps else torch.empty)((T, self.out_width), dtype=dt, device=dev)
        for name, m, scale, a, b in zip(self.names, self.members, self.scales, self.in_at, self.out_at):
            m.core(proj[:, a:a + m.in_width], step, _member_views(views, name), mixed[:, b:b + m.out_width], scale)
        out = torch.empty((T, self.D), dtype=torch.float32, device=dev)
        ops.linear(mixed, self.w_o, out)
        return out

    def forward(self, h, step, cache) -> torch.Tensor:
        """float32 [rows, hidden].  `cache`: {"mixer.<member>": view, "mixer.<member>.state": view}."""
        views = cache if isinstance(cache, dict) else {}
        if self.joint:
            return self._forward_joint(h, step, views)
        out = None
        for i, (name, m) in enumerate(zip(self.names, self.members)):
            y = m.forward(h, step, _member_views(views, name))
            if i == 0:
                out, first = y, self.scales[0]
            else:
                # out <- first * out + scale * y in 32-bit (the first member's factor is applied with the second's sum)
                ops.weighted_pair(out, first, y, self.scales[i], out)
                first = 1.0
        return out
