"""Norms.

`rmsnorm`: out = x / sqrt(mean(x^2) + eps) * w, the sum and the scale in
32-bit; eps inside the root, the weight applied plainly (no 1 + w)
(crates/allpaca-cpu/src/kernels.rs:492-507).  With `scalar` the weight is a single
number: out = x / sqrt(mean(x^2) + eps) * g.

`dynamic_tanh`: out = tanh(alpha * x) * w + b, element by element and in 32-bit: no mean, no variance, no eps.  alpha is
one number (a tensor without dimensions), w and b have the row's size."""
from __future__ import annotations

from typing import Dict, Mapping, Optional

import torch

from ..kernels import ops
from .base import NORMS, Norm, Runtime, to_device
from .spec import ParamSpec


@NORMS.register("rmsnorm")
class RMSNorm(Norm):
    graph_safe = True

    def __init__(self, size: int, eps: float, name: str = "weight", scalar: bool = False):
        self.size, self.eps, self.name = int(size), float(eps), name     # `name`: the weight's tensor name
        self.scalar = bool(scalar)     # the weight is one number for all coordinates (a tensor without dimensions)

    def param_specs(self) -> Dict[str, ParamSpec]:
        return {self.name: ParamSpec(() if self.scalar else (self.size,), store="float32")}

    def bind(self, tensors: Mapping[str, torch.Tensor], rt: Runtime) -> None:
        self.rt = rt
        w = tensors[self.name].to(torch.float32)
        if self.scalar:                # kept as a row of equal numbers: the kernels and the folded forms are the same
            w = w.reshape(1).expand(self.size)
        self.weight = to_device(w, rt, torch.float32)

    def forward(self, x: torch.Tensor, out: torch.Tensor, rows: Optional[torch.Tensor] = None) -> None:
        ops.rmsnorm_rows(x, self.weight, self.eps, out, rows)

    def rms_params(self):
        return self.weight, self.eps

    def add_normed(self, x, y, then=None, h=None) -> None:
        ops.rmsnorm_add(y, self.weight, self.eps, 1.0, x)
        if then is not None:
            then.forward(x, h)

    def native_desc(self):
        return {"kind": "rmsnorm", "weight": self.weight, "eps": self.eps} if type(self) is RMSNorm else None


@NORMS.register("dynamic_tanh")
class DynamicTanh(Norm):
    graph_safe = True

    def __init__(self, size: int, name: str = "weight", alpha_name: Optional[str] = None,
                 bias_name: Optional[str] = None):
        self.size, self.name = int(size), name
        self.alpha_name, self.bias_name = alpha_name or name + ".alpha", bias_name or name + ".b"

    def param_specs(self) -> Dict[str, ParamSpec]:
        return {self.name: ParamSpec((self.size,), store="float32"),
                self.bias_name: ParamSpec((self.size,), store="float32", init="zeros"),
                self.alpha_name: ParamSpec((), store="float32", init=1.0)}

    def bind(self, tensors: Mapping[str, torch.Tensor], rt: Runtime) -> None:
        self.rt = rt
        self.weight = to_device(tensors[self.name], rt, torch.float32)
        self.bias = to_device(tensors[self.bias_name], rt, torch.float32)
        self.alpha = float(tensors[self.alpha_name].to(torch.float32))

    def tanh_params(self):
        return self.alpha, self.weight, self.bias

    def forward(self, x: torch.Tensor, out: torch.Tensor, rows: Optional[torch.Tensor] = None) -> None:
        ops.tanh_norm(x, self.tanh_params(), out, rows, exact=self.rt.is_float32)

    def add_normed(self, x, y, then=None, h=None) -> None:
        if isinstance(then, DynamicTanh):       # the sum and the next norm in one pass over the row
            ops.tanh_norm_add(x, y, self.tanh_params(), then.tanh_params(), h, exact=self.rt.is_float32)
            return
        ops.tanh_norm_add(x, y, self.tanh_params(), exact=self.rt.is_float32)
        if then is not None:
            then.forward(x, h)
