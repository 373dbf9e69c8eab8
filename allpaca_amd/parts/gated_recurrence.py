"""A recurrent block around a real-gated linear recurrence (the block and the unit of Griffin, De et al. 2024).

Per row, with h the mixer's input and `width` channels C:
  y = gelu(Wy h + by),  x = Wx h + bx
  u = conv(x) + bc                                    a short causal convolution over time on every channel, zeros ahead
                                                      of the sequence
  u in `blocks` equal parts: r = sigmoid(Ra_b u_b + ra_b), i = sigmoid(Ri_b u_b + ri_b)      (square matrices a part)
  log a = -8 r softplus(lam);  S <- a S + sqrt(1 - a^2) i u;  out = Wo (S * y)
S is float32 state of the request (a slot, zero when a request starts: the first row is no special case), and so are the
convolution's last taps - 1 inputs (with their bias).  The gates, a, the root and the state are 32-bit; x, u, y and S * y
are held in the run's element type."""
from __future__ import annotations

from typing import Dict, List, Mapping, Optional

import torch

from ..kernels import ops
from .base import MIXERS, FixedState, Mixer, Runtime, as_normed, to_device
from .spec import ParamSpec

RATE = -8.0      # log a at r = 1, in units of softplus(lam)


@MIXERS.register("gated_recurrence")
class GatedRecurrence(Mixer):
    graph_safe = True

    def __init__(self, hidden_size: int, width: int, blocks: int, conv_taps: int,
                 names: Optional[Mapping[str, str]] = None):
        self.D, self.C, self.B, self.taps = int(hidden_size), int(width), int(blocks), int(conv_taps)
        if min(self.D, self.C, self.B, self.taps) < 1 or self.C % self.B:
            raise ValueError(f"gated recurrence: {blocks} equal parts of {width} channels, a convolution of at least one tap")
        self.w = self.C // self.B
        self.names = {"y": "y", "x": "x", "bias": ".b", "conv": "conv", "conv_bias": "conv.b", "ra": "ra", "ri": "ri",
                      "lam": "lam", "o": "o", **dict(names or {})}
        self.in_width, self.out_width = 2 * self.C, self.C

    def param_specs(self) -> Dict[str, ParamSpec]:
        n, C, B, w = self.names, self.C, self.B, self.w
        out = {n["conv"]: ParamSpec((C, self.taps), store="float32", init="normal"),
               n["conv_bias"]: ParamSpec((C,), store="float32", init="zeros"),
               n["lam"]: ParamSpec((C,), store="float32", init="normal"),
               n["o"]: ParamSpec((self.D, C))}
        for p in ("y", "x"):
            out[n[p]] = ParamSpec((C, self.D))
            out[n[p] + n["bias"]] = ParamSpec((C,), store="float32", init="zeros")
        for p in ("ra", "ri"):
            out[n[p]] = ParamSpec((B, w, w))
            out[n[p] + n["bias"]] = ParamSpec((B, w), store="float32", init="zeros")
        return out

    def cache_need(self):
        return FixedState((self.C,), "float32")

    def state_need(self):
        return FixedState((self.taps - 1, self.C), "float32") if self.taps > 1 else None

    # ---- the pieces around `core`: a caller with several mixers side by side may put their matrices together
    def in_matrices(self, tensors: Mapping[str, torch.Tensor]) -> List[torch.Tensor]:
        """Matrices [.., hidden] whose outputs one below the other are the `in_width` columns `core` reads: y, then x."""
        return [tensors[self.names["y"]], tensors[self.names["x"]]]

    def out_matrix(self, tensors: Mapping[str, torch.Tensor]) -> torch.Tensor:
        return tensors[self.names["o"]]

    def bind_core(self, tensors: Mapping[str, torch.Tensor], rt: Runtime) -> None:
        self.rt = rt
        n, B, w = self.names, self.B, self.w
        # a part's two square matrices one below the other: one product gives r's and i's logits
        gates = torch.cat([to_device(tensors[n[p]], rt) for p in ("ra", "ri")], dim=1).contiguous()
        self.w_gates = ops.prepare_heads(gates, rt.dtype, w, 2 * w)
        self.gates_b = torch.cat([to_device(tensors[n[p] + n["bias"]], rt, torch.float32).view(B, w)
                                  for p in ("ra", "ri")], dim=1).reshape(-1).contiguous()
        self.y_b, self.x_b = (to_device(tensors[n[p] + n["bias"]], rt, torch.float32) for p in ("y", "x"))
        self.conv_w = to_device(tensors[n["conv"]], rt, torch.float32)
        self.conv_b = to_device(tensors[n["conv_bias"]], rt, torch.float32)
        lam = tensors[n["lam"]].to(torch.float64)
        self.rate = to_device((RATE * torch.nn.functional.softplus(lam, threshold=40.0)).to(torch.float32), rt)

    def core(self, proj: torch.Tensor, step, cache, out: torch.Tensor, scale: float = 1.0) -> None:
        """`proj` [rows, in_width] (y and x without their biases) -> `out` [rows, out_width], what Wo multiplies, times
        `scale`."""
        state, conv = (cache.get("mixer"), cache.get("mixer.state")) if isinstance(cache, dict) else (cache, None)
        if state is None or not state.writes:
            raise ValueError("a recurrent mixer needs a state of its own")
        T, dev, C = proj.shape[0], proj.device, self.C
        u = torch.empty((T, C), dtype=self.rt.dtype, device=dev)
        ops.conv_channels(proj[:, C:], C, self.conv_w, self.conv_b, conv.state if conv is not None else None, step,
                          conv.slots if conv is not None else None, "none", u, in_bias=self.x_b)
        z = torch.empty((T, 2 * C), dtype=torch.float32, device=dev)
        ops.heads_linear(u, self.w, self.w_gates, z, 2 * self.w)
        ops.gated_recurrence(u, z, self.gates_b, self.B, self.rate, proj[:, :C], self.y_b, state.state, step,
                             state.slots, out, scale)

    # ---- the mixer by itself
    def bind(self, tensors: Mapping[str, torch.Tensor], rt: Runtime) -> None:
        self.bind_core(tensors, rt)
        mats = self.in_matrices(tensors)
        dt = mats[0].dtype if all(m.dtype == mats[0].dtype for m in mats) else torch.float32
        self.w_in = ops.prepare_matrix(torch.cat([to_device(m, rt, dt) for m in mats], dim=0), rt.dtype)
        self.w_o = ops.prepare_matrix(to_device(self.out_matrix(tensors), rt), rt.dtype)

    def forward(self, h, step, cache) -> torch.Tensor:
        """float32 [rows, hidden]: the mixer's output.  `cache`: the state's view, or {"mixer": the state,
        "mixer.state": the convolution's inputs}."""
        h = as_normed(h).tensor()
        T, dev, dt = h.shape[0], h.device, self.rt.dtype
        proj = torch.empty((T, self.in_width), dtype=dt, device=dev)
        ops.linear(h, self.w_in, proj)
        mixed = torch.empty((T, self.out_width), dtype=dt, device=dev)
        self.core(proj, step, cache, mixed)
        out = torch.empty((T, self.D), dtype=torch.float32, device=dev)
        ops.linear(mixed, self.w_o, out)
        return out
