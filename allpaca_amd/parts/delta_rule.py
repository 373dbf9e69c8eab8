"""Gated delta rule: linear attention whose write replaces what the state already gives for a key, with a decay per head.

Per row, with h the mixer's input, H heads of values over G heads of queries and keys (head h uses q/k head h // (H / G)):
  q = Wq h, k = Wk h  (G x key_dim),  v = Wv h  (H x value_dim);  each through a short causal convolution over time on
  every channel (zeros ahead of the sequence) and silu
  q and k of a head divided by sqrt(sum of squares + 1e-6), q also times key_dim^(-1/2)
  beta = sigmoid(Wb h),  g = exp(-exp(A_log) softplus(Wa h + dt_bias))          one number a head each
  S <- g S;  u = beta (v - S^T k);  S <- S + k u^T;  o = S^T q                    S [key_dim, value_dim]
  o divided by its root mean square over the head (eps), times a weight [value_dim] of all heads, times silu(Wg h); Wo
S is float32 state of the request (a slot, zero when a request starts), and so are the convolutions' last taps - 1
inputs.  Everything behind the projections and the convolutions with their silu is 32-bit up to the gated norm."""
from __future__ import annotations

from typing import Dict, Mapping, Optional

import torch

from ..kernels import ops
from .base import MIXERS, FixedState, Mixer, Runtime, as_normed, to_device
from .spec import ParamSpec


@MIXERS.register("gated_delta_rule")
class GatedDeltaRule(Mixer):
    graph_safe = True

    def __init__(self, hidden_size: int, num_heads: int, num_kv_heads: int, key_dim: int, value_dim: int,
                 conv_taps: int, norm_eps: float = 1e-6, names: Optional[Mapping[str, str]] = None):
        if num_heads % num_kv_heads:
            raise ValueError(f"delta rule: {num_heads} heads are not a multiple of {num_kv_heads} query/key heads")
        self.D, self.H, self.G = int(hidden_size), int(num_heads), int(num_kv_heads)
        self.dk, self.dv, self.taps, self.eps = int(key_dim), int(value_dim), int(conv_taps), float(norm_eps)
        if min(self.dk, self.dv, self.taps) < 1:
            raise ValueError("delta rule: every size must be positive (a convolution has at least one tap)")
        self.names = {"q": "q", "k": "k", "v": "v", "conv": ".conv", "b": "b", "a": "a", "A_log": "A_log",
                      "dt_bias": "dt_bias", "norm": "norm", "gate": "g", "o": "o", **dict(names or {})}
        self.projections = [("q", self.G * self.dk), ("k", self.G * self.dk), ("v", self.H * self.dv)]
        self.q_off, self.k_off, self.v_off = 0, self.G * self.dk, 2 * self.G * self.dk
        self.channels = self.v_off + self.H * self.dv          # through the convolutions
        # columns behind them, each from a multiple of 8 on: the gate's logits, then a, then b
        self.g_off = -(-self.channels // 8) * 8
        self.a_off = -(-(self.g_off + self.H * self.dv) // 8) * 8
        self.width = -(-(self.a_off + 2 * self.H) // 8) * 8

    def param_specs(self) -> Dict[str, ParamSpec]:
        n, H, N = self.names, self.H, self.H * self.dv
        out: Dict[str, ParamSpec] = {}
        for p, rows in self.projections:
            out[n[p]] = ParamSpec((rows, self.D))
            out[n[p] + n["conv"]] = ParamSpec((rows, self.taps), store="float32", init="normal")
        out[n["a"]] = out[n["b"]] = ParamSpec((H, self.D))
        out[n["A_log"]] = out[n["dt_bias"]] = ParamSpec((H,), store="float32", init="normal")
        out[n["norm"]] = ParamSpec((self.dv,), store="float32")
        out[n["gate"]] = ParamSpec((N, self.D))
        out[n["o"]] = ParamSpec((self.D, N))
        return out

    def cache_need(self):
        return FixedState((self.H, self.dk, self.dv), "float32")

    def state_need(self):
        return FixedState((self.taps - 1, self.channels), "float32") if self.taps > 1 else None

    def bind(self, tensors: Mapping[str, torch.Tensor], rt: Runtime) -> None:
        self.rt = rt
        n = self.names
        mats = [(self.q_off, "q"), (self.k_off, "k"), (self.v_off, "v"), (self.g_off, "gate"), (self.a_off, "a"),
                (self.a_off + self.H, "b")]
        mats = [(at, tensors[n[p]]) for at, p in mats]
        dt = mats[0][1].dtype if all(m.dtype == mats[0][1].dtype for _, m in mats) else torch.float32
        # one [width, D] matrix (rows of zeros between the pieces): a single product gives everything of a row
        w_in = torch.zeros((self.width, self.D), dtype=dt, device=rt.device)
        for at, m in mats:
            w_in[at:at + m.shape[0]] = to_device(m, rt, dt)
        self.w_in = ops.prepare_matrix(w_in, rt.dtype)
        self.w_o = ops.prepare_matrix(to_device(tensors[n["o"]], rt), rt.dtype)
        self.conv_w = torch.cat([to_device(tensors[n[p] + n["conv"]], rt, torch.float32)
                                 for p, _ in self.projections], dim=0).contiguous()
        self.A = to_device(torch.exp(tensors[n["A_log"]].to(torch.float64)).to(torch.float32), rt)
        self.dt_bias = to_device(tensors[n["dt_bias"]], rt, torch.float32)
        # the head's weight once for every head: what the norm of groups reads
        self.norm_w = to_device(tensors[n["norm"]], rt, torch.float32).repeat(self.H).contiguous()

    def forward(self, h, step, cache) -> torch.Tensor:
        """float32 [rows, hidden]: the mixer's output.  `cache`: the state's view, or {"mixer": the state,
        "mixer.state": the convolutions' inputs}."""
        state, conv = (cache.get("mixer"), cache.get("mixer.state")) if isinstance(cache, dict) else (cache, None)
        if state is None or not state.writes:
            raise ValueError("a recurrent mixer needs a state of its own")
        h = as_normed(h).tensor()
        T, dev, dt, N = h.shape[0], h.device, self.rt.dtype, self.H * self.dv
        proj = torch.empty((T, self.width), dtype=dt, device=dev)
        ops.linear(h, self.w_in, proj)
        act = torch.empty((T, self.channels), dtype=dt, device=dev)
        ops.conv_channels(proj, self.channels, self.conv_w, None, conv.state if conv is not None else None, step,
                          conv.slots if conv is not None else None, "silu", act)
        o = torch.empty((T, N), dtype=torch.float32, device=dev)
        ops.delta_rule(act, self.q_off, self.k_off, self.v_off, self.H, self.G, self.dk, self.dv, proj, self.a_off,
                       self.a_off + self.H, self.A, self.dt_bias, state.state, step, state.slots, o)
        a = torch.empty((T, N), dtype=dt, device=dev)
        ops.gated_rmsnorm(o, self.norm_w, self.eps, proj[:, self.g_off:self.g_off + N], a, group=self.dv, gate_act="silu")
        out = torch.empty((T, self.D), dtype=torch.float32, device=dev)
        ops.linear(a, self.w_o, out)
        return out
