"""Attention over cached latents.

Per row, with h the mixer's input, H heads, dn unrotated and dr rotated elements of a query or key head, R the size of
the latent of keys and values:
  q = Wq h                                     heads of [dn, dr]
  [c' | kr'] = Wdkv h                          R, dr
  c = rms_norm(c') * dkv.norm;  kr = rotate(kr')          one rotated key part, shared by all heads
  key of head j = [(Wuk c)_j, kr], value of head j = (Wuv c)_j;  s = (q . k) * scale, causal softmax;  out = Wo (sum p v)
The pages hold c and kr alone (`PagedLatents`), and keys and values are never written out: the two up-projections are
applied to the queries and to the outputs instead,
  q . k = (Wuk_j^T q[:dn]) . c + rotate(q[dn:]) . kr,     sum_t p_t (Wuv_j c_t) = Wuv_j (sum_t p_t c_t),
so all heads read one row of R + dr elements a position, and what a head attends with is a query of that size.
`q_rank` Q: the queries come through a latent of their own, cq = rms_norm(Wdq h) * dq.norm, q = Wuq cq (tensors "dq",
"dq.norm", "uq" in place of "q").  `gate`: the concatenated heads leave multiplied element by element with
sigmoid(Wg h), ahead of Wo (tensor "g" [heads * value_dim, hidden]).
`shares_kv`: the mixer has no Wdkv and reads another layer's pages with its own q, Wuk, Wuv.
Pairs of the rotation are (i, i + dr/2), or neighbours (2i, 2i + 1) with `rope_interleaved`: then the rows of Wq and Wdkv
that make the rotated elements are put in the other order when the weights are bound, once and on both sides of the
score, which keeps every score as it is and needs no second rotation kernel."""
from __future__ import annotations

from typing import Dict, Mapping, Optional

import torch

from ..kernels import ops
from .base import MIXERS, Mixer, PagedLatents, Runtime, as_normed, to_device
from .rope import rotary_table
from .spec import ParamSpec


@MIXERS.register("absorbed_latent_attention")
class AbsorbedLatentAttention(Mixer):
    graph_safe = True

    def __init__(self, hidden_size: int, num_heads: int, head_dim: int, rot_dim: int, value_dim: int, kv_rank: int,
                 scale: float, rope_theta: float = 10000.0, rope_scaling: Optional[Mapping] = None,
                 rope_interleaved: bool = False, norm_eps: float = 1e-6, shares_kv: bool = False,
                 names: Optional[Mapping[str, str]] = None, q_rank: int = 0, gate: bool = False):
        self.D, self.H = int(hidden_size), int(num_heads)
        self.dn, self.dr, self.dv, self.R = int(head_dim), int(rot_dim), int(value_dim), int(kv_rank)
        if self.dr % 2 or self.dr < 0 or min(self.dn, self.dv, self.R, self.H) < 1:
            raise ValueError(f"latent attention: rot_dim {rot_dim} must be even, every other size positive")
        self.dq, self.row = self.dn + self.dr, self.R + self.dr
        self.scale, self.theta, self.eps = float(scale), float(rope_theta), float(norm_eps)
        self.rope_scaling = dict(rope_scaling) if rope_scaling else None
        self.interleaved, self.shares_kv = bool(rope_interleaved), bool(shares_kv)
        self.Q, self.gate = int(q_rank), bool(gate)
        if self.Q < 0:
            raise ValueError(f"latent attention: q_rank {q_rank} must not be negative")
        self.names = {"q": "q", "dq": "dq", "dq_norm": "dq.norm", "uq": "uq", "dkv": "dkv", "dkv_norm": "dkv.norm",
                      "uk": "uk", "uv": "uv", "gate": "g", "o": "o", **dict(names or {})}
        # columns of the first product's rows: the queries or their latent, the latent of keys and values with the
        # rotated key part, the gate's logits, each from a multiple of 8 on (rows of zeros in the matrix between them)
        def up8(n: int) -> int:
            return -(-n // 8) * 8

        self.c_off = up8(self.Q) if self.Q else self.H * self.dq
        self.g_off = up8(self.c_off + (0 if self.shares_kv else self.row))
        self.width = self.g_off + self.H * self.dv if self.gate else self.c_off + (0 if self.shares_kv else self.row)
        self.stride = up8(self.width)

    def param_specs(self) -> Dict[str, ParamSpec]:
        n = self.names
        if self.Q:
            out = {n["dq"]: ParamSpec((self.Q, self.D)), n["dq_norm"]: ParamSpec((self.Q,), store="float32"),
                   n["uq"]: ParamSpec((self.H * self.dq, self.Q))}
        else:
            out = {n["q"]: ParamSpec((self.H * self.dq, self.D))}
        if not self.shares_kv:
            out[n["dkv"]] = ParamSpec((self.row, self.D))
            out[n["dkv_norm"]] = ParamSpec((self.R,), store="float32")
        out[n["uk"]] = ParamSpec((self.H * self.dn, self.R))
        out[n["uv"]] = ParamSpec((self.H * self.dv, self.R))
        if self.gate:
            out[n["gate"]] = ParamSpec((self.H * self.dv, self.D))
        out[n["o"]] = ParamSpec((self.D, self.H * self.dv))
        return out

    def cache_need(self):
        return PagedLatents(self.R, self.dr)

    def _halves(self, w: torch.Tensor) -> torch.Tensor:
        """[.., dr, D] rows of rotated elements, neighbouring pairs -> pairs (i, i + dr/2)."""
        return torch.cat([w[..., 0::2, :], w[..., 1::2, :]], dim=-2) if self.interleaved else w

    def bind(self, tensors: Mapping[str, torch.Tensor], rt: Runtime) -> None:
        self.rt = rt
        n, H, dn, dr, dv, R = self.names, self.H, self.dn, self.dr, self.dv, self.R
        q = tensors[n["uq"] if self.Q else n["q"]]
        q = q.reshape(H, self.dq, q.shape[-1])
        q = torch.cat([q[:, :dn], self._halves(q[:, dn:])], dim=1).reshape(H * self.dq, q.shape[-1])
        self.norm_w = None
        mats = [(0, tensors[n["dq"]] if self.Q else q)]          # (first column of its outputs, matrix)
        if not self.shares_kv:
            down = tensors[n["dkv"]]
            mats += [(self.c_off, down[:R]), (self.c_off + R, self._halves(down[R:]))]
            self.norm_w = to_device(tensors[n["dkv_norm"]], rt, torch.float32)
        if self.gate:
            mats.append((self.g_off, tensors[n["gate"]]))
        dt = mats[0][1].dtype if all(m.dtype == mats[0][1].dtype for _, m in mats) else torch.float32
        # one [width, D] matrix: a single product gives q (or its latent), the latent, the shared key part and the gate
        w_in = torch.zeros((self.width, self.D), dtype=dt, device=rt.device)
        for at, m in mats:
            w_in[at:at + m.shape[0]] = to_device(m, rt, dt)
        self.w_in = ops.prepare_matrix(w_in, rt.dtype)
        self.w_uq = self.q_norm_w = None
        if self.Q:
            self.w_uq = ops.prepare_matrix(to_device(q, rt), rt.dtype)
            self.q_norm_w = to_device(tensors[n["dq_norm"]], rt, torch.float32)
        uk = to_device(tensors[n["uk"]], rt).view(H, dn, R)
        self.w_uk = ops.prepare_heads(uk.transpose(1, 2).contiguous(), rt.dtype, self.dq, self.row)     # a head: [R, dn]
        self.w_uv = ops.prepare_heads(to_device(tensors[n["uv"]], rt).view(H, dv, R), rt.dtype, R, dv)
        self.w_o = ops.prepare_matrix(to_device(tensors[n["o"]], rt), rt.dtype)
        self.cos_sin = rotary_table(dr, self.theta, rt, self.rope_scaling) if dr else None

    def forward(self, h, step, cache) -> torch.Tensor:
        """float32 [rows, hidden]: the mixer's output."""
        pages = cache.get("mixer") if isinstance(cache, dict) else cache
        if pages.writes == self.shares_kv:
            raise ValueError("latent attention: a layer with latents of its own needs pages of its own, a layer "
                             "without them another entry's")
        h = as_normed(h).tensor()
        T, dev, dt = h.shape[0], h.device, self.rt.dtype
        H, R = self.H, self.R
        proj = torch.empty((T, self.stride), dtype=dt, device=dev)[:, :self.width]
        ops.linear(h, self.w_in, proj)
        queries = proj
        if self.Q:
            cq = torch.empty((T, self.Q), dtype=dt, device=dev)
            ops.rmsnorm_rows(proj[:, :self.Q], self.q_norm_w, self.eps, cq)
            queries = torch.empty((T, H * self.dq), dtype=dt, device=dev)
            ops.linear(cq, self.w_uq, queries)
        q = torch.empty((T, H * self.row), dtype=dt, device=dev)          # a head: [R, dr]
        ops.latent_rows(queries, H, self.dn, self.dr, None if self.shares_kv else self.c_off, R, self.norm_w, self.eps,
                        self.cos_sin, step, pages.block_table, pages.kv, pages.page_tokens, q, kv=proj)
        ops.heads_linear(queries, self.dq, self.w_uk, q, self.row)
        o = torch.empty((T, H * R), dtype=dt, device=dev)
        ops.latent_attention(q, o, H, R, self.dr, pages.kv, pages.page_tokens, pages.block_table, step, self.scale)
        attn = torch.empty((T, H * self.dv), dtype=dt, device=dev)
        ops.heads_linear(o, R, self.w_uv, attn, self.dv,
                         gate=proj[:, self.g_off:self.g_off + H * self.dv] if self.gate else None)
        out = torch.empty((T, self.D), dtype=torch.float32, device=dev)
        ops.linear(attn, self.w_o, out)
        return out
