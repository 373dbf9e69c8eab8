"""A plain, slow reading of the Muvorax decoder in numpy (float64), one function per mechanism.  It shares no code with
the engine: tests compare the engine's parts and whole steps with it.

Notation: T tokens of one sequence at positions 0 .. T-1, D the model's width, H heads, dn / dr the plain and the
rotated elements of a query or key head, dv a value head's, R the size of the latent of keys and values, C channels and
N states of the selective scan, E experts of which a token uses K.  `rnd` (where a function takes it) rounds a stored
activation: the identity for the exact model, a rounding to bfloat16 for the estimate of what 16-bit activations cost.

Keys and values are always written out here, head by head, from the latents (the engine never does that).  Two forms of
everything that carries something from token to token stand side by side: over a whole sequence (`forward`), and in
portions with what is carried kept in a dict (`Stepper`); the tests hold the one against the other."""
from __future__ import annotations

import json
import math
import os
import struct
from typing import Callable, Dict, List, Optional

import numpy as np


def exact(x):
    return x


def to_bf16(x):
    """Round to the nearest bfloat16 (ties to even), returned as float64."""
    a = np.ascontiguousarray(np.asarray(x, dtype=np.float32))
    u = a.view(np.uint32).astype(np.uint64)
    u = ((u + 0x7FFF + ((u >> 16) & 1)) >> 16) << 16
    return u.astype(np.uint32).view(np.float32).astype(np.float64).reshape(a.shape)


# ---------------------------------------------------------------------------------------------- single mechanisms
def squash(x: np.ndarray, alpha, w: np.ndarray, b: np.ndarray) -> np.ndarray:
    """The norm of this design: element by element, no mean and no variance."""
    return np.tanh(float(alpha) * x) * w + b


def unit_rms(x: np.ndarray, eps: float) -> np.ndarray:
    """x over its root mean square along the last axis, eps inside the root."""
    return x / np.sqrt(np.mean(x * x, axis=-1, keepdims=True) + eps)


def sigmoid(z):
    return 0.5 * (1.0 + np.tanh(0.5 * np.asarray(z)))


def silu(z):
    return z * sigmoid(z)


def softplus(z):
    return np.logaddexp(0.0, z)


def gelu_tanh(z):
    return 0.5 * z * (1.0 + np.tanh(math.sqrt(2.0 / math.pi) * (z + 0.044715 * z ** 3)))


def relu2(z):
    return np.maximum(z, 0.0) ** 2


def short_conv(u: np.ndarray, w: np.ndarray, before: Optional[np.ndarray] = None) -> np.ndarray:
    """u [T, C], w [C, n]: y[t] = sum_j w[:, j] * u[t - (n - 1) + j], with `before` [n - 1, C] (zeros if None) standing
    in front of the sequence.  The last column of w is the current token's."""
    T, C = u.shape
    n = w.shape[1]
    pad = np.zeros((n - 1, C)) if before is None else np.asarray(before, dtype=np.float64)
    full = np.concatenate([pad, u], axis=0)
    y = np.zeros((T, C))
    for j in range(n):
        y += w[:, j][None, :] * full[j:j + T]
    return y


def frequencies(rot: dict) -> tuple:
    """(frequency of every pair, what cosines and sines are multiplied with) of a rotation {"base", "dims", "scaling"}."""
    r, base = int(rot["dims"]), float(rot["base"])
    i = np.arange(r // 2, dtype=np.float64)
    f = np.power(base, -2.0 * i / r)
    sc = rot.get("scaling")
    if not sc:
        return f, 1.0
    factor, orig = float(sc["factor"]), float(sc["original"])

    def dim_at(turns):
        return r * math.log(orig / (2.0 * math.pi * turns)) / (2.0 * math.log(base))

    lo = max(math.floor(dim_at(float(sc["fast"]))), 0)
    hi = min(math.ceil(dim_at(float(sc["slow"]))), r - 1)
    ramp = np.clip((i - lo) / max(hi - lo, 0.001), 0.0, 1.0)
    return f / factor * ramp + f * (1.0 - ramp), 0.1 * math.log(factor) + 1.0


def rotate_pairs(v: np.ndarray, positions, rot: dict) -> np.ndarray:
    """v [T, ..., r]: elements 2i and 2i+1 are a pair, turned by the angle position * frequency_i."""
    r = int(rot["dims"])
    if r == 0:
        return v
    f, mag = frequencies(rot)
    ang = np.asarray(positions, dtype=np.float64)[:, None] * f[None, :]
    shape = (ang.shape[0],) + (1,) * (v.ndim - 2) + (r // 2,)
    c, s = (np.cos(ang) * mag).reshape(shape), (np.sin(ang) * mag).reshape(shape)
    out = np.empty_like(v)
    a, b = v[..., 0::2], v[..., 1::2]
    out[..., 0::2] = a * c - b * s
    out[..., 1::2] = b * c + a * s
    return out


def softmax_attention(q: np.ndarray, k: np.ndarray, v: np.ndarray, scale: float, q_pos0: int = 0) -> np.ndarray:
    """q [Tq, H, d] stand at positions q_pos0 .. of the keys k [Tk, H, d] with values v [Tk, H, dv]; causal."""
    Tq, H = q.shape[0], q.shape[1]
    out = np.zeros((Tq, H, v.shape[2]))
    p = q_pos0 + np.arange(Tq)
    hidden = np.arange(k.shape[0])[None, :] > p[:, None]
    for h in range(H):
        s = (q[:, h] @ k[:, h].T) * scale
        s[hidden] = -np.inf
        e = np.exp(s - s.max(axis=1, keepdims=True))
        out[:, h] = (e / e.sum(axis=1, keepdims=True)) @ v[:, h]
    return out


def decayed_sums(q: np.ndarray, k: np.ndarray, v: np.ndarray, decay, S0: Optional[np.ndarray] = None):
    """q, k [T, H, dk], v [T, H, dv]: S_t = decay_h S_(t-1) + k_t v_t^T, o_t = S_t^T q_t.  Returns (o, last S)."""
    T, H, dk = q.shape
    dv = v.shape[2]
    S = np.zeros((H, dk, dv)) if S0 is None else np.array(S0, dtype=np.float64)
    d = np.asarray(decay, dtype=np.float64)[:, None, None]
    o = np.zeros((T, H, dv))
    for t in range(T):
        S = d * S + k[t][:, :, None] * v[t][:, None, :]
        o[t] = np.einsum("hkv,hk->hv", S, q[t])
    return o, S


def selective_scan(x: np.ndarray, dt: np.ndarray, A: np.ndarray, B: np.ndarray, C: np.ndarray, Dw: np.ndarray,
                   S0: Optional[np.ndarray] = None):
    """x, dt [T, C]; A [C, N]; B, C [T, N]: S[c, n] <- exp(dt_c A[c, n]) S[c, n] + dt_c x_c B_n;
    y_c = sum_n S[c, n] C_n + D_c x_c.  Returns (y, last S)."""
    T, ch = x.shape
    S = np.zeros(A.shape) if S0 is None else np.array(S0, dtype=np.float64)
    y = np.zeros((T, ch))
    for t in range(T):
        S = np.exp(dt[t][:, None] * A) * S + (dt[t] * x[t])[:, None] * B[t][None, :]
        y[t] = S @ C[t] + Dw * x[t]
    return y, S


def route(z: np.ndarray, correction: np.ndarray, top: int, scale: float = 1.0, groups: int = 1, keep: int = 1):
    """One token's choice.  s = sigmoid(z), c = s + correction.  The outputs form `groups` equal runs of neighbours; a
    run's score is the sum of its two largest c, and only outputs of the `keep` best runs can be chosen.  The `top`
    largest c among them (lower index first on a tie).  Weights: s of the chosen over their sum, times `scale`."""
    s = sigmoid(z)
    c = s + correction
    n = len(z) // groups
    if keep < groups:
        scores = [np.sort(c[g * n:(g + 1) * n])[-2:].sum() for g in range(groups)]
        best = np.argsort(-np.asarray(scores), kind="stable")[:keep]
        allowed = np.zeros(len(z), dtype=bool)
        for g in best:
            allowed[g * n:(g + 1) * n] = True
        c = np.where(allowed, c, -np.inf)
    ids = np.argsort(-c, kind="stable")[:top]
    return ids, s[ids] / (s[ids].sum() + 1e-20) * scale


# ---------------------------------------------------------------------------------------------- mixers, feed-forwards
def latent_rows(h, W, p, m, eps, positions, rnd: Callable = exact):
    """(latents [T, R], the rotated key part of all heads [T, dr]) of the rows, as the cache holds them."""
    R = m["kv_rank"]
    a = h @ W[p + "dkv"].T
    return rnd(unit_rms(a[:, :R], eps) * W[p + "dkv.norm"]), rnd(rotate_pairs(a[:, R:], positions, m["rot"]))


def latent_mixer(h, W, p, m, positions, c, kr, rnd: Callable = exact):
    """Attention of the rows at `positions` over all latents c [Tk, R] and rotated key parts kr [Tk, dr] so far."""
    T, Tk = h.shape[0], c.shape[0]
    H, dn, dr, dv = m["heads"], m["dim"], m["rot_dim"], m["vdim"]
    q = rnd(h @ W[p + "q"].T).reshape(T, H, dn + dr)
    q = np.concatenate([q[..., :dn], rnd(rotate_pairs(q[..., dn:], positions, m["rot"]))], axis=-1)
    k = np.concatenate([rnd(c @ W[p + "uk"].T).reshape(Tk, H, dn),
                        np.broadcast_to(kr[:, None, :], (Tk, H, dr))], axis=-1)
    v = rnd(c @ W[p + "uv"].T).reshape(Tk, H, dv)
    o = softmax_attention(q, k, v, m["scale"], q_pos0=int(positions[0]))
    return rnd(o).reshape(T, H * dv) @ W[p + "o"].T


def scan_mixer(h, W, p, m, state=None, rnd: Callable = exact):
    """The selective scan.  `state`: {"conv": the last inputs, "S": the scan's state}; returns (output, new state)."""
    C, N, R = m["inner"], m["state"], m["dt_rank"]
    state = state or {}
    xz = rnd(h @ W[p + "in"].T)
    x_in, z = xz[:, :C], xz[:, C:]
    x = rnd(silu(short_conv(x_in, W[p + "conv"], state.get("conv")) + W[p + "conv.b"]))
    low = rnd(x @ W[p + "x"][:R].T)
    bc = x @ W[p + "x"][R:].T
    dt = softplus(low @ W[p + "dt"].T + W[p + "dt.b"])
    y, S = selective_scan(x, dt, -np.exp(W[p + "A_log"]), bc[:, :N], bc[:, N:], W[p + "D"], state.get("S"))
    taps = W[p + "conv"].shape[1]
    held = np.concatenate([state.get("conv", np.zeros((taps - 1, C))), x_in])[-(taps - 1):] if taps > 1 else None
    return rnd(y * silu(z)) @ W[p + "o"].T, {"conv": held, "S": S}


def lightning_mixer(h, W, p, m, eps, S0=None, rnd: Callable = exact):
    T = h.shape[0]
    H, dk, dv = m["heads"], m["dim"], m["vdim"]
    q = rnd(silu(rnd(h @ W[p + "q"].T))).reshape(T, H, dk)
    k = rnd(silu(rnd(h @ W[p + "k"].T))).reshape(T, H, dk)
    v = rnd(silu(rnd(h @ W[p + "v"].T))).reshape(T, H, dv)
    o, S = decayed_sums(q, k, v, m["decay"], S0)
    g = rnd(h @ W[p + "g"].T)
    return rnd(unit_rms(o.reshape(T, H * dv), eps) * W[p + "norm"] * sigmoid(g)) @ W[p + "o"].T, S


def dense_ff(h, W, p, rnd: Callable = exact):
    return rnd(gelu_tanh(h @ W[p + "up"].T)) @ W[p + "down"].T


def expert_ff(h, W, p, f, rnd: Callable = exact):
    r = f["router"]
    g = r.get("groups") or {}
    z = h @ W[p + "router"].T
    out = np.zeros_like(h)
    for t in range(h.shape[0]):
        ids, w = route(z[t], W[p + "correction"], r["top"], r.get("scale", 1.0), g.get("count", 1), g.get("keep", 1))
        for e, we in zip(ids, w):
            out[t] += we * (rnd(relu2(W[f"{p}e{e}.up"] @ h[t])) @ W[f"{p}e{e}.down"].T)
    return out


# ---------------------------------------------------------------------------------------------- the model
class Stepper:
    """The model fed in portions of any size: latents, rotated key parts, last inputs and states are kept here between
    calls, as a cache would keep them."""

    def __init__(self, cfg: dict, W: Dict[str, np.ndarray], rnd: Callable = exact):
        self.cfg, self.W, self.n, self.rnd = cfg, W, 0, rnd
        self.kept: Dict[int, dict] = {i: {} for i in range(len(cfg["layers"]))}

    def norm(self, x, name):
        W = self.W
        return squash(x, W[name + ".alpha"], W[name], W[name + ".b"])

    def feed(self, tokens, taps: Optional[list] = None) -> np.ndarray:
        cfg, W, rnd = self.cfg, self.W, self.rnd
        eps = cfg["norm"]["eps"]
        pos = np.arange(self.n, self.n + len(tokens))
        x = W["embed"][np.asarray(tokens)]
        for i, layer in enumerate(cfg["layers"]):
            p, m, st = f"l{i}.mix.", layer["mixer"], self.kept[i]
            h = rnd(self.norm(x, f"l{i}.norm1"))
            if layer["type"] == "latent_attention":
                src = m.get("kv_from")
                if src is None:
                    c, kr = latent_rows(h, W, p, m, eps, pos, rnd)
                    st["c"] = c if st.get("c") is None else np.concatenate([st["c"], c])
                    st["kr"] = kr if st.get("kr") is None else np.concatenate([st["kr"], kr])
                owner = self.kept[i if src is None else src]
                y = latent_mixer(h, W, p, m, pos, owner["c"], owner["kr"], rnd)
            elif layer["type"] == "mamba1":
                y, self.kept[i] = scan_mixer(h, W, p, m, st, rnd)
            elif layer["type"] == "lightning":
                y, st["S"] = lightning_mixer(h, W, p, m, eps, st.get("S"), rnd)
            else:
                raise ValueError(layer["type"])
            x = x + self.norm(y, f"l{i}.norm1b")
            f = layer.get("mlp")
            if f is not None:
                h = rnd(self.norm(x, f"l{i}.norm2"))
                y = dense_ff(h, W, f"l{i}.mlp.", rnd) if f["kind"] == "dense" else expert_ff(h, W, f"l{i}.mlp.", f, rnd)
                x = x + self.norm(y, f"l{i}.norm2b")
            if taps is not None:
                taps.append(x.copy())
        self.n += len(tokens)
        return rnd(self.norm(x, "final.norm")) @ W["embed"].T


def forward(cfg: dict, W: Dict[str, np.ndarray], tokens, rnd: Callable = exact, taps: Optional[list] = None):
    """Logits [T, vocab] of one whole sequence; `taps` (a list) receives the residual stream after every layer."""
    return Stepper(cfg, W, rnd).feed(tokens, taps)


# ---------------------------------------------------------------------------------------------- tensors and folders
def tensor_shapes(cfg: dict) -> Dict[str, tuple]:
    D, V = cfg["width"], cfg["vocab"]
    out = {"embed": (V, D)}

    def norm(name):
        out[name], out[name + ".b"], out[name + ".alpha"] = (D,), (D,), ()

    norm("final.norm")
    for i, layer in enumerate(cfg["layers"]):
        p, m = f"l{i}.mix.", layer["mixer"]
        norm(f"l{i}.norm1"), norm(f"l{i}.norm1b")
        if layer["type"] == "latent_attention":
            H, dn, dr, dv, R = m["heads"], m["dim"], m["rot_dim"], m["vdim"], m["kv_rank"]
            out[p + "q"], out[p + "uk"], out[p + "uv"], out[p + "o"] = (H * (dn + dr), D), (H * dn, R), (H * dv, R), (D, H * dv)
            if m.get("kv_from") is None:
                out[p + "dkv"], out[p + "dkv.norm"] = (R + dr, D), (R,)
        elif layer["type"] == "mamba1":
            C, N, R = m["inner"], m["state"], m["dt_rank"]
            out[p + "in"], out[p + "conv"], out[p + "conv.b"] = (2 * C, D), (C, m["conv"]), (C,)
            out[p + "x"], out[p + "dt"], out[p + "dt.b"] = (R + 2 * N, C), (C, R), (C,)
            out[p + "A_log"], out[p + "D"], out[p + "o"] = (C, N), (C,), (D, C)
        else:
            H, dk, dv = m["heads"], m["dim"], m["vdim"]
            out[p + "q"] = out[p + "k"] = (H * dk, D)
            out[p + "v"] = out[p + "g"] = (H * dv, D)
            out[p + "o"], out[p + "norm"] = (D, H * dv), (H * dv,)
        f = layer.get("mlp")
        if f is not None:
            norm(f"l{i}.norm2"), norm(f"l{i}.norm2b")
            if f["kind"] == "dense":
                out[f"l{i}.mlp.up"], out[f"l{i}.mlp.down"] = (f["ff"], D), (D, f["ff"])
            else:
                E = f["router"]["experts"]
                out[f"l{i}.mlp.router"], out[f"l{i}.mlp.correction"] = (E, D), (E,)
                for e in range(E):
                    out[f"l{i}.mlp.e{e}.up"], out[f"l{i}.mlp.e{e}.down"] = (f["expert"]["ff"], D), (D, f["expert"]["ff"])
    return out


def read_safetensors(path: str) -> Dict[str, np.ndarray]:
    """A reader of its own: 8 bytes of length, that many of JSON, then the data (F32 and BF16)."""
    with open(path, "rb") as f:
        (n,) = struct.unpack("<Q", f.read(8))
        meta = json.loads(f.read(n))
        data = f.read()
    out = {}
    for name, e in meta.items():
        if name == "__metadata__":
            continue
        a, b = e["data_offsets"]
        if e["dtype"] == "F32":
            v = np.frombuffer(data[a:b], dtype="<f4").astype(np.float64)
        elif e["dtype"] == "BF16":
            v = (np.frombuffer(data[a:b], dtype="<u2").astype(np.uint32) << 16).view(np.float32).astype(np.float64)
        else:
            raise ValueError(f"{name}: element type {e['dtype']}")
        out[name] = v.reshape(e["shape"])
    return out


def read_model_folder(path: str):
    with open(os.path.join(path, "config.json")) as f:
        cfg = json.load(f)
    return cfg, read_safetensors(os.path.join(path, "model.safetensors"))


def greedy(cfg: dict, W: Dict[str, np.ndarray], prompt, n: int) -> List[int]:
    st, out = Stepper(cfg, W), []
    logits = st.feed(list(prompt))
    for i in range(n):
        out.append(int(np.argmax(logits[-1])))
        if i + 1 < n:
            logits = st.feed(out[-1:])
    return out
