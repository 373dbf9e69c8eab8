"""A plain, slow reading of the Natenex decoder in numpy (float64), one function per mechanism.  It shares no code with
the engine: tests compare the engine's parts and whole steps with it.

Notation: T tokens of one sequence at positions 0 .. T-1, D the model's width, H query heads over G key/value heads,
d / e the sizes of a key and of a value, R the size of the latent of keys and values, C channels of the gated linear
recurrence.  `rnd` (where a function takes it) rounds a stored activation: the identity for the exact model, a rounding
to bfloat16 for the estimate of what 16-bit activations cost.

Keys and values of the latent attention are always written out here, head by head (the engine never does that), and the
delta rule and the gated recurrence walk token by token with the state as a matrix (the engine takes chunks).  Two forms
of everything that carries something from token to token stand side by side: over a whole sequence (`forward`), and in
portions with what is carried kept in a dict (`Stepper`)."""
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
def rms_norm(x: np.ndarray, w, eps: float) -> np.ndarray:
    """x over its root mean square along the last axis (eps inside the root), times w."""
    return x / np.sqrt(np.mean(x * x, axis=-1, keepdims=True) + eps) * w


def unit(x: np.ndarray, eps: float = 1e-6) -> np.ndarray:
    """A vector of length 1 along the last axis: a sum under the root, not a mean."""
    return x / np.sqrt(np.sum(x * x, axis=-1, keepdims=True) + eps)


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


def last_inputs(u: np.ndarray, n: int, before: Optional[np.ndarray] = None) -> Optional[np.ndarray]:
    """The n - 1 rows that a convolution of n taps needs of the past of the next row."""
    if n <= 1:
        return None
    pad = np.zeros((n - 1, u.shape[1])) if before is None else before
    return np.concatenate([pad, u], axis=0)[-(n - 1):]


def frequencies(rot: dict) -> np.ndarray:
    """The frequency of every pair of a rotation {"base", "dims", "scaling": {"factor", "low", "high", "original"}}."""
    r = int(rot["dims"])
    f = np.array([float(rot["base"]) ** (-2.0 * i / r) for i in range(r // 2)])
    sc = rot.get("scaling")
    if not sc:
        return f
    out = []
    for x in f:
        wave = 2.0 * math.pi / x
        if wave < sc["original"] / sc["high"]:
            out.append(x)
        elif wave > sc["original"] / sc["low"]:
            out.append(x / sc["factor"])
        else:
            s = (sc["original"] / wave - sc["low"]) / (sc["high"] - sc["low"])
            out.append((1.0 - s) * x / sc["factor"] + s * x)
    return np.array(out)


def rotate_halves(v: np.ndarray, positions, rot: dict) -> np.ndarray:
    """v [T, ..., n]: elements i and i + dims/2 of the first `dims` are a pair, turned by position * frequency_i."""
    r = int(rot["dims"])
    if r == 0:
        return v
    ang = np.asarray(positions, dtype=np.float64)[:, None] * frequencies(rot)[None, :]
    shape = (ang.shape[0],) + (1,) * (v.ndim - 2) + (r // 2,)
    c, s = np.cos(ang).reshape(shape), np.sin(ang).reshape(shape)
    out = np.array(v, dtype=np.float64)
    a, b = v[..., :r // 2], v[..., r // 2:r]
    out[..., :r // 2] = a * c - b * s
    out[..., r // 2:r] = b * c + a * s
    return out


def visible(i: int, j: int, mask: Optional[dict]) -> bool:
    """Whether the row at position i sees the key at position j: all earlier ones, or with a mask {"size",
    "keep_first"} the last `size` (the row's own among them) and the first `keep_first` of the sequence."""
    if j > i:
        return False
    return mask is None or i - j < mask["size"] or j < mask["keep_first"]


def softmax_attention(q, k, v, scale: float, q_pos0: int = 0, mask: Optional[dict] = None) -> np.ndarray:
    """q [Tq, H, d] stand at positions q_pos0 .. of the keys k [Tk, G, d] with values v [Tk, G, e]."""
    Tq, H = q.shape[0], q.shape[1]
    per = H // k.shape[1]
    see = np.array([[visible(q_pos0 + i, j, mask) for j in range(k.shape[0])] for i in range(Tq)])
    out = np.zeros((Tq, H, v.shape[2]))
    for h in range(H):
        s = np.where(see, (q[:, h] @ k[:, h // per].T) * scale, -np.inf)
        p = np.exp(s - s.max(axis=1, keepdims=True))
        out[:, h] = (p / p.sum(axis=1, keepdims=True)) @ v[:, h // per]
    return out


def gated_recurrence(u, r, i, lam, S0: Optional[np.ndarray] = None):
    """u, r, i [T, C], lam [C]: a = exp(-8 r softplus(lam)); S <- a S + sqrt(1 - a^2) i u.  Returns (S of every row, the
    last S); the first row is no special case."""
    S = np.zeros(u.shape[1]) if S0 is None else np.array(S0, dtype=np.float64)
    out = np.zeros_like(u)
    for t in range(u.shape[0]):
        log_a = -8.0 * r[t] * softplus(lam)
        S = np.exp(log_a) * S + np.sqrt(-np.expm1(2.0 * log_a)) * i[t] * u[t]
        out[t] = S
    return out, S


def delta_rule(q, k, v, beta, g, S0: Optional[np.ndarray] = None):
    """q, k [T, H, d], v [T, H, e], beta, g [T, H], S [H, d, e]: S <- g S, then what S gives for k is moved towards v by
    beta, then o is what the new S gives for q.  Returns (o [T, H, e], last S)."""
    T, H, d = q.shape
    S = np.zeros((H, d, v.shape[2])) if S0 is None else np.array(S0, dtype=np.float64)
    o = np.zeros((T, H, v.shape[2]))
    for t in range(T):
        for h in range(H):
            S[h] = g[t, h] * S[h]
            w = beta[t, h] * (v[t, h] - S[h].T @ k[t, h])
            S[h] = S[h] + np.outer(k[t, h], w)
            o[t, h] = S[h].T @ q[t, h]
    return o, S


# ---------------------------------------------------------------------------------------------- mixers, feed-forward
def window_keys(h, W, p, m, eps, positions, rnd: Callable = exact):
    """(keys [T, G, d] normed and rotated, values [T, G, e]) of the rows, as the cache holds them."""
    T, G = h.shape[0], m["kv_heads"]
    k = rms_norm(rnd(h @ W[p + "k"].T).reshape(T, G, m["dim"]), W[p + "k.norm"], eps)
    return rnd(rotate_halves(k, positions, m["rot"])), rnd(h @ W[p + "v"].T).reshape(T, G, m["vdim"])


def window_mixer(h, W, p, m, eps, positions, k, v, rnd: Callable = exact):
    T, H = h.shape[0], m["heads"]
    q = rms_norm(rnd(h @ W[p + "q"].T).reshape(T, H, m["dim"]), W[p + "q.norm"], eps)
    q = rnd(rotate_halves(q, positions, m["rot"]))
    o = softmax_attention(q, k, v, m["scale"], int(positions[0]), m.get("mask"))
    return rnd(o).reshape(T, H * m["vdim"]) @ W[p + "o"].T


def griffin_mixer(h, W, p, m, state: dict, rnd: Callable = exact):
    """The recurrent block.  `state`: {"conv": the last inputs, "S"}; returns (output, new state)."""
    T, B = h.shape[0], m["blocks"]
    y = rnd(gelu_tanh(h @ W[p + "y"].T + W[p + "y.b"]))
    x = rnd(h @ W[p + "x"].T + W[p + "x.b"])
    w = W[p + "conv"]
    u = rnd(short_conv(x, w, state.get("conv")) + W[p + "conv.b"])
    parts = u.reshape(T, B, -1)

    def gate(name):
        z = np.stack([parts[:, b] @ W[p + name][b].T for b in range(B)], axis=1) + W[p + name + ".b"]
        return sigmoid(z).reshape(T, -1)

    s, S = gated_recurrence(u, gate("ra"), gate("ri"), W[p + "lam"], state.get("S"))
    return rnd(s * y) @ W[p + "o"].T, {"conv": last_inputs(x, w.shape[1], state.get("conv")), "S": S}


def latent_rows(h, W, p, m, eps, positions, rnd: Callable = exact):
    """(latents [T, R], the rotated key part of all heads) of the rows, as the cache holds them."""
    R = m["kv_rank"]
    a = rnd(h @ W[p + "dkv"].T)
    return rnd(rms_norm(a[:, :R], W[p + "dkv.norm"], eps)), rnd(rotate_halves(a[:, R:], positions, m["rot"]))


def latent_mixer(h, W, p, m, eps, positions, c, kr, rnd: Callable = exact):
    """Attention of the rows at `positions` over all latents c [Tk, R] and rotated key parts kr so far."""
    T, Tk, H, dn, dr = h.shape[0], c.shape[0], m["heads"], m["dim"], m["rot_dim"]
    cq = rnd(rms_norm(rnd(h @ W[p + "dq"].T), W[p + "dq.norm"], eps))
    q = rnd(cq @ W[p + "uq"].T).reshape(T, H, dn + dr)
    q = np.concatenate([q[..., :dn], rnd(rotate_halves(q[..., dn:], positions, m["rot"]))], axis=-1)
    k = np.concatenate([rnd(c @ W[p + "uk"].T).reshape(Tk, H, dn), np.broadcast_to(kr[:, None], (Tk, H, dr))], axis=-1)
    v = rnd(c @ W[p + "uv"].T).reshape(Tk, H, m["vdim"])
    o = rnd(softmax_attention(q, k, v, m["scale"], int(positions[0]))).reshape(T, -1)
    return rnd(o * sigmoid(rnd(h @ W[p + "g"].T))) @ W[p + "o"].T


def delta_mixer(h, W, p, m, eps, state: dict, rnd: Callable = exact):
    """`state`: {"q", "k", "v": the convolutions' last inputs, "S"}; returns (output, new state)."""
    T, H, G, d, e = h.shape[0], m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    new, act = {}, {}
    for n in "qkv":
        u, w = rnd(h @ W[p + n].T), W[p + n + ".conv"]
        act[n] = rnd(silu(rnd(short_conv(u, w, state.get(n)))))
        new[n] = last_inputs(u, w.shape[1], state.get(n))
    q = np.repeat(unit(act["q"].reshape(T, G, d)) * d ** -0.5, H // G, axis=1)
    k = np.repeat(unit(act["k"].reshape(T, G, d)), H // G, axis=1)
    beta = sigmoid(h @ W[p + "b"].T)
    g = np.exp(-np.exp(W[p + "A_log"]) * softplus(h @ W[p + "a"].T + W[p + "dt_bias"]))
    o, new["S"] = delta_rule(q, k, act["v"].reshape(T, H, e), beta, g, state.get("S"))
    o = rms_norm(o, W[p + "norm"], eps).reshape(T, H * e)
    return rnd(o * silu(rnd(h @ W[p + "g"].T))) @ W[p + "o"].T, new


def dense_ff(h, W, p, rnd: Callable = exact):
    return rnd(relu2(h @ W[p + "up"].T)) @ W[p + "down"].T


# ---------------------------------------------------------------------------------------------- the model
class Stepper:
    """The model fed in portions of any size: keys, values, latents, last inputs and states are kept here between calls,
    as a cache would keep them; every layer of the list has its own, also one that uses another's weights."""

    def __init__(self, cfg: dict, W: Dict[str, np.ndarray], rnd: Callable = exact):
        self.cfg, self.W, self.n, self.rnd = cfg, W, 0, rnd
        self.kept: Dict[int, dict] = {i: {} for i in range(len(cfg["layers"]))}

    def feed(self, tokens, taps: Optional[list] = None) -> np.ndarray:
        cfg, W, rnd = self.cfg, self.W, self.rnd
        eps = cfg["norm"]["eps"]
        pos = np.arange(self.n, self.n + len(tokens))
        x = W["embed"][np.asarray(tokens)] * cfg["embedding"]["scale"]

        def grow(st, **new):
            for key, rows in new.items():
                st[key] = rows if key not in st else np.concatenate([st[key], rows])

        for i, layer in enumerate(cfg["layers"]):
            j = i
            while cfg["layers"][j].get("weights_of") is not None:
                j = cfg["layers"][j]["weights_of"]
            p, m, st = f"l{j}.mix.", layer["mixer"], self.kept[i]
            h = rnd(x)
            if layer["type"] == "parallel":
                l, lp = m["left"], p + "left."
                k, v = window_keys(h, W, lp, l, eps, pos, rnd)
                grow(st, k=k, v=v)
                left = window_mixer(h, W, lp, l, eps, pos, st["k"], st["v"], rnd)
                right, st["right"] = griffin_mixer(h, W, p + "right.", m["right"], st.get("right", {}), rnd)
                y = m["left_scale"] * left + m["right_scale"] * right
            elif layer["type"] == "latent_attention":
                c, kr = latent_rows(h, W, p, m, eps, pos, rnd)
                grow(st, c=c, kr=kr)
                y = latent_mixer(h, W, p, m, eps, pos, st["c"], st["kr"], rnd)
            elif layer["type"] == "delta":
                y, self.kept[i] = delta_mixer(h, W, p, m, eps, st, rnd)
            else:
                raise ValueError(layer["type"])
            x = x + rms_norm(y, W[f"l{j}.norm1"], eps)
            if layer.get("mlp") is not None:
                x = x + rms_norm(dense_ff(rnd(x), W, f"l{j}.mlp.", rnd), W[f"l{j}.norm2"], eps)
            if taps is not None:
                taps.append(x.copy())
        self.n += len(tokens)
        return rnd(rms_norm(x, W["final.norm"], eps)) @ W["embed"].T


def forward(cfg: dict, W: Dict[str, np.ndarray], tokens, rnd: Callable = exact, taps: Optional[list] = None):
    """Logits [T, vocab] of one whole sequence; `taps` (a list) receives the residual stream after every layer."""
    return Stepper(cfg, W, rnd).feed(tokens, taps)


# ---------------------------------------------------------------------------------------------- tensors and folders
def tensor_shapes(cfg: dict) -> Dict[str, tuple]:
    D, V = cfg["width"], cfg["vocab"]
    out = {"embed": (V, D), "final.norm": (D,)}
    for i, layer in enumerate(cfg["layers"]):
        if layer.get("weights_of") is not None:
            continue
        p, m = f"l{i}.mix.", layer["mixer"]
        out[f"l{i}.norm1"] = (D,)
        if layer["type"] == "parallel":
            l, r, a, b = m["left"], m["right"], p + "left.", p + "right."
            H, G, d, e, C, B = l["heads"], l["kv_heads"], l["dim"], l["vdim"], r["width"], r["blocks"]
            out[a + "q"], out[a + "k"], out[a + "v"], out[a + "o"] = (H * d, D), (G * d, D), (G * e, D), (D, H * e)
            out[a + "q.norm"] = out[a + "k.norm"] = (d,)
            out[b + "y"] = out[b + "x"] = (C, D)
            out[b + "y.b"] = out[b + "x.b"] = out[b + "conv.b"] = out[b + "lam"] = (C,)
            out[b + "conv"], out[b + "o"] = (C, r["conv"]), (D, C)
            out[b + "ra"] = out[b + "ri"] = (B, C // B, C // B)
            out[b + "ra.b"] = out[b + "ri.b"] = (B, C // B)
        elif layer["type"] == "latent_attention":
            H, dn, dr, e, R, Q = (m[x] for x in ("heads", "dim", "rot_dim", "vdim", "kv_rank", "q_rank"))
            out[p + "dq"], out[p + "dq.norm"], out[p + "uq"] = (Q, D), (Q,), (H * (dn + dr), Q)
            out[p + "dkv"], out[p + "dkv.norm"] = (R + dr, D), (R,)
            out[p + "uk"], out[p + "uv"], out[p + "g"], out[p + "o"] = (H * dn, R), (H * e, R), (H * e, D), (D, H * e)
        else:
            H, G, d, e, n = (m[x] for x in ("heads", "kv_heads", "dim", "vdim", "conv"))
            out[p + "q"] = out[p + "k"] = (G * d, D)
            out[p + "v"] = out[p + "g"] = (H * e, D)
            out[p + "q.conv"] = out[p + "k.conv"] = (G * d, n)
            out[p + "v.conv"] = (H * e, n)
            out[p + "a"] = out[p + "b"] = (H, D)
            out[p + "A_log"] = out[p + "dt_bias"] = (H,)
            out[p + "norm"], out[p + "o"] = (e,), (D, H * e)
        if layer.get("mlp") is not None:
            out[f"l{i}.norm2"] = (D,)
            out[f"l{i}.mlp.up"], out[f"l{i}.mlp.down"] = (layer["mlp"]["ff"], D), (D, layer["mlp"]["ff"])
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
