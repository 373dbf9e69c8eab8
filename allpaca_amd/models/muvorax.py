"""The Muvorax decoder described with parts (config.json "architecture": "Muvorax").

Token rows as the table holds them.  A layer norms the input and the output of each of its sublayers,
x += norm1b(mixer(norm1(x))), x += norm2b(ff(norm2(x))), and a norm is tanh(alpha x) * w + b element by element.  Its
mixer is one of three: an attention whose keys and values are a low-rank latent and one rotated key part for all heads
(both cached as they are; neighbouring elements are the rotation's pairs, with a frequency rule for longer contexts;
optionally the latents of an earlier layer), a selective scan, or a linear attention with a fixed decay a head (silu on
q, k and v, a root mean square over the row, a sigmoid gate).  Its feed-forward is two matrices around a gelu, routed
experts without a gate (squared relu; sigmoid scores with a correction of the choice, groups of experts, weights
divided by their sum and scaled), or none.  Final norm, head tied to the table.  Tensor names: `embed`,
`l<i>.norm1|norm1b|norm2|norm2b` (+ `.alpha`, `.b`), `l<i>.mix.q|dkv|dkv.norm|uk|uv|o`,
`l<i>.mix.in|conv|conv.b|x|dt|dt.b|A_log|D|o`, `l<i>.mix.q|k|v|g|norm|o`, `l<i>.mlp.up|down`,
`l<i>.mlp.router|correction`, `l<i>.mlp.e<j>.up|down`, `final.norm`."""
from __future__ import annotations

from ..config.muvorax import MuvoraxConfig, MuvoraxDense, MuvoraxLatent, MuvoraxScan, sizes_from_tensors
from ..parts.spec import BlockSpec, ModelSpec, PartSpec, PlanEntry
from . import ARCHITECTURES, Architecture


def _norm(cfg: MuvoraxConfig, name: str) -> PartSpec:
    return PartSpec("dynamic_tanh", dict(size=cfg.width, name=name))


def muvorax_spec(cfg: MuvoraxConfig) -> ModelSpec:
    D = cfg.width
    blocks, plan = [], []
    for i, layer in enumerate(cfg.layers):
        m = layer.mixer
        cache_of = None
        if isinstance(m, MuvoraxLatent):
            scaling = None
            if m.scaling is not None:
                scaling = dict(rope_type="yarn", factor=m.scaling.factor, original=m.scaling.original,
                               fast=m.scaling.fast, slow=m.scaling.slow)
            mixer = PartSpec("absorbed_latent_attention", dict(
                hidden_size=D, num_heads=m.heads, head_dim=m.dim, rot_dim=m.rot_dim, value_dim=m.vdim,
                kv_rank=m.kv_rank, scale=m.scale, rope_theta=m.rot_base, rope_scaling=scaling, rope_interleaved=True,
                norm_eps=cfg.eps, shares_kv=m.kv_from is not None), "mix.")
            cache_of = m.kv_from
        elif isinstance(m, MuvoraxScan):
            mixer = PartSpec("selective_scan", dict(hidden_size=D, inner=m.inner, state=m.state, dt_rank=m.dt_rank,
                                                    conv_taps=m.conv), "mix.")
        else:
            mixer = PartSpec("decay_linear_attention", dict(
                hidden_size=D, num_heads=m.heads, key_dim=m.dim, value_dim=m.vdim, decay=m.decay, norm_eps=cfg.eps,
                activation="silu", gate=True), "mix.")
        parts = {"mixer_norm": _norm(cfg, "norm1"), "mixer": mixer, "mixer_post": _norm(cfg, "norm1b")}
        f = layer.mlp
        if f is not None:
            parts["ffn_norm"], parts["ffn_post"] = _norm(cfg, "norm2"), _norm(cfg, "norm2b")
            if isinstance(f, MuvoraxDense):
                parts["ffn"] = PartSpec("mlp", dict(hidden_size=D, intermediate_size=f.ff, activation="gelu_tanh"), "mlp.")
            else:
                parts["ffn"] = PartSpec("routed_experts", dict(
                    hidden_size=D, intermediate_size=f.ff, experts=f.experts, top=f.top, identity=0, correction=True,
                    renormalize=True, activation="relu2", score="sigmoid", groups=f.groups, keep_groups=f.keep,
                    weight_scale=f.scale), "mlp.")
        blocks.append(BlockSpec(arrangement="sandwich_norm", weight_prefix=f"l{i}.", parts=parts))
        plan.append(PlanEntry(i, cache_of=cache_of))
    return ModelSpec(
        hidden_size=D,
        vocab_size=cfg.vocab,
        max_positions=cfg.max_positions,
        embedding=PartSpec("token_table", dict(vocab_size=cfg.vocab, hidden_size=D, name="embed")),
        blocks=blocks,
        plan=plan,
        final_norm=_norm(cfg, "final.norm"),
        head=PartSpec("linear", dict(vocab_size=cfg.vocab, hidden_size=D, tied=True)),
    )


ARCHITECTURES.register("Muvorax", Architecture("muvorax", MuvoraxConfig.from_dict, muvorax_spec, sizes_from_tensors))
