"""The Natenex decoder described with parts (config.json "architecture": "Natenex").

Token rows times a scale.  A layer norms the output of each of its sublayers only, x += norm1(mixer(x)),
x += norm2(ff(x)), with RMS norms.  Its mixer is one of three: two mixers side by side, an attention over a sliding
window with kept first tokens (norm per head, partial rotation with the llama3 frequency rule) beside a recurrent block
with a real-gated linear recurrence, added with constant factors; an attention over cached latents whose queries come
through a latent too and whose heads leave through a sigmoid gate; or a gated delta rule.  Its feed-forward is two
matrices around a squared relu, or none.  A layer may use an earlier or later layer's tensors with a cache of its own.
Final norm, head tied to the table (without its scale).  Tensor names: `embed`, `l<i>.norm1|norm2`,
`l<i>.mix.left.q|k|v|o` (+ `.norm`), `l<i>.mix.right.y|x|conv|ra|ri` (+ `.b`) `|lam|o`,
`l<i>.mix.dq|dq.norm|uq|dkv|dkv.norm|uk|uv|g|o`, `l<i>.mix.q|k|v` (+ `.conv`) `|a|b|A_log|dt_bias|norm|g|o`,
`l<i>.mlp.up|down`, `final.norm`."""
from __future__ import annotations

from typing import Optional

from ..config.natenex import NatenexConfig, NatenexLatent, NatenexParallel, NatenexScaling, sizes_from_tensors
from ..parts.spec import BlockSpec, ModelSpec, PartSpec, PlanEntry
from . import ARCHITECTURES, Architecture


def _norm(cfg: NatenexConfig, name: str) -> PartSpec:
    return PartSpec("rmsnorm", dict(size=cfg.width, eps=cfg.eps, name=name))


def _rope_scaling(s: Optional[NatenexScaling]) -> Optional[dict]:
    if s is None:
        return None
    return dict(rope_type="llama3", factor=s.factor, low_freq_factor=s.low, high_freq_factor=s.high,
                original_max_position_embeddings=s.original)


def natenex_spec(cfg: NatenexConfig) -> ModelSpec:
    D = cfg.width
    blocks, block_of = [], {}
    for i, layer in enumerate(cfg.layers):
        if layer.weights_of is not None:
            continue
        m = layer.mixer
        if isinstance(m, NatenexParallel):
            l, r = m.left, m.right
            mixer = PartSpec("parallel", dict(members=[
                dict(name="left", kind="sink_attention", scale=m.left_scale, params=dict(
                    hidden_size=D, num_heads=l.heads, num_kv_heads=l.kv_heads, key_dim=l.dim, value_dim=l.vdim,
                    scale=l.scale, rotary_dim=l.rot_dims, rope_theta=l.rot_base, rope_scaling=_rope_scaling(l.scaling),
                    mask="window" if l.window else "causal", mask_size=l.window, keep_first=l.keep_first,
                    learned_sink=False, qk_norm=True, norm_eps=cfg.eps)),
                dict(name="right", kind="gated_recurrence", scale=m.right_scale, params=dict(
                    hidden_size=D, width=r.width, blocks=r.blocks, conv_taps=r.conv)),
            ]), "mix.")
        elif isinstance(m, NatenexLatent):
            mixer = PartSpec("absorbed_latent_attention", dict(
                hidden_size=D, num_heads=m.heads, head_dim=m.dim, rot_dim=m.rot_dim, value_dim=m.vdim,
                q_rank=m.q_rank, kv_rank=m.kv_rank, scale=m.scale, rope_theta=m.rot_base,
                rope_scaling=_rope_scaling(m.scaling), norm_eps=cfg.eps, gate=True), "mix.")
        else:
            mixer = PartSpec("gated_delta_rule", dict(
                hidden_size=D, num_heads=m.heads, num_kv_heads=m.kv_heads, key_dim=m.dim, value_dim=m.vdim,
                conv_taps=m.conv, norm_eps=cfg.eps), "mix.")
        parts = {"mixer": mixer, "mixer_norm": _norm(cfg, "norm1"), "scale": PartSpec("scaled", dict(mult=1.0))}
        if layer.ff:
            parts["ffn"] = PartSpec("mlp", dict(hidden_size=D, intermediate_size=layer.ff, activation="relu2"), "mlp.")
            parts["ffn_norm"] = _norm(cfg, "norm2")
        block_of[i] = len(blocks)
        blocks.append(BlockSpec(arrangement="sublayer_norm", weight_prefix=f"l{i}.", parts=parts))
    plan = [PlanEntry(block_of[i if layer.weights_of is None else layer.weights_of]) for i, layer in enumerate(cfg.layers)]
    return ModelSpec(
        hidden_size=D,
        vocab_size=cfg.vocab,
        max_positions=cfg.max_positions,
        embedding=PartSpec("token_table", dict(vocab_size=cfg.vocab, hidden_size=D, name="embed",
                                               scale=cfg.embedding_scale)),
        blocks=blocks,
        plan=plan,
        final_norm=_norm(cfg, "final.norm"),
        head=PartSpec("linear", dict(vocab_size=cfg.vocab, hidden_size=D, tied=True)),
    )


ARCHITECTURES.register("Natenex", Architecture("natenex", NatenexConfig.from_dict, natenex_spec, sizes_from_tensors))
