"""Sisepel as a `ModelSpec`: a norm before and one after each sub-layer, a mixer that is windowed
attention and retention side by side (each normed by itself), a GELU-gated feed-forward or
routed experts, and a side input of every token into every layer.  The factor on the logits is
part of the final norm's weight.

Tensor names: 'embed', 'side.embed', 'final.norm', 'head', and per layer i 'l<i>.norm1',
'l<i>.norm1b', 'l<i>.norm2', 'l<i>.norm2b', 'l<i>.mix.*' (the two mixers' under '.left.' and
'.right.'), 'l<i>.mlp.*', 'l<i>.side.*'.
"""

from __future__ import annotations

from tokensprint_amd.config.registry import register_architecture
from tokensprint_amd.config.sisepel_config import (ARCHITECTURE, AttentionSizes, DenseFF,
                                                   RetentionSizes, SisepelConfig)
from tokensprint_amd.models.spec import LayerSpec, ModelSpec, PartSpec, Run
from tokensprint_amd.parts.attention import SoftmaxAttention


def _attention_spec(m: AttentionSizes, pre: str, cfg: SisepelConfig, positions: dict) -> PartSpec:
    name = None
    if m.rot is not None:
        head, s = SoftmaxAttention.padded_head(m.dim, m.vdim), m.rot.scaling
        # one table per rotation and head size, shared by the layers that use it
        name = f"rot_{m.rot!r}_{head}"
        positions.setdefault(name, PartSpec("rope_partial", {
            "dims": m.rot.dims, "base": m.rot.base, "head_dim": head, "pairs": "neighbours",
            "max_position": cfg.max_position,
            "scaling": None if s is None else {
                "kind": "wavelength", "factor": s.factor, "low": s.low, "high": s.high,
                "original": s.original}}))
    # (norms without weights and rotations commute: a rotation keeps a head's length)
    return PartSpec("softmax_attention", {
        "prefix": pre, "heads": m.heads, "kv_heads": m.kv_heads, "dim": m.dim, "vdim": m.vdim,
        "scale": m.scale, "position": name, "window": m.window, "softcap": m.softcap,
        "sink": True, "qk_norm": "plain", "qk_norm_eps": cfg.eps, "wide_output": True})


def _retention_spec(m: RetentionSizes, pre: str, cfg: SisepelConfig, positions: dict) -> PartSpec:
    name = f"turn_{m.rot.base!r}_{m.rot.dims}"
    positions.setdefault(name, PartSpec("rope_interleaved", {
        "dims": m.rot.dims, "base": m.rot.base, "pairs": "halves",
        "max_position": cfg.max_position}))
    return PartSpec("retention", {
        "prefix": pre, "heads": m.heads, "dim": m.dim, "vdim": m.vdim, "decay": m.decay,
        "eps": cfg.eps, "position": name, "state": "retention"})


def _ff_spec(mlp, pre: str) -> PartSpec:
    if isinstance(mlp, DenseFF):
        return PartSpec("swiglu", {"prefix": pre, "inner_dim": mlp.ff, "act": "gelu_tanh",
                                   "names": ("gate", "up", "down"), "wide_output": True})
    return PartSpec("routed_experts", {
        "prefix": pre, "inner_dim": mlp.ff, "experts": mlp.experts, "top": mlp.top,
        "gated": "silu", "router_bias": True, "shared_inner": mlp.shared_ff})


def sisepel_spec(cfg: SisepelConfig) -> ModelSpec:
    positions: dict[str, PartSpec] = {}
    layers = []

    def norm(name, **more):
        return PartSpec("rmsnorm", {"dim": cfg.width, "eps": cfg.eps, "weight": name, **more})

    for i, layer in enumerate(cfg.layers):
        pre, mix = f"l{i}.", f"l{i}.mix."
        parts = dict(
            mixer_norm=norm(pre + "norm1"),
            mixer=PartSpec("side_by_side", {
                "left": _attention_spec(layer.mixer.left, mix + "left.", cfg, positions),
                "right": _retention_spec(layer.mixer.right, mix + "right.", cfg, positions),
                "left_scale": 0.5, "right_scale": 0.5,
                "norms": (mix + "left.out", mix + "right.out"), "norm_eps": cfg.eps}),
            mixer_post_norm=norm(pre + "norm1b"))
        if layer.mlp is not None:
            parts.update(ffn_norm=norm(pre + "norm2"),
                         feed_forward=_ff_spec(layer.mlp, pre + "mlp."),
                         ffn_post_norm=norm(pre + "norm2b"))
        if cfg.side_dim is not None:
            parts.update(
                side=PartSpec("gated_token_table", {
                    "prefix": pre + "side.", "table": "side.embed", "vocab_size": cfg.vocab_size,
                    "dim": cfg.side_dim, "parts": len(cfg.layers), "index": i}),
                side_post_norm=norm(pre + "side.norm"))
        layers.append(LayerSpec("sandwich_norm", **parts))
    return ModelSpec(
        architecture=ARCHITECTURE, width=cfg.width, vocab_size=cfg.vocab_size,
        embedding=PartSpec("embedding", {"weight": "embed", "vocab_size": cfg.vocab_size}),
        positions=positions, layers=tuple(layers),
        order=tuple(Run(i) for i in range(len(layers))),
        final_norm=norm("final.norm", scale=cfg.logit_scale),
        head=PartSpec("head", {"weight": "head", "vocab_size": cfg.vocab_size}),
        max_position=cfg.max_position, eos_token_id=cfg.eos_token_id,
    )


register_architecture(ARCHITECTURE, parse_config=SisepelConfig.from_dict, build_spec=sisepel_spec)
