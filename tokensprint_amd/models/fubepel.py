"""Fubepel as a `ModelSpec`: post-norm layers (the sub-layers read the stream as it is, their
outputs are normed before they are added) with three kinds of mixer, a gated feed-forward with
clamped inputs, and a side input of every token into every layer.  A latent-attention layer
may read the latents of an earlier one: its run names that layer's run as the owner of its
cache.

Tensor names: 'embed', 'side.embed', 'final.norm', 'head', and per layer i 'l<i>.norm1',
'l<i>.norm2', 'l<i>.mix.*', 'l<i>.mlp.*', 'l<i>.side.*'.
"""

from __future__ import annotations

from tokensprint_amd.config.fubepel_config import (ARCHITECTURE, DeltaSizes, FubepelConfig,
                                                   LatentSizes)
from tokensprint_amd.config.registry import register_architecture
from tokensprint_amd.models.spec import LayerSpec, ModelSpec, PartSpec, Run


def _mixer_spec(m, pre: str, cfg: FubepelConfig, positions: dict) -> PartSpec:
    if isinstance(m, DeltaSizes):
        return PartSpec("gated_delta", {
            "prefix": pre, "heads": m.heads, "kv_heads": m.kv_heads, "dim": m.dim,
            "vdim": m.vdim, "conv": m.conv, "eps": cfg.eps})
    if isinstance(m, LatentSizes):
        # one rotation per (base, dims), shared by the layers that use it
        name = f"rot_{m.rot_base!r}_{m.rot_dims}"
        positions.setdefault(name, PartSpec("rope_interleaved", {
            "dims": m.rot_dims, "base": m.rot_base, "pairs": "halves"}))
        return PartSpec("latent_attention", {
            "prefix": pre, "heads": m.heads, "dim": m.dim, "rot_dim": m.rot_dim, "vdim": m.vdim,
            "kv_rank": m.kv_rank, "scale": m.scale, "eps": cfg.eps, "position": name,
            "sink": True, "own_kv": m.kv_from is None})
    return PartSpec("softmax_attention", {
        "prefix": pre, "heads": m.heads, "kv_heads": m.kv_heads, "dim": m.dim, "vdim": m.vdim,
        "scale": m.scale, "position": None, "window": m.window, "keep_first": m.keep_first,
        "qk_norm": "plain", "qk_norm_eps": cfg.eps, "wide_output": True})


def fubepel_spec(cfg: FubepelConfig) -> ModelSpec:
    positions: dict[str, PartSpec] = {}
    layers, order = [], []

    def norm(name):
        return PartSpec("rmsnorm", {"dim": cfg.width, "eps": cfg.eps, "weight": name})

    for i, layer in enumerate(cfg.layers):
        pre = f"l{i}."
        parts = dict(mixer=_mixer_spec(layer.mixer, pre + "mix.", cfg, positions),
                     mixer_post_norm=norm(pre + "norm1"))
        if layer.mlp is not None:
            parts.update(
                feed_forward=PartSpec("swiglu", {
                    "prefix": pre + "mlp.", "inner_dim": layer.mlp.ff, "limit": layer.mlp.limit,
                    "names": ("gate", "up", "down"), "wide_output": True}),
                ffn_post_norm=norm(pre + "norm2"))
        if cfg.side_dim is not None:
            parts.update(
                side=PartSpec("gated_token_table", {
                    "prefix": pre + "side.", "table": "side.embed", "vocab_size": cfg.vocab_size,
                    "dim": cfg.side_dim, "parts": len(cfg.layers), "index": i}),
                side_post_norm=norm(pre + "side.norm"))
        layers.append(LayerSpec("post_norm", **parts))
        # layers run once each, in order: a layer's index is its run's
        order.append(Run(i, cache_of=getattr(layer.mixer, "kv_from", None)))
    return ModelSpec(
        architecture=ARCHITECTURE, width=cfg.width, vocab_size=cfg.vocab_size,
        embedding=PartSpec("embedding", {"weight": "embed", "vocab_size": cfg.vocab_size,
                                         "scale": cfg.embed_scale}),
        positions=positions, layers=tuple(layers), order=tuple(order),
        final_norm=norm("final.norm"),
        head=PartSpec("head", {"weight": "head", "vocab_size": cfg.vocab_size}),
        max_position=cfg.max_position, eos_token_id=cfg.eos_token_id,
    )


register_architecture(ARCHITECTURE, parse_config=FubepelConfig.from_dict, build_spec=fubepel_spec)
