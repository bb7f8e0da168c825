"""Typed Fubepel configuration read from config.json.

A Fubepel model is a list of layers whose sub-layers read the residual stream as it is and
whose outputs are normed before they are added.  Mixers: `delta` (gated delta rule, one decay
per head and token), `attention` (grouped-query attention without positions, queries and keys
normed per head without weights, a window beside which the sequence's first tokens stay
visible) and `latent_attention` (a low-rank latent and a rotated key part shared by the heads,
a sink in the softmax; a layer may read the latents an earlier layer keeps: `kv_from`).  The
optional feed-forward is a gated unit with clamped inputs; with `token_side` every layer also
takes in a part of its own of each token's row of a second table.  Every size and every
constant that may differ between two models is read here.
"""

from __future__ import annotations

from dataclasses import dataclass, field
from typing import Any

from tokensprint_amd.config.model_config import ConfigError
from tokensprint_amd.config.palelix_config import _need, _number, _pos_int

ARCHITECTURE = "Fubepel"
MIXER_TYPES = ("delta", "attention", "latent_attention")


@dataclass(frozen=True)
class DeltaSizes:
    heads: int                   # value heads
    kv_heads: int                # query/key heads
    dim: int
    vdim: int
    conv: int                    # taps of the short convolutions


@dataclass(frozen=True)
class AttentionSizes:
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    scale: float
    window: int | None           # a query sees itself and the window - 1 tokens before it
    keep_first: int              # and the sequence's first so many tokens


@dataclass(frozen=True)
class LatentSizes:
    heads: int
    dim: int                     # unrotated query/key dimensions per head
    rot_dim: int                 # rotated query/key dimensions per head (the key's are shared)
    vdim: int
    kv_rank: int
    scale: float
    rot_base: float
    rot_dims: int                # leading dimensions of the rotated part that are rotated
    kv_from: int | None          # the layer whose latents this one reads, None: its own


@dataclass(frozen=True)
class DenseFF:
    ff: int
    limit: float


@dataclass(frozen=True)
class FubepelLayer:
    type: str
    mixer: DeltaSizes | AttentionSizes | LatentSizes
    mlp: DenseFF | None


@dataclass(frozen=True)
class FubepelConfig:
    width: int
    vocab_size: int
    eps: float
    embed_scale: float
    side_dim: int | None         # columns of the side table per layer, None: there is none
    layers: tuple[FubepelLayer, ...]
    eos_token_id: int | None = None
    max_position: int = 1 << 20
    architecture: str = ARCHITECTURE
    raw: dict = field(default_factory=dict, compare=False, repr=False)

    @classmethod
    def from_dict(cls, raw: dict[str, Any]) -> "FubepelConfig":
        width = _pos_int(raw, "width", "config")
        vocab = _pos_int(raw, "vocab", "config")
        eps = _number(_need(raw, "norm", "config"), "eps", "norm", positive=True)
        emb, side = raw.get("embedding"), raw.get("token_side")
        embed_scale = _number(emb, "scale", "embedding") \
            if emb is not None and "scale" in emb else 1.0
        entries = _need(raw, "layers", "config")
        if not isinstance(entries, list) or not entries:
            raise ConfigError("config.json: 'layers' must be a non-empty list")
        read = {"delta": cls._delta, "attention": cls._attention, "latent_attention": cls._latent}
        layers = []
        for i, entry in enumerate(entries):
            where = f"layers[{i}]"
            kind = _need(entry, "type", where)
            if kind not in MIXER_TYPES:
                raise ConfigError(f"config.json: {where}.type={kind!r}; Fubepel has "
                                  f"{', '.join(MIXER_TYPES)}")
            mixer = read[kind](_need(entry, "mixer", where), where + ".mixer")
            layers.append(FubepelLayer(kind, mixer, cls._mlp(entry.get("mlp"), where + ".mlp")))
        for i, layer in enumerate(layers):
            source = getattr(layer.mixer, "kv_from", None)
            if source is None:
                continue
            where = f"layers[{i}].mixer.kv_from={source!r}"
            if not isinstance(source, int) or isinstance(source, bool) or not 0 <= source < i:
                raise ConfigError(f"config.json: {where} names no earlier layer")
            src, m = layers[source].mixer, layer.mixer
            if not isinstance(src, LatentSizes) or src.kv_from is not None:
                raise ConfigError(f"config.json: {where}: that layer keeps no latents of its own")
            if (src.kv_rank, src.rot_dim, src.rot_base, src.rot_dims) != \
                    (m.kv_rank, m.rot_dim, m.rot_base, m.rot_dims):
                raise ConfigError(f"config.json: {where}: the two layers' latents differ in rank "
                                  "or rotation")
        return cls(width=width, vocab_size=vocab, eps=eps, embed_scale=embed_scale,
                   side_dim=_pos_int(side, "dim", "token_side") if side is not None else None,
                   layers=tuple(layers), eos_token_id=raw.get("eos_token_id"),
                   # rotation angles are computed in float32, which is exact for positions up to
                   # here, and there is no table to run out of
                   max_position=int(raw.get("max_position", 1 << 20)), raw=dict(raw))

    @staticmethod
    def _grouped(m, where):
        heads, kv = _pos_int(m, "heads", where), _pos_int(m, "kv_heads", where)
        if heads % kv:
            raise ConfigError(f"config.json: {where}: heads={heads} is not a multiple of "
                              f"kv_heads={kv}")
        return dict(heads=heads, kv_heads=kv, dim=_pos_int(m, "dim", where),
                    vdim=_pos_int(m, "vdim", where))

    @classmethod
    def _delta(cls, m, where) -> DeltaSizes:
        return DeltaSizes(**cls._grouped(m, where), conv=_pos_int(m, "conv", where))

    @classmethod
    def _attention(cls, m, where) -> AttentionSizes:
        mask, keep = m.get("mask"), 0
        if mask is not None:
            keep = mask.get("keep_first") or 0
            if not isinstance(keep, int) or isinstance(keep, bool) or keep < 0:
                raise ConfigError(f"config.json: {where}.mask.keep_first={keep!r} is no count")
        return AttentionSizes(
            **cls._grouped(m, where), scale=_number(m, "scale", where, positive=True),
            window=_pos_int(mask, "size", where + ".mask") if mask is not None else None,
            keep_first=keep)

    @staticmethod
    def _latent(m, where) -> LatentSizes:
        rot = _need(m, "rot", where)
        s = LatentSizes(
            heads=_pos_int(m, "heads", where), dim=_pos_int(m, "dim", where),
            rot_dim=_pos_int(m, "rot_dim", where), vdim=_pos_int(m, "vdim", where),
            kv_rank=_pos_int(m, "kv_rank", where), scale=_number(m, "scale", where, positive=True),
            rot_base=_number(rot, "base", where + ".rot", positive=True),
            rot_dims=_pos_int(rot, "dims", where + ".rot"), kv_from=m.get("kv_from"))
        if s.rot_dims % 2 or s.rot_dims > s.rot_dim:
            raise ConfigError(f"config.json: {where}.rot.dims={s.rot_dims} must be even and at "
                              f"most rot_dim={s.rot_dim}")
        return s

    @staticmethod
    def _mlp(mlp, where) -> DenseFF | None:
        if mlp is None:
            return None
        kind = _need(mlp, "kind", where)
        if kind != "dense":
            raise ConfigError(f"config.json: {where}.kind={kind!r}; Fubepel has dense")
        return DenseFF(ff=_pos_int(mlp, "ff", where),
                       limit=_number(mlp, "limit", where, positive=True))
