"""Typed Sisepel configuration read from config.json.

A Sisepel model is a list of layers with a norm before and one after each sub-layer.  The
mixer (`parallel`) is two side by side, each output normed by itself: windowed grouped-query
attention (queries and keys rotated and then normed per head without weights, capped scores, a
sink) on the left, retention (linear attention with a fixed decay per head) on the right.  The
optional feed-forward is a dense GELU-gated unit or routed experts beside a shared one; with
`token_side` every layer also takes in a part of its own of each token's row of a second
table.  Every size and every constant that may differ between two models is read here; what a
config.json leaves out (a window, a cap, a frequency scaling, a shared expert, a factor on the
logits) takes its mechanism along.
"""

from __future__ import annotations

from dataclasses import dataclass, field
from typing import Any

from tokensprint_amd.config.model_config import ConfigError
from tokensprint_amd.config.palelix_config import _need, _number, _pos_int

ARCHITECTURE = "Sisepel"
MIXER_TYPES = ("parallel",)


@dataclass(frozen=True)
class FrequencyScaling:
    """Stretches frequencies whose wavelength is long beside the `original` context."""

    factor: float
    low: float                   # wavelengths above original / low are stretched in full,
    high: float                  # those below original / high not at all
    original: float


@dataclass(frozen=True)
class Rotation:
    base: float
    dims: int                    # leading dimensions of a head that are rotated
    scaling: FrequencyScaling | None = None


@dataclass(frozen=True)
class AttentionSizes:
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    scale: float
    rot: Rotation | None
    window: int | None           # a query sees itself and the window - 1 tokens before it
    softcap: float | None


@dataclass(frozen=True)
class RetentionSizes:
    heads: int
    dim: int
    vdim: int
    decay: tuple[float, ...]     # one per head
    rot: Rotation


@dataclass(frozen=True)
class ParallelSizes:
    left: AttentionSizes
    right: RetentionSizes


@dataclass(frozen=True)
class DenseFF:
    ff: int


@dataclass(frozen=True)
class RoutedFF:
    ff: int                      # inner size of one expert
    experts: int
    top: int
    shared_ff: int | None        # inner size of the expert every token uses, None: there is none


@dataclass(frozen=True)
class SisepelLayer:
    type: str
    mixer: ParallelSizes
    mlp: DenseFF | RoutedFF | None


@dataclass(frozen=True)
class SisepelConfig:
    width: int
    vocab_size: int
    eps: float
    logit_scale: float
    side_dim: int | None         # columns of the side table per layer, None: there is none
    layers: tuple[SisepelLayer, ...]
    eos_token_id: int | None = None
    max_position: int = 1 << 17
    architecture: str = ARCHITECTURE
    raw: dict = field(default_factory=dict, compare=False, repr=False)

    @classmethod
    def from_dict(cls, raw: dict[str, Any]) -> "SisepelConfig":
        width = _pos_int(raw, "width", "config")
        vocab = _pos_int(raw, "vocab", "config")
        eps = _number(_need(raw, "norm", "config"), "eps", "norm", positive=True)
        side = raw.get("token_side")
        logit_scale = _number(raw, "logit_scale", "config") \
            if raw.get("logit_scale") is not None else 1.0
        entries = _need(raw, "layers", "config")
        if not isinstance(entries, list) or not entries:
            raise ConfigError("config.json: 'layers' must be a non-empty list")
        layers = []
        for i, entry in enumerate(entries):
            where = f"layers[{i}]"
            kind = _need(entry, "type", where)
            if kind not in MIXER_TYPES:
                raise ConfigError(f"config.json: {where}.type={kind!r}; Sisepel has "
                                  f"{', '.join(MIXER_TYPES)}")
            m, at = _need(entry, "mixer", where), where + ".mixer"
            mixer = ParallelSizes(left=cls._attention(_need(m, "left", at), at + ".left"),
                                  right=cls._retention(_need(m, "right", at), at + ".right"))
            layers.append(SisepelLayer(kind, mixer, cls._mlp(entry.get("mlp"), where + ".mlp")))
        return cls(width=width, vocab_size=vocab, eps=eps, logit_scale=logit_scale,
                   side_dim=_pos_int(side, "dim", "token_side") if side is not None else None,
                   layers=tuple(layers), eos_token_id=raw.get("eos_token_id"),
                   max_position=int(raw.get("max_position", 1 << 17)), raw=dict(raw))

    @staticmethod
    def _rotation(rot, where, dim) -> Rotation:
        r = Rotation(base=_number(rot, "base", where, positive=True),
                     dims=_pos_int(rot, "dims", where))
        if r.dims % 2 or r.dims > dim:
            raise ConfigError(f"config.json: {where}.dims={r.dims} must be even and at most "
                              f"dim={dim}")
        s, at = rot.get("scaling"), where + ".scaling"
        if s is None:
            return r
        scaling = FrequencyScaling(*(_number(s, key, at, positive=True)
                                     for key in ("factor", "low", "high", "original")))
        if scaling.high < scaling.low:
            raise ConfigError(f"config.json: {at}.high={scaling.high} is below low={scaling.low}")
        return Rotation(r.base, r.dims, scaling)

    @classmethod
    def _attention(cls, m, where) -> AttentionSizes:
        heads, kv = _pos_int(m, "heads", where), _pos_int(m, "kv_heads", where)
        if heads % kv:
            raise ConfigError(f"config.json: {where}: heads={heads} is not a multiple of "
                              f"kv_heads={kv}")
        dim, mask, rot = _pos_int(m, "dim", where), m.get("mask"), m.get("rot")
        return AttentionSizes(
            heads=heads, kv_heads=kv, dim=dim, vdim=_pos_int(m, "vdim", where),
            scale=_number(m, "scale", where, positive=True),
            rot=cls._rotation(rot, where + ".rot", dim) if rot is not None else None,
            window=_pos_int(mask, "size", where + ".mask") if mask is not None else None,
            softcap=_number(m, "softcap", where, positive=True)
            if m.get("softcap") is not None else None)

    @classmethod
    def _retention(cls, m, where) -> RetentionSizes:
        heads, dim = _pos_int(m, "heads", where), _pos_int(m, "dim", where)
        decay = _need(m, "decay", where)
        if not isinstance(decay, list) or len(decay) != heads:
            raise ConfigError(f"config.json: {where}.decay must list one number per head")
        rot = cls._rotation(_need(m, "rot", where), where + ".rot", dim)
        if rot.scaling is not None:
            raise ConfigError(f"config.json: {where}.rot.scaling: retention's rotation has none")
        return RetentionSizes(heads=heads, dim=dim, vdim=_pos_int(m, "vdim", where),
                              decay=tuple(float(d) for d in decay), rot=rot)

    @staticmethod
    def _mlp(mlp, where) -> DenseFF | RoutedFF | None:
        if mlp is None:
            return None
        kind = _need(mlp, "kind", where)
        if kind == "dense":
            return DenseFF(ff=_pos_int(mlp, "ff", where))
        if kind != "moe":
            raise ConfigError(f"config.json: {where}.kind={kind!r}; Sisepel has dense and moe")
        router, shared = _need(mlp, "router", where), mlp.get("shared")
        f = RoutedFF(ff=_pos_int(_need(mlp, "expert", where), "ff", where + ".expert"),
                     experts=_pos_int(router, "experts", where + ".router"),
                     top=_pos_int(router, "top", where + ".router"),
                     shared_ff=_pos_int(shared, "ff", where + ".shared")
                     if shared is not None else None)
        if f.top > f.experts:
            raise ConfigError(f"config.json: {where}.router: {f.experts} experts cannot give "
                              f"{f.top}")
        return f
