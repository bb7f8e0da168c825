"""Plain Sisepel forward: one function per mechanism, whole sequences, no cache, CPU torch.

Everything runs over a whole sequence [T, ...] in one precision (float64 by default):
attention as full T x T tables of scores with the mask written out, the recurrence a token
at a time, rotations position by position and pair by pair, the router token by token, so
that a mistake in the engine's cache, window, state or batch handling cannot be mirrored
here.  Nothing imports the engine package.

Notation: T tokens, D model width, eps the model's norm epsilon; a linear weight W is
[out, in] and applied as x W^T; H query heads, G key/value heads.
"""

from __future__ import annotations

import json
import math
from pathlib import Path

import torch
from safetensors import safe_open


def read_model_dir(model_dir, dtype=torch.float64):
    model_dir = Path(model_dir)
    cfg = json.loads((model_dir / "config.json").read_text())
    tensors = {}
    for file in sorted(model_dir.glob("*.safetensors")):
        with safe_open(str(file), framework="pt", device="cpu") as f:
            for key in f.keys():
                t = f.get_tensor(key)
                tensors[key] = t.to(dtype) if t.is_floating_point() else t
    return cfg, tensors


# --------------------------------------------------------------------------- small pieces


def over_rms(x, eps):
    return x / torch.sqrt(x.pow(2).mean(-1, keepdim=True) + eps)


def silu(x):
    return x / (1.0 + torch.exp(-x))


def gelu_tanh(z):
    return 0.5 * z * (1.0 + torch.tanh(math.sqrt(2.0 / math.pi) * (z + 0.044715 * z ** 3)))


# --------------------------------------------------------------------------- rotations


def frequencies(base, dims):
    return [base ** (-2.0 * i / dims) for i in range(dims // 2)]


def stretch_long_waves(freqs, scaling):
    """Frequencies whose wave is longer than original/low are divided by factor, those whose
    wave is shorter than original/high stay, and between the two the blend is linear in
    original over the wavelength."""
    if scaling is None:
        return freqs
    out = []
    for f in freqs:
        wave = 2.0 * math.pi / f
        if wave < scaling["original"] / scaling["high"]:
            out.append(f)
        elif wave > scaling["original"] / scaling["low"]:
            out.append(f / scaling["factor"])
        else:
            s = (scaling["original"] / wave - scaling["low"]) / (scaling["high"] - scaling["low"])
            out.append((1.0 - s) * f / scaling["factor"] + s * f)
    return out


def turn(x, freqs, pair_of):
    """x [T, n, d]: for every frequency i the two dimensions pair_of(i) of each vector are
    turned by position * freqs[i]; the others stay."""
    out = x.clone()
    for p in range(x.shape[0]):
        for i, f in enumerate(freqs):
            a, b = pair_of(i)
            c, s = math.cos(p * f), math.sin(p * f)
            u, v = x[p, :, a], x[p, :, b]
            out[p, :, a] = u * c - v * s
            out[p, :, b] = v * c + u * s
    return out


def turn_neighbours(x, rot):
    freqs = stretch_long_waves(frequencies(rot["base"], rot["dims"]), rot.get("scaling"))
    return turn(x, freqs, lambda i: (2 * i, 2 * i + 1))


def turn_halves(x, rot):
    half = rot["dims"] // 2
    return turn(x, frequencies(rot["base"], rot["dims"]), lambda i: (i, i + half))


# --------------------------------------------------------------------------- attention


def visible(T, window=None):
    """[T, T] bool: query i sees itself and the window - 1 keys before it (None: every key
    before it)."""
    i = torch.arange(T)[:, None]
    j = torch.arange(T)[None, :]
    seen = j <= i
    return seen if window is None else seen & (i - j < window)


def capped(scores, cap):
    return scores if cap is None else cap * torch.tanh(scores / cap)


def softmax_with_sink(scores, seen, sink):
    """scores [T, T] -> weights over the visible keys; exp(sink) joins every denominator and
    belongs to no key."""
    s = torch.where(seen, scores, torch.full_like(scores, -math.inf))
    top = torch.clamp(s.max(-1, keepdim=True).values, min=float(sink))
    e = torch.exp(s - top)
    return e / (e.sum(-1, keepdim=True) + torch.exp(sink - top))


def window_attention(h, w, pre, m, eps):
    """Queries and keys are rotated (neighbours in pairs, long waves stretched), then divided
    by their root mean square; capped scores, a window, a sink."""
    T = h.shape[0]
    H, G, d, dv = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q = over_rms(turn_neighbours((h @ w[pre + "q"].T).view(T, H, d), m["rot"]), eps)
    k = over_rms(turn_neighbours((h @ w[pre + "k"].T).view(T, G, d), m["rot"]), eps)
    v = (h @ w[pre + "v"].T).view(T, G, dv)
    mask = m.get("mask")
    seen = visible(T, mask["size"] if mask is not None else None)
    out = torch.zeros(T, H, dv, dtype=h.dtype)
    for j in range(H):
        g = j // (H // G)
        scores = capped((q[:, j] @ k[:, g].T) * m["scale"], m.get("softcap"))
        out[:, j] = softmax_with_sink(scores, seen, w[pre + "sink"][j]) @ v[:, g]
    return out.reshape(T, H * dv) @ w[pre + "o"].T


# --------------------------------------------------------------------------- retention


def fading_memory(q, k, v, decay):
    """q, k [T, H, dk], v [T, H, dv], decay [H]: S <- decay S + k v^T, then o = S^T q, a token
    at a time from S = 0."""
    T, H, dk = q.shape
    S = torch.zeros(H, dk, v.shape[-1], dtype=q.dtype)
    out = torch.zeros(T, H, v.shape[-1], dtype=q.dtype)
    for t in range(T):
        for j in range(H):
            S[j] = decay[j] * S[j] + k[t, j][:, None] * v[t, j][None, :]
            out[t, j] = S[j].T @ q[t, j]
    return out


def retention(h, w, pre, m, eps):
    T = h.shape[0]
    H, dk, dv = m["heads"], m["dim"], m["vdim"]
    q = turn_halves((h @ w[pre + "q"].T).view(T, H, dk), m["rot"])
    k = turn_halves((h @ w[pre + "k"].T).view(T, H, dk), m["rot"]) / math.sqrt(dk)
    v = (h @ w[pre + "v"].T).view(T, H, dv)
    o = over_rms(fading_memory(q, k, v, m["decay"]), eps).reshape(T, H * dv)
    return (o * silu(h @ w[pre + "g"].T)) @ w[pre + "o"].T


def both_mixers(h, w, pre, m, eps):
    """Half the sum of the two mixers' outputs, each normed over the width first."""
    left = window_attention(h, w, pre + "left.", m["left"], eps)
    right = retention(h, w, pre + "right.", m["right"], eps)
    return 0.5 * (over_rms(left, eps) * w[pre + "left.out"]
                  + over_rms(right, eps) * w[pre + "right.out"])


# --------------------------------------------------------------------------- feed-forwards


def gelu_ff(h, w, pre):
    return (gelu_tanh(h @ w[pre + "gate"].T) * (h @ w[pre + "up"].T)) @ w[pre + "down"].T


def silu_ff(h, w, pre):
    return (silu(h @ w[pre + "gate"].T) * (h @ w[pre + "up"].T)) @ w[pre + "down"].T


def route(z, top):
    """z [E] -> {expert: weight}: the `top` largest logits and the softmax over them alone."""
    chosen = sorted(range(z.shape[0]), key=lambda e: (-float(z[e]), e))[:top]
    best = max(float(z[e]) for e in chosen)
    raw = {e: math.exp(float(z[e]) - best) for e in chosen}
    total = sum(raw.values())
    return {e: r / total for e, r in raw.items()}


def expert_ff(h, w, pre, mlp):
    out = torch.zeros(h.shape[0], w[pre + "router"].shape[1], dtype=h.dtype)
    z = h @ w[pre + "router"].T + w[pre + "router.b"]
    for t in range(h.shape[0]):
        for e, weight in route(z[t], mlp["router"]["top"]).items():
            out[t] += weight * silu_ff(h[t:t + 1], w, f"{pre}e{e}.")[0]
    if mlp.get("shared") is not None:
        out = out + silu_ff(h, w, pre + "shared.")
    return out


# --------------------------------------------------------------------------- the rest of a layer


def side_input(x, w, tokens, i, dim, eps):
    """What the tokens themselves bring into layer i: the layer's part of every token's row,
    gated by the stream, projected and normed."""
    e = w["side.embed"][torch.as_tensor(tokens, dtype=torch.long)][:, i * dim:(i + 1) * dim]
    pre = f"l{i}.side."
    y = (gelu_tanh(x @ w[pre + "gate"].T) * e) @ w[pre + "proj"].T
    return over_rms(y, eps) * w[pre + "norm"]


def forward(cfg, w, tokens, layer_outputs=None):
    """Logits [T, vocab] of a whole sequence; `layer_outputs`: a list that receives the
    stream after every layer."""
    eps = float(cfg["norm"]["eps"])

    def norm(x, name):
        return over_rms(x, eps) * w[name]

    x = w["embed"][torch.as_tensor(tokens, dtype=torch.long)]
    for i, layer in enumerate(cfg["layers"]):
        pre = f"l{i}."
        out = both_mixers(norm(x, pre + "norm1"), w, pre + "mix.", layer["mixer"], eps)
        x = x + norm(out, pre + "norm1b")
        mlp = layer.get("mlp")
        if mlp is not None:
            h = norm(x, pre + "norm2")
            out = gelu_ff(h, w, pre + "mlp.") if mlp["kind"] == "dense" \
                else expert_ff(h, w, pre + "mlp.", mlp)
            x = x + norm(out, pre + "norm2b")
        if cfg.get("token_side") is not None:
            x = x + side_input(x, w, tokens, i, int(cfg["token_side"]["dim"]), eps)
        if layer_outputs is not None:
            layer_outputs.append(x.clone())
    return (norm(x, "final.norm") @ w["head"].T) * float(cfg["logit_scale"])
