"""Plain Fubepel forward: one function per mechanism, whole sequences, no cache, CPU torch.

Everything runs over a whole sequence [T, ...] in one precision (float64 by default):
attention as full T x T tables of scores with the mask written out, the recurrence a token
at a time, the rotation and the convolutions position by position, so that a mistake in the
engine's cache, window, state or batch handling cannot be mirrored here.  Nothing imports
the engine package.

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


def over_length(x):
    """Every vector of the last axis divided by the root of its sum of squares plus 1e-6."""
    return x / torch.sqrt(x.pow(2).sum(-1, keepdim=True) + 1e-6)


def sigmoid(x):
    return 1.0 / (1.0 + torch.exp(-x))


def silu(x):
    return x * sigmoid(x)


def softplus(x):
    return torch.clamp(x, min=0.0) + torch.log1p(torch.exp(-x.abs()))


def gelu_tanh(z):
    return 0.5 * z * (1.0 + torch.tanh(math.sqrt(2.0 / math.pi) * (z + 0.044715 * z ** 3)))


# --------------------------------------------------------------------------- attention


def visible(T, window=None, keep_first=0):
    """[T, T] bool: query i sees key j <= i that is among the last `window` (itself counted)
    or among the sequence's `keep_first` first tokens."""
    i = torch.arange(T)[:, None]
    j = torch.arange(T)[None, :]
    seen = j <= i
    if window is not None:
        seen = seen & ((i - j < window) | (j < keep_first))
    return seen


def softmax_with_sink(scores, seen, sink=None):
    """scores [H, T, T] -> weights over the visible keys; `sink` [H]: exp(sink) joins every
    denominator of the head and belongs to no key."""
    s = torch.where(seen, scores, torch.full_like(scores, -math.inf))
    top = s.max(-1, keepdim=True).values
    if sink is not None:
        top = torch.maximum(top, sink[:, None, None])
    e = torch.exp(s - top)
    total = e.sum(-1, keepdim=True)
    if sink is not None:
        total = total + torch.exp(sink[:, None, None] - top)
    return e / total


def window_attention(h, w, pre, m, eps):
    """'attention': per-head norms without weights on queries and keys, no positions, a
    window that keeps the sequence's first tokens."""
    T = h.shape[0]
    H, G, d, dv = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q = over_rms((h @ w[pre + "q"].T).view(T, H, d), eps)
    k = over_rms((h @ w[pre + "k"].T).view(T, G, d), eps)
    v = (h @ w[pre + "v"].T).view(T, G, dv)
    mask = m.get("mask")
    seen = visible(T) if mask is None else visible(T, mask["size"], mask.get("keep_first", 0))
    out = torch.zeros(T, H, dv, dtype=h.dtype)
    for j in range(H):
        g = j // (H // G)
        p = softmax_with_sink(((q[:, j] @ k[:, g].T) * m["scale"])[None], seen)[0]
        out[:, j] = p @ v[:, g]
    return out.reshape(T, H * dv) @ w[pre + "o"].T


def turn_halves(x, base, dims):
    """x [T, n, r]: dimension i < dims/2 of every vector is paired with i + dims/2 and turned
    by position * base^(-2i/dims); dimensions from `dims` on stay."""
    half = dims // 2
    out = x.clone()
    for p in range(x.shape[0]):
        for i in range(half):
            a = p * base ** (-2.0 * i / dims)
            c, s = math.cos(a), math.sin(a)
            u, v = x[p, :, i], x[p, :, i + half]
            out[p, :, i] = u * c - v * s
            out[p, :, i + half] = v * c + u * s
    return out


def latent_of(h, w, pre, m, eps):
    """What a latent layer keeps per token: (latent c [T, R], rotated key part [T, r])."""
    R = m["kv_rank"]
    down = h @ w[pre + "dkv"].T
    c = over_rms(down[:, :R], eps) * w[pre + "dkv.norm"]
    k_rot = turn_halves(down[:, None, R:], m["rot"]["base"], m["rot"]["dims"])[:, 0]
    return c, k_rot


def latent_attention(h, w, pre, m, kept):
    """'latent_attention' over what a latent layer (this one or an earlier one) keeps: keys
    and values are expanded from the latent with this layer's matrices."""
    T = h.shape[0]
    H, d, r, dv = m["heads"], m["dim"], m["rot_dim"], m["vdim"]
    c, k_rot = kept
    q = (h @ w[pre + "q"].T).view(T, H, d + r)
    q_plain, q_rot = q[..., :d], turn_halves(q[..., d:], m["rot"]["base"], m["rot"]["dims"])
    k = (c @ w[pre + "uk"].T).view(T, H, d)
    v = (c @ w[pre + "uv"].T).view(T, H, dv)
    scores = torch.stack([q_plain[:, j] @ k[:, j].T + q_rot[:, j] @ k_rot.T for j in range(H)])
    p = softmax_with_sink(scores * m["scale"], visible(T), w[pre + "sink"])
    out = torch.stack([p[j] @ v[:, j] for j in range(H)], dim=1)
    return out.reshape(T, H * dv) @ w[pre + "o"].T


# --------------------------------------------------------------------------- recurrence


def short_conv(x, taps_w):
    """Causal convolution over time per channel: x [T, C], taps_w [C, taps]; the last column
    weighs the current token, zeros stand in front of the sequence."""
    taps = taps_w.shape[1]
    out = torch.zeros_like(x)
    for t in range(x.shape[0]):
        for back in range(taps):
            if t - back >= 0:
                out[t] += x[t - back] * taps_w[:, taps - 1 - back]
    return out


def delta_rule(q, k, v, beta, g):
    """q, k [T, H, dk], v [T, H, dv], beta and g [T, H].  Per head and token, in this order:
    S <- g S; u = beta (v - S^T k); S <- S + k u^T; o = S^T q."""
    T, H, dk = q.shape
    S = torch.zeros(H, dk, v.shape[-1], dtype=q.dtype)
    out = torch.zeros(T, H, v.shape[-1], dtype=q.dtype)
    for t in range(T):
        S = S * g[t, :, None, None]
        read = torch.einsum("hkv,hk->hv", S, k[t])
        u = beta[t, :, None] * (v[t] - read)
        S = S + k[t, :, :, None] * u[:, None, :]
        out[t] = torch.einsum("hkv,hk->hv", S, q[t])
    return out


def delta_mixer(h, w, pre, m, eps):
    T = h.shape[0]
    H, G, dk, dv = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q, k, v = (silu(short_conv(h @ w[pre + n].T, w[pre + n + ".conv"])) for n in "qkv")
    q = over_length(q.view(T, G, dk)) * dk ** -0.5
    k = over_length(k.view(T, G, dk))
    head_of = torch.arange(H) // (H // G)
    beta = sigmoid(h @ w[pre + "b"].T)
    step = softplus(h @ w[pre + "a"].T + w[pre + "dt_bias"])
    g = torch.exp(-torch.exp(w[pre + "A_log"]) * step)
    o = delta_rule(q[:, head_of], k[:, head_of], v.view(T, H, dv), beta, g)
    o = over_rms(o, eps) * w[pre + "norm"]
    o = o.reshape(T, H * dv) * silu(h @ w[pre + "g"].T)
    return o @ w[pre + "o"].T


# --------------------------------------------------------------------------- the rest of a layer


def clamped_ff(h, w, pre, limit):
    g = torch.clamp(h @ w[pre + "gate"].T, max=limit)
    u = torch.clamp(h @ w[pre + "up"].T, min=-limit, max=limit)
    return (g * sigmoid(1.702 * g) * (u + 1.0)) @ w[pre + "down"].T


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
    x = w["embed"][torch.as_tensor(tokens, dtype=torch.long)] * float(cfg["embedding"]["scale"])
    kept = {}                                   # latent layers' latents, by layer
    for i, layer in enumerate(cfg["layers"]):
        pre, m = f"l{i}.mix.", layer["mixer"]
        if layer["type"] == "delta":
            out = delta_mixer(x, w, pre, m, eps)
        elif layer["type"] == "attention":
            out = window_attention(x, w, pre, m, eps)
        else:
            source = i if m.get("kv_from") is None else m["kv_from"]
            if source == i:
                kept[i] = latent_of(x, w, pre, m, eps)
            out = latent_attention(x, w, pre, m, kept[source])
        x = x + over_rms(out, eps) * w[f"l{i}.norm1"]
        if layer.get("mlp") is not None:
            out = clamped_ff(x, w, f"l{i}.mlp.", float(layer["mlp"]["limit"]))
            x = x + over_rms(out, eps) * w[f"l{i}.norm2"]
        if cfg.get("token_side") is not None:
            x = x + side_input(x, w, tokens, i, int(cfg["token_side"]["dim"]), eps)
        if layer_outputs is not None:
            layer_outputs.append(x.clone())
    return (over_rms(x, eps) * w["final.norm"]) @ w["head"].T
