"""Softmax attention over a shared low-rank latent, kept in a paged cache.

Per token the part caches one vector [c | k_r]: c, the normalised key/value latent of
`kv_rank` elements, and k_r, `rot_dim` rotated key elements shared by all heads.  Head j's
key is [U_k,j c | k_r] and its value U_v,j c, so with q_j = [q_n | q_r] (the rotated part
rotated like k_r)

    score_j(i, t) = scale * ((U_k,j^T q_n) . c_t + q_r . k_r,t)
    out_j(i)      = U_v,j  sum_t softmax_t(score_j(i, t)) c_t

and neither keys nor values are ever expanded: queries are carried into the latent's space
before attention, and its output back out of it afterwards.  Both steps are folded into the
weights when they are loaded (products taken in float64, rounded once to the run's dtype):
the query up-projection becomes [U_k,j^T U_q,j ; U_q,j's rotated rows] per head, a plain
product from the query latent straight to q', and the output projection becomes
W_o,j U_v,j per head, a plain product from the attention's latent-space result to the
model width.  Queries come through a latent of their own (down, RMS norm, up), or straight
from the mixer's input; then queries and latent are one product.  A window W lets position
i see positions i-W+1..i.  A run may read the latents another run keeps, with queries and
up-projections of its own.
"""

from __future__ import annotations

import torch

from tokensprint_amd.parts.base import MIXERS, Mixer, PagedLatentNeed, TensorDecl, register


@register(MIXERS, "latent_attention")
class LatentAttention(Mixer):
    """params: prefix, heads, dim, rot_dim, vdim, q_rank (None: queries come from the input by
    one projection, '<prefix>q'), kv_rank, scale, eps, window (None = all earlier tokens),
    position (name of a shared 'rope_interleaved' rotation), sink ('<prefix>sink': a number per
    head that joins the softmax's denominator as one more score, not scaled, without key or
    value), own_kv (False: the run has no 'dkv' and reads the cache of another; q_rank None)."""

    def __init__(self, params, ctx):
        super().__init__(params, ctx)
        p = params
        self.prefix = p["prefix"]
        self.heads, self.dim, self.rot_dim = int(p["heads"]), int(p["dim"]), int(p["rot_dim"])
        self.q_rank = int(p["q_rank"]) if p.get("q_rank") is not None else None
        self.vdim, self.kv_rank = int(p["vdim"]), int(p["kv_rank"])
        self.scale, self.eps = float(p["scale"]), float(p["eps"])
        self.window = p.get("window")
        self.has_sink, self.own_kv = bool(p.get("sink", False)), bool(p.get("own_kv", True))
        self.position = ctx.positions[p["position"]]
        if self.position.dims > self.rot_dim:
            raise ValueError(f"{self.prefix}: the rotation covers {self.position.dims} "
                             f"dimensions, the rotated part has {self.rot_dim}")
        if not self.own_kv and self.q_rank is not None:
            raise ValueError(f"{self.prefix}: reading another run's latents is built for queries "
                             "that come straight from the input")
        self.w_down = self.w_query = self.w_out = None
        self.q_norm = self.kv_norm = self.sink = None

    def tensors(self):
        W, pre, H = self.ctx.width, self.prefix, self.heads
        t = {pre + "uk": TensorDecl((H * self.dim, self.kv_rank)),
             pre + "uv": TensorDecl((H * self.vdim, self.kv_rank)),
             pre + "o": TensorDecl((W, H * self.vdim))}
        if self.q_rank is None:
            t[pre + "q"] = TensorDecl((H * (self.dim + self.rot_dim), W))
        else:
            t[pre + "dq"] = TensorDecl((self.q_rank, W))
            t[pre + "dq.norm"] = TensorDecl((self.q_rank,), role="vector")
            t[pre + "uq"] = TensorDecl((H * (self.dim + self.rot_dim), self.q_rank))
        if self.own_kv:
            t[pre + "dkv"] = TensorDecl((self.kv_rank + self.rot_dim, W))
            t[pre + "dkv.norm"] = TensorDecl((self.kv_rank,), role="vector")
        if self.has_sink:
            t[pre + "sink"] = TensorDecl((H,), role="vector", init=(-1.0, 2.0))
        return t

    def load(self, get):
        pre = self.prefix
        H, dn, dr, R, dv = self.heads, self.dim, self.rot_dim, self.kv_rank, self.vdim
        turned = self.position.layout(dr)        # the rotated part's places
        dkv = None
        if self.own_kv:
            dkv = get(pre + "dkv")
            dkv = torch.cat([dkv[:R], dkv[R:][turned]], dim=0)
            self.kv_norm = get(pre + "dkv.norm")
        uq = get(pre + ("q" if self.q_rank is None else "uq"))
        uk, uv, wo = get(pre + "uk"), get(pre + "uv"), get(pre + "o")
        uq64 = uq.double().view(H, dn + dr, -1)
        carried = torch.matmul(uk.double().view(H, dn, R).transpose(1, 2).contiguous(),
                               uq64[:, :dn].contiguous())
        w_query = torch.cat([carried, uq64[:, dn:][:, turned]], dim=1) \
            .reshape(H * (R + dr), -1).to(uq.dtype)
        self.w_out = torch.matmul(wo.double().view(-1, H, dv).transpose(0, 1).contiguous(),
                                  uv.double().view(H, dv, R)).transpose(0, 1) \
            .reshape(-1, H * R).to(wo.dtype).contiguous()
        if self.q_rank is None:
            if dkv is not None and dkv.dtype != w_query.dtype:
                raise ValueError(f"{pre}: q and dkv are stored in different dtypes")
            rows = [w_query] if dkv is None else [w_query, dkv]
            self.w_query = torch.cat(rows, dim=0).contiguous()       # [queries | latent | key part]
        else:
            dq = get(pre + "dq")
            if dq.dtype != dkv.dtype:
                raise ValueError(f"{pre}: the two down projections are stored in different dtypes")
            self.w_down = torch.cat([dq, dkv], dim=0).contiguous()
            self.q_norm = get(pre + "dq.norm")
            self.w_query = w_query.contiguous()
        if self.has_sink:
            self.sink = get(pre + "sink").float().contiguous()

    def cache_need(self):
        return PagedLatentNeed(self.kv_rank + self.rot_dim, self.window)

    def forward(self, h, batch, cache, write_cache):
        if cache is None or cache.k_pages is None:
            raise RuntimeError("latent_attention needs a paged latent cache")
        if write_cache != self.own_kv:
            raise RuntimeError(f"{self.prefix}: " + (
                "a run without a latent of its own cannot own a cache" if write_cache
                else "reading another run's latents is a layer's without 'dkv'"))
        ops, T = self.ops, h.shape[0]
        table = batch.tables[cache.group]
        freqs, rot_dims = self.position.frequencies(), self.position.dims
        sizes = dict(kv_rank=self.kv_rank, rot_dim=self.rot_dim)
        if self.q_rank is None:
            qa = ops.linear(h, self.w_query, torch.float32)
            ops.latent_rows(qa, batch, table, cache, heads=self.heads, own=self.own_kv,
                            kv_norm=self.kv_norm, eps=self.eps, freqs=freqs, rot_dims=rot_dims,
                            **sizes)
        else:
            proj = ops.linear(h, self.w_down, torch.float32)
            cq = ops.latent_prepare(proj, batch, table, cache, q_rank=self.q_rank,
                                    q_norm=self.q_norm, kv_norm=self.kv_norm, eps=self.eps,
                                    freqs=freqs, rot_dims=rot_dims, out_dtype=self.ctx.dtype,
                                    **sizes)
            qa = ops.linear(cq, self.w_query, torch.float32).view(T, self.heads,
                                                                  self.kv_rank + self.rot_dim)
            ops.rotate_interleaved_inplace(qa, batch.positions, freqs, rot_dims,
                                           offset=self.kv_rank)
        more = {"sink": self.sink} if self.has_sink else {}
        ol = ops.latent_attention(qa, batch, table, cache, heads=self.heads, scale=self.scale,
                                  window=self.window, out_dtype=self.ctx.dtype, **sizes, **more)
        return ops.linear(ol.view(T, self.heads * self.kv_rank), self.w_out, torch.float32)
