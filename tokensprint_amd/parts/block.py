"""Arrangements of a layer's parts around the residual stream.

Pre-norm arrangement: x = x + mixer(norm(x)); x = x + ffn(norm(x))
(engine/nn/layers.py:111-121).  Each residual add is fused into the following norm.
A layer may leave out one of the two sub-layers (its part and its norm together)."""

from __future__ import annotations

import torch

from tokensprint_amd.kernels.stream import (NormAhead, NormedPair, NormedRows, RowsAhead, StreamRows,
                                            fused_rmsnorm_of)
from tokensprint_amd.parts.base import (BLOCKS, FEED_FORWARDS, FILTERS, MIXERS, NORMS, SIDES, Block,
                                        StreamFilter, TensorDecl, SlotStateNeed, register)


@register(BLOCKS, "pre_norm")
class PreNormBlock(Block):
    ROLES = {"mixer_norm": (NORMS, False), "mixer": (MIXERS, False),
             "ffn_norm": (NORMS, False), "feed_forward": (FEED_FORWARDS, False)}

    def __init__(self, parts, ctx):
        super().__init__(parts, ctx)
        if (self.mixer is None) != (self.mixer_norm is None) or \
                (self.feed_forward is None) != (self.ffn_norm is None):
            raise ValueError("pre_norm: a sub-layer and its norm come together")
        if self.mixer is None and self.feed_forward is None:
            raise ValueError("pre_norm: a layer needs a mixer or a feed-forward")

    def entry_hint(self):
        if self.mixer is not None:
            return self.mixer.stream_hint(self.mixer_norm)
        return self.feed_forward.stream_hint(self.ffn_norm)

    def forward(self, resid, delta, batch, cache, write_cache, next_hint=None):
        if self.mixer is not None:
            hint = self.feed_forward.stream_hint(self.ffn_norm) \
                if self.feed_forward is not None else next_hint
            delta, resid = self.mixer.forward_from_stream(
                resid, delta, self.mixer_norm, batch, cache, write_cache, hint=hint)
        if self.feed_forward is not None:
            delta, resid = self.feed_forward.forward_from_stream(
                resid, delta, self.ffn_norm, batch, hint=next_hint)
        return resid, delta


@register(BLOCKS, "sandwich_norm")
class SandwichNormBlock(Block):
    """A norm before and one after each sub-layer:
    x = x + post1(mixer(filter(norm1(x)))); x = x + post2(ffn(norm2(x))); then, where the layer
    has a side input, x = x + post3(side(x, tokens)).
    The filter (what the mixer reads passes through it, e.g. a token shift), the feed-forward
    with its two norms and the side input with its norm may be left out.  With RMS norms the
    add of a sub-layer's normalised output and whatever reads the stream next are one kernel:
    the norm in front of the feed-forward, the rows of the side input's product, or the norm
    in front of the next layer's mixer (where that layer is of a kind that asks for it); and
    so are the norm in front of the mixer and the filter.  The stream leaves the block summed
    up (no delta is handed on)."""

    ROLES = {"mixer_norm": (NORMS, True), "mixer_filter": (FILTERS, False),
             "mixer": (MIXERS, True), "mixer_post_norm": (NORMS, True),
             "ffn_norm": (NORMS, False), "feed_forward": (FEED_FORWARDS, False),
             "ffn_post_norm": (NORMS, False), "side": (SIDES, False),
             "side_post_norm": (NORMS, False)}

    def __init__(self, parts, ctx):
        super().__init__(parts, ctx)
        ffn = (self.ffn_norm, self.feed_forward, self.ffn_post_norm)
        if any(p is None for p in ffn) and any(p is not None for p in ffn):
            raise ValueError("sandwich_norm: a feed-forward comes with both of its norms")
        if (self.side is None) != (self.side_post_norm is None):
            raise ValueError("sandwich_norm: a side input and its norm come together")

    def entry_hint(self):
        fused = fused_rmsnorm_of(self.mixer_norm) if self.mixer_filter is None else None
        return None if fused is None else NormAhead(fused[0], fused[1])

    def _post_add(self, resid, out, post, then=None, rows=False):
        """resid += post(out); then, if given, the norm `then` (weight, eps) of the sum, or with
        `rows` the sum's rows in the activation dtype."""
        ops, dtype = self.ctx.ops, self.ctx.dtype
        fused = fused_rmsnorm_of(post)
        weight, eps = then or (None, 0.0)
        if isinstance(out, NormedPair):
            if fused is not None:
                return ops.pair_postnorm_add(resid, out, fused[0], fused[1], weight, eps,
                                             dtype if then or rows else None)
            out = ops.normed_pair(out, torch.float32)
        if fused is None:            # another kind of norm: its own forward, then a plain add
            ops.stream_add(resid, post.forward(out), None, None)
            if then:
                return ops.rmsnorm(resid, weight, eps, dtype)
            return ops.stream_rows(resid, dtype) if rows else None
        if then:
            return ops.postnorm_add_norm(resid, out, fused[0], fused[1], weight, eps, dtype)
        if rows:
            return ops.postnorm_add_rows(resid, out, fused[0], fused[1], dtype)
        ops.postnorm_add(resid, out, fused[0], fused[1])
        return None

    def forward(self, resid, delta, batch, cache, write_cache, next_hint=None):
        if isinstance(delta, NormedRows):
            h = delta.rows
        elif self.mixer_filter is not None:
            if delta is not None:
                # a block in front that hands on a delta (with a filter this one gives no entry
                # hint, so it is a plain tensor): added through the mixer's norm, whose output
                # is not used
                self.mixer_norm.add_forward(resid, delta)
            h = self.mixer_filter.forward_from_stream(resid, self.mixer_norm, batch, cache)
        else:
            h = self.mixer_norm.forward(resid) if delta is None \
                else self.mixer_norm.add_forward(resid, delta)
        # the norm the next block opens with, for this block's last add (a row that enters in
        # front of that block would have to be added first)
        ahead = (next_hint.norm_weight, next_hint.eps) \
            if isinstance(next_hint, NormAhead) and next_hint.row is None else None
        side_reads = self.side is not None
        out = self.mixer.forward(h, batch, cache, write_cache)
        if self.feed_forward is None:
            h = self._post_add(resid, out, self.mixer_post_norm,
                               None if side_reads else ahead, rows=side_reads)
        else:
            norm = fused_rmsnorm_of(self.ffn_norm)
            h = self._post_add(resid, out, self.mixer_post_norm, norm)
            if norm is None:
                h = self.ffn_norm.forward(resid)
            out = self.feed_forward.forward(h, batch)
            h = self._post_add(resid, out, self.ffn_post_norm,
                               None if side_reads else ahead, rows=side_reads)
        if side_reads:
            h = self._post_add(resid, self.side.forward(h, batch), self.side_post_norm, ahead)
        return resid, NormedRows(h, False) if ahead else None


@register(BLOCKS, "post_norm")
class PostNormBlock(Block):
    """A norm behind every sub-layer and none in front: the sub-layers read the stream itself,
    x = x + post(mixer(x)); x = x + post(ffn(x)); then, where the layer has a side input,
    x = x + post(side(x, tokens)).  Feed-forward and side input may be left out, each with its
    norm.  The add of a normalised output also writes the rows the next sub-layer (or the next
    block of this kind) reads; the stream leaves the block summed up (no delta is handed
    on)."""

    ROLES = {"mixer": (MIXERS, True), "mixer_post_norm": (NORMS, True),
             "feed_forward": (FEED_FORWARDS, False), "ffn_post_norm": (NORMS, False),
             "side": (SIDES, False), "side_post_norm": (NORMS, False)}

    def __init__(self, parts, ctx):
        super().__init__(parts, ctx)
        if (self.feed_forward is None) != (self.ffn_post_norm is None) or \
                (self.side is None) != (self.side_post_norm is None):
            raise ValueError("post_norm: a sub-layer and its norm come together")

    def entry_hint(self):
        return RowsAhead()

    def _post_add(self, resid, out, post, want_rows):
        """resid += post(out); the rows of the sum in the activation dtype if wanted."""
        ops, dtype = self.ctx.ops, self.ctx.dtype
        fused = fused_rmsnorm_of(post)
        if fused is None:            # another kind of norm: its own forward, then a plain add
            ops.stream_add(resid, post.forward(out), None, None)
            return ops.stream_rows(resid, dtype) if want_rows else None
        if not want_rows:
            ops.postnorm_add(resid, out, fused[0], fused[1])
            return None
        return ops.postnorm_add_rows(resid, out, fused[0], fused[1], dtype)

    def forward(self, resid, delta, batch, cache, write_cache, next_hint=None):
        if isinstance(delta, StreamRows):
            h = delta.rows
        else:
            if delta is not None:
                self.ctx.ops.stream_add(resid, delta, None, None)
            h = self.ctx.ops.stream_rows(resid, self.ctx.dtype)
        onward = isinstance(next_hint, RowsAhead)
        out = self.mixer.forward(h, batch, cache, write_cache)
        h = self._post_add(resid, out, self.mixer_post_norm,
                           self.feed_forward is not None or self.side is not None or onward)
        if self.feed_forward is not None:
            out = self.feed_forward.forward(h, batch)
            h = self._post_add(resid, out, self.ffn_post_norm, self.side is not None or onward)
        if self.side is not None:
            out = self.side.forward(h, batch)
            h = self._post_add(resid, out, self.side_post_norm, onward)
        return resid, StreamRows(h) if onward else None


@register(BLOCKS, "parallel_residual")
class ParallelResidualBlock(Block):
    """One norm whose output both sub-layers read: with h = norm(x),
    x <- x + (mixer(h) + ffn(h)).  The feed-forward may be left out.  The stream leaves the
    block summed up (no delta is handed on); where a block of this kind follows, the sum and
    that block's norm (and a row that enters in front of it) are one kernel, and the normed
    rows travel in delta's place."""

    ROLES = {"mixer_norm": (NORMS, True), "mixer": (MIXERS, True),
             "feed_forward": (FEED_FORWARDS, False)}

    def entry_hint(self):
        fused = fused_rmsnorm_of(self.mixer_norm)
        if fused is None or not hasattr(self.ctx.ops, "stream_add_norm"):
            return None
        return NormAhead(fused[0], fused[1])

    def forward(self, resid, delta, batch, cache, write_cache, next_hint=None):
        if isinstance(delta, NormedRows):
            h = delta.rows
        else:
            h = self.mixer_norm.forward(resid) if delta is None \
                else self.mixer_norm.add_forward(resid, delta)
        mixed = self.mixer.forward(h, batch, cache, write_cache)
        fed = self.feed_forward.forward(h, batch) if self.feed_forward is not None else None
        if isinstance(next_hint, NormAhead):
            rows = self.ctx.ops.stream_add_norm(resid, mixed, fed, next_hint.row,
                                                next_hint.norm_weight, next_hint.eps,
                                                self.ctx.dtype)
            return resid, NormedRows(rows, next_hint.row is not None)
        self.ctx.ops.stream_add(resid, mixed, fed, None)
        return resid, None


@register(FILTERS, "token_shift")
class TokenShift(StreamFilter):
    """h_t <- h_t + (h_(t-1) - h_t) * w, element by element, with h the norm of the stream
    and h_(t-1) the previous token's h before this replacement (zeros in front of a
    sequence's first token).  The last token's h (float32) is kept in the request's state
    slot between steps.

    params: weight (tensor name), dim."""

    def __init__(self, params, ctx):
        super().__init__(params, ctx)
        self.name, self.dim = params["weight"], int(params["dim"])
        self.weight = None

    def tensors(self):
        return {self.name: TensorDecl((self.dim,), role="vector", init=(0.0, 1.0))}

    def load(self, get):
        self.weight = get(self.name)

    def cache_need(self):
        return SlotStateNeed((self.dim,), torch.float32, "shift")

    def forward_from_stream(self, resid, norm, batch, cache):
        fused = fused_rmsnorm_of(norm)
        if fused is None:
            raise ValueError("token_shift is built behind an RMS norm")
        if cache is None or "shift" not in cache.states:
            raise RuntimeError("token_shift needs its per-request state")
        return self.ops.norm_token_shift(resid, fused[0], fused[1], self.weight, batch,
                                         cache.states["shift"], self.ctx.dtype)
