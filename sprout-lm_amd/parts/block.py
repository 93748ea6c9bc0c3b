"""Arrangement of parts in a layer (reference: src/qwen.ts:164-202)."""
from __future__ import annotations

import torch

from .. import ops
from .base import Block, register_part


@register_part("block", "pre_norm")
class PreNormBlock(Block):
    """x += mixer(norm(x)); x += feed_forward(norm(x)).  The residual stream x is float32.  `ffn` (and its norm) may
    be absent: the layer is then its mixer alone.  `mixer_conv`: a part that stands between the norm and the mixer (a
    short convolution over time, which keeps its last inputs per request): the mixer reads mixer_conv(norm(x))."""

    graph_safe = True

    graph_safe_portions = True

    def __init__(self, mixer_norm, mixer, ffn_norm=None, ffn=None, mixer_conv=None):
        self.mixer_norm, self.mixer, self.ffn_norm, self.ffn, self.mixer_conv = mixer_norm, mixer, ffn_norm, ffn, mixer_conv

    def parts(self):
        named = {"mixer_norm": self.mixer_norm, "mixer": self.mixer}
        if self.mixer_conv is not None:
            named["mixer_conv"] = self.mixer_conv
        if self.ffn is not None:
            named.update({"ffn_norm": self.ffn_norm, "ffn": self.ffn})
        return named

    def forward(self, ctx, residual, caches):
        T, H = residual.shape
        cache = caches.get("mixer")
        h = ctx.buffer("normed", (T, H), ctx.act_dtype)
        if self.mixer_conv is not None:
            self.mixer_norm.forward(ctx, residual, h)
            mixed_in = ctx.buffer("normed_conv", (T, H), ctx.act_dtype)
            self.mixer_conv.forward(ctx, h, mixed_in, caches.get("mixer_conv"))
            self.mixer.forward(ctx, mixed_in, residual, cache)
        elif not self.mixer.forward_from_residual(ctx, self.mixer_norm, residual, cache):
            self.mixer_norm.forward(ctx, residual, h)
            self.mixer.forward(ctx, h, residual, cache)
        if self.ffn is None:
            return
        if not self.ffn.forward_from_residual(ctx, self.ffn_norm, residual):
            self.ffn_norm.forward(ctx, residual, h)
            self.ffn.forward(ctx, h, residual)


@register_part("block", "parallel")
class ParallelBlock(Block):
    """x += mixer(norm_a(x)) + feed_forward(norm_b(x)): both norms read the same x, so both are taken before
    either part adds into the float32 residual stream.  `ffn` (and its norm) may be absent.  A feed-forward without a
    norm of its own (`ffn_norm` None) reads norm_a(x), the mixer's input: where both sublayers can (`Mixer.joins`,
    `FeedForward.joins`, bfloat16), their first products are then one product, whose feed-forward columns leave it activated,
    and their last products one product over both sublayers' rows side by side."""

    graph_safe = True

    graph_safe_portions = True

    def __init__(self, mixer_norm, mixer, ffn_norm=None, ffn=None):
        self.mixer_norm, self.mixer, self.ffn_norm, self.ffn = mixer_norm, mixer, ffn_norm, ffn
        self.w_first = None

    def join(self, dtype):
        if (dtype != torch.bfloat16 or self.ffn is None or self.ffn_norm is not None or not self.mixer.joins() or not self.ffn.joins()
                or self.mixer.middle_width % 8 or self.ffn.inner % 8):
            return
        rows, width = self.mixer.first_rows() + self.ffn.inner, self.ffn.hidden
        if self.mixer.first_rows() % 8 or width % 64 or not ops.joined_takes(1, rows, width) or not ops.joined_takes(65, rows, width):
            return
        first, bias, last = self.mixer.give_matrices()
        up, down = self.ffn.give_matrices()
        self.w_first = torch.cat([first, up], dim=0).contiguous()
        self.w_last = torch.cat([last, down], dim=1).contiguous()
        self.split, self.b_first = first.shape[0], None
        if bias is not None:
            self.b_first = torch.cat([bias.to(torch.float32), torch.zeros(up.shape[0], device=bias.device)]).contiguous()

    def _forward_joined(self, ctx, h, residual, cache):
        T = h.shape[0]
        proj = ctx.buffer("parallel_first", (T, self.split), ctx.act_dtype)
        middle = ctx.buffer("parallel_middle", (T, self.w_last.shape[1]), ctx.act_dtype)
        if T <= 64:      # few tokens: a launch less
            ops.gemm_joined(h, self.w_first, self.b_first, proj, self.split, middle, self.mixer.middle_width, self.ffn.activation)
        else:      # (many: the two shapes each find tiles that fit them better than their sum does)
            ops.gemm(h, self.w_first[:self.split], proj, bias=None if self.b_first is None else self.b_first[:self.split])
            ops.gemm_joined(h, self.w_first[self.split:], None, None, 0, middle, self.mixer.middle_width, self.ffn.activation)
        self.mixer.forward_middle(ctx, proj, cache, middle)
        ops.gemm(middle, self.w_last, residual, accumulate=True)

    def parts(self):
        named = {"mixer_norm": self.mixer_norm, "mixer": self.mixer}
        if self.ffn_norm is not None:
            named["ffn_norm"] = self.ffn_norm
        if self.ffn is not None:
            named["ffn"] = self.ffn
        return named

    def forward(self, ctx, residual, caches):
        T, H = residual.shape
        h = h2 = ctx.buffer("normed", (T, H), ctx.act_dtype)
        if self.ffn is None or self.ffn_norm is None:
            self.mixer_norm.forward(ctx, residual, h)
        else:
            h2 = ctx.buffer("normed_ffn", (T, H), ctx.act_dtype)
            pair = getattr(self.mixer_norm, "forward_pair", None)      # norms that share their statistics take one pass
            if pair is None or not pair(ctx, self.ffn_norm, residual, h, h2):
                self.mixer_norm.forward(ctx, residual, h)
                self.ffn_norm.forward(ctx, residual, h2)
        if self.w_first is not None:
            self._forward_joined(ctx, h, residual, caches.get("mixer"))
            return
        self.mixer.forward(ctx, h, residual, caches.get("mixer"))
        if self.ffn is not None:
            self.ffn.forward(ctx, h2, residual)


@register_part("block", "parallel_scaled")
class ScaledParallelBlock(Block):
    """x += scale_a(mixer(norm(x))) + scale_b(feed_forward(norm(x))): ONE norm whose output both sublayers read, and each
    sublayer's result goes through a part of its own (a learned vector, a constant) before the sum.  The sublayers add
    into float32 rows of their own, which are cleared first; `ffn` (and its scale) may be absent."""

    graph_safe = True

    graph_safe_portions = True

    def __init__(self, mixer_norm, mixer, mixer_scale, ffn=None, ffn_scale=None):
        self.mixer_norm, self.mixer, self.mixer_scale, self.ffn, self.ffn_scale = mixer_norm, mixer, mixer_scale, ffn, ffn_scale

    def parts(self):
        named = {"mixer_norm": self.mixer_norm, "mixer": self.mixer, "mixer_scale": self.mixer_scale}
        if self.ffn is not None:
            named.update({"ffn": self.ffn, "ffn_scale": self.ffn_scale})
        return named

    def forward(self, ctx, residual, caches):
        T, H = residual.shape
        h = ctx.buffer("normed", (T, H), ctx.act_dtype)
        self.mixer_norm.forward(ctx, residual, h)
        both = ctx.buffer("branches", (2, T, H), torch.float32)
        if self.ffn is None:
            both[0].zero_()
            self.mixer.forward(ctx, h, both[0], caches.get("mixer"))
            self.mixer_scale.add(ctx, residual, both[0])
            return
        both.zero_()
        self.mixer.forward(ctx, h, both[0], caches.get("mixer"))
        self.ffn.forward(ctx, h, both[1])
        self.mixer_scale.add(ctx, residual, both[0], self.ffn_scale, both[1])
