"""Differential attention: two softmax maps per head over the same values, the second taken off the first."""
from __future__ import annotations

import torch

from .. import ops
from ..cache.spec import PagedKVSpec
from ..config.base import ConfigError
from ..weights.loader import TensorSpec
from .base import Mixer, register_part
from .sink_attention import padded_width


@register_part("mixer", "differential_attention")
class DifferentialAttention(Mixer):
    """q = W_q h (+ b), heads x 2 maps of dim numbers; k = W_k h (+ b), kv_heads x 2 maps; v = W_v h (+ b), kv_heads x vdim; query
    head n reads key/value head n // (heads / kv_heads).  `position` (a rotary part with "halves" pairing, or one that turns
    nothing) turns the first rotary_dim numbers of every map.  Map s of a head is softmax(q_s . k_s * scale) over the keys of
    the window (None: all earlier ones) applied to the head's values, a_s.  With the layer's number
    l = exp(sum lq1 lk1) - exp(sum lq2 lk2) + diff, o = a_1 - l a_2 is divided by its root mean square over vdim (`eps` inside
    the root) and multiplied by 1 - diff; W_o mixes the heads.

    The two maps of a key lie side by side as ONE cached key of 2 dim numbers, beside values of vdim (both at `width`
    numbers, zeros behind), so values are kept once and the attention kernels see 2 heads query heads over kv_heads
    key/value heads: a query of map s stands where that map's key does, zeros elsewhere.

    `tensors`: local names of q, k, v, o, the biases' suffix, and the four vectors of l.
    """

    graph_safe = True

    graph_safe_portions = True

    def __init__(self, hidden: int, heads: int, kv_heads: int, dim: int, vdim: int, scale: float, diff: float, eps: float, position,
                 qkv_bias: bool = True, window: int | None = None, page_tokens: int | None = None,
                 tensors: tuple = ("q", "k", "v", "o", ".b", "lq1", "lk1", "lq2", "lk2")):
        if min(hidden, heads, kv_heads, dim, vdim) <= 0 or heads % kv_heads:
            raise ConfigError(f"Attention needs positive sizes and heads in whole groups, got heads={heads} kv_heads={kv_heads} "
                              f"dim={dim} vdim={vdim}.")
        if window is not None and window <= 0:
            raise ConfigError(f"window must be positive, got {window!r}.")
        rotary = getattr(position, "rotary_dim", 0)
        if rotary and (getattr(position, "pairing", None) != "halves" or rotary > dim or rotary % 2):
            raise ConfigError(f"This mixer turns the first {rotary} numbers of a map of {dim} in halves; the position encoding "
                              f"must pair them so and fit.")
        self.width = padded_width(2 * dim, vdim)
        try:
            ops.check_attention_sizes(2 * heads, kv_heads, self.width)
        except ops.KernelError as error:
            raise ConfigError(str(error)) from None
        self.hidden, self.heads, self.kv_heads, self.dim, self.vdim = hidden, heads, kv_heads, dim, vdim
        self.scale, self.diff, self.eps, self.position = float(scale), float(diff), float(eps), position
        self.qkv_bias, self.window, self.page_tokens = bool(qkv_bias), window, page_tokens
        self.names = tuple(tensors)
        self.middle_width = heads * vdim

    # ------------------------------------------------------------------ what it keeps and costs
    def cache_spec(self):
        return PagedKVSpec(self.kv_heads, self.width, self.window, self.page_tokens)

    def cache_elements_per_token(self) -> int:
        return 2 * self.kv_heads * self.width

    def flops(self, tokens: int, pairs: int = 0) -> float:
        q, k, v = 2 * self.heads * self.dim, 2 * self.kv_heads * self.dim, self.kv_heads * self.vdim
        return 2.0 * tokens * self.hidden * (q + k + v + self.heads * self.vdim) + 4.0 * self.heads * (self.dim + self.vdim) * pairs

    def tensors(self):
        q, k, v, o, b, *vectors = self.names
        H, G, D, V = self.heads, self.kv_heads, self.dim, self.vdim
        out = {}
        for name, rows in ((q, H * 2 * D), (k, G * 2 * D), (v, G * V)):
            out[name] = TensorSpec((rows, self.hidden))
            if self.qkv_bias:
                out[name + b] = TensorSpec((rows,), "vector")
        out[o] = TensorSpec((self.hidden, H * V))
        out.update({name: TensorSpec((D,), "vector") for name in vectors})
        return out

    def bind(self, tensors):
        q, k, v, o, b, lq1, lk1, lq2, lk2 = self.names
        self.w_qkv = torch.cat([tensors[q], tensors[k], tensors[v]], dim=0).contiguous()
        self.b_qkv = torch.cat([tensors[q + b], tensors[k + b], tensors[v + b]], dim=0).contiguous() if self.qkv_bias else None
        dot = lambda x, y: torch.sum(tensors[x].to(torch.float64) * tensors[y].to(torch.float64))
        self.factor = (torch.exp(dot(lq1, lk1)) - torch.exp(dot(lq2, lk2)) + self.diff).to(torch.float32).reshape(1).contiguous()
        self.w_o = tensors[o]
        self.w = {}

    def prepare(self, device, dtype):
        self.position.prepare(device, dtype)

    def subparts(self):
        return [self.position]

    # ------------------------------------------------------------------ the step
    def joins(self):
        return True

    def first_rows(self):
        return self.w_qkv.shape[0]

    def give_matrices(self):
        given, self.w_qkv, self.w_o = (self.w_qkv, self.b_qkv, self.w_o), None, None
        return given

    def forward(self, ctx, h, residual, cache):
        T = h.shape[0]
        proj = ctx.buffer("qkv", (T, self.w_qkv.shape[0]), ctx.act_dtype)
        ops.gemm(h, self.w_qkv, proj, bias=self.b_qkv)
        mixed = ctx.buffer("map_difference", (T, self.middle_width), ctx.act_dtype)
        self.forward_middle(ctx, proj, cache, mixed)
        ops.gemm(mixed, self.w_o, residual, accumulate=True)

    def forward_middle(self, ctx, proj, cache, out):
        T, H, G, W = proj.shape[0], self.heads, self.kv_heads, self.width
        queries = ctx.buffer("padded_q", (T, 2 * H * W), ctx.act_dtype)
        writes = cache.writes
        rotary = getattr(self.position, "rotary_dim", 0)
        ops.qkv_prepare(proj, 2 * H, G, self.dim, self.vdim, W, queries, positions=ctx.positions,
                        inv_freq=self.position.inv_freq if rotary else None,
                        inv_freq_tail=getattr(self.position, "inv_freq_tail", None) if rotary and proj.dtype == torch.float32 else None,
                        rotary_dim=rotary, slot_mapping=cache.slot_mapping if writes else None,
                        k_pool=cache.k if writes else None, v_pool=cache.v if writes else None,
                        magnitude=getattr(self.position, "magnitude", 1.0) if rotary else 1.0, maps=2)
        maps = ctx.buffer("attn", (T, 2 * H * W), ctx.act_dtype)
        ops.attention(queries, 2 * H * W, cache.k, cache.v, cache.block_tables, ctx.attention, maps, 2 * H, G, W, self.window,
                      self.scale, workspace=lambda n: ctx.buffer("attention_partials", (n,), torch.float32), kind=ctx.attention_kind)
        ops.map_difference(maps, W, self.factor, self.eps, 1.0 - self.diff, out, H, self.vdim)
