"""Attention over a cached latent: per token one low-rank latent and one rotated key part serve every head."""
from __future__ import annotations

import torch

from .. import ops
from ..cache.spec import PagedKVSpec
from ..config.base import ConfigError
from ..weights.loader import TensorSpec
from .base import Mixer, register_part
from .sink_attention import padded_width


@register_part("mixer", "latent_attention")
class LatentAttention(Mixer):
    """Head h scores key j as (q_h[:dim] . (U_k,h c_j) + turn(q_h[dim:]) . turn(r_j)) * scale and sums values
    U_v,h c_j, where c_j (kv_rank numbers, RMS-normed) and r_j (rot_dim numbers) come from one down projection of
    token j; the head's output is multiplied by sigmoid(gate_h) where `gated`, and W_o mixes the heads.
    q_rank: the queries come through a latent of their own, q = W_uq norm(W_dq h) (None: q = W_q h).  sinks: the softmax's
    denominator also holds exp(sink_h), a tensor of one number per head that has no key and no value.

    Only c and turn(r) are cached, and attention runs on them directly: since q . (U_k c) = (U_k^T q) . c, the
    queries are carried into the latent's space by a per-head product, the attention kernels see ONE key/value
    head of width kv_rank + rot_dim shared by all query heads (key [c, turn(r)], value c in the same width), and a
    second per-head product with U_v (and the gate) brings the weighted latents to value size.  A decoded token
    reads kv_rank + rot_dim numbers per key instead of heads * (dim + rot_dim + vdim).

    hidden, heads, dim, rot_dim, vdim, kv_rank: sizes.  scale: the factor on q . k, used as given.  window: None,
    or how many of the latest keys (itself included) a query sees.  position: a PositionEncoding whose `freq`
    (float64 table), `rotary_dim` (how many of the rot_dim numbers turn), `pairing` and `magnitude` the turning kernel
    takes.  eps: of the latents' RMS norms.  `tensors`: local names of the query,
    down, latent-norm, key-up, value-up, gate and output tensors; then of the query latent's down, norm and up tensors and
    of the sinks.

    Keys lie in the cache at `width` numbers, zeros behind (`padded_width`: a size the matrix-core kernels take).
    """

    graph_safe = True

    graph_safe_portions = True

    def __init__(self, hidden: int, heads: int, dim: int, rot_dim: int, vdim: int, kv_rank: int, scale: float, eps: float,
                 position, window: int | None = None, gated: bool = True, page_tokens: int | None = None,
                 q_rank: int | None = None, sinks: bool = False, tensors: tuple = ()):
        if min(hidden, heads, dim, vdim, kv_rank) <= 0 or rot_dim < 0:
            raise ConfigError(f"Latent attention needs positive sizes, got heads={heads} dim={dim} rot_dim={rot_dim} "
                              f"vdim={vdim} kv_rank={kv_rank}.")
        if q_rank is not None and q_rank <= 0:
            raise ConfigError(f"A query latent has a positive size, got {q_rank!r}.")
        if getattr(position, "rotary_dim", 0) and getattr(position, "pairing", None) not in ops.LATENT_PAIRINGS:
            raise ConfigError(f"Latent attention turns numbers in pairs {sorted(ops.LATENT_PAIRINGS)}; its position encoding must "
                              f"pair them so.")
        if getattr(position, "rotary_dim", 0) > rot_dim:
            raise ConfigError(f"{position.rotary_dim} numbers cannot turn in a rotated part of {rot_dim}.")
        self.key_width = kv_rank + rot_dim
        self.width = padded_width(self.key_width, self.key_width)
        try:      # one key/value head of this width under all query heads
            ops.check_attention_sizes(heads, 1, self.width)
        except ops.KernelError as error:
            raise ConfigError(str(error)) from None
        self.hidden, self.heads, self.dim, self.rot_dim, self.vdim, self.kv_rank = hidden, heads, dim, rot_dim, vdim, kv_rank
        self.scale, self.eps, self.position, self.window, self.gated = float(scale), float(eps), position, window, gated
        self.page_tokens, self.q_rank, self.sinks = page_tokens, q_rank, bool(sinks)
        defaults = ("q", "dkv", "dkv.norm", "uk", "uv", "g", "o", "dq", "dq.norm", "uq", "sink")
        self.names = tuple(tensors) + defaults[len(tensors):]
        self.middle_width = heads * vdim

    # ------------------------------------------------------------------ what it keeps and costs
    def cache_spec(self):
        return PagedKVSpec(1, self.width, self.window, self.page_tokens)

    def cache_elements_per_token(self) -> int:
        return 2 * self.width

    def flops(self, tokens: int, pairs: int = 0) -> float:
        H = self.heads
        query_rows = H * (self.dim + self.rot_dim)
        rows_in = (self.q_rank or query_rows) + self.key_width + (H if self.gated else 0)
        products = rows_in * self.hidden + (self.q_rank or 0) * query_rows + H * self.dim * self.kv_rank \
            + H * self.kv_rank * self.vdim + H * self.vdim * self.hidden
        return 2.0 * tokens * products + 2.0 * H * (self.key_width + self.kv_rank) * pairs

    def tensors(self):
        q, dkv, norm, uk, uv, g, o, dq, dq_norm, uq, sink = self.names
        H, rows = self.heads, self.heads * (self.dim + self.rot_dim)
        if self.q_rank is None:
            out = {q: TensorSpec((rows, self.hidden))}
        else:
            out = {dq: TensorSpec((self.q_rank, self.hidden)), dq_norm: TensorSpec((self.q_rank,), "vector", "one_plus_normal"),
                   uq: TensorSpec((rows, self.q_rank))}
        out.update({dkv: TensorSpec((self.key_width, self.hidden)),
                    norm: TensorSpec((self.kv_rank,), "vector", "one_plus_normal"),
                    uk: TensorSpec((H * self.dim, self.kv_rank)),
                    uv: TensorSpec((H * self.vdim, self.kv_rank)),
                    o: TensorSpec((self.hidden, H * self.vdim))})
        if self.gated:
            out[g] = TensorSpec((H, self.hidden))
        if self.sinks:
            out[sink] = TensorSpec((H,), "vector")
        return out

    def bind(self, tensors):
        q, dkv, norm, uk, uv, g, o, dq, dq_norm, uq, sink = self.names
        H = self.heads
        # one product for everything that reads the mixer's input: queries (or their latent), latent + rotated key part,
        # gates (rows of zeros behind them bring a row of results to a multiple of 8 numbers: every token's row, and with
        # head sizes in eights every head's part of it, then starts at a multiple of 16 bytes for the per-head products)
        first = tensors[q if self.q_rank is None else dq]
        stacked = [first, tensors[dkv]] + ([tensors[g]] if self.gated else [])
        rows = sum(t.shape[0] for t in stacked)
        if rows % 8:
            stacked.append(torch.zeros(8 - rows % 8, self.hidden, dtype=first.dtype, device=first.device))
        self.w_in = torch.cat(stacked, dim=0).contiguous()
        self.q_off, self.dkv_off = 0, first.shape[0]
        self.gate_off = self.dkv_off + self.key_width
        self.w_norm = tensors[norm]
        self.w_q_norm, self.w_uq = (None, None) if self.q_rank is None else (tensors[dq_norm], tensors[uq])
        self.sink = tensors[sink].to(torch.float32).contiguous() if self.sinks else None
        # U_k per head as [kv_rank, dim]: the product that carries a query into the latent's space
        self.w_uk_t = tensors[uk].view(H, self.dim, self.kv_rank).transpose(1, 2).contiguous()
        self.w_uv = tensors[uv].view(H, self.vdim, self.kv_rank).contiguous()
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
        return self.w_in.shape[0]

    def give_matrices(self):
        given, self.w_in, self.w_o = (self.w_in, None, self.w_o), None, None
        return given

    def forward(self, ctx, h, residual, cache):
        T = h.shape[0]
        proj = ctx.buffer("latent_proj", (T, self.w_in.shape[0]), ctx.act_dtype)
        ops.gemm(h, self.w_in, proj)
        values = ctx.buffer("latent_values", (T, self.middle_width), ctx.act_dtype)
        self.forward_middle(ctx, proj, cache, values)
        ops.gemm(values, self.w_o, residual, accumulate=True)

    def forward_middle(self, ctx, proj, cache, out):
        T, H, W = proj.shape[0], self.heads, self.width
        queries = ctx.buffer("latent_q", (T, H * W), ctx.act_dtype)
        writes = cache.writes
        turn = (ctx.positions, self.position.freq, self.position.rotary_dim, self.position.magnitude, self.position.pairing)
        latent = (proj, self.dkv_off, self.w_norm, cache.slot_mapping, cache.k, cache.v) if writes else None
        rows = proj
        if self.q_rank is None:
            ops.latent_prepare(H, self.dim, self.rot_dim, self.kv_rank, W, self.eps, *turn, latent=latent,
                               queries=(proj, self.q_off, queries))
        else:      # both latents in one launch, the queries' product, then their turn
            c_q = ctx.buffer("latent_cq", (T, self.q_rank), ctx.act_dtype)
            ops.latent_prepare(H, self.dim, self.rot_dim, self.kv_rank, W, self.eps, *turn, latent=latent,
                               query_latent=(proj, self.q_off, self.w_q_norm, c_q))
            rows = ctx.buffer("latent_uq", (T, self.w_uq.shape[0]), ctx.act_dtype)
            ops.gemm(c_q, self.w_uq, rows)
            ops.latent_prepare(H, self.dim, self.rot_dim, self.kv_rank, W, self.eps, *turn, queries=(rows, 0, queries))
        ops.head_gemm(rows, self.q_off, self.dim + self.rot_dim, self.w_uk_t, queries, 0, W)
        mixed = ctx.buffer("latent_mixed", (T, H * W), ctx.act_dtype)
        ops.attention(queries, H * W, cache.k, cache.v, cache.block_tables, ctx.attention, mixed, H, 1, W, self.window,
                      self.scale, workspace=lambda n: ctx.buffer("attention_partials", (n,), torch.float32),
                      kind=ctx.attention_kind, sinks=self.sink)
        ops.head_gemm(mixed, 0, W, self.w_uv, out, 0, self.vdim, gate=proj if self.gated else None, gate_offset=self.gate_off)
