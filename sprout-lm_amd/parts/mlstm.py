"""A matrix memory with exponential gates (mLSTM): its memory is one float32 matrix and one vector per head and request, and
the running maximum of the gates' logarithms that keeps both in range."""
from __future__ import annotations

import torch

from .. import ops
from ..cache.spec import StateSpec
from ..config.base import ConfigError
from ..weights.loader import TensorSpec
from .base import Mixer, register_part


@register_part("mixer", "mlstm")
class MatrixLSTM(Mixer):
    """q = dim^(-1/2) W_q h, k = W_k h (heads x dim), v = W_v h (heads x vdim), no biases.  Per head two gates' logarithms,
    i = cap tanh((W_i h + b_i) / cap) and f = logsigmoid(cap tanh((W_f h + b_f) / cap)), cap = gate_cap; with a running maximum
    m (0 before the first token) m' = max(f + m, i), and S and n (zeros before the first token) fade by exp(f + m - m') and take
    exp(i - m') k v^T and exp(i - m') k.  o = S^T q / (max(|n . q|, exp(-m')) + 1e-6).  Every head's o is divided by its root mean
    square over vdim (`eps` inside the root), the heads are multiplied by a weight over all of them and by sigmoid(W_g h), and
    W_o projects them.  All of a request's state is float32.

    `tensors`: local names of W_q, W_k, W_v, W_g, W_i, W_f, the biases' suffix, the norm's weight and W_o.
    """

    graph_safe = True

    graph_safe_portions = True

    def __init__(self, hidden: int, heads: int, dim: int, vdim: int, gate_cap: float, eps: float,
                 tensors: tuple = ("q", "k", "v", "g", "i", "f", ".b", "norm", "o")):
        if min(hidden, heads, dim, vdim) <= 0 or not gate_cap > 0:
            raise ConfigError(f"A matrix memory needs positive sizes and a positive cap on its gates, got heads={heads} dim={dim} "
                              f"vdim={vdim} gate_cap={gate_cap!r}.")
        if 2 * dim + vdim > 15000:
            raise ConfigError(f"No kernel for a matrix memory with heads of {dim} and {vdim} numbers.")
        self.hidden, self.heads, self.dim, self.vdim, self.gate_cap, self.eps = hidden, heads, dim, vdim, float(gate_cap), float(eps)
        self.names = tuple(tensors)
        self.middle_width = heads * vdim

    # ------------------------------------------------------------------ what it keeps and costs
    def cache_spec(self):
        # the memory a row per value number, the normaliser n as its last row
        return {"memory": StateSpec((self.heads, self.vdim + 1, self.dim), "float32"), "max": StateSpec((self.heads,), "float32")}

    def tensors(self):
        q, k, v, g, i, f, b, norm, o = self.names
        H, D, V, W = self.heads, self.dim, self.vdim, self.hidden
        return {q: TensorSpec((H * D, W)), k: TensorSpec((H * D, W)), v: TensorSpec((H * V, W)), g: TensorSpec((H * V, W)),
                i: TensorSpec((H, W)), i + b: TensorSpec((H,), "vector"), f: TensorSpec((H, W)), f + b: TensorSpec((H,), "vector"),
                norm: TensorSpec((H * V,), "vector", "one_plus_normal"), o: TensorSpec((W, H * V))}

    def flops(self, tokens: int, pairs: int = 0) -> float:
        H, D, V = self.heads, self.dim, self.vdim
        return 2.0 * tokens * self.hidden * (2 * H * D + 3 * H * V + 2 * H) + 4.0 * tokens * H * D * (V + 1)

    def bind(self, tensors):
        q, k, v, g, i, f, b, norm, o = self.names
        rows, self.at, width = [], {}, 0
        for name in (q, k, v, g, i, f):      # one product; each begins at a column in whole eights (16 bytes)
            self.at[name] = width
            rows.append(tensors[name])
            width += tensors[name].shape[0]
            if width % 8:
                rows.append(torch.zeros(8 - width % 8, self.hidden, dtype=tensors[q].dtype, device=tensors[q].device))
                width += 8 - width % 8
        self.w_in = torch.cat(rows, dim=0).contiguous()
        f32 = lambda name: tensors[name].to(torch.float32).contiguous()
        self.b_i, self.b_f, self.w_norm = f32(i + b), f32(f + b), f32(norm)
        self.w_o = tensors[o]
        self.w = {}

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
        proj = ctx.buffer("mlstm_in", (T, self.w_in.shape[0]), ctx.act_dtype)
        ops.gemm(h, self.w_in, proj)
        out = ctx.buffer("mlstm_out", (T, self.middle_width), ctx.act_dtype)
        self.forward_middle(ctx, proj, cache, out)
        ops.gemm(out, self.w_o, residual, accumulate=True)

    def forward_middle(self, ctx, proj, cache, out):
        q, k, v, g, i, f, *_ = self.names
        ops.mlstm(proj, *(self.at[name] for name in (q, k, v, g, i, f)), self.heads, self.dim, self.vdim, self.gate_cap, self.b_i,
                  self.b_f, self.w_norm, self.eps, ctx.q_start, ctx.q_len, ctx.state_slots, ctx.n_seqs, cache["memory"].state,
                  cache["max"].state, out, max_q_len=ctx.max_q_len,
                  workspace=lambda n: ctx.buffer("mlstm_chunks", (n,), torch.float32))
