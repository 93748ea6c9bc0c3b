"""Varunex on the GPU: every mechanism alone against its plain function, then whole models cut into steps in different
ways, then generation through the engine's entry point and scheduler."""
import json
import os
import subprocess
import sys

import numpy as np
import pytest
import torch

from tests import traces
from tests import varunex_helpers as VH
from tests.plain import varunex_plain as V
from tests.test_gpu_megozen import dev
from tests.test_gpu_morarax import close, rounded, run_in_portions, specs_of, store_of

pytestmark = pytest.mark.gpu
DEV = "cuda"
ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
DTYPES = [torch.float32, torch.bfloat16]
# single tokens, short portions, both sides of the step kernel's longest portion and of a chunk's length
PORTIONS = [(16, 1), (5, 17), (1, 1), (2, 3), (33, 16), (1, 2), (40, 64), (1, 1), (1, 1), (63, 65), (250, 250)]
LENGTHS_ALONE = (380, 350)


def weights_for(part, rng, dtype, prefix="mix."):
    out = {}
    for name, spec in part.tensors().items():
        a = VH.random_array(rng, prefix + name, spec.shape)
        if spec.kind == "matrix":
            a = a * 1.5
        out[name] = rounded(a, dtype).reshape(spec.shape)
    return out


def bind(part, weights, dtype):
    part.bind({name: dev(a, dtype) for name, a in weights.items()})
    part.prepare(DEV, dtype)


def position_of(turn, size):
    from sprout_lm_amd.parts import make_part
    if not turn["dims"]:
        return make_part("position", "none", head_dim=size)
    return make_part("position", "rotary_neox", head_dim=size, theta=turn["base"], rotary_dim=turn["dims"], scaling=turn.get("scaling"))


# ---------------------------------------------------------------------------------------------- mechanisms alone
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("T,hidden,inner", [(1, 64, 128), (3, 100, 36), (17, 128, 256), (70, 64, 64), (300, 192, 320), (700, 256, 512)])
def test_square_of_relu_feed_forward(dtype, T, hidden, inner):
    from sprout_lm_amd.parts import make_part
    rng = np.random.default_rng(T)
    part = make_part("feed_forward", "mlp", hidden=hidden, inner=inner, activation="relu_squared", bias=None)
    w = {name: rounded(rng.normal(0, 2 * hidden ** -0.5, spec.shape), dtype) for name, spec in part.tensors().items()}
    bind(part, w, dtype)
    x = rounded(rng.standard_normal((T, hidden)), dtype)
    residual = dev(np.zeros((T, hidden), np.float32))
    part.forward(Scratch(dtype), dev(x, dtype), residual)
    close(residual.cpu().numpy(), V.dense_ff(w, "", x, store_of(dtype)), dtype, "feed-forward", f32=2e-5, bf16=1e-2)


@pytest.mark.parametrize("T", [1, 16, 17, 64, 65, 300])
@pytest.mark.parametrize("split,second,K,bias", [(0, 64, 64, False), (40, 96, 128, True), (136, 24, 192, False), (256, 260, 64, True)])
def test_two_products_of_one_input(T, split, second, K, bias):
    """Rows of one matrix that go to two tensors, the second activated and between other columns, for few and many tokens."""
    from sprout_lm_amd import ops
    rng = np.random.default_rng(T + split)
    x, w = (rounded(rng.standard_normal(shape), torch.bfloat16) for shape in ((T, K), (split + second, K)))
    b = rng.standard_normal(split + second).astype(np.float32) if bias else None
    out = torch.full((T, max(split, 4)), 7.0, dtype=torch.bfloat16, device=DEV)
    rows = torch.full((T, second + 12), 7.0, dtype=torch.bfloat16, device=DEV)
    ops.gemm_joined(dev(x, torch.bfloat16), dev(w, torch.bfloat16), None if b is None else dev(b), out if split else None, split, rows, 8,
                    "relu_squared")
    y = x.astype(np.float64) @ w.astype(np.float64).T + (0.0 if b is None else b)
    got = rows.float().cpu().numpy()
    if split:
        close(out.float().cpu().numpy(), y[:, :split], torch.bfloat16, "first product", bf16=2.0 ** -8)
    close(got[:, 8:8 + second], np.maximum(y[:, split:], 0.0) ** 2, torch.bfloat16, "second product", bf16=2.0 ** -8)
    assert np.all(got[:, :8] == 7.0) and np.all(got[:, 8 + second:] == 7.0)


@pytest.mark.parametrize("page,window,keep,sinks", [(16, None, 0, True), (8, 100, 0, True), (16, 70, 5, False), (12, 100, 0, False), (32, None, 0, False)])
@pytest.mark.parametrize("width", [160, 192, 256])
def test_wide_heads(width, page, window, keep, sinks):
    """Heads above 128 numbers in bfloat16: portions, single queries and long contexts beside each other, every number of heads
    over a key head that changes how a block is cut, windows, kept first keys, sinks, pages of a power of two and not."""
    from sprout_lm_amd import ops
    from sprout_lm_amd.ops.kernels import AttentionBatch
    rng = np.random.default_rng(width + page)
    lens, ctx = [33, 1, 1, 5, 150, 1], [300, 400, 7, 1400, 150, 1]
    T, table, pages = sum(lens), [], 0
    order = rng.permutation(sum(-(-c // page) for c in ctx))
    for c in ctx:
        n = -(-c // page)
        table.append(list(order[pages:pages + n]) + [0] * (-(-max(ctx) // page) - n))
        pages += n
    for nq, nkv in ((1, 1), (2, 1), (3, 1), (6, 1), (16, 1), (20, 1), (4, 2)):
        q = rounded(rng.standard_normal((T, nq, width)), torch.bfloat16)
        k, v = (rounded(rng.standard_normal((pages * page, nkv, width)), torch.bfloat16) for _ in range(2))
        k_pool = dev(k.reshape(pages, page, nkv, width).transpose(0, 2, 1, 3), torch.bfloat16).contiguous()
        v_pool = dev(v.reshape(pages, page, nkv, width).transpose(0, 2, 3, 1), torch.bfloat16).contiguous()
        sink = rng.normal(2, 2, nq).astype(np.float32) if sinks else None
        out = torch.full((T, nq * width), float("nan"), dtype=torch.bfloat16, device=DEV)
        ops.attention(dev(q.reshape(T, -1), torch.bfloat16), nq * width, k_pool, v_pool, torch.tensor(table, dtype=torch.int32, device=DEV),
                      AttentionBatch.build(lens, ctx, DEV), out, nq, nkv, width, window, 1.5 * width ** -0.5,
                      sinks=None if sink is None else dev(sink), keep_first=keep)
        got, first = out.float().cpu().numpy().reshape(T, nq, width), 0
        for s, (n, c) in enumerate(zip(lens, ctx)):
            slots = np.array([table[s][p // page] * page + p % page for p in range(c)])
            pos, key = np.arange(c - n, c)[:, None], np.arange(c)[None, :]
            mask = (key <= pos) & ((pos - key < (window or c)) | (key < keep))
            for h in range(nq):
                g = h // (nq // nkv)
                score = q[first:first + n, h].astype(np.float64) @ k[slots, g].astype(np.float64).T * (1.5 * width ** -0.5)
                want = V.softmax(score, mask, None if sink is None else float(sink[h])) @ v[slots, g].astype(np.float64)
                close(got[first:first + n, h], want, torch.bfloat16, f"{nq} over {nkv}, request {s}, head {h}", bf16=1.5e-2)
            first += n


class Scratch:
    """What a part asks of a step that carries no sequences."""

    def __init__(self, dtype):
        self.act_dtype = dtype

    def buffer(self, name, shape, dtype):
        return torch.empty(shape, dtype=dtype, device=DEV)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("ff", [None, 48])
def test_one_norm_for_both_sublayers(dtype, ff):
    """A parallel layer whose feed-forward has no norm: x + (mixer(n(x)) + ff(n(x))), rows whose mean is far from zero."""
    import sprout_lm_amd as S
    from sprout_lm_amd.models.plan import ModelParts
    from sprout_lm_amd.registry import build_model_plan
    cfg = VH.model(40, 9, [VH.layer(VH.memory(2, 8, 12, 4.0), ff)], eps=1e-4)
    parts = ModelParts(build_model_plan(S.config_from_dict(cfg)))
    w = {name: rounded(a, dtype) for name, a in VH.random_weights(cfg, 5).items()}
    parts.bind({name: dev(a, dtype) for name, a in w.items()}, DEV, dtype)
    block = parts.blocks[0]
    rng = np.random.default_rng(2)
    x = (rng.standard_normal((30, 40)) + rng.uniform(-20, 20, (30, 1))).astype(np.float32)

    class Whole:
        """The block as a mixer of its own, for the harness."""
        cache_spec = staticmethod(block.mixer.cache_spec)

        @staticmethod
        def forward(ctx, h, residual, cache):
            residual.copy_(dev(x[at[0]:at[0] + residual.shape[0]]))
            at[0] += residual.shape[0]
            block.forward(ctx, residual, {"mixer": cache})

    at = [0]
    got = run_in_portions(Whole, specs_of(block.mixer), dtype, [x], [(11,), (1,), (18,)], 40)[0]
    store = store_of(dtype)
    h = store(V.layer_norm(x, w["l0.norm1"], w["l0.norm1.b"], 1e-4))
    want = x + V.mlstm_mixer(w, "l0.mix.", cfg["layers"][0]["mixer"], h, 1e-4, store) + (V.dense_ff(w, "l0.mlp.", h, store) if ff else 0.0)
    close(got, want, dtype, "layer", f32=3e-5, bf16=2e-2)


# sizes no fast kernel takes; few and many lanes to a row; several rows a thread; heads whose memory stays in memory
MEMORIES = [(3, 7, 9, 6.0), (5, 32, 48, 11.0), (2, 16, 24, 3.0), (1, 128, 256, 10.0), (2, 48, 40, 15.0), (2, 12, 100, 1.0), (1, 256, 72, 8.0),
            (1, 64, 512, 14.0), (1, 260, 12, 5.0), (1, 256, 512, 9.0), (5, 4, 3, 7.0)]


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("heads,dim,vdim,cap", MEMORIES)
def test_memory_alone_in_portions(dtype, heads, dim, vdim, cap):
    from sprout_lm_amd.parts import make_part
    hidden, eps = 48, 1e-5
    m = VH.memory(heads, dim, vdim, cap)["mixer"]
    rng = np.random.default_rng(dim * 10 + vdim)
    part = make_part("mixer", "mlstm", hidden=hidden, eps=eps, **m)
    w = weights_for(part, rng, dtype)
    bind(part, w, dtype)
    inputs = [rounded(rng.standard_normal((n, hidden)), dtype) for n in LENGTHS_ALONE]
    got = run_in_portions(part, specs_of(part), dtype, inputs, PORTIONS, hidden)
    for i, x in enumerate(inputs):
        close(got[i], V.mlstm_mixer(w, "", m, x, eps, store_of(dtype)), dtype, f"request {i}", f32=1e-4, bf16=6e-2)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("heads,dim,vdim", [(3, 16, 8), (2, 32, 72), (2, 128, 128), (1, 128, 256), (1, 256, 512), (2, 48, 200), (2, 20, 12), (1, 9, 5)])
def test_memory_kernels_from_a_state_with_extreme_gates(dtype, heads, dim, vdim):
    """The recurrence on rows as they are, from memories that are not empty and maxima far from zero: tokens that wipe the
    memory, tokens that all but leave it, inputs weaker and stronger than all before by many powers of e, in one chunk and
    across chunks.  States (float32, from inputs both storage types hold exactly) keep their digits; whole and in pieces."""
    from sprout_lm_amd import ops
    rng = np.random.default_rng(dim + vdim)
    H, D, W, cap, eps = heads, dim, vdim, 30.0, 1e-5
    lens = [150, 1, 64, 33]
    T, starts, slots = sum(lens), [0, 150, 151, 215], [2, 0, 4, 3]
    at = np.cumsum([0, H * D, H * D, H * W, H * W, H])
    pad = lambda n: -(-n // 8) * 8
    off, width = [], 0
    for n in (H * D, H * D, H * W, H * W, H, H):
        off.append(width)
        width += pad(n)
    rows = rng.standard_normal((T, width)).astype(np.float32)
    gates = rng.normal(0, 6, (T, 2, H))
    gates[::13, 1] = -40.0           # everything before is forgotten
    gates[1::4, 1] = 40.0            # all but nothing is
    gates[::7, 0] = -35.0            # a whisper ...
    gates[60:70, 0] = 25.0           # ... and inputs that drown what came before
    rows[:, off[4]:off[4] + H], rows[:, off[5]:off[5] + H] = gates[:, 0], gates[:, 1]
    rows[8, off[0]:off[0] + H * D] = 0.0      # a query of zeros reads nothing: the floor of the share
    rows = rounded(rows, torch.bfloat16)
    bias_i, bias_f = rng.normal(0, 1, H).astype(np.float32), rng.normal(1, 1, H).astype(np.float32)
    norm = (1 + 0.1 * rng.standard_normal(H * W)).astype(np.float32)
    memory0 = rng.standard_normal((6, H, W + 1, D)).astype(np.float32)
    max0 = rng.normal(0, 8, (6, H)).astype(np.float32)
    ints = lambda a: torch.tensor(a, dtype=torch.int32, device=DEV)
    scratch = []

    def workspace(n):
        scratch.append(n)
        return torch.full((n,), float("nan"), device=DEV)

    def run(lengths, first, begin, memory, maxima, chosen):
        n = sum(lengths)
        out = torch.empty(n, H * W, dtype=dtype, device=DEV)
        ops.mlstm(dev(rows[begin:begin + n], dtype), *off, H, D, W, cap, dev(bias_i), dev(bias_f), dev(norm), eps, ints(first),
                  ints(lengths), ints(chosen), len(lengths), memory, maxima, out, max(lengths), workspace)
        return out.float().cpu().numpy()

    memory, maxima = dev(memory0), dev(max0)
    whole = run(lens, starts, 0, memory, maxima, slots)
    assert bool(scratch) == (dtype == torch.bfloat16 and dim % 16 == 0 and vdim % 8 == 0), "the chunks' kernels did not run, or did"
    for i, (s, l) in enumerate(zip(starts, lens)):
        x = rows[s:s + l].astype(np.float64)
        part = lambda j, n: x[:, off[j]:off[j] + H * n].reshape(l, H, n)
        i_gate = cap * np.tanh((x[:, off[4]:off[4] + H] + bias_i) / cap)
        f_gate = -np.logaddexp(0.0, -cap * np.tanh((x[:, off[5]:off[5] + H] + bias_f) / cap))
        S0 = memory0[slots[i]].astype(np.float64)
        o, (S, n, m) = V.mlstm(part(0, D) * D ** -0.5, part(1, D), part(2, W), i_gate, f_gate,
                               (S0[:, :W].transpose(0, 2, 1), S0[:, W], max0[slots[i]].astype(np.float64)))
        got = memory[slots[i]].cpu().numpy()
        close(got[:, :W].transpose(0, 2, 1), S, torch.float32, f"memory of request {i}", f32=2e-5)
        close(got[:, W], n, torch.float32, f"normaliser of request {i}", f32=2e-5)
        close(maxima[slots[i]].cpu().numpy(), m, torch.float32, f"maximum of request {i}", f32=2e-6)
        want = (V.rms(o, eps) * norm.reshape(H, W) * V.sigmoid(part(3, W))).reshape(l, H * W)
        close(whole[s:s + l], want, dtype, f"request {i}", f32=2e-4, bf16=2.0 ** -7)
    for free in (1, 5):      # nobody's slots
        assert torch.equal(memory[free].cpu(), torch.from_numpy(memory0[free])) and torch.equal(maxima[free].cpu(), torch.from_numpy(max0[free]))
    pieces, pmax, done = dev(memory0), dev(max0), 0
    for n in (1, 63, 1, 20, 2, 63):      # the first request again, through both kernels in turn
        got = run([n], [0], done, pieces, pmax, slots[:1])
        close(got, whole[done:done + n], dtype, f"tokens {done} on, alone", f32=2e-4, bf16=2.0 ** -6)
        done += n
    close(pieces[slots[0]].cpu().numpy(), memory[slots[0]].cpu().numpy(), torch.float32, "memory", f32=2e-5)
    close(pmax[slots[0]].cpu().numpy(), maxima[slots[0]].cpu().numpy(), torch.float32, "maximum", f32=2e-6)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("far", [1, 63, 64, 65, 128, 500])
def test_a_value_far_back_is_read(dtype, far):
    """One early token writes a value under a key that only the reader asks for; a head that keeps everything returns it from
    `far` tokens back (inside a chunk, at its edges, many chunks back), a head that forgets has lost it unless it was just
    written.  The reader last in a portion and decoded alone."""
    from sprout_lm_amd.parts import make_part
    hidden, dim, vdim, heads = 16, 16, 8, 2
    m = VH.memory(heads, dim, vdim, 20.0)["mixer"]
    part = make_part("mixer", "mlstm", hidden=hidden, eps=1e-6, **m)
    w = {name: np.zeros(spec.shape, np.float32) for name, spec in part.tensors().items()}
    for n in range(heads):
        w["k"][n * dim + 0, 0] = 1.0         # everybody's key but the writer's
        w["k"][n * dim + 1, 1] = 4.0         # the writer's key
        w["q"][n * dim + 1, 2] = 4.0         # the reader asks for the writer's
        w["q"][n * dim + 0, 5] = 4.0         # the others for everybody's
        w["v"][n * vdim:(n + 1) * vdim, 3] = (4.0, -3.0, 2.0, 1.0, -1.0, 0.5, 3.0, -2.0)
        w["v"][n * vdim, 6] = 0.25
    w["g"][:, 4] = 3.0                       # an open gate
    w["norm"][:] = 1.0
    w["f.b"][:] = (18.0, 0.0)                # the first head keeps, the second halves
    w["o"][:] = rounded(np.random.default_rng(0).normal(0, 0.3, w["o"].shape), dtype)
    bind(part, w, dtype)
    n, writer = 560, 20
    reader = writer + far
    x = np.zeros((n, hidden), np.float32)
    x[:, 0] = x[:, 4] = x[:, 5] = x[:, 6] = 1.0
    x[writer, 0], x[writer, 1], x[writer, 3] = 0.0, 1.0, 1.0
    x[reader, 2], x[reader, 5] = 1.0, 0.0
    want = V.mlstm_mixer(w, "", m, x, 1e-6, store_of(dtype))
    heads_out = np.linalg.lstsq(w["o"].astype(np.float64), want[reader], rcond=None)[0]
    assert np.abs(heads_out[1:vdim]).max() > 0.5
    for steps in ([(reader + 1,), (n,)], [(reader,), (1,), (n,)], [(writer + 1,), (n,)], [(19,), (2,), (n,)]):
        got = run_in_portions(part, specs_of(part), dtype, [x], steps, hidden)[0]
        close(got, want, dtype, f"steps {steps}", f32=3e-5, bf16=2e-2)


def latent_part(hidden, m, eps):
    from sprout_lm_amd.parts import make_part
    sizes = {key: value for key, value in m.items() if key != "rot"}
    return make_part("mixer", "latent_attention", hidden=hidden, eps=eps, sinks=True, position=position_of(m["rot"], m["rot_dim"]), **sizes)


LATENTS = [(3, 10, 6, 14, 9, 20, VH.rot(6, 30.0), 8), (4, 16, 16, 32, 64, 48, VH.rot(16, 1000.0, (8.0, 1.0, 4.0, 64.0)), 16),
           (20, 8, 24, 8, 40, 112, VH.rot(24, 100.0), 4), (2, 24, 0, 16, 16, 32, VH.rot(0, 10.0), 8), (6, 40, 32, 24, 24, 96, VH.rot(32, 500.0), 16),
           (2, 8, 8, 24, 1, 1, VH.rot(8, 20.0), 8), (6, 64, 32, 64, 96, 160, VH.rot(32, 10000.0), 16), (4, 16, 16, 16, 32, 240, VH.rot(16, 100.0), 12),
           (1, 16, 64, 16, 48, 400, VH.rot(64, 100.0), 8), (5, 24, 64, 40, 56, 512, VH.rot(64, 1000.0), 16)]


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("heads,dim,rot_dim,vdim,q_rank,kv_rank,turn,page", LATENTS)
def test_latent_attention_alone_in_portions(dtype, heads, dim, rot_dim, vdim, q_rank, kv_rank, turn, page):
    """Query latents, halves that turn, sinks and gates; keys of 9 to 576 numbers, padded and not."""
    hidden, eps = 40, 1e-5
    m = VH.latent(heads, dim, rot_dim, vdim, q_rank, kv_rank, 1.2 / np.sqrt(dim + rot_dim), turn)["mixer"]
    rng = np.random.default_rng(heads * 10 + kv_rank)
    part = latent_part(hidden, m, eps)
    w = weights_for(part, rng, dtype)
    bind(part, w, dtype)
    inputs = [rounded(rng.standard_normal((n, hidden)), dtype) for n in LENGTHS_ALONE]
    got = run_in_portions(part, specs_of(part), dtype, inputs, PORTIONS, hidden, page=page)
    for i, x in enumerate(inputs):
        close(got[i], V.latent_attention(w, "", m, x, np.arange(len(x)), eps, store_of(dtype)), dtype, f"request {i}", f32=3e-5, bf16=3e-2)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("page,kv_rank", [(8, 48), (16, 112), (4, 26)])
def test_latent_attention_finds_one_key_and_weighs_its_sink(dtype, page, kv_rank):
    """One flagged key outweighs everything: far back, at a page's first and last place, the first tokens; and sinks of every
    strength: heads that see their keys alone, heads that give half to the sink, heads that it silences."""
    hidden, heads, n = 24, 4, 300
    m = VH.latent(heads, 16, 8, 12, 32, kv_rank, 0.8, VH.rot(8, 100.0))["mixer"]
    part = latent_part(hidden, m, 1e-5)
    rng = np.random.default_rng(5)
    w = weights_for(part, rng, dtype)
    # feature 0 flags a key, feature 1 a reader: the latents' first numbers, which the unturned part alone looks at
    w["dkv"][0], w["dq"][0] = 0.0, 0.0
    w["dkv"][0, 0] = w["dq"][0, 1] = 2.0
    w["uk"].reshape(heads, 16, kv_rank)[:, :, 0] = 1.5
    w["uq"].reshape(heads, 24, 32)[:, :16, 0] = 0.02
    w["sink"][:] = (-30.0, 12.0, 18.0, 60.0)
    w = {name: rounded(a, dtype) for name, a in w.items()}
    bind(part, w, dtype)
    for reader, key in ((200, 4), (255, 128), (256, 127), (299, 0), (1, 0), (0, 0), (97, 96), (64, 63), (270, 269)):
        x = rounded(rng.standard_normal((n, hidden)) * 0.3, dtype)
        x[:, :2] = 0.0
        x[key, 0] = 6.0
        x[reader, 1] = 6.0
        run = lambda weights, rows: V.latent_attention(weights, "", m, rows, np.arange(n), 1e-5, store_of(dtype))
        want = run(w, x)
        if key != reader:
            assert np.abs(want[reader] - run(w, np.where(np.arange(n)[:, None] == key, 0.0, x))[reader]).max() > 0.02
        assert np.abs(want[reader] - run(dict(w, sink=w["sink"] - 100.0), x)[reader]).max() > 0.02
        for steps in ([(reader + 1,), (n,)], [(reader,), (1,), (n,)], [(33,), (reader - 33,), (1,), (1,), (n,)]):
            if any(s[0] <= 0 for s in steps):
                continue
            got = run_in_portions(part, specs_of(part), dtype, [x], steps, hidden, page=page)[0]
            err = np.abs(got[reader] - want[reader]).max()
            assert err <= (2e-5 if dtype == torch.float32 else 2e-2), f"reader {reader}, key {key}, steps {steps}: off by {err:.3e}"


def difference_part(hidden, m, eps):
    from sprout_lm_amd.parts import make_part
    sizes = {key: value for key, value in m.items() if key not in ("rot", "mask")}
    return make_part("mixer", "differential_attention", hidden=hidden, eps=eps, window=m["mask"]["size"] if m.get("mask") else None,
                     position=position_of(m["rot"], m["dim"]), **sizes)


DIFFERENCES = [(6, 3, 6, 10, 4, 7, 8), (2, 2, 12, 5, 0, None, 8), (4, 1, 16, 32, 8, 24, 16), (3, 1, 5, 18, 2, 1, 4), (4, 2, 32, 64, 32, 100, 16),
               (6, 1, 40, 80, 20, 129, 16), (2, 1, 64, 128, 64, None, 16), (2, 1, 64, 64, 16, 300, 24), (10, 1, 32, 16, 16, 65, 8),
               (2, 2, 80, 40, 80, 50, 8), (1, 1, 8, 200, 8, 33, 12), (2, 1, 72, 128, 8, None, 12),
               (1, 1, 40, 530, 16, 70, 16)]


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("heads,kv_heads,dim,vdim,rot_dims,window,page", DIFFERENCES)
def test_difference_of_two_maps_alone_in_portions(dtype, heads, kv_heads, dim, vdim, rot_dims, window, page):
    hidden, eps = 40, 1e-4
    turn = VH.rot(rot_dims, 200.0, (4.0, 1.0, 4.0, 90.0) if rot_dims > 4 else None)
    m = VH.difference(heads, kv_heads, dim, vdim, 1.5 / np.sqrt(dim), 0.3, turn, window)["mixer"]
    rng = np.random.default_rng(heads * 10 + dim)
    part = difference_part(hidden, m, eps)
    w = weights_for(part, rng, dtype)
    bind(part, w, dtype)
    inputs = [rounded(rng.standard_normal((n, hidden)), dtype) for n in LENGTHS_ALONE]
    got = run_in_portions(part, specs_of(part), dtype, inputs, PORTIONS, hidden, page=page)
    for i, x in enumerate(inputs):
        close(got[i], V.differential_attention(w, "", m, x, np.arange(len(x)), eps, store_of(dtype)), dtype, f"request {i}", f32=5e-5,
              bf16=4e-2)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("page,dim,flagged", [(8, 16, 0), (16, 32, 1), (4, 10, 0), (16, 16, 1)])
def test_each_map_finds_its_key_at_the_window_s_edges(dtype, page, dim, flagged):
    """One map looks for a flagged key, the other does not: just inside the window, just outside, far back, at a page's first
    and last place, the first tokens; the reader in a portion of a prompt and decoded alone."""
    hidden, window, heads = 24, 36, 4
    m = VH.difference(heads, 2, dim, 2 * dim, 1.0, 0.4, VH.rot(8, 100.0), window)["mixer"]
    part = difference_part(hidden, m, 1e-5)
    rng = np.random.default_rng(5)
    w = weights_for(part, rng, dtype)
    # feature 0 flags a key, feature 1 a reader: both point along the unturned dimensions of one of a head's two maps
    for name, column in (("k", 0), ("q", 1)):
        w[name] = (w[name] * 0.1).astype(np.float32)
        w[name].reshape(-1, 2, dim, hidden)[:, flagged, 8:, column] = 3.0
        w[name + ".b"][:] = 0.0
        w[name] = rounded(w[name], dtype)
    bind(part, w, dtype)
    n = 260
    for reader, key in ((200, 165), (200, 164), (200, 4), (227, 192), (227, 191), (96, 61), (91, 56), (91, 55), (259, 224), (259, 223),
                        (40, 5), (40, 4), (35, 0), (36, 0), (0, 0), (1, 0)):
        x = rounded(rng.standard_normal((n, hidden)) * 0.3, dtype)
        x[:, :2] = 0.0
        x[key, 0] = 4.0
        x[reader, 1] = 4.0
        run = lambda rows: V.differential_attention(w, "", m, rows, np.arange(n), 1e-5, store_of(dtype))
        want = run(x)
        if key != reader and reader >= 35:      # (among a sequence's first few keys any of them weighs much)
            moved = np.abs(want[reader] - run(np.where(np.arange(n)[:, None] == key, 0.0, x))[reader]).max()
            assert (moved > 0.02) == (reader - key < window), (reader, key, moved)
        for steps in ([(reader + 1,), (n,)], [(reader,), (1,), (n,)], [(33,), (reader - 33,), (1,), (1,), (n,)]):
            if any(s[0] <= 0 for s in steps):
                continue
            got = run_in_portions(part, specs_of(part), dtype, [x], steps, hidden, page=page)[0]
            err = np.abs(got[reader] - want[reader]).max()
            assert err <= (3e-5 if dtype == torch.float32 else 4e-2), f"reader {reader}, key {key}, steps {steps}: off by {err:.3e}"


# ---------------------------------------------------------------------------------------------- whole models
@pytest.fixture(scope="module")
def folders(tmp_path_factory):
    root = str(tmp_path_factory.mktemp("varunex"))
    return {name: VH.make_folder(root, name) for name in VH.CONFIGS}


def requests_for(name, lengths, seed=100):
    vocab = VH.CONFIGS[name]["vocab"]
    return {f"r{i}": VH.random_tokens(vocab, n, seed + i) for i, n in enumerate(lengths)}


def replay(folder, name, dtype, trace, max_tokens, page=None, slots=4, reused=None):
    """The engine's trace session on a pool of `max_tokens`; per step the logits rows."""
    from sprout_lm_amd.engine import ModelRunner
    from sprout_lm_amd.engine.trace import TraceSession
    page = page or VH.PAGE[name]
    runner = ModelRunner.from_folder(folder, dtype, block_size=page, num_blocks=-(-max_tokens // page), max_sequences=slots,
                                     prefix_caching=False)
    session = TraceSession(runner)
    out, owners, holders = [], {}, {}
    for record in trace.steps:
        logits = session.run_step(record)
        out.append(None if logits is None or not logits.shape[0] else logits.cpu().numpy().copy())
        for rid, seq in session.live.items():
            if rid not in holders.setdefault(seq.state_slot, []):
                holders[seq.state_slot].append(rid)
            for g, blocks in enumerate(seq.blocks):
                for page_id in blocks:
                    if page_id >= 0 and rid not in owners.setdefault((g, page_id), []):
                        owners[(g, page_id)].append(rid)
    if reused is not None:
        reused["pages"] = sum(len(r) > 1 for r in owners.values())
        reused["slots"] = sum(len(r) > 1 for r in holders.values())
    assert all(free == total for free, total in zip(runner.cache.free_pages(), [g.pool.num_pages for g in runner.cache.groups]))
    assert not session.live
    return out


def check(folder, dtype, requests, trace, results):
    worst = 0.0
    for step, (rows, got) in enumerate(zip(trace.expected, results)):
        if not rows:
            assert got is None
            continue
        assert got.shape[0] == len(rows)
        for i, (rid, pos) in enumerate(rows):
            want = VH.plain_logits(folder, dtype, requests[rid])[pos]
            err = float(np.abs(got[i] - want).max())
            worst = max(worst, err)
            bound = VH.tolerance(dtype, want)
            if dtype == "bfloat16":     # how far bfloat16 rounding moves this row on the plain side itself
                bound += float(np.abs(want - VH.plain_logits(folder, "float32", requests[rid])[pos]).max())
            assert err <= bound, f"step {step} request {rid} position {pos}: error {err:.3e}"
    return worst


LENGTHS = {"odd": [1, 2, 21, 70, 45, 97], "general": [1, 9, 40, 97, 150, 33, 2, 75], "states": [9, 40, 97, 33, 130, 3],
           "wide": [2, 70, 97, 33, 64, 120]}
CASES = [(n, d) for d in ("float32", "bfloat16") for n in VH.CONFIGS]


@pytest.mark.parametrize("name,dtype", CASES)
@pytest.mark.parametrize("family", ["whole", "tail", "portions", "mixed"])
def test_replay_family(folders, name, dtype, family):
    """Whole prompts; a prompt and its last 48 tokens one by one; portions down to two tokens; four live requests in a
    pool and on state slots that hold no more, so that pages and slots are used again."""
    requests = requests_for(name, LENGTHS[name])
    roomy = 4 * 64 * (1 + max(LENGTHS[name]) // 64)
    if family == "whole":
        trace, pool = traces.whole(requests), roomy
    elif family == "tail":
        trace, pool = traces.tail_decoded(requests, tail=48), roomy
    elif family == "portions":
        trace, pool = traces.portions(requests), roomy
    else:
        trace = traces.mixed(requests, seed=7)
        pool = sum(sorted(-(-len(t) // 64) * 64 for t in requests.values())[-4:])
    reused = {}
    results = replay(folders[name], name, dtype, trace, pool, reused=reused)
    if family == "mixed":
        assert reused["slots"] >= 1, f"no state slot was used again: {reused}"
        if name != "states":      # (a model without pages)
            assert reused["pages"] >= 2, f"no page was used again: {reused}"
    worst = check(folders[name], dtype, requests, trace, results)
    print(f"{family} {name} {dtype}: {len(trace.steps)} steps, worst error {worst:.3e}")


@pytest.mark.parametrize("name,page,dtype", [("general", 12, "float32"), ("odd", 4, "float32"), ("wide", 64, "float32"),
                                             ("general", 24, "bfloat16")])
def test_replay_with_other_page_sizes(folders, name, page, dtype):
    requests = requests_for(name, LENGTHS[name], seed=300)
    trace = traces.mixed(requests, seed=11)
    pool = sum(sorted(-(-len(t) // 192) * 192 for t in requests.values())[-4:])
    results = replay(folders[name], name, dtype, trace, pool, page=page)
    check(folders[name], dtype, requests, trace, results)


@pytest.mark.parametrize("name,dtype", [("general", "float32"), ("states", "float32"), ("wide", "float32"), ("general", "bfloat16"),
                                        ("states", "bfloat16")])
def test_long_prompts_in_long_portions(folders, name, dtype):
    """Prompts of 700 tokens whole, in long uneven portions, and two requests' long portions beside each other and beside
    single tokens."""
    requests = requests_for(name, [700, 333], seed=500)
    cut = traces.portions(requests, sizes=(200, 129, 65, 2, 64, 190, 1, 70))
    both = traces.Trace()
    a, b = requests["r0"], requests["r1"]
    both.add([("r0", 0, a[:400], range(390, 400)), ("r1", 0, b[:150], [149])])
    both.add([("r0", 400, a[400:401], [0]), ("r1", 150, b[150:], range(0, 183, 7))], end=["r1"])
    both.add([("r0", 401, a[401:], range(0, 299, 5))], end=["r0"])
    for trace in (traces.whole(requests), cut, both):
        results = replay(folders[name], name, dtype, trace, 1280)
        check(folders[name], dtype, requests, trace, results)


def test_windows_give_pages_back_while_latents_stay(folders):
    """A long request: the pages of the layers with a window are given back as it passes them, those of the latents stay."""
    from sprout_lm_amd.engine import ModelRunner, StepEntry
    name, dtype = "general", "float32"
    tokens = VH.random_tokens(VH.CONFIGS[name]["vocab"], 600, 900)
    runner = ModelRunner.from_folder(folders[name], dtype, block_size=16, num_blocks=48, max_sequences=1, prefix_caching=False)
    seq = runner.cache.create()
    want, done = VH.plain_logits(folders[name], dtype, tokens), 0
    for i in range(400):
        n = min((50, 1, 1, 33, 2, 70)[i % 6], 600 - done)
        if n == 0:
            break
        assert runner.cache.reserve(seq, done + n)
        got = runner.step([StepEntry(seq, tokens[done:done + n], list(range(n)))]).cpu().numpy()
        for j in range(n):
            assert np.abs(got[j] - want[done + j]).max() <= VH.tolerance(dtype, want[done + j]), f"position {done + j}"
        done += n
    kept = {group.spec.window: sum(page >= 0 for page in blocks) for group, blocks in zip(runner.cache.groups, seq.blocks)}
    assert kept[None] == 38 and kept[24] <= 3 and kept[100] <= 8, kept
    seq.release()


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_cuts_agree_with_each_other(folders, dtype):
    """Whole, token-by-token and portioned replays give the same logits beyond rounding."""
    name = "general"
    requests = requests_for(name, [90])
    rows_of = {}
    for family, trace in (("whole", traces.whole(requests)), ("tail", traces.tail_decoded(requests, tail=89)),
                          ("portions", traces.portions(requests))):
        results = replay(folders[name], name, dtype, trace, 256)
        rows_of[family] = {key: got[i] for expect, got in zip(trace.expected, results) for i, key in enumerate(expect)}
    bound = 1e-5 if dtype == "float32" else 3e-2
    for key, row in rows_of["whole"].items():
        for other in ("tail", "portions"):
            if key in rows_of[other]:
                assert np.abs(row - rows_of[other][key]).max() <= bound * max(1.0, np.abs(row).max()), (key, other)


def test_first_tokens_and_long_decoding(folders):
    """Positions 0, 1, 2, ... fed one by one from the very first token, 260 in a row."""
    from sprout_lm_amd.engine import ModelRunner, StepEntry
    for name, dtype in (("general", "float32"), ("odd", "float32"), ("states", "bfloat16")):
        tokens = VH.random_tokens(VH.CONFIGS[name]["vocab"], 260, 9)
        runner = ModelRunner.from_folder(folders[name], dtype, block_size=8, num_blocks=40, max_sequences=2,
                                         prefix_caching=False)
        seq = runner.cache.create()
        want = VH.plain_logits(folders[name], dtype, tokens)
        for p, token in enumerate(tokens):
            assert runner.cache.reserve(seq, p + 1)
            got = runner.step([StepEntry(seq, [token], [0])]).cpu().numpy()[0]
            assert np.abs(got - want[p]).max() <= VH.tolerance(dtype, want[p]), f"{name} {dtype} position {p}"
        seq.release()


def test_a_state_slot_starts_from_zero_again(folders):
    """A request that takes over the slot of a finished one computes what it computes on a fresh engine."""
    from sprout_lm_amd.engine import ModelRunner, StepEntry
    name, dtype = "states", "float32"
    runner = ModelRunner.from_folder(folders[name], dtype, block_size=8, num_blocks=16, max_sequences=1, prefix_caching=False)
    vocab = VH.CONFIGS[name]["vocab"]
    for seed in (1, 2, 3):
        tokens = VH.random_tokens(vocab, 50, seed)
        seq = runner.cache.create()
        assert seq.state_slot == 0 and runner.cache.reserve(seq, 50)
        got = runner.step([StepEntry(seq, tokens, [49])]).cpu().numpy()[0]
        want = VH.plain_logits(folders[name], dtype, tokens)[49]
        assert np.abs(got - want).max() <= VH.tolerance(dtype, want)
        seq.release()


def test_trace_replay_program_beside_the_plain_one(folders, tmp_path):
    """The replay program as a user runs it, on a model it picks by the folder's config.json, and the plain side of the same trace."""
    name, dtype = "odd", "float32"
    requests = requests_for(name, [33, 70, 20, 64, 45])
    trace = traces.mixed(requests, seed=3)
    pool = sum(sorted(-(-len(t) // 64) * 64 for t in requests.values())[-4:])
    out = tmp_path / "logits"
    proc = subprocess.Popen([sys.executable, os.path.join(ROOT, "bin", "trace_run"), "--model", folders[name],
                             "--dtype", dtype, "--out", str(out), "--max-tokens", str(pool)],
                            stdin=subprocess.PIPE, stdout=subprocess.PIPE, text=True, bufsize=1)
    try:
        for record in trace.steps:
            proc.stdin.write(json.dumps(record) + "\n")
            proc.stdin.flush()
            assert proc.stdout.readline().strip() == f"done {record['step']}"
        proc.stdin.close()
        assert proc.wait(timeout=60) == 0
    finally:
        if proc.poll() is None:
            proc.kill()
    vocab = VH.CONFIGS[name]["vocab"]
    results = [np.fromfile(out / f"{r['step']}.f32", dtype="<f4").reshape(len(rows), vocab) if rows else None
               for r, rows in zip(trace.steps, trace.expected)]
    check(folders[name], dtype, requests, trace, results)
    from tests.plain import trace_plain
    cfg, weights, logits_of = trace_plain.plain_side(folders[name], dtype)
    trace_plain.replay(cfg, weights, dtype, trace.steps[:6], str(tmp_path / "plain"), logits_of)
    for record, rows in zip(trace.steps[:6], trace.expected):
        if rows:
            theirs = np.fromfile(tmp_path / "plain" / f"{record['step']}.f32", dtype="<f4").reshape(len(rows), vocab)
            assert np.abs(theirs - results[record["step"]]).max() <= VH.tolerance(dtype, theirs)


# ---------------------------------------------------------------------------------------------- generation
def plain_greedy(folder, dtype, prompt, steps):
    history, out = list(prompt), []
    for _ in range(steps):
        token = int(np.argmax(VH.plain_logits(folder, dtype, history)[-1]))
        history.append(token)
        out.append(token)
    return out


def test_greedy_generation_through_the_entry_point(folders):
    """Prompts of 1 to 70 tokens in portions of 16, 20 greedy tokens each, float32: every token is the plain side's."""
    from sprout_lm_amd.engine import Engine
    for name in ("general", "odd", "states"):
        engine = Engine.from_folder(folders[name], "float32", block_size=VH.PAGE[name], num_blocks=64, max_sequences=4,
                                    max_batch_tokens=48, prefill_chunk_size=16, record_trace=True)
        vocab = VH.CONFIGS[name]["vocab"]
        prompts = [VH.random_tokens(vocab, n, 40 + i) for i, n in enumerate((1, 9, 40, 70))]
        outputs = engine.generate(prompts, max_new_tokens=20, ignore_eos=True)
        for prompt, got in zip(prompts, outputs):
            assert got == plain_greedy(folders[name], "float32", prompt, 20), f"{name}, prompt of {len(prompt)}"
        assert all(free == g.pool.num_pages for free, g in zip(engine.cache.free_pages(), engine.cache.groups))


def test_scheduling_never_changes_generation(folders):
    """Too few pages (preemption: the state slot is given back, then the prompt and what was generated are computed again
    from a cleared slot) and a late arrival give what each request generates alone."""
    from sprout_lm_amd.engine import Engine
    name, dtype = "wide", "float32"      # no layer has a window: pages are never given back
    vocab = VH.CONFIGS[name]["vocab"]
    prompts = {"A": VH.random_tokens(vocab, 33, 78), "B": VH.random_tokens(vocab, 29, 79),
               "C": VH.random_tokens(vocab, 40, 80), "D": VH.random_tokens(vocab, 3, 81)}
    want = {k: plain_greedy(folders[name], dtype, p, 14) for k, p in prompts.items()}
    for num_blocks, expect_preemption in ((64, False), (12, True)):
        engine = Engine.from_folder(folders[name], dtype, block_size=8, num_blocks=num_blocks, max_sequences=4,
                                    max_batch_tokens=24, prefill_chunk_size=16, record_trace=True)
        engine.add("A", prompts["A"], 14, ignore_eos=True)
        engine.step(); engine.step(); engine.step()
        for k in "BCD":
            engine.add(k, prompts[k], 14, ignore_eos=True)
        ticks = 0
        while engine.pending:
            ticks += 1
            assert ticks < 2000
            engine.step()
        for k in prompts:
            assert engine.result(k)["output"] == want[k], f"request {k} with {num_blocks} pages"
        assert any(e["type"] == "preempted" for e in engine.trace) == expect_preemption


def test_recorded_steps_equal_eager_steps(folders):
    """Steps replayed from recorded graphs (decoded tokens with the sampler inside, portions of recurring shapes) give
    the tokens of eagerly launched steps: the states go through the graphs' buffers unharmed."""
    from sprout_lm_amd.engine import Engine
    name = "general"
    vocab = VH.CONFIGS[name]["vocab"]
    prompts = [VH.random_tokens(vocab, n, 60 + i) for i, n in enumerate((7, 21, 3, 40, 12))]

    def run(use_graphs):
        engine = Engine.from_folder(folders[name], "float32", block_size=16, num_blocks=48, max_sequences=4,
                                    max_batch_tokens=32, prefill_chunk_size=16)
        engine.model.use_graphs = use_graphs
        engine.add("r0", prompts[0], 30, ignore_eos=True)
        engine.add("r1", prompts[1], 25, ignore_eos=True)
        steps = 0
        while engine.pending:
            steps += 1
            if steps == 6:
                engine.add("r2", prompts[2], 20, temperature=0.8, seed=5, ignore_eos=True)
            if steps == 15:
                engine.add("r3", prompts[3], 10, ignore_eos=True)
                engine.add("r4", prompts[4], 28, temperature=1.2, seed=9, ignore_eos=True)
            engine.step()
        replays = engine.model._graphs.replays if engine.model._graphs else 0
        return [engine.result(f"r{i}")["output"] for i in range(5)], replays

    eager, none = run(False)
    graphed, replays = run(True)
    assert none == 0 and replays > 40
    assert graphed == eager


def test_command_line_generates(folders):
    done = subprocess.run([sys.executable, "-m", "sprout_lm_amd", "generate", folders["general"], "--prompt-ids",
                           "3,1,4,1,5,9,2,6", "--dtype", "float32", "--ignore-eos"], cwd=ROOT,
                          env=dict(os.environ, MAX_NEW_TOKENS="6"), capture_output=True, text=True, timeout=120)
    assert done.returncode == 0, done.stderr
    final = json.loads(done.stdout.strip().splitlines()[-1])
    assert final["output"] == plain_greedy(folders["general"], "float32", [3, 1, 4, 1, 5, 9, 2, 6], 6)


def test_a_preset_written_to_a_folder_is_read_back(tmp_path):
    """Random weights written as a model folder (the command line's `init`): the folder's configuration is the preset's."""
    path = tmp_path / "preset.json"
    path.write_text(json.dumps(dict(VH.GENERAL, vocab=64)))
    folder = tmp_path / "model"
    done = subprocess.run([sys.executable, "-m", "sprout_lm_amd", "init", "--config", str(path), "--out", str(folder), "--seed", "3"],
                          cwd=ROOT, capture_output=True, text=True, timeout=120)
    assert done.returncode == 0, done.stderr
    import sprout_lm_amd as S
    assert S.load_config(str(folder)) == S.config_from_dict(dict(VH.GENERAL, vocab=64))
    tokens = VH.random_tokens(64, 20, 1)
    from sprout_lm_amd.engine import ModelRunner, StepEntry
    runner = ModelRunner.from_folder(str(folder), "float32", block_size=8, num_blocks=16, max_sequences=1)
    seq = runner.cache.create()
    assert runner.cache.reserve(seq, 20)
    got = runner.step([StepEntry(seq, tokens, [19])]).cpu().numpy()[0]
    config, weights = V.load_folder(str(folder))
    want = V.forward(weights, config, tokens)[19]
    assert np.abs(got - want).max() <= VH.tolerance("float32", want)
