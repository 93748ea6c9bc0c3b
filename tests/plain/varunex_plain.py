"""Plain Varunex forward pass: whole sequence, no cache, float64 arithmetic, one function per mechanism.

Shares no code with the engine.  `store` is an optional rounding function applied wherever the bfloat16 engine keeps a
tensor in bfloat16 (normed activations, projection outputs, what enters an output projection); with the default
(float32 rounding) everything is float32 storage over float64 sums.  What the design computes in 32 bits (angles,
scores and weights, norms, the gates and the state of the recurrence, the residual sum) is never rounded by `store`.

Notation.  x: the residual stream [tokens, width], x = embed[token] before the first layer.  A layer reads its norm once,
  h = ln(x),  x <- x + (mixer(h) + ff(h))        (the feed-forward may be absent),
  ln(x) = (x - mean x) / sqrt(mean (x - mean x)^2 + eps) * w + b.
Mixers:
  "latent_attention"  queries come through a latent of q_rank numbers, keys and values through one of kv_rank that is kept
                      beside one turned key part shared by all heads; the softmax's denominator has a learned term per
                      head; a gate per head on the output.
  "mlstm"             per head a matrix S [dim, vdim] and a vector n [dim], fed through exponential gates that a running
                      maximum m keeps in range; what is read is divided by |n . q|.
  "attention"         two softmax maps per head over the same values; the second is taken off with one learned factor;
                      grouped heads, a window, biases, angles with blended frequencies.
Feed-forward: W_down relu(W_up h)^2.  Logits: head ln(x).
"""
from __future__ import annotations

import math

import numpy as np

from tests.plain.kodezen_plain import bf16_round, f32, linear, load_folder, rms  # noqa: F401


# ---------------------------------------------------------------------------------------------- small functions
def sigmoid(x):
    return 0.5 * (1.0 + np.tanh(0.5 * np.asarray(x, dtype=np.float64)))


def layer_norm(x, w, b, eps):
    x = np.asarray(x, dtype=np.float64)
    d = x - np.mean(x, axis=-1, keepdims=True)
    return d / np.sqrt(np.mean(d * d, axis=-1, keepdims=True) + eps) * np.asarray(w, dtype=np.float64) + np.asarray(b, dtype=np.float64)


def frequencies(dims: int, base: float, scaling=None):
    """The angle per position of every pair.  `scaling`: long wavelengths are stretched by `factor`, short ones kept, and
    between original / high and original / low the two are mixed in proportion to original / wavelength."""
    f = float(base) ** (-2.0 * np.arange(dims // 2) / dims) if dims else np.zeros(0)
    if not scaling:
        return f
    original, low, high, factor = (float(scaling[k]) for k in ("original", "low", "high", "factor"))
    out = []
    for one in f:
        length = 2.0 * math.pi / one
        if length < original / high:
            out.append(one)
        elif length > original / low:
            out.append(one / factor)
        else:
            s = (original / length - low) / (high - low)
            out.append((1.0 - s) * one / factor + s * one)
    return np.array(out)


def turn_halves(x, positions, freq):
    """Number i of the last axis turns with number i + len(freq), by position * freq[i]; x [T, heads, numbers]."""
    out = np.array(x, dtype=np.float64)
    half = len(freq)
    if half == 0:
        return out
    angle = np.asarray(positions, dtype=np.float64)[:, None] * freq[None, :]
    cos, sin = np.cos(angle)[:, None, :], np.sin(angle)[:, None, :]
    u, v = out[..., :half].copy(), out[..., half:2 * half].copy()
    out[..., :half] = u * cos - v * sin
    out[..., half:2 * half] = v * cos + u * sin
    return out


def in_window(T: int, size):
    """[T, T] mask: query i sees key j."""
    i, j = np.arange(T)[:, None], np.arange(T)[None, :]
    return (j <= i) & (i - j < (T if size is None else size))


def softmax(scores, mask, sink=None):
    """Weights of the visible keys; `sink`: a term of the denominator that has no key."""
    s = np.where(mask, scores, -np.inf)
    top = np.max(s, axis=-1, keepdims=True)
    if sink is not None:
        top = np.maximum(top, sink)
    e = np.exp(s - top)
    return e / (np.sum(e, axis=-1, keepdims=True) + (0.0 if sink is None else np.exp(sink - top)))


# ---------------------------------------------------------------------------------------------- mixers
def latent_attention(w, pre: str, m, h, positions, eps, store=f32):
    T = h.shape[0]
    H, D, R, V, K = m["heads"], m["dim"], m["rot_dim"], m["vdim"], m["kv_rank"]
    freq = frequencies(m["rot"]["dims"], m["rot"]["base"], m["rot"].get("scaling"))
    c_q = store(rms(store(linear(h, w[pre + "dq"])), eps) * np.asarray(w[pre + "dq.norm"], dtype=np.float64))
    q = store(linear(c_q, w[pre + "uq"])).reshape(T, H, D + R)
    q_turned = store(turn_halves(q[..., D:], positions, freq))
    down = store(linear(h, w[pre + "dkv"]))
    c = store(rms(down[:, :K], eps) * np.asarray(w[pre + "dkv.norm"], dtype=np.float64))
    k_turned = store(turn_halves(down[:, None, K:], positions, freq))[:, 0]
    k = store(linear(c, w[pre + "uk"])).reshape(T, H, D)
    v = store(linear(c, w[pre + "uv"])).reshape(T, H, V)
    gate = sigmoid(store(linear(h, w[pre + "g"])))
    mask = in_window(T, None)
    out = np.zeros((T, H, V))
    for n in range(H):
        score = (q[:, n, :D] @ k[:, n].T + q_turned[:, n] @ k_turned.T) * float(m["scale"])
        out[:, n] = softmax(score, mask, float(np.asarray(w[pre + "sink"])[n])) @ v[:, n] * gate[:, n:n + 1]
    return linear(store(out.reshape(T, H * V)), w[pre + "o"])


def mlstm_gates(h, w, pre: str, cap: float):
    """(log input gate, log forget gate) [T, heads]."""
    squash = lambda name: cap * np.tanh(linear(h, w[pre + name], w[pre + name + ".b"]) / cap)
    return squash("i"), -np.logaddexp(0.0, -squash("f"))


def mlstm(q, k, v, i, f, state=None):
    """o [T, heads, vdim] and the last (S, n, m).  q, k [T, heads, dim], v [T, heads, vdim], gates [T, heads]."""
    T, H, D = q.shape
    S, n, m = state if state is not None else (np.zeros((H, D, v.shape[-1])), np.zeros((H, D)), np.zeros(H))
    out = np.zeros((T, H, v.shape[-1]))
    for t in range(T):
        top = np.maximum(f[t] + m, i[t])
        keep, take = np.exp(f[t] + m - top), np.exp(i[t] - top)
        S = keep[:, None, None] * S + take[:, None, None] * k[t][:, :, None] * v[t][:, None, :]
        n = keep[:, None] * n + take[:, None] * k[t]
        m = top
        share = np.maximum(np.abs(np.einsum("hd,hd->h", n, q[t])), np.exp(-m)) + 1e-6
        out[t] = np.einsum("hdv,hd->hv", S, q[t]) / share[:, None]
    return out, (S, n, m)


def mlstm_mixer(w, pre: str, m, h, eps, store=f32):
    T = h.shape[0]
    H, D, V = m["heads"], m["dim"], m["vdim"]
    q = store(linear(h, w[pre + "q"])).reshape(T, H, D) * D ** -0.5
    k = store(linear(h, w[pre + "k"])).reshape(T, H, D)
    v = store(linear(h, w[pre + "v"])).reshape(T, H, V)
    i, f = mlstm_gates(h, w, pre, float(m["gate_cap"]))
    o, _ = mlstm(q, k, v, i, f)
    o = rms(o, eps).reshape(T, H * V) * np.asarray(w[pre + "norm"], dtype=np.float64)
    return linear(store(o * sigmoid(store(linear(h, w[pre + "g"])))), w[pre + "o"])


def difference_factor(w, pre: str, diff: float) -> float:
    dot = lambda a, b: float(np.dot(np.asarray(w[pre + a], dtype=np.float64), np.asarray(w[pre + b], dtype=np.float64)))
    return math.exp(dot("lq1", "lk1")) - math.exp(dot("lq2", "lk2")) + diff


def differential_attention(w, pre: str, m, h, positions, eps, store=f32):
    T = h.shape[0]
    H, G, D, V, diff = m["heads"], m["kv_heads"], m["dim"], m["vdim"], float(m["diff"])
    freq = frequencies(m["rot"]["dims"], m["rot"]["base"], m["rot"].get("scaling"))
    project = lambda name: store(linear(h, w[pre + name], w[pre + name + ".b"]))
    q = store(turn_halves(project("q").reshape(T, H * 2, D), positions, freq)).reshape(T, H, 2, D)
    k = store(turn_halves(project("k").reshape(T, G * 2, D), positions, freq)).reshape(T, G, 2, D)
    v = project("v").reshape(T, G, V)
    mask = in_window(T, m["mask"]["size"] if m.get("mask") else None)
    factor = difference_factor(w, pre, diff)
    out = np.zeros((T, H, V))
    for n in range(H):
        g = n // (H // G)
        a1, a2 = (softmax((q[:, n, s] @ k[:, g, s].T) * float(m["scale"]), mask) @ v[:, g] for s in (0, 1))
        out[:, n] = rms(a1 - factor * a2, eps) * (1.0 - diff)
    return linear(store(out.reshape(T, H * V)), w[pre + "o"])


# ---------------------------------------------------------------------------------------------- feed-forward
def dense_ff(w, pre: str, h, store=f32):
    return linear(store(np.maximum(linear(h, w[pre + "up"]), 0.0) ** 2), w[pre + "down"])


# ---------------------------------------------------------------------------------------------- the model
def forward(w, cfg, tokens, store=f32, rows=None, streams=None):
    """Logits [len(rows) or T, vocab] of the whole sequence.  `streams`: a list that receives x after every layer."""
    eps = float(cfg["norm"]["eps"])
    x = np.asarray(w["embed"], dtype=np.float64)[np.asarray(tokens)]
    positions = np.arange(len(tokens))
    for i, layer in enumerate(cfg["layers"]):
        pre, m = f"l{i}.", layer["mixer"]
        h = store(layer_norm(x, w[pre + "norm1"], w[pre + "norm1.b"], eps))
        if layer["type"] == "latent_attention":
            mixed = latent_attention(w, pre + "mix.", m, h, positions, eps, store)
        elif layer["type"] == "mlstm":
            mixed = mlstm_mixer(w, pre + "mix.", m, h, eps, store)
        elif layer["type"] == "attention":
            mixed = differential_attention(w, pre + "mix.", m, h, positions, eps, store)
        else:
            raise ValueError(layer["type"])
        x = x + (mixed + (dense_ff(w, pre + "mlp.", h, store) if layer.get("mlp") else 0.0))
        if streams is not None:
            streams.append(x.copy())
    if rows is not None:
        x = x[np.asarray(rows)]
    return linear(store(layer_norm(x, w["final.norm"], w["final.norm.b"], eps)), w["head"]).astype(np.float32)
