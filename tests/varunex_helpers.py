"""Tiny Varunex configurations, model folders with weights of the tests' own making, and the plain side's logits."""
from __future__ import annotations

import copy
import os

import numpy as np

from tests.kodezen_helpers import random_tokens, tolerance, write_folder  # noqa: F401
from tests.plain import varunex_plain as V


def rot(dims, base, scaling=None):
    """`scaling`: (factor, low, high, original) or None."""
    out = {"dims": dims, "base": base}
    if scaling is not None:
        out["scaling"] = dict(zip(("factor", "low", "high", "original"), scaling))
    return out


def latent(heads, dim, rot_dim, vdim, q_rank, kv_rank, scale, turn):
    return {"type": "latent_attention", "mixer": {"heads": heads, "dim": dim, "rot_dim": rot_dim, "vdim": vdim, "q_rank": q_rank,
                                                  "kv_rank": kv_rank, "scale": scale, "rot": turn}}


def memory(heads, dim, vdim, cap):
    return {"type": "mlstm", "mixer": {"heads": heads, "dim": dim, "vdim": vdim, "gate_cap": cap}}


def difference(heads, kv_heads, dim, vdim, scale, diff, turn, window=None):
    m = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale, "diff": diff, "rot": turn}
    if window is not None:
        m["mask"] = {"size": window}
    return {"type": "attention", "mixer": m}


def layer(mix, ff=None):
    out = copy.deepcopy(mix)
    out["mlp"] = None if ff is None else {"kind": "dense", "ff": ff}
    return out


def model(width, vocab, layers, eps=1e-5):
    return {"architecture": "Varunex", "vocab": vocab, "width": width, "norm": {"eps": eps}, "layers": layers}


# no size in whole eights; windows of one key, of seven and none; heads that turn in part, whole and not at all; frequencies
# that are blended and that are not; keys wider and narrower than values; several query heads over one key head; no feed-forward
ODD = model(100, 77, [
    layer(difference(6, 3, 6, 10, 0.4, 0.2, rot(4, 50.0, (3.0, 0.5, 6.0, 40.0)), 7), 28),
    layer(latent(3, 10, 6, 14, 9, 20, 0.3, rot(6, 30.0))),
    layer(memory(3, 7, 9, 6.0), 36),
    layer(difference(2, 2, 12, 5, 0.3, 0.7, rot(0, 10.0)), 20),
    layer(memory(2, 12, 22, 3.0)),
    layer(difference(3, 1, 5, 18, 0.5, -0.1, rot(2, 10.0), 1), 12),
], eps=1e-3)
# sizes the matrix-core kernels take; four query heads over one key head; a latent whose keys are 64 wide
GENERAL = model(128, 300, [
    layer(latent(4, 16, 16, 32, 64, 48, 0.2, rot(16, 1000.0, (8.0, 1.0, 4.0, 64.0))), 96),
    layer(difference(4, 1, 16, 32, 0.3, 0.35, rot(8, 250.0), 24), 64),
    layer(memory(3, 32, 56, 10.0), 64),
    layer(difference(4, 2, 32, 64, 0.2, 0.5, rot(32, 5000.0, (4.0, 1.0, 4.0, 128.0)), 100), 80),
    layer(memory(2, 16, 40, 15.0), 48),
], eps=1e-6)
# the memory alone: a model whose requests hold no pages, only state slots
STATES = model(64, 150, [layer(memory(2, 16, 24, 8.0), 64), layer(memory(1, 48, 16, 2.0))])
# every layer sees every earlier key; a latent whose keys no matrix-core size fits, more heads than a block of the one-query
# kernel holds, no rotated part at all
WIDE = model(96, 211, [
    layer(latent(20, 8, 24, 8, 40, 112, 0.15, rot(24, 100.0)), 64),
    layer(latent(2, 24, 0, 16, 16, 32, 0.2, rot(0, 10.0)), 32),
    layer(difference(2, 1, 40, 24, 0.15, 0.1, rot(24, 300.0)), 32),
])

CONFIGS = {"odd": ODD, "general": GENERAL, "states": STATES, "wide": WIDE}
PAGE = {"odd": 16, "general": 16, "states": 8, "wide": 4}
SEED = {"odd": 54, "general": 55, "states": 56, "wide": 57}


def random_array(rng, name: str, shape) -> np.ndarray:
    """Values for the tensor `name` by the last pieces of its name: the table N(0, 1), matrices N(0, 0.1), norm weights around
    one, biases N(0, 0.3), forget gates' biases N(2, 2), sinks N(1, 1.5), the vectors of the difference's factor N(0, 0.2), gates'
    matrices N(0, 0.05): where one token drowns all others, what a head reads is that token's value times the SIGN of k . q, and
    a sign near zero is any rounding's to turn."""
    pieces = name.split(".")
    last = pieces[-1]
    if name == "embed":
        return rng.normal(0.0, 1.0, shape)
    if last == "b":
        return rng.normal(2.0, 2.0, shape) if pieces[-2] == "f" else rng.normal(0.0, 0.3, shape)
    if last in ("norm1", "norm"):
        return 1.0 + rng.normal(0.0, 0.1, shape)
    if last == "sink":
        return rng.normal(1.0, 1.5, shape)
    if last in ("lq1", "lk1", "lq2", "lk2"):
        return rng.normal(0.0, 0.2, shape)
    if last in ("i", "f"):
        return rng.normal(0.0, 0.05, shape)
    return rng.normal(0.0, 0.1, shape)


def random_weights(cfg: dict, seed: int) -> dict:
    """name -> float32 array for every tensor the configuration needs (shapes asked from the engine's plan, values the
    tests' own), rounded to what bfloat16 holds."""
    import sprout_lm_amd as S
    from sprout_lm_amd.registry import build_model_plan
    expected = build_model_plan(S.config_from_dict(cfg)).expected_tensors()
    rng = np.random.default_rng(seed)
    out = {}
    for name in sorted(expected):
        shape = tuple(expected[name].shape)
        out[name] = V.bf16_round(np.asarray(random_array(rng, name, shape), dtype=np.float32)).reshape(shape)
    return out


def make_folder(root: str, name: str) -> str:
    folder = os.path.join(root, "varunex_" + name)
    if not os.path.exists(os.path.join(folder, "model.safetensors")):
        write_folder(folder, CONFIGS[name], random_weights(CONFIGS[name], SEED[name]))
    return folder


_MODELS: dict = {}
_LOGITS: dict = {}


def plain_logits(folder: str, dtype: str, tokens) -> np.ndarray:
    """The plain implementation's logits at every position of `tokens`."""
    key = (folder, dtype, tuple(tokens))
    if key not in _LOGITS:
        if folder not in _MODELS:
            _MODELS[folder] = V.load_folder(folder)
        cfg, w = _MODELS[folder]
        _LOGITS[key] = V.forward(w, cfg, list(tokens), store=V.bf16_round if dtype == "bfloat16" else V.f32)
    return _LOGITS[key]
