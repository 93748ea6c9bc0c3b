"""Varunex without a GPU: configuration, the plan's tensors and cache slots, and properties of the plain implementation."""
import copy
import math

import numpy as np
import pytest

import sprout_lm_amd as S
from sprout_lm_amd.cache.spec import PagedKVSpec, StateSpec
from sprout_lm_amd.config.base import ConfigError
from sprout_lm_amd.registry import build_model_plan
from tests import varunex_helpers as VH
from tests.plain import varunex_plain as V


@pytest.mark.parametrize("name", list(VH.CONFIGS))
def test_configuration_round_trip(name):
    cfg = S.config_from_dict(VH.CONFIGS[name])
    assert cfg.architecture == "Varunex"
    assert cfg.to_dict() == VH.CONFIGS[name]
    assert S.config_from_dict(cfg.to_dict()) == cfg


@pytest.mark.parametrize("path,value", [
    (("width",), 0), (("vocab",), True), (("norm", "eps"), -1.0), (("layers",), []), (("layers", 0, "type"), "delta"),
    (("layers", 0, "mlp", "kind"), "moe"), (("layers", 0, "mlp", "ff"), 0), (("layers", 0, "mixer", "kv_heads"), 4),
    (("layers", 0, "mixer", "rot", "dims"), 5), (("layers", 0, "mixer", "rot", "dims"), 8), (("layers", 0, "mixer", "mask", "size"), 0),
    (("layers", 0, "mixer", "rot", "scaling", "factor"), 0), (("layers", 0, "mixer", "rot", "scaling", "low"), 9.0),
    (("layers", 0, "mixer", "diff"), None), (("layers", 0, "mixer", "scale"), 0), (("layers", 1, "mixer", "q_rank"), 0),
    (("layers", 1, "mixer", "rot", "dims"), 8), (("layers", 2, "mixer", "gate_cap"), 0.0), (("layers", 2, "mixer"), None)])
def test_configuration_refusals(path, value):
    raw = copy.deepcopy(VH.ODD)
    at = raw
    for key in path[:-1]:
        at = at[key]
    at[path[-1]] = value
    with pytest.raises(ConfigError):
        S.config_from_dict(raw)


def test_plan_names_tensors_and_cache_slots():
    plan = build_model_plan(S.config_from_dict(VH.ODD))
    parts = plan.instantiate()
    expected = {name: tuple(spec.shape) for name, spec in parts.expected_tensors().items()}
    assert expected["l0.norm1"] == expected["l0.norm1.b"] == expected["final.norm.b"] == (100,)
    assert not any(".norm2" in name for name in expected)      # one norm a layer
    assert expected["l0.mix.q"] == (72, 100) and expected["l0.mix.q.b"] == (72,) and expected["l0.mix.k"] == (36, 100)
    assert expected["l0.mix.v"] == (30, 100) and expected["l0.mix.o"] == (100, 60) and expected["l0.mix.lk2"] == (6,)
    assert expected["l1.mix.dq"] == (9, 100) and expected["l1.mix.dq.norm"] == (9,) and expected["l1.mix.uq"] == (48, 9)
    assert expected["l1.mix.dkv"] == (26, 100) and expected["l1.mix.uk"] == (30, 20) and expected["l1.mix.uv"] == (42, 20)
    assert expected["l1.mix.sink"] == (3,) and expected["l1.mix.g"] == (3, 100) and "l1.mlp.up" not in expected
    assert expected["l2.mix.i"] == (3, 100) and expected["l2.mix.f.b"] == (3,) and expected["l2.mix.norm"] == (27,)
    assert expected["l2.mix.g"] == (27, 100) and expected["l2.mlp.up"] == (36, 100) and expected["l2.mlp.down"] == (100, 36)
    assert len([n for n in expected if n.startswith("l0.")]) == 2 + 11 + 2
    specs = parts.cache_slot_specs
    paged = [(s.kv_heads, s.head_dim, s.window) for s in specs if isinstance(s, PagedKVSpec)]
    assert paged == [(3, 16, 7), (1, 32, None), (2, 32, None), (1, 32, 1)]      # a key holds both maps; latents are padded
    assert [s.shape for s in specs if isinstance(s, StateSpec)] == [(3, 10, 7), (3,), (2, 23, 12), (2,)]
    assert not parts.prefix_sharing and parts.graph_safe and parts.graph_safe_portions
    pages_only = build_model_plan(S.config_from_dict(VH.WIDE)).instantiate()
    assert pages_only.prefix_sharing      # nothing but pages is kept: requests may share those of a common prefix


def test_sizes_that_are_refused():
    from sprout_lm_amd.parts import make_part
    none = make_part("position", "none", head_dim=4)
    for kind, good, bads in (
            ("mlstm", dict(hidden=8, heads=2, dim=4, vdim=4, gate_cap=5.0, eps=1e-5), (dict(gate_cap=0.0), dict(vdim=0), dict(dim=8000))),
            ("differential_attention", dict(hidden=8, heads=2, kv_heads=1, dim=4, vdim=4, scale=1.0, diff=0.1, eps=1e-5, position=none),
             (dict(kv_heads=3), dict(window=0), dict(dim=330), dict(position=make_part("position", "rotary_interleaved", rotary_dim=4, theta=9.0)))),
            ("latent_attention", dict(hidden=8, heads=2, dim=4, rot_dim=4, vdim=4, kv_rank=8, scale=1.0, eps=1e-5, position=none),
             (dict(q_rank=0), dict(kv_rank=0), dict(kv_rank=700), dict(position=make_part("position", "rotary_neox", head_dim=8, theta=9.0))))):
        make_part("mixer", kind, **good)
        for bad in bads:
            with pytest.raises(ConfigError):
                make_part("mixer", kind, **dict(good, **bad))


@pytest.mark.parametrize("dims,base,scaling", [(10, 30000.0, (6.0, 1.0, 5.0, 400.0)), (8, 100.0, (16.0, 0.5, 3.0, 60.0)), (6, 20.0, (2.0, 2.0, 2.0, 30.0)),
                                               (16, 1e6, None)])
def test_frequencies_blended_by_wavelength(dims, base, scaling):
    """The engine's table and the plain one, which decides by wavelength; short waves kept, long ones stretched."""
    from sprout_lm_amd.parts import make_part
    named = dict(zip(("factor", "low", "high", "original"), scaling)) if scaling else None
    part = make_part("position", "rotary_neox", head_dim=dims, theta=base, rotary_dim=dims, scaling=named)
    got, want = part.frequencies().numpy(), V.frequencies(dims, base, named)
    assert np.abs(got / want - 1.0).max() < 1e-12 and part.magnitude == 1.0
    if scaling:
        bare = V.frequencies(dims, base)
        length = 2 * math.pi / bare
        factor, low, high, original = scaling
        assert np.allclose(got[length < original / high], bare[length < original / high])
        assert np.allclose(got[length > original / low], bare[length > original / low] / factor)


# ---------------------------------------------------------------------------------------------- the plain implementation
def test_memory_by_hand():
    """One head of one number: gates that are wide open and a forget gate of one make S and n plain sums, scaled by the
    maximum; the floor exp(-m) counts while |n q| is small; a maximum starts at 0, so a weak first input stays weak."""
    ones = np.ones((3, 1, 1))
    i, f = np.full((3, 1), 2.0), np.zeros((3, 1))
    o, (S, n, m) = V.mlstm(ones, ones, ones * [[[1.0]], [[3.0]], [[5.0]]], i, f)
    assert np.allclose(m, 2.0) and np.allclose(S, 9.0) and np.allclose(n, 3.0)
    assert np.allclose(o[:, 0, 0], [1.0, 2.0, 3.0], rtol=1e-5)
    o, (S, n, m) = V.mlstm(ones[:1], ones[:1], ones[:1], np.full((1, 1), -4.0), np.zeros((1, 1)))
    assert np.allclose(m, 0.0) and np.allclose(n, math.exp(-4.0)) and np.allclose(o, math.exp(-4.0) / (1.0 + 1e-6))
    # a forget gate of almost nothing: only the last token is left
    o, (S, n, m) = V.mlstm(ones[:2], ones[:2], ones[:2] * [[[7.0]], [[2.0]]], np.zeros((2, 1)), np.full((2, 1), -50.0))
    assert np.allclose(o[1], 2.0, rtol=1e-5) and np.allclose(m, 0.0)


def test_memory_in_two_parts_is_the_whole():
    rng = np.random.default_rng(3)
    q, k, v = rng.standard_normal((20, 2, 5)), rng.standard_normal((20, 2, 5)), rng.standard_normal((20, 2, 7))
    i, f = rng.normal(0, 4, (20, 2)), -np.abs(rng.normal(0, 3, (20, 2)))
    whole, last = V.mlstm(q, k, v, i, f)
    first, state = V.mlstm(q[:9], k[:9], v[:9], i[:9], f[:9])
    second, end = V.mlstm(q[9:], k[9:], v[9:], i[9:], f[9:], state)
    assert np.allclose(np.concatenate([first, second]), whole) and all(np.allclose(a, b) for a, b in zip(last, end))


def test_softmax_with_a_sink_and_the_difference():
    mask = np.ones((1, 2), bool)
    w = V.softmax(np.array([[1.0, 3.0]]), mask, 2.0)
    e = np.exp([1.0, 3.0, 2.0])
    assert np.allclose(w[0], e[:2] / e.sum()) and np.allclose(V.softmax(np.array([[1.0, 3.0]]), mask).sum(), 1.0)
    weights = {"lq1": np.array([0.5]), "lk1": np.array([2.0]), "lq2": np.array([1.0]), "lk2": np.array([0.0])}
    assert abs(V.difference_factor(weights, "", 0.25) - (math.e - 1.0 + 0.25)) < 1e-12


@pytest.mark.parametrize("name", list(VH.CONFIGS))
def test_causality_and_every_constant_matters(name, tmp_path):
    folder = VH.make_folder(str(tmp_path), name)
    cfg, w = V.load_folder(folder)
    tokens = VH.random_tokens(cfg["vocab"], 40, 1)
    base = V.forward(w, cfg, tokens)
    changed = list(tokens)
    changed[30] = (changed[30] + 1) % cfg["vocab"]
    other = V.forward(w, cfg, changed)
    assert np.abs(other[:30] - base[:30]).max() < 1e-6 and np.abs(other[30:] - base[30:]).max() > 1e-3

    def differs(change):
        raw = copy.deepcopy(cfg)
        change(raw)
        return np.abs(V.forward(w, raw, tokens) - base).max() > 1e-5

    def scaled(*path):
        def change(raw):
            at = raw
            for key in path[:-1]:
                at = at[key]
            at[path[-1]] *= 1.5
        return change

    assert differs(scaled("norm", "eps")) or cfg["norm"]["eps"] < 1e-4
    for i, entry in enumerate(cfg["layers"]):
        m = entry["mixer"]
        if m.get("mask", {}).get("size") == 1:
            continue      # a softmax over one key is one, whatever its score
        for key in ("scale", "diff", "gate_cap"):
            if key in m:
                assert differs(scaled("layers", i, "mixer", key)), (i, key)
        if m.get("rot", {}).get("dims"):
            assert differs(scaled("layers", i, "mixer", "rot", "base")) or m["rot"]["dims"] == 2, i
            for key in m["rot"].get("scaling", {}):
                assert differs(scaled("layers", i, "mixer", "rot", "scaling", key)) or key in ("low", "high"), (i, key)
        if "mask" in m and m["mask"]["size"] < 39:
            def wider(raw, i=i):
                raw["layers"][i]["mixer"]["mask"]["size"] += 1
            assert differs(wider), i
