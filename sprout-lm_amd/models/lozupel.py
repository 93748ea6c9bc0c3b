"""Lozupel as a plan of parts.

Tensor names: `embed`, `final.norm`, `head`, `loop.step` (what a pass over the repeated layers adds to the stream); layer
i's start with `l<i>.`: `norm1`, `norm2` (one number each); the mixer's under `mix.` (delta: `q`, `k`, `v` and their `.conv`,
`b`, `a`, `g`, `A_log`, `dt_bias`, `norm`, `o`; parallel: under `left.` `q`, `k`, `v`, `temp`, `pb`, `g`, `o`, `out`, under `right.`
the delta rule's with `a1`, `a2`, `g1`, `g2` for `a` and `g`, and `out`); the feed-forward's under `mlp.` (`gate`, `up`, `down`).
"""
from __future__ import annotations

from ..config.base import ConfigError
from ..config.lozupel import AttentionSizes, DeltaSizes, LozupelConfig
from .plan import LayerPlan, ModelPlan, PartPlan, run_schedule

# The design gives no position limit; the engine's bookkeeping wants one.
MAX_POSITIONS = 1 << 22


def _norm(cfg: LozupelConfig, tensor: str, prefix: str = "") -> PartPlan:
    return PartPlan("norm", "rmsnorm", {"size": cfg.width, "eps": cfg.eps, "tensor": tensor, "single": True}, prefix)


def _delta(cfg: LozupelConfig, m: DeltaSizes, **kind) -> PartPlan:
    return PartPlan("mixer", "gated_delta", {"hidden": cfg.width, "heads": m.heads, "kv_heads": m.kv_heads, "dim": m.dim,
                                             "vdim": m.vdim, "taps": m.conv, "eps": cfg.eps, **kind})


def _attention(cfg: LozupelConfig, m: AttentionSizes) -> PartPlan:
    position = PartPlan("position", "rotary_neox", {"head_dim": m.dim, "theta": m.rot_base, "rotary_dim": m.rot_dims}) \
        if m.rot_dims else PartPlan("position", "none", {"head_dim": m.dim})
    return PartPlan("mixer", "sink_attention", {
        "hidden": cfg.width, "heads": m.heads, "kv_heads": m.kv_heads, "dim": m.dim, "vdim": m.vdim, "scale": m.scale,
        "position": position, "window": m.window, "sinks": False, "head_gate": True, "sigmoid_weights": True, "temperature": True})


def _mixer(cfg: LozupelConfig, i: int, prefix: str) -> PartPlan:
    entry = cfg.layers[i]
    if entry.kind == "delta":
        plan = _delta(cfg, entry.mixer)
    else:
        right = entry.mixer.right
        if right.decay_rank is None or right.gate_rank is None:
            raise ConfigError(f"Layer {i} of a Lozupel model: neither its configuration (mixer.right.decay_rank, gate_rank) nor a "
                              f"checkpoint (the shapes of l{i}.mix.right.a1 and g1) gives the ranks of its two-matrix projections.")
        plan = PartPlan("mixer", "side_by_side", {
            "hidden": cfg.width, "eps": cfg.eps, "factor": 0.5, "left": _attention(cfg, entry.mixer.left),
            "right": _delta(cfg, right, decay="channel", gate="sigmoid", decay_rank=right.decay_rank, gate_rank=right.gate_rank)})
    plan.prefix = prefix
    return plan


def _layer(cfg: LozupelConfig, i: int) -> LayerPlan:
    base = f"l{i}."
    parts = {"mixer_norm": _norm(cfg, "norm1", base), "mixer": _mixer(cfg, i, base + "mix.")}
    if cfg.layers[i].ff is not None:
        parts["ffn_norm"] = _norm(cfg, "norm2", base)
        parts["ffn"] = PartPlan("feed_forward", "gated_mlp", {"hidden": cfg.width, "inner": cfg.layers[i].ff, "activation": "gelu_tanh",
                                                              "tensors": ("gate", "up", "down")}, base + "mlp.")
    return LayerPlan("pre_norm", parts)


def _entry(cfg: LozupelConfig, t: int) -> LayerPlan:
    """Pass t's place ahead of the repeated layers: the embedding (from the second pass on) and the pass's vector join the
    stream."""
    return LayerPlan("stream_entry", {"entry": PartPlan("stream", "pass_entry", {
        "size": cfg.width, "passes": cfg.loop.times, "index": t, "embedding": t > 0}, "loop.")})


def _run_order(cfg: LozupelConfig) -> list[int]:
    """Layer numbers in the order in which they run; pass t's entry is number len(layers) + t."""
    n, loop = len(cfg.layers), cfg.loop
    if loop is None:
        return list(range(n))
    order = list(range(loop.start))
    for t in range(loop.times):
        order += [n + t] + list(range(loop.start, loop.stop))
    return order + list(range(loop.stop, n))


def build_lozupel(cfg: LozupelConfig) -> ModelPlan:
    layers = [_layer(cfg, i) for i in range(len(cfg.layers))]
    if cfg.loop is not None:
        layers += [_entry(cfg, t) for t in range(cfg.loop.times)]
    return ModelPlan(
        architecture=cfg.architecture, config=cfg, hidden_size=cfg.width, vocab_size=cfg.vocab, max_positions=MAX_POSITIONS,
        eos_token_ids=(), embedding=PartPlan("embedding", "token_embedding", {"vocab": cfg.vocab, "hidden": cfg.width,
                                                                              "tensor": "embed", "scale": cfg.embedding_scale}),
        layers=layers, schedule=run_schedule(layers, _run_order(cfg)), final_norm=_norm(cfg, "final.norm"),
        head=PartPlan("head", "linear_head", {"vocab": cfg.vocab, "hidden": cfg.width, "tied": False, "tensor": "head",
                                              "softcap": cfg.logit_softcap}))
