"""Varunex as a plan of parts.

Tensor names: `embed`, `final.norm`, `final.norm.b`, `head`; layer i's start with `l<i>.`: `norm1`, `norm1.b`; the mixer's under
`mix.` (latent_attention: `dq`, `dq.norm`, `uq`, `dkv`, `dkv.norm`, `uk`, `uv`, `sink`, `g`, `o`; mlstm: `q`, `k`, `v`, `g`, `i`,
`i.b`, `f`, `f.b`, `norm`, `o`; attention: `q`, `k`, `v` with `.b`, `lq1`, `lk1`, `lq2`, `lk2`, `o`); the feed-forward's under
`mlp.` (`up`, `down`).
"""
from __future__ import annotations

from ..config.varunex import RotarySizes, VarunexConfig
from .plan import LayerPlan, ModelPlan, PartPlan, run_schedule

# The design gives no position limit; the engine's bookkeeping wants one.
MAX_POSITIONS = 1 << 22


def _norm(cfg: VarunexConfig, name: str, prefix: str = "") -> PartPlan:
    return PartPlan("norm", "layernorm", {"size": cfg.width, "eps": cfg.eps, "tensor": name, "bias": name + ".b"}, prefix)


def _position(rot: RotarySizes, size: int) -> PartPlan:
    if not rot.dims:
        return PartPlan("position", "none", {"head_dim": size})
    return PartPlan("position", "rotary_neox", {"head_dim": size, "theta": rot.base, "rotary_dim": rot.dims,
                                                "scaling": rot.scaling_dict()})


def _mixer(cfg: VarunexConfig, i: int, prefix: str) -> PartPlan:
    kind, m = cfg.layers[i].kind, cfg.layers[i].mixer
    if kind == "latent_attention":
        return PartPlan("mixer", "latent_attention", {
            "hidden": cfg.width, "heads": m.heads, "dim": m.dim, "rot_dim": m.rot_dim, "vdim": m.vdim, "kv_rank": m.kv_rank,
            "q_rank": m.q_rank, "scale": m.scale, "eps": cfg.eps, "position": _position(m.rot, m.rot_dim), "gated": True,
            "sinks": True}, prefix)
    if kind == "mlstm":
        return PartPlan("mixer", "mlstm", {"hidden": cfg.width, "heads": m.heads, "dim": m.dim, "vdim": m.vdim,
                                           "gate_cap": m.gate_cap, "eps": cfg.eps}, prefix)
    return PartPlan("mixer", "differential_attention", {
        "hidden": cfg.width, "heads": m.heads, "kv_heads": m.kv_heads, "dim": m.dim, "vdim": m.vdim, "scale": m.scale,
        "diff": m.diff, "eps": cfg.eps, "position": _position(m.rot, m.dim), "qkv_bias": True, "window": m.window}, prefix)


def _layer(cfg: VarunexConfig, i: int) -> LayerPlan:
    base = f"l{i}."
    parts = {"mixer_norm": _norm(cfg, "norm1", base), "mixer": _mixer(cfg, i, base + "mix.")}
    if cfg.layers[i].ff is not None:      # no norm of its own: it reads the mixer's
        parts["ffn"] = PartPlan("feed_forward", "mlp", {"hidden": cfg.width, "inner": cfg.layers[i].ff, "activation": "relu_squared",
                                                        "bias": None}, base + "mlp.")
    return LayerPlan("parallel", parts)


def build_varunex(cfg: VarunexConfig) -> ModelPlan:
    layers = [_layer(cfg, i) for i in range(len(cfg.layers))]
    return ModelPlan(
        architecture=cfg.architecture, config=cfg, hidden_size=cfg.width, vocab_size=cfg.vocab, max_positions=MAX_POSITIONS,
        eos_token_ids=(), embedding=PartPlan("embedding", "token_embedding", {"vocab": cfg.vocab, "hidden": cfg.width, "tensor": "embed"}),
        layers=layers, schedule=run_schedule(layers, range(len(layers))), final_norm=_norm(cfg, "final.norm"),
        head=PartPlan("head", "linear_head", {"vocab": cfg.vocab, "hidden": cfg.width, "tied": False, "tensor": "head"}))
