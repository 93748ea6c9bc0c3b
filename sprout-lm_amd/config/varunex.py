"""Configuration of the Varunex decoder: a list of parallel layers under one norm whose mixers are latent attention with query
latents and sinks, a matrix memory with exponential gates, or differential attention."""
from __future__ import annotations

import math
from dataclasses import dataclass
from typing import Any, ClassVar, Mapping

from .base import ConfigError, ModelConfig, positive_float, positive_int

_WHAT = "Invalid Varunex config: "


def _section(raw: Mapping, key: str, where: str, optional: bool = False):
    value = raw.get(key)
    if value is None and optional:
        return None
    if not isinstance(value, Mapping):
        raise ConfigError(f"{_WHAT}{where}{key} must be an object, got {value!r}.")
    return value


def _count(raw: Mapping, key: str, where: str, least: int = 1) -> int:
    value = raw.get(key)
    if isinstance(value, bool) or not isinstance(value, int) or value < least:
        raise ConfigError(f"{_WHAT}{where}{key} must be an integer of at least {least}, got {value!r}.")
    return value


def _number(raw: Mapping, key: str, where: str, positive: bool = True) -> float:
    value = raw.get(key)
    if isinstance(value, bool) or not isinstance(value, (int, float)) or not math.isfinite(value) or (positive and value <= 0):
        raise ConfigError(f"{_WHAT}{where}{key} must be a {'positive ' if positive else ''}finite number, got {value!r}.")
    return float(value)


@dataclass(frozen=True)
class RotarySizes:
    """scaling: (factor, low, high, original) of frequencies blended by wavelength, or None."""

    dims: int
    base: float
    scaling: tuple | None

    KEYS: ClassVar[tuple[str, ...]] = ("factor", "low", "high", "original")

    @classmethod
    def parse(cls, raw: Mapping, where: str, most: int) -> "RotarySizes":
        dims = _count(raw, "dims", where, 0)
        if dims % 2 or dims > most:
            raise ConfigError(f"{_WHAT}{where}dims must be even and at most {most}, got {dims}.")
        scaling = _section(raw, "scaling", where, optional=True)
        if scaling is not None:
            scaling = tuple(_number(scaling, key, where + "scaling.") for key in cls.KEYS)
            if scaling[1] > scaling[2]:
                raise ConfigError(f"{_WHAT}{where}scaling.low {scaling[1]} exceeds scaling.high {scaling[2]}.")
        return cls(dims, _number(raw, "base", where), scaling)

    def scaling_dict(self) -> dict | None:
        return None if self.scaling is None else dict(zip(self.KEYS, self.scaling))

    def to_dict(self) -> dict:
        out = {"base": self.base, "dims": self.dims}
        if self.scaling is not None:
            out["scaling"] = self.scaling_dict()
        return out


@dataclass(frozen=True)
class LatentSizes:
    """Latent attention: queries through q_rank numbers, keys and values through kv_rank and a turned part of rot_dim."""

    heads: int
    dim: int
    rot_dim: int
    vdim: int
    q_rank: int
    kv_rank: int
    scale: float
    rot: RotarySizes

    @classmethod
    def parse(cls, raw: Mapping, where: str) -> "LatentSizes":
        rot_dim = _count(raw, "rot_dim", where, 0)
        return cls(_count(raw, "heads", where), _count(raw, "dim", where), rot_dim, _count(raw, "vdim", where),
                   _count(raw, "q_rank", where), _count(raw, "kv_rank", where), _number(raw, "scale", where),
                   RotarySizes.parse(_section(raw, "rot", where), where + "rot.", rot_dim))

    def to_dict(self) -> dict:
        return {"dim": self.dim, "heads": self.heads, "kv_rank": self.kv_rank, "q_rank": self.q_rank, "rot": self.rot.to_dict(),
                "rot_dim": self.rot_dim, "scale": self.scale, "vdim": self.vdim}


@dataclass(frozen=True)
class MemorySizes:
    """The matrix memory with exponential gates."""

    heads: int
    dim: int
    vdim: int
    gate_cap: float

    @classmethod
    def parse(cls, raw: Mapping, where: str) -> "MemorySizes":
        return cls(*(_count(raw, key, where) for key in ("heads", "dim", "vdim")), _number(raw, "gate_cap", where))

    def to_dict(self) -> dict:
        return {"dim": self.dim, "gate_cap": self.gate_cap, "heads": self.heads, "vdim": self.vdim}


@dataclass(frozen=True)
class DifferenceSizes:
    """Differential attention.  window None: every earlier key is seen."""

    heads: int
    kv_heads: int
    dim: int
    vdim: int
    scale: float
    diff: float
    rot: RotarySizes
    window: int | None

    @classmethod
    def parse(cls, raw: Mapping, where: str) -> "DifferenceSizes":
        heads, kv_heads, dim, vdim = (_count(raw, k, where) for k in ("heads", "kv_heads", "dim", "vdim"))
        if heads % kv_heads:
            raise ConfigError(f"{_WHAT}{where}heads {heads} are no whole multiple of kv_heads {kv_heads}.")
        mask = _section(raw, "mask", where, optional=True)
        return cls(heads, kv_heads, dim, vdim, _number(raw, "scale", where), _number(raw, "diff", where, positive=False),
                   RotarySizes.parse(_section(raw, "rot", where), where + "rot.", dim),
                   None if mask is None else _count(mask, "size", where + "mask."))

    def to_dict(self) -> dict:
        out = {"diff": self.diff, "dim": self.dim, "heads": self.heads, "kv_heads": self.kv_heads, "rot": self.rot.to_dict(),
               "scale": self.scale, "vdim": self.vdim}
        if self.window is not None:
            out["mask"] = {"size": self.window}
        return out


_MIXERS = {"latent_attention": LatentSizes, "mlstm": MemorySizes, "attention": DifferenceSizes}


@dataclass(frozen=True)
class VarunexLayer:
    kind: str                        # a key of _MIXERS
    mixer: object
    ff: int | None                   # None for a layer without feed-forward

    def to_dict(self) -> dict:
        return {"mixer": self.mixer.to_dict(), "mlp": None if self.ff is None else {"ff": self.ff, "kind": "dense"}, "type": self.kind}


@dataclass(frozen=True)
class VarunexConfig(ModelConfig):
    """Every size and constant of a Varunex model, as config.json gives them; nothing has a default."""

    architecture: ClassVar[str] = "Varunex"

    vocab: int
    width: int
    eps: float
    layers: tuple[VarunexLayer, ...]

    @property
    def vocab_size(self) -> int:
        return self.vocab

    @property
    def hidden_size(self) -> int:
        return self.width

    @classmethod
    def from_dict(cls, raw: Mapping[str, Any]) -> "VarunexConfig":
        if not isinstance(raw, Mapping):
            raise ConfigError(_WHAT + "expected a JSON object.")
        if raw.get("architecture") != cls.architecture:
            raise ConfigError(f"Not a Varunex config: architecture is {raw.get('architecture')!r}.")
        vocab, width = positive_int(raw, "vocab"), positive_int(raw, "width")
        eps = positive_float(_section(raw, "norm", ""), "eps")
        entries = raw.get("layers")
        if not isinstance(entries, list) or not entries:
            raise ConfigError(_WHAT + "layers must be a non-empty list.")
        layers = []
        for i, entry in enumerate(entries):
            where = f"layers[{i}]."
            if not isinstance(entry, Mapping):
                raise ConfigError(f"{_WHAT}layers[{i}] must be an object.")
            kind = entry.get("type")
            if kind not in _MIXERS:
                raise ConfigError(f"{_WHAT}{where}type {kind!r} is no mixer of this design {tuple(_MIXERS)}.")
            mixer = _MIXERS[kind].parse(_section(entry, "mixer", where), where + "mixer.")
            mlp = _section(entry, "mlp", where, optional=True)
            if mlp is not None and mlp.get("kind") != "dense":
                raise ConfigError(f"{_WHAT}{where}mlp.kind must be 'dense', got {mlp.get('kind')!r}.")
            layers.append(VarunexLayer(kind, mixer, None if mlp is None else _count(mlp, "ff", where + "mlp.")))
        return cls(vocab, width, eps, tuple(layers))

    def to_dict(self) -> dict:
        return {"architecture": self.architecture, "layers": [layer.to_dict() for layer in self.layers],
                "norm": {"eps": self.eps}, "vocab": self.vocab, "width": self.width}
