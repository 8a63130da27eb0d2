"""Typed configuration of the Tipezen decoder, read from its config.json keys.

A Tipezen config.json names the design in `architecture` and gives `vocab`, `width`, `norm.eps`, `streams` (the number of
parallel residual streams) and `layers`: a list with one entry per layer, each with `type`, `mixer` and `mlp` (null for no
feed-forward, or kind 'dense' with ff).  The mixers by type:

  attention   heads, kv_heads (absent: heads), dim, vdim, scale, softcap (absent: no cap), mask.size (no mask: every earlier
              token), rot.{base, dims, scaling.{factor, original, fast, slow} or none}, v_mix (absent: false)
  retention   heads, dim, vdim, decay[heads], rot.{base, dims}
"""
from __future__ import annotations

from dataclasses import dataclass
from typing import Any, Mapping

from .base import ConfigError, KeyReader
from .pekasun import RotationConfig


def _object(data: Mapping[str, Any], key: str, where: str, required: bool = True):
    v = data.get(key)
    if v is None:
        if required:
            raise ConfigError(f"{where}: required key '{key}' (an object) is missing")
        return None
    if not isinstance(v, Mapping):
        raise ConfigError(f"{where}: '{key}' must be an object{'' if required else ' or null'}")
    return v


def _rotation(data: Mapping[str, Any], where: str, dim: int, stretched: bool) -> RotationConfig | None:
    raw = _object(data, "rot", where, required=False)
    if raw is None:
        return None
    rot = RotationConfig.from_dict(raw, where + ".rot")
    if rot.dims > dim:
        raise ConfigError(f"{where}.rot: 'dims' ({rot.dims}) is larger than the head size {dim}")
    if rot.factor is not None and not stretched:
        raise ConfigError(f"{where}.rot: this mixer's rotation has no 'scaling'")
    return rot if rot.dims > 0 else None


@dataclass(frozen=True)
class CappedAttentionConfig:
    """`window` None: every earlier token; `softcap` None: scores are not capped."""

    heads: int
    kv_heads: int
    dim: int
    vdim: int
    scale: float
    softcap: float | None
    window: int | None
    rotation: RotationConfig | None
    mixes_values: bool

    @classmethod
    def from_dict(cls, data: Mapping[str, Any], where: str) -> "CappedAttentionConfig":
        r = KeyReader(data, where)
        heads = r.integer("heads", minimum=1)
        kv_heads = r.integer("kv_heads", heads, minimum=1)
        if heads % kv_heads:
            raise ConfigError(f"{where}: 'heads' ({heads}) must be a multiple of 'kv_heads' ({kv_heads})")
        dim = r.integer("dim", minimum=1)
        mask = _object(data, "mask", where, required=False)
        window = None if mask is None else KeyReader(mask, where + ".mask").integer("size", minimum=1)
        return cls(heads, kv_heads, dim, r.integer("vdim", minimum=1), r.number("scale"), r.number("softcap", None, positive=True),
                   window, _rotation(data, where, dim, stretched=True), r.boolean("v_mix", False))


@dataclass(frozen=True)
class RetentionConfig:
    heads: int
    dim: int
    vdim: int
    decay: tuple[float, ...]
    rotation: RotationConfig | None

    @classmethod
    def from_dict(cls, data: Mapping[str, Any], where: str) -> "RetentionConfig":
        r = KeyReader(data, where)
        heads = r.integer("heads", minimum=1)
        dim = r.integer("dim", minimum=1)
        raw = data.get("decay")
        if not isinstance(raw, list) or len(raw) != heads or any(isinstance(v, bool) or not isinstance(v, (int, float)) for v in raw):
            raise ConfigError(f"{where}: 'decay' must be a list of {heads} numbers, one per head")
        return cls(heads, dim, r.integer("vdim", minimum=1), tuple(float(v) for v in raw), _rotation(data, where, dim, stretched=False))


@dataclass(frozen=True)
class TipezenLayer:
    type: str                    # 'attention' or 'retention'
    mixer: CappedAttentionConfig | RetentionConfig
    ff: int | None               # the inner width of the feed-forward; None: the layer has none


MIXER_TYPES = {"attention": CappedAttentionConfig, "retention": RetentionConfig}


@dataclass(frozen=True)
class TipezenConfig:
    architecture: str
    vocab: int
    width: int
    eps: float
    streams: int
    layers: tuple[TipezenLayer, ...]

    @classmethod
    def from_dict(cls, data: Mapping[str, Any], where: str = "config.json") -> "TipezenConfig":
        r = KeyReader(data, where)
        architecture = r.string("architecture")
        eps = KeyReader(_object(data, "norm", where), where + ".norm").number("eps", positive=True)
        raw = data.get("layers")
        if not isinstance(raw, list) or not raw:
            raise ConfigError(f"{where}: required key 'layers' (a list of layers) is missing or empty")
        layers: list[TipezenLayer] = []
        first = None                 # the first layer that mixes values
        for i, entry in enumerate(raw):
            at = f"{where}.layers[{i}]"
            if not isinstance(entry, Mapping):
                raise ConfigError(f"{at}: must be an object")
            kind = KeyReader(entry, at).string("type", check=lambda v: v in MIXER_TYPES)
            m = MIXER_TYPES[kind].from_dict(_object(entry, "mixer", at), at + ".mixer")
            if getattr(m, "mixes_values", False):
                if first is None:
                    first = (i, m)
                elif (m.kv_heads, m.vdim) != (first[1].kv_heads, first[1].vdim):
                    raise ConfigError(f"{at}.mixer: values of {m.kv_heads} heads of {m.vdim} cannot be mixed with layer {first[0]}'s "
                                      f"{first[1].kv_heads} heads of {first[1].vdim}")
            mlp = _object(entry, "mlp", at, required=False)
            ff = None
            if mlp is not None:
                mk = KeyReader(mlp, at + ".mlp")
                mk.string("kind", check=lambda v: v == "dense")
                ff = mk.integer("ff", minimum=1)
            layers.append(TipezenLayer(kind, m, ff))
        return cls(architecture, r.integer("vocab", minimum=1), r.integer("width", minimum=1), eps, r.integer("streams", minimum=1),
                   tuple(layers))
