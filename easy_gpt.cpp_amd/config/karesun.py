"""Typed configuration of the Karesun decoder, read from its config.json keys.

A Karesun config.json names the design in `architecture` and gives `vocab`, `width`, `max_positions` (the rows of the learned
position table), `norm.eps`, `embedding.scale` (absent: 1) and `layers`: a list with one entry per layer, each with `type`
('attention'), `mixer` (heads, kv_heads (absent: heads), dim: the size of one of a head's two maps, vdim, scale, diff, softcap
(absent: no cap), mask.size (no mask: every earlier token), and kv_from: the layer whose keys and values it reads instead of
making its own) and `mlp` (null for no feed-forward; kind 'dense' with ff; or kind 'moe' with expert.ff and router.{experts,
top, scale (absent: 1), identity (absent: 0), groups.{count, keep} or no groups}).
"""
from __future__ import annotations

from dataclasses import dataclass
from typing import Any, Mapping

from .base import ConfigError, KeyReader


def _object(data: Mapping[str, Any], key: str, where: str, required: bool = True):
    v = data.get(key)
    if v is None:
        if required:
            raise ConfigError(f"{where}: required key '{key}' (an object) is missing")
        return None
    if not isinstance(v, Mapping):
        raise ConfigError(f"{where}: '{key}' must be an object{'' if required else ' or null'}")
    return v


@dataclass(frozen=True)
class DifferentialAttentionConfig:
    """`window` None: every earlier token; `softcap` None: scores are not capped; `kv_from` None: keys and values of its own."""

    heads: int
    kv_heads: int
    dim: int                     # the size of one map's query and key; a head has two
    vdim: int
    scale: float
    diff: float
    softcap: float | None
    window: int | None
    kv_from: int | None

    @classmethod
    def from_dict(cls, data: Mapping[str, Any], where: str) -> "DifferentialAttentionConfig":
        r = KeyReader(data, where)
        heads = r.integer("heads", minimum=1)
        kv_heads = r.integer("kv_heads", heads, minimum=1)
        if heads % kv_heads:
            raise ConfigError(f"{where}: 'heads' ({heads}) must be a multiple of 'kv_heads' ({kv_heads})")
        mask = _object(data, "mask", where, required=False)
        window = None if mask is None else KeyReader(mask, where + ".mask").integer("size", minimum=1)
        return cls(heads, kv_heads, r.integer("dim", minimum=1), r.integer("vdim", minimum=1), r.number("scale"), r.number("diff"),
                   r.number("softcap", None, positive=True), window, r.integer("kv_from", None, minimum=0))


@dataclass(frozen=True)
class FeedForwardConfig:
    kind: str                    # 'dense' or 'moe'
    ff: int                      # inner width (of one expert for 'moe')
    experts: int = 0             # experts with tensors
    top: int = 0
    scale: float = 1.0
    identities: int = 0          # router outputs behind them that hand on their input
    groups: int = 1              # experts and identity experts together form this many groups of neighbours
    keep_groups: int = 1

    @classmethod
    def from_dict(cls, data: Mapping[str, Any], where: str) -> "FeedForwardConfig":
        kind = KeyReader(data, where).string("kind", check=lambda v: v in ("dense", "moe"))
        if kind == "dense":
            return cls(kind, KeyReader(data, where).integer("ff", minimum=1))
        at = where + ".router"
        raw = _object(data, "router", where)
        router = KeyReader(raw, at)
        experts, top, identities = router.integer("experts", minimum=1), router.integer("top", minimum=1), router.integer("identity", 0, minimum=0)
        outputs = experts + identities
        groups = keep = 1
        parts = _object(raw, "groups", at, required=False)
        if parts is not None:
            g = KeyReader(parts, at + ".groups")
            groups, keep = g.integer("count", minimum=1), g.integer("keep", minimum=1)
            if outputs % groups:
                raise ConfigError(f"{at}.groups: 'count' ({groups}) must divide the {outputs} experts and identity experts")
            if keep > groups:
                raise ConfigError(f"{at}.groups: 'keep' ({keep}) is larger than 'count' ({groups})")
        if top > outputs // groups * keep:
            raise ConfigError(f"{at}: 'top' ({top}) is larger than the {outputs // groups * keep} experts that can be chosen")
        ff = KeyReader(_object(data, "expert", where), where + ".expert").integer("ff", minimum=1)
        return cls(kind, ff, experts, top, router.number("scale", 1.0), identities, groups, keep)


@dataclass(frozen=True)
class KaresunLayer:
    mixer: DifferentialAttentionConfig
    mlp: FeedForwardConfig | None


@dataclass(frozen=True)
class KaresunConfig:
    architecture: str
    vocab: int
    width: int
    max_positions: int
    eps: float
    embedding_scale: float
    layers: tuple[KaresunLayer, ...]

    @classmethod
    def from_dict(cls, data: Mapping[str, Any], where: str = "config.json") -> "KaresunConfig":
        r = KeyReader(data, where)
        architecture = r.string("architecture")
        eps = KeyReader(_object(data, "norm", where), where + ".norm").number("eps", positive=True)
        embedding = _object(data, "embedding", where, required=False)
        scale = 1.0 if embedding is None else KeyReader(embedding, where + ".embedding").number("scale", 1.0)
        raw = data.get("layers")
        if not isinstance(raw, list) or not raw:
            raise ConfigError(f"{where}: required key 'layers' (a list of layers) is missing or empty")
        layers: list[KaresunLayer] = []
        for i, entry in enumerate(raw):
            at = f"{where}.layers[{i}]"
            if not isinstance(entry, Mapping):
                raise ConfigError(f"{at}: must be an object")
            KeyReader(entry, at).string("type", check=lambda v: v == "attention")
            m = DifferentialAttentionConfig.from_dict(_object(entry, "mixer", at), at + ".mixer")
            if m.kv_from is not None:
                src = layers[m.kv_from].mixer if m.kv_from < i else None
                if src is None or src.kv_from is not None:
                    raise ConfigError(f"{at}.mixer: 'kv_from' ({m.kv_from}) must name an earlier layer with keys and values of its own")
                if (src.kv_heads, src.dim, src.vdim) != (m.kv_heads, m.dim, m.vdim):
                    raise ConfigError(f"{at}.mixer: kv_heads, dim and vdim must equal those of layer {m.kv_from}, whose keys and values it reads")
            mlp = _object(entry, "mlp", at, required=False)
            layers.append(KaresunLayer(m, None if mlp is None else FeedForwardConfig.from_dict(mlp, at + ".mlp")))
        return cls(architecture, r.integer("vocab", minimum=1), r.integer("width", minimum=1), r.integer("max_positions", minimum=1),
                   eps, scale, tuple(layers))
