"""Tipezen decoder: typed configuration -> ModelSpec.

Tensor names: `embed`, `l<i>.norm1`, `l<i>.norm2`, `l<i>.mix.{q,k,v,g,o}` (attention that mixes values also `vmix`),
`l<i>.mlp.{gate,up,down}`, `l<i>.ls1`, `l<i>.ls2`, `l<i>.hc1.{in,out,mix}`, `l<i>.hc2.{in,out,mix}`, `final.norm`, `head`.

A layer is the pre-norm arrangement on several parallel residual streams, each branch with a factor per coordinate on
what it adds; its mixer is softmax attention (rotation of neighbouring pairs, a window, a cap on the scores, a constant
sink, a gate per head, values mixed with the first such layer's) or retention (rotation of the halves, a decay per head);
its feed-forward, if it has one, is the gated one with the tanh form of gelu.
"""
from __future__ import annotations

from ..config.registry import Architecture, register_architecture
from ..config.tipezen import TipezenConfig, TipezenLayer
from ..parts.spec import LayerSpec, ModelSpec, PartSpec, RunSpec

MAX_POSITION = 2**31 - 2        # the design names no longest sequence: positions are 32-bit integers
SINK_SCORE = 0.0                # the softmax's denominator holds one more term, exp(0) = 1


def _norm(prefix: str, name: str, eps: float) -> PartSpec:
    return PartSpec("rmsnorm", dict(eps=eps, name=name), prefix=prefix)


def _rotation(rot, kind: str) -> PartSpec | None:
    if rot is None:
        return None
    scaling = None if rot.factor is None else dict(factor=rot.factor, original=rot.original, fast=rot.fast, slow=rot.slow)
    return PartSpec(kind, dict(theta=rot.base, rotary_dim=rot.dims, scaling=scaling, exact_frequencies=True))


def _mixer_spec(layer: TipezenLayer, p: str, eps: float) -> PartSpec:
    m = layer.mixer
    if layer.type == "attention":
        return PartSpec(
            "normed_attention",
            dict(n_heads=m.heads, n_kv_heads=m.kv_heads, key_dim=m.dim, value_dim=m.vdim, scale=m.scale, eps=eps, window=m.window,
                 norm_queries_keys=False, position=_rotation(m.rotation, "rope_interleaved"), sink=SINK_SCORE, gated="heads",
                 softcap=m.softcap, mixes_values=m.mixes_values,
                 names=dict(q="q", k="k", v="v", o="o", gate="g", value_mix="vmix")),
            prefix=p)
    return PartSpec(
        "constant_decay_attention",
        dict(n_heads=m.heads, key_dim=m.dim, value_dim=m.vdim, decay=m.decay, eps=eps, activated=False,
             position=_rotation(m.rotation, "rope_half_split"), key_scale=m.dim ** -0.5, norm_heads=True, norm_weighted=False,
             gate_act="silu"),
        prefix=p)


def _layer_spec(layer: TipezenLayer, index: int, cfg: TipezenConfig) -> LayerSpec:
    p, eps = f"l{index}.", cfg.eps

    def connection(branch: int) -> PartSpec:
        hc = f"hc{branch}."
        return PartSpec("hyper_connection", dict(streams=cfg.streams, names=dict(read=hc + "in", write=hc + "out", mix=hc + "mix"),
                                                 scale_name=f"ls{branch}"), prefix=p)

    mixer = _mixer_spec(layer, p + "mix.", eps)
    norms, connections = {"mixer": _norm(p, "norm1", eps)}, {"mixer": connection(1)}
    if layer.ff is None:
        return LayerSpec(block="connected_mixer_only", mixer=mixer, feed_forward=None, norms=norms, connections=connections)
    norms["feed_forward"], connections["feed_forward"] = _norm(p, "norm2", eps), connection(2)
    ff = PartSpec("swiglu", dict(intermediate_size=layer.ff, activation="gelu_tanh", names=("gate", "up", "down"), unrounded=True),
                  prefix=p + "mlp.")
    return LayerSpec(block="connected", mixer=mixer, feed_forward=ff, norms=norms, connections=connections)


def tipezen_spec(cfg: TipezenConfig) -> ModelSpec:
    layers = tuple(_layer_spec(layer, i, cfg) for i, layer in enumerate(cfg.layers))
    runs = tuple(RunSpec(layer=i, cache=i) if layer.type == "attention" else RunSpec(layer=i, state=i)
                 for i, layer in enumerate(cfg.layers))
    return ModelSpec(
        hidden_size=cfg.width,
        vocab_size=cfg.vocab,
        max_position=MAX_POSITION,
        embedding=PartSpec("token_embedding_scaled", dict(scale=1.0, name="embed"), prefix=""),
        layers=layers,
        run_order=runs,
        final_norm=PartSpec("rmsnorm_stream_sum", dict(eps=cfg.eps, streams=cfg.streams, name="final.norm"), prefix=""),
        output_head=PartSpec("linear_head", dict(tied=False, name="head"), prefix=""),
    )


TIPEZEN = register_architecture(
    Architecture(name="Tipezen", config_class=TipezenConfig, build_spec=tipezen_spec, model_types=("tipezen",)),
    replace=True,
)
