"""Karesun decoder: typed configuration -> ModelSpec.

Tensor names: `embed`, `pos`, `l<i>.norm1`, `l<i>.norm2`, `l<i>.mix.{q,k,v,lq1,lk1,lq2,lk2,o}` (without `k`, `v` where the layer
reads another's keys and values), `l<i>.mlp.*` (dense: `up`, `down`; experts: `e<j>.{gate,up,down}`, `router`, `correction`),
`final.norm`, `head`.

A layer is the pre-norm arrangement with RMS norms whose weights are stored as their distance from one; its mixer is window
attention without rotation whose heads are the difference of two maps with capped scores; its feed-forward is dense with a
squared relu, or a mixture of gated experts chosen within groups, some of which are the identity.
"""
from __future__ import annotations

from ..config.karesun import KaresunConfig, KaresunLayer
from ..config.registry import Architecture, register_architecture
from ..parts.spec import LayerSpec, ModelSpec, PartSpec, RunSpec


def _norm(prefix: str, name: str, eps: float) -> PartSpec:
    return PartSpec("rmsnorm", dict(eps=eps, name=name, weight_offset=1.0), prefix=prefix)


def _layer_spec(layer: KaresunLayer, p: str, eps: float) -> LayerSpec:
    m, f = layer.mixer, layer.mlp
    mixer = PartSpec(
        "normed_attention",
        dict(n_heads=m.heads, n_kv_heads=m.kv_heads, key_dim=m.dim, value_dim=m.vdim, scale=m.scale, eps=eps, window=m.window,
             norm_queries_keys=False, softcap=m.softcap, difference=m.diff, shares_cache=m.kv_from is not None,
             names=dict(q="q", k="k", v="v", o="o", lambda_q1="lq1", lambda_k1="lk1", lambda_q2="lq2", lambda_k2="lk2")),
        prefix=p + "mix.")
    norms = {"mixer": _norm(p, "norm1", eps)}
    if f is None:
        return LayerSpec(block="pre_norm_mixer_only", mixer=mixer, feed_forward=None, norms=norms)
    norms["feed_forward"] = _norm(p, "norm2", eps)
    if f.kind == "dense":
        ff = PartSpec("activated", dict(intermediate_size=f.ff, activation="relu2", names=("up", "down")), prefix=p + "mlp.")
    else:
        ff = PartSpec("expert_mixture",
                      dict(n_experts=f.experts, top=f.top, intermediate_size=f.ff, router_bias=False, routing="softmax_all",
                           weight_scale=f.scale, identities=f.identities, groups=f.groups, keep_groups=f.keep_groups, normalized=False),
                      prefix=p + "mlp.")
    return LayerSpec(block="pre_norm", mixer=mixer, feed_forward=ff, norms=norms)


def karesun_spec(cfg: KaresunConfig) -> ModelSpec:
    runs = []
    for i, layer in enumerate(cfg.layers):
        src = layer.mixer.kv_from
        runs.append(RunSpec(layer=i, cache=i if src is None else src, writes_cache=src is None))
    return ModelSpec(
        hidden_size=cfg.width,
        vocab_size=cfg.vocab,
        max_position=cfg.max_positions,
        embedding=PartSpec("token_embedding_positions",
                           dict(max_positions=cfg.max_positions, name="embed", position_name="pos", scale=cfg.embedding_scale,
                                any_stream=True), prefix=""),
        layers=tuple(_layer_spec(layer, f"l{i}.", cfg.eps) for i, layer in enumerate(cfg.layers)),
        run_order=tuple(runs),
        final_norm=_norm("", "final.norm", cfg.eps),
        output_head=PartSpec("linear_head", dict(tied=False, name="head"), prefix=""),
    )


KARESUN = register_architecture(
    Architecture(name="Karesun", config_class=KaresunConfig, build_spec=karesun_spec, model_types=("karesun",)),
    replace=True,
)
