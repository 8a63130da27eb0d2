"""Small Karesun configurations and weights for the tests: sizes that differ in every respect, weights drawn so that attention
is peaked and its cap bends the largest scores, the second map takes a visible share that differs from layer to layer, norm
weights stand well away from one, and the router's scores are spread (with weights of N(0, 0.02) a key that is wrongly seen would
hardly move the logits).  The tensor names are written out here, not taken from the engine."""
from __future__ import annotations

import json
import os

import torch

from easy_gpt.cpp_amd.weights import write_safetensors


def mixer(heads, kv_heads, dim, vdim, scale, diff, window=None, softcap=None, kv_from=None):
    m = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale, "diff": diff}
    if window:
        m["mask"] = {"size": window}
    if softcap:
        m["softcap"] = softcap
    if kv_from is not None:
        m["kv_from"] = kv_from
    return m


def dense(ff):
    return {"kind": "dense", "ff": ff}


def moe(ff, experts, top, scale=1.0, identity=0, groups=None):
    r = {"experts": experts, "top": top, "scale": scale, "identity": identity}
    if groups:
        r["groups"] = {"count": groups[0], "keep": groups[1]}
    return {"kind": "moe", "expert": {"ff": ff}, "router": r}


def config(vocab, width, max_positions, eps, scale, layers):
    return {"architecture": "Karesun", "vocab": vocab, "width": width, "max_positions": max_positions, "norm": {"eps": eps},
            "embedding": {"scale": scale}, "layers": [{"type": "attention", "mixer": m, "mlp": f} for m, f in layers]}


# every kind of layer; two layers read the first one's keys and values through windows that are narrower and wider than its own
CONFIG_A = config(300, 64, 300, 1e-6, 1.5, [
    (mixer(4, 2, 16, 24, 0.25, 0.4, 12, 5.0), dense(96)),
    (mixer(4, 2, 16, 24, 0.3, 0.2, 7, 8.0, kv_from=0), moe(40, 6, 2, 1.7, 2, (4, 2))),
    (mixer(6, 3, 8, 16, 0.35, 0.6, 33, 6.0), None),
    (mixer(2, 2, 16, 24, 0.2, 0.75, 21, 12.0, kv_from=0), moe(24, 5, 4, 0.8)),
    (mixer(6, 3, 8, 16, 0.4, 0.1, 5, 9.0, kv_from=2), dense(56)),
])
# multiples of nothing: a width of 100, odd map and value sizes, no window, no cap, a window of one token; one query head per
# key/value head; identity experts alone in a group; one group; values of 70
CONFIG_B = config(257, 100, 1000, 1e-5, 0.7, [
    (mixer(3, 3, 11, 13, 0.35, 0.3, 1, None), dense(50)),
    (mixer(5, 1, 7, 70, 0.5, 0.5, None, 6.0), moe(33, 7, 3, 2.2, 2, (3, 2))),
    (mixer(5, 1, 7, 70, 0.4, 0.0, 17, 4.0, kv_from=1), moe(10, 3, 1, 1.0, 1, (1, 1))),
    (mixer(2, 1, 20, 17, 0.3, 0.9, 700, None), None),
    (mixer(3, 3, 11, 13, 0.3, 0.45, None, 3.0, kv_from=0), dense(41)),
])
# multiples of 16, so that the matrix-core attention runs: maps of 64, 32, 24 and 16, windows of 44 (no multiple of a page or of a
# chunk of keys) and of 64 (a page's and a chunk's edge), a reader whose window is wider than the writer's
CONFIG_C = config(411, 128, 1200, 1e-6, 2.0, [
    (mixer(8, 2, 64, 64, 0.1, 0.35, 44, 12.0), dense(192)),
    (mixer(4, 2, 32, 64, 0.18, 0.6, 64, 9.0), moe(64, 12, 4, 2.0, 4, (4, 2))),
    (mixer(8, 2, 64, 64, 0.12, 0.2, 100, 7.0, kv_from=0), moe(48, 6, 2, 1.2, 2, (2, 1))),
    (mixer(6, 1, 24, 96, 0.2, 0.5, None, 10.0), dense(160)),
    (mixer(4, 2, 16, 48, 0.25, 0.15, 64, None), None),
])
# one kind of layer alone: experts without groups or identities, and every layer on the first one's keys
CONFIG_D = config(199, 96, 700, 1e-5, 1.0, [
    (mixer(6, 2, 16, 32, 0.25, 0.5, 40, 8.0), moe(32, 4, 4, 0.6)),
    (mixer(6, 2, 16, 32, 0.25, 0.5, 40, 8.0, kv_from=0), moe(32, 4, 3, 0.6)),
    (mixer(6, 2, 16, 32, 0.25, 0.5, 40, 8.0, kv_from=0), moe(32, 4, 1, 0.9)),
])
# dense layers alone: no router, so that bfloat16 has no close call
CONFIG_F = config(211, 192, 900, 1e-5, 1.2, [
    (mixer(6, 2, 32, 48, 0.12, 0.25, 70, 9.0), dense(264)),
    (mixer(6, 2, 32, 48, 0.15, 0.5, 33, 14.0, kv_from=0), dense(304)),
    (mixer(3, 1, 9, 21, 0.3, 0.6, 48, 6.0), dense(100)),
])
CONFIGS = {"A": (CONFIG_A, 5), "B": (CONFIG_B, 6), "C": (CONFIG_C, 7), "D": (CONFIG_D, 8), "F": (CONFIG_F, 10)}


def draw_weights(cfg: dict, seed: int, sharp: float = 2.0) -> dict[str, torch.Tensor]:
    """name -> float32 tensor whose values are bfloat16 numbers (so that both precisions load the same model)."""
    g = torch.Generator().manual_seed(seed)
    width = cfg["width"]

    def matrix(out_f, in_f, gain=1.0):
        return torch.randn(out_f, in_f, generator=g) * (gain / in_f ** 0.5)

    def around_zero(m):
        return 0.25 * torch.randn(m, generator=g)

    w = {"embed": torch.randn(cfg["vocab"], width, generator=g), "pos": 0.5 * torch.randn(cfg["max_positions"], width, generator=g),
         "final.norm": around_zero(width), "head": matrix(cfg["vocab"], width, 2.0)}
    for i, entry in enumerate(cfg["layers"]):
        p, m, q = f"l{i}.", entry["mixer"], f"l{i}.mix."
        nh, hk, dim, vdim = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
        w[p + "norm1"] = around_zero(width)
        w[q + "q"] = matrix(nh * 2 * dim, width, sharp)
        if m.get("kv_from") is None:
            w[q + "k"], w[q + "v"] = matrix(hk * 2 * dim, width, 1.5), matrix(hk * vdim, width)
        # the exponents' sums lie around 0.25 - 0.15 i and -0.1: lambda is some tenths for every layer and never near 1.  With a
        # lambda of 1 and one key in sight (a request's first token) the maps' difference would vanish, and the norm behind it
        # make a unit vector of what the rounding left
        w[q + "lq1"], w[q + "lq2"] = 1.0 + 0.3 * torch.randn(dim, generator=g), 1.0 + 0.3 * torch.randn(dim, generator=g)
        w[q + "lk1"] = (0.25 - 0.15 * i + 0.1 * torch.randn(dim, generator=g)) / dim
        w[q + "lk2"] = (-0.1 + 0.1 * torch.randn(dim, generator=g)) / dim
        w[q + "o"] = matrix(width, nh * vdim)
        f = entry.get("mlp")
        if f is None:
            continue
        w[p + "norm2"] = around_zero(width)
        if f["kind"] == "dense":
            w[p + "mlp.up"], w[p + "mlp.down"] = matrix(f["ff"], width), matrix(width, f["ff"])
            continue
        r, ff = f["router"], f["expert"]["ff"]
        for e in range(r["experts"]):
            pe = f"{p}mlp.e{e}."
            w[pe + "gate"], w[pe + "up"], w[pe + "down"] = matrix(ff, width, 2.0), matrix(ff, width), matrix(width, ff)
        outputs = r["experts"] + r.get("identity", 0)
        w[p + "mlp.router"] = matrix(outputs, width, 1.5)
        # corrections as large as the scores, some negative: the choice is often another than by the scores alone
        w[p + "mlp.correction"] = 0.3 * torch.randn(outputs, generator=g)
    return {k: v.to(torch.bfloat16).to(torch.float32) for k, v in w.items()}


def write_model(model_dir: str, cfg: dict, seed: int, change=None, **kw) -> str:
    """Writes config.json and model.safetensors (bfloat16); `change(weights)` may edit the drawn tensors first."""
    os.makedirs(model_dir, exist_ok=True)
    with open(os.path.join(model_dir, "config.json"), "w") as f:
        json.dump(cfg, f)
    w = draw_weights(cfg, seed, **kw)
    if change is not None:
        change(w)
    write_safetensors(os.path.join(model_dir, "model.safetensors"), {k: v.to(torch.bfloat16) for k, v in w.items()})
    return model_dir
