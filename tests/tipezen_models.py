"""Small Tipezen configurations and weights for the tests: sizes that differ in every respect, weights drawn so that the
streams differ from one another and mix visibly, attention is peaked and its cap bends the largest scores, the denominator's
constant term takes a visible share, decays lie well inside (0, 1), and the gates and layer scales are neither 0 nor 1 (with
weights of N(0, 0.02) a key that is wrongly seen or a lost state would hardly move the logits).  The tensor names are written
out here, not taken from the engine."""
from __future__ import annotations

import json
import os

import torch

from easy_gpt.cpp_amd.weights import write_safetensors


def rotation(base, dims, scaling=None):
    r = {"base": base, "dims": dims}
    if scaling is not None:
        r["scaling"] = dict(zip(("factor", "original", "fast", "slow"), scaling))
    return r


def attention(heads, kv_heads, dim, vdim, scale, rot, window=None, softcap=None, v_mix=False):
    m = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale, "rot": rot, "v_mix": v_mix}
    if window:
        m["mask"] = {"size": window}
    if softcap:
        m["softcap"] = softcap
    return "attention", m


def retention(dim, vdim, decay, rot):
    return "retention", {"heads": len(decay), "dim": dim, "vdim": vdim, "decay": list(decay), "rot": rot}


def layer(mixer, ff):
    return {"type": mixer[0], "mixer": mixer[1], "mlp": None if ff is None else {"kind": "dense", "ff": ff}}


def config(vocab, width, eps, streams, layers):
    return {"architecture": "Tipezen", "vocab": vocab, "width": width, "norm": {"eps": eps}, "streams": streams, "layers": layers}


# both kinds of layer with and without a feed-forward; three attentions that mix values (the first of them the second layer);
# two streams; rotation over part of a head; windows of 12 and 33
CONFIG_A = config(300, 64, 1e-6, 2, [
    layer(retention(16, 24, (0.9, 0.97, 0.6), rotation(10000.0, 8)), 96),
    layer(attention(4, 2, 16, 24, 0.25, rotation(10000.0, 8, (4.0, 64, 8.0, 1.0)), 12, 5.0, True), 80),
    layer(attention(6, 2, 24, 24, 0.2, rotation(500.0, 24), 33, 8.0, True), None),
    layer(retention(20, 8, (0.95, 0.5), rotation(300.0, 20)), None),
    layer(attention(2, 2, 8, 24, 0.35, rotation(10000.0, 4), None, 4.0, True), 48),
])
# multiples of nothing: a width of 100, odd head sizes, no rotation, no window, no cap, no mixing; a window of one token;
# one stream; one query head per key/value head; a decay of zero and one of one; values of 70 and 14
CONFIG_B = config(257, 100, 1e-5, 1, [
    layer(attention(3, 3, 11, 13, 0.35, rotation(777.0, 10), 1, None, False), 50),
    layer(retention(10, 14, (0.8, 1.0, 0.0), rotation(1000.0, 6)), None),
    layer(attention(5, 1, 7, 9, 0.5, rotation(10000.0, 0), None, 6.0, False), 33),
    layer(retention(9, 70, (0.99,), rotation(50.0, 0)), 64),
    layer(attention(2, 1, 20, 17, 0.3, rotation(50.0, 6, (2.0, 20, 3.0, 0.5)), 700, None, True), 40),
])
# multiples of 16, so that the matrix-core attention runs: heads of 64 and 32, windows of 44 (no multiple of a page or of a
# chunk of keys) and of 64 (a page's and a chunk's edge); states of 64 x 80, 32 x 64 and 48 x 32; four streams
CONFIG_C = config(411, 128, 1e-6, 4, [
    layer(attention(8, 2, 64, 64, 0.1, rotation(500000.0, 32, (6.0, 256, 16.0, 2.0)), 44, 12.0, True), 192),
    layer(retention(64, 80, (0.7, 0.995), rotation(10000.0, 64)), 160),
    layer(attention(4, 2, 32, 64, 0.18, rotation(10000.0, 32), 64, 9.0, True), None),
    layer(retention(32, 64, (0.9, 0.97, 0.999), rotation(10000.0, 16)), None),
    layer(retention(48, 32, (0.98, 0.8), rotation(2e6, 48)), 96),
])
# retention alone; then attention alone (no state: every step may replay from a graph)
CONFIG_D = config(199, 96, 1e-5, 3, [
    layer(retention(16, 16, (0.5, 0.9, 0.998), rotation(10000.0, 16)), 80),
    layer(retention(40, 48, (0.96, 0.99), rotation(10000.0, 40)), None),
    layer(retention(8, 12, (0.7, 0.8, 0.9, 0.95), rotation(300.0, 2)), 64),
])
CONFIG_F = config(150, 72, 1e-5, 5, [
    layer(attention(2, 1, 16, 16, 0.3, rotation(10000.0, 16), 20, 7.0, True), 40),
    layer(attention(3, 1, 24, 16, 0.2, rotation(64.0, 2, (3.0, 100, 32.0, 1.0)), 7, 5.0, True), None),
    layer(attention(6, 3, 4, 12, 0.5, rotation(2e6, 4), None, 10.0, False), 56),
])
CONFIGS = {"A": (CONFIG_A, 5), "B": (CONFIG_B, 6), "C": (CONFIG_C, 7), "D": (CONFIG_D, 8), "F": (CONFIG_F, 10)}


def draw_weights(cfg: dict, seed: int, sharp: float = 2.0) -> dict[str, torch.Tensor]:
    """name -> float32 tensor whose values are bfloat16 numbers (so that both precisions load the same model)."""
    g = torch.Generator().manual_seed(seed)
    width, n = cfg["width"], cfg["streams"]

    def matrix(out_f, in_f, gain=1.0):
        return torch.randn(out_f, in_f, generator=g) * (gain / in_f ** 0.5)

    def gains(m):
        return 1.0 + 0.2 * torch.randn(m, generator=g)

    w = {"embed": torch.randn(cfg["vocab"], width, generator=g), "final.norm": gains(width), "head": matrix(cfg["vocab"], width, 2.0)}

    def connection(p, branch):
        w[f"{p}ls{branch}"] = 0.8 + 0.3 * torch.randn(width, generator=g)
        hc = f"{p}hc{branch}."
        w[hc + "in"] = (1.0 + 0.5 * torch.randn(n, generator=g)) / n
        w[hc + "out"] = 1.0 + 0.5 * torch.randn(n, generator=g)
        w[hc + "mix"] = 0.8 * torch.eye(n) + 0.2 / n + 0.1 * torch.randn(n, n, generator=g)

    for i, entry in enumerate(cfg["layers"]):
        p, m, q = f"l{i}.", entry["mixer"], f"l{i}.mix."
        w[p + "norm1"] = gains(width)
        connection(p, 1)
        nh, dim, vdim = m["heads"], m["dim"], m["vdim"]
        if entry["type"] == "attention":
            hk = m["kv_heads"]
            w[q + "q"], w[q + "k"], w[q + "v"] = matrix(nh * dim, width, sharp), matrix(hk * dim, width, 1.5), matrix(hk * vdim, width)
            w[q + "g"] = matrix(nh, width, 2.0)
            if m.get("v_mix"):
                w[q + "vmix"] = torch.tensor(0.3 + 0.1 * i)
        else:
            # keys lean towards the queries: with independent ones a state that holds few keys (a request's first tokens, a
            # small decay) may answer with a sum that nearly cancels, and the norm behind it makes a unit vector of what the
            # rounding left
            w[q + "q"] = matrix(nh * dim, width)
            w[q + "k"] = 0.8 * w[q + "q"] + matrix(nh * dim, width, 0.6)
            w[q + "v"], w[q + "g"] = matrix(nh * vdim, width), matrix(nh * vdim, width, 2.0)
        w[q + "o"] = matrix(width, nh * vdim)
        if entry.get("mlp") is None:
            continue
        ff = entry["mlp"]["ff"]
        w[p + "norm2"] = gains(width)
        connection(p, 2)
        w[p + "mlp.gate"], w[p + "mlp.up"], w[p + "mlp.down"] = matrix(ff, width, 2.0), matrix(ff, width), matrix(width, ff)
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
