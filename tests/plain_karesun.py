"""A plain, slow Karesun decoder: whole sequences, no cache, one function per mechanism, float64 on the CPU.

It shares no code with the engine: it reads a model folder with its own few lines and knows the tensor names
itself.  Notation: x [T, W] is the residual stream of one sequence, positions count from 0, a linear weight is
[out, in] and applied as x W^T.

The design: x = scale * embed[token] + pos[position]; a layer is pre-norm, x <- x + mixer(N1(x)), x <- x + ff(N2(x)), with
RMS norms whose weights are stored as the distance from one.  The mixer is a differential attention behind a sliding window:
a head has two query/key maps over the same values, each a softmax of its own over capped scores, and what goes on is the
first map's output minus lambda times the second's, divided by its root mean square and multiplied by 1 - diff; such a layer
may read another layer's keys and values.  The feed-forward is dense with a squared relu, or a mixture of gated experts
that are chosen within groups, some of which hand their input on as it is.  A last norm and the output matrix.
"""
from __future__ import annotations

import json
import math
import os
import struct

import numpy as np
import torch

F64 = torch.float64


def read_safetensors(path: str) -> dict[str, torch.Tensor]:
    with open(path, "rb") as f:
        raw = f.read()
    (hlen,) = struct.unpack("<Q", raw[:8])
    header = json.loads(raw[8 : 8 + hlen])
    base = 8 + hlen
    out = {}
    for name, info in header.items():
        if name == "__metadata__":
            continue
        b, e = info["data_offsets"]
        buf = raw[base + b : base + e]
        if info["dtype"] == "F32":
            a = torch.from_numpy(np.frombuffer(buf, dtype="<f4").copy())
        elif info["dtype"] == "BF16":
            u16 = np.frombuffer(buf, dtype="<u2").astype(np.uint32) << 16
            a = torch.from_numpy(u16.view(np.float32).copy())
        else:
            raise ValueError(info["dtype"])
        out[name] = a.reshape(info["shape"]).to(F64)
    return out


def read_model(model_dir: str):
    with open(os.path.join(model_dir, "config.json")) as f:
        cfg = json.load(f)
    return cfg, read_safetensors(os.path.join(model_dir, "model.safetensors"))


# ----------------------------------------------------------------------------- norms
def unit_rms(x, eps):
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def offset_norm(x, weight, eps):
    """The weight is stored as its distance from one."""
    return unit_rms(x, eps) * (1.0 + weight)


# ----------------------------------------------------------------------------- differential attention
def capped_window_map(q, k, v, scale, softcap=None, window=None):
    """One map: q [T, heads, d], k [T, kv heads, d], v [T, kv heads, dv] -> [T, heads, dv].  Query head h reads key/value
    head h // (heads / kv heads); a score is softcap * tanh(q.k scale / softcap); key j is seen if 0 <= i - j < window."""
    t, nq, _ = q.shape
    nkv = k.shape[1]
    i, j = torch.arange(t)[:, None], torch.arange(t)[None, :]
    seen = j <= i
    if window is not None:
        seen = seen & (i - j < window)
    heads = []
    for head in range(nq):
        g = head // (nq // nkv)
        s = (q[:, head] @ k[:, g].T) * scale
        if softcap is not None:
            s = softcap * torch.tanh(s / softcap)
        heads.append(torch.softmax(s.masked_fill(~seen, -math.inf), dim=-1) @ v[:, g])
    return torch.stack(heads, dim=1)


def map_weight(w, p, diff):
    """lambda, the factor on the second map's output: one number for the layer."""
    return float(torch.exp((w[p + "lq1"] * w[p + "lk1"]).sum()) - torch.exp((w[p + "lq2"] * w[p + "lk2"]).sum()) + diff)


def two_maps(q, k, v, scale, softcap, window, lam, diff, eps):
    """q [T, heads, 2, d], k [T, kv heads, 2, d], v [T, kv heads, dv] -> [T, heads, dv]."""
    a1 = capped_window_map(q[:, :, 0], k[:, :, 0], v, scale, softcap, window)
    a2 = capped_window_map(q[:, :, 1], k[:, :, 1], v, scale, softcap, window)
    return unit_rms(a1 - lam * a2, eps) * (1.0 - diff)


def keys_and_values(h, w, p, m):
    t = h.shape[0]
    return (h @ w[p + "k"].T).view(t, m["kv_heads"], 2, m["dim"]), (h @ w[p + "v"].T).view(t, m["kv_heads"], m["vdim"])


def attention(h, w, p, m, eps, k, v):
    """The mixer on its input h [T, W] with the keys and values it is given."""
    t = h.shape[0]
    q = (h @ w[p + "q"].T).view(t, m["heads"], 2, m["dim"])
    window = m["mask"]["size"] if m.get("mask") else None
    o = two_maps(q, k, v, m["scale"], m.get("softcap"), window, map_weight(w, p, m["diff"]), m["diff"], eps)
    return o.reshape(t, -1) @ w[p + "o"].T


# ----------------------------------------------------------------------------- feed-forwards
def squared_relu(h, w, p):
    return (torch.relu(h @ w[p + "up"].T) ** 2) @ w[p + "down"].T


def gated_expert(h, w, p):
    z = h @ w[p + "gate"].T
    return (z * torch.sigmoid(z) * (h @ w[p + "up"].T)) @ w[p + "down"].T


def route_scores(z, correction, router):
    """Chosen outputs [T, top] and their weights from the router's logits z [T, experts + identity]."""
    s = torch.softmax(z, dim=-1)
    choice = s + correction
    groups = router.get("groups")
    if groups:
        t, n = choice.shape
        split = choice.view(t, groups["count"], n // groups["count"])
        best = torch.argsort(-split.max(-1).values, dim=-1, stable=True)[:, : groups["keep"]]
        allowed = torch.zeros(t, groups["count"], dtype=torch.bool)
        allowed.scatter_(1, best, True)
        choice = split.masked_fill(~allowed[:, :, None], -math.inf).reshape(t, n)
    idx = torch.argsort(-choice, dim=-1, stable=True)[:, : router["top"]]
    return idx, torch.gather(s, -1, idx) * router.get("scale", 1.0)


def expert_mixture(h, w, p, mlp):
    r = mlp["router"]
    idx, weight = route_scores(h @ w[p + "router"].T, w[p + "correction"], r)
    out = torch.zeros_like(h)
    for t in range(h.shape[0]):
        for e, a in zip(idx[t].tolist(), weight[t]):
            out[t] += a * (h[t] if e >= r["experts"] else gated_expert(h[t : t + 1], w, f"{p}e{e}.")[0])
    return out


# ----------------------------------------------------------------------------- the model
def forward(cfg, w, tokens, collect=None):
    """Logits [T, vocab] (float64) of one sequence; collect, if a list, gets the stream after every layer."""
    eps = cfg["norm"]["eps"]
    t = len(tokens)
    x = w["embed"][torch.as_tensor(tokens, dtype=torch.long)] * cfg["embedding"]["scale"] + w["pos"][:t]
    kept = {}
    for i, layer in enumerate(cfg["layers"]):
        p, m = f"l{i}.", layer["mixer"]
        h = offset_norm(x, w[p + "norm1"], eps)
        if layer["type"] != "attention":
            raise ValueError(layer["type"])
        if m.get("kv_from") is None:
            kept[i] = keys_and_values(h, w, p + "mix.", m)
        k, v = kept[i if m.get("kv_from") is None else m["kv_from"]]
        x = x + attention(h, w, p + "mix.", m, eps, k, v)
        mlp = layer.get("mlp")
        if mlp is not None:
            h = offset_norm(x, w[p + "norm2"], eps)
            if mlp["kind"] == "dense":
                x = x + squared_relu(h, w, p + "mlp.")
            elif mlp["kind"] == "moe":
                x = x + expert_mixture(h, w, p + "mlp.", mlp)
            else:
                raise ValueError(mlp["kind"])
        if collect is not None:
            collect.append(x.clone())
    return offset_norm(x, w["final.norm"], eps) @ w["head"].T
