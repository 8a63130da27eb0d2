"""A plain, slow Tipezen decoder: whole sequences, no cache, one function per mechanism, float64 on the CPU.

It shares no code with the engine: it reads a model folder with its own few lines and knows the tensor names
itself.  Notation: one sequence of T tokens, positions count from 0, a linear weight is [out, in] and applied as
x W^T.

The design keeps s parallel residual streams X [s, T, W], all of them embed[token] at the start.  A sublayer reads
u = sum_i in_i X_i, computes y = scale * f(rms_norm(u)) (`scale` a vector of the width) and leaves
X'_j = sum_i mix_ij X_i + out_j y.  A layer has a mixer sublayer and, unless its 'mlp' is null, a feed-forward sublayer.
The mixer is grouped-query softmax attention behind a sliding window ('attention': interleaved rotation with stretched
frequencies, a tanh cap on the scores, one in the softmax's denominator, values mixed with those of the first layer that
mixes values, a gate per head) or a linear attention whose state decays by a constant per head ('retention': rotation
of the halves, heads divided by their root mean square, a silu gate).  The feed-forward is gated with the tanh form of
gelu.  At the end the streams are summed, normed and multiplied by the head.
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


# ----------------------------------------------------------------------------- small pieces
def rms_norm(x, weight, eps):
    y = x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)
    return y if weight is None else y * weight


def silu(z):
    return z * torch.sigmoid(z)


def gelu_tanh(z):
    return 0.5 * z * (1.0 + torch.tanh(math.sqrt(2.0 / math.pi) * (z + 0.044715 * z ** 3)))


def rotation_frequencies(rot: dict) -> tuple[list[float], float]:
    """(f_i for i < dims / 2, the factor on cosines and sines): f_i = base^(-2i / dims); with `scaling` {factor, original,
    fast, slow} the frequencies from a pair on are divided by the factor, with a linear ramp before it."""
    dims, base = rot["dims"], rot["base"]
    f = [base ** (-2.0 * i / dims) for i in range(dims // 2)]
    sc = rot.get("scaling")
    if not sc:
        return f, 1.0

    def place(turns):
        return dims * math.log(sc["original"] / (2 * math.pi * turns)) / (2 * math.log(base))

    lo = max(math.floor(place(sc["fast"])), 0)
    hi = min(math.ceil(place(sc["slow"])), dims - 1)
    out = []
    for i, fi in enumerate(f):
        ramp = min(max((i - lo) / max(hi - lo, 0.001), 0.0), 1.0)
        out.append(fi / sc["factor"] * ramp + fi * (1.0 - ramp))
    return out, 0.1 * math.log(sc["factor"]) + 1.0


def rotate(x, positions, rot: dict, layout: str):
    """x [T, heads, d]: the first rot['dims'] places of every head turn by position * f_i; 'interleaved' pairs the
    places (2i, 2i + 1), 'half' the places (i, i + dims / 2).  The rest passes."""
    dims = rot["dims"]
    if dims == 0:
        return x
    freq, magnitude = rotation_frequencies(rot)
    out = x.clone()
    for i, fi in enumerate(freq):
        a, b = (2 * i, 2 * i + 1) if layout == "interleaved" else (i, i + dims // 2)
        angle = positions.to(F64) * fi
        c, s = (torch.cos(angle) * magnitude)[:, None], (torch.sin(angle) * magnitude)[:, None]
        u, v = x[..., a], x[..., b]
        out[..., a] = u * c - v * s
        out[..., b] = v * c + u * s
    return out


# ----------------------------------------------------------------------------- mixers
def capped_window_attention(q, k, v, scale, softcap=None, window=None):
    """q [T, heads, dk], k [T, kv heads, dk], v [T, kv heads, dv] -> [T, heads, dv].  Query head h reads key/value head
    h // (heads / kv heads); a score is softcap * tanh(q.k scale / softcap); the softmax's denominator holds one more term
    exp(0)."""
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
        s = s.masked_fill(~seen, -math.inf)
        top = s.max(-1, keepdim=True).values.clamp(min=0.0)
        e = torch.exp(s - top)
        heads.append((e / (torch.exp(-top) + e.sum(-1, keepdim=True))) @ v[:, g])
    return torch.stack(heads, dim=1)


def attention(h, w, p, m, first_values):
    """(output [T, W], the layer's values before any mixing); first_values: the values to mix in, or None."""
    t = h.shape[0]
    nh, dim, vdim = m["heads"], m["dim"], m["vdim"]
    g = m.get("kv_heads") or nh
    positions = torch.arange(t)
    q = rotate((h @ w[p + "q"].T).view(t, nh, dim), positions, m["rot"], "interleaved")
    k = rotate((h @ w[p + "k"].T).view(t, g, dim), positions, m["rot"], "interleaved")
    v = (h @ w[p + "v"].T).view(t, g, vdim)
    used = v
    if first_values is not None:
        lam = w[p + "vmix"].reshape(())
        used = (1.0 - lam) * v + lam * first_values
    window = m["mask"]["size"] if m.get("mask") else None
    o = capped_window_attention(q, k, used, m["scale"], m.get("softcap"), window)
    o = o * torch.sigmoid(h @ w[p + "g"].T)[:, :, None]
    return o.reshape(t, nh * vdim) @ w[p + "o"].T, v


def constant_decay_scan(q, k, v, decay, state=None):
    """Per head S_t = decay_h S_(t-1) + k_t v_t^T, o_t = S_t^T q_t.  q, k [T, heads, dk]; v [T, heads, dv]."""
    t, nh, dk = q.shape
    s = torch.zeros(nh, dk, v.shape[-1], dtype=F64) if state is None else state.clone()
    d = torch.as_tensor(decay, dtype=F64)[:, None, None]
    out = torch.zeros(t, nh, v.shape[-1], dtype=F64)
    for i in range(t):
        s = d * s + k[i][:, :, None] * v[i][:, None, :]
        out[i] = torch.einsum("hkv,hk->hv", s, q[i])
    return out, s


def retention(h, w, p, m, eps):
    t = h.shape[0]
    nh, dim, vdim = m["heads"], m["dim"], m["vdim"]
    positions = torch.arange(t)
    q = rotate((h @ w[p + "q"].T).view(t, nh, dim), positions, m["rot"], "half")
    k = rotate((h @ w[p + "k"].T).view(t, nh, dim), positions, m["rot"], "half") * dim ** -0.5
    v = (h @ w[p + "v"].T).view(t, nh, vdim)
    o, _ = constant_decay_scan(q, k, v, m["decay"])
    o = rms_norm(o, None, eps).reshape(t, nh * vdim)
    return (o * silu(h @ w[p + "g"].T)) @ w[p + "o"].T


def gated_feed_forward(h, w, p):
    return (gelu_tanh(h @ w[p + "gate"].T) * (h @ w[p + "up"].T)) @ w[p + "down"].T


# ----------------------------------------------------------------------------- streams
def read_streams(x, w, p):
    """u = sum_i in_i X_i for X [s, T, W]."""
    return torch.einsum("i,itw->tw", w[p + "in"], x)


def write_streams(x, y, w, p):
    """X'_j = sum_i mix[i, j] X_i + out_j y."""
    return torch.einsum("ij,itw->jtw", w[p + "mix"], x) + w[p + "out"][:, None, None] * y[None]


# ----------------------------------------------------------------------------- the model
def forward(cfg, w, tokens, collect=None):
    """Logits [T, vocab] (float64) of one sequence; collect, if a list, gets the streams' sum after every layer."""
    eps = cfg["norm"]["eps"]
    x = w["embed"][torch.as_tensor(tokens, dtype=torch.long)][None].expand(cfg["streams"], -1, -1).clone()
    first_values = None
    for i, layer in enumerate(cfg["layers"]):
        p, m = f"l{i}.", layer["mixer"]
        h = rms_norm(read_streams(x, w, p + "hc1."), w[p + "norm1"], eps)
        if layer["type"] == "retention":
            y = retention(h, w, p + "mix.", m, eps)
        elif layer["type"] == "attention":
            mixes = bool(m.get("v_mix"))
            y, v = attention(h, w, p + "mix.", m, first_values if mixes else None)
            if mixes and first_values is None:
                first_values = v
        else:
            raise ValueError(layer["type"])
        x = write_streams(x, y * w[p + "ls1"], w, p + "hc1.")
        if layer.get("mlp") is not None:
            if layer["mlp"]["kind"] != "dense":
                raise ValueError(layer["mlp"]["kind"])
            h = rms_norm(read_streams(x, w, p + "hc2."), w[p + "norm2"], eps)
            y = gated_feed_forward(h, w, p + "mlp.")
            x = write_streams(x, y * w[p + "ls2"], w, p + "hc2.")
        if collect is not None:
            collect.append(x.sum(0))
    return rms_norm(x.sum(0), w["final.norm"], eps) @ w["head"].T
