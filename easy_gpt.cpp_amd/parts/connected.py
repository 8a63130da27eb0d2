"""Layers connected by several parallel residual streams.

In place of one stream x there are n, X_1 .. X_n, all equal to the embedding's output at the start.  A branch (a mixer or
a feed-forward behind its norm) reads a weighted sum of them, u = sum_s read_s X_s, and its output y = scale * f(norm(u))
(`scale` a vector of the width, one number per coordinate) rewrites all of them at once:
X'_t = sum_s mix[s, t] X_s + write_t y.  A model ends with the norm of the streams' sum (`rmsnorm_stream_sum`).

The streams are float32 [n, T, H] ([T, H] while they are all equal) and everything here is float32.  A branch's rewriting is
left to whoever reads the streams next, as the pending update that a block hands on as its delta: one kernel
(`kernels.connect_streams`) adds up the branch's product, rewrites the streams, sums them for the next branch and norms.
"""
from __future__ import annotations

import torch

from .. import kernels
from .base import Block, StreamConnection, register_part
from .norm import RMSNorm
from .spec import ParamSpec


class HyperConnection(StreamConnection):
    graph_safe = True

    def __init__(self, prefix: str, hidden_size: int, streams: int, names: dict | None = None, scale_name: str | None = None):
        """names: the tensors behind `prefix` of read [n], write [n] and mix [n, n] (from, to); scale_name: the tensor of the
        branch's factor per coordinate [H] (None: there is none)."""
        if int(streams) < 1:
            raise ValueError(f"a connection of {streams} streams: there is at least one")
        self.prefix, self.hidden_size, self.streams = prefix, int(hidden_size), int(streams)
        self.names = dict(read="in", write="out", mix="mix")
        self.names.update(names or {})
        self.scale_name = scale_name
        self.read_weights = self.write_weights = self.mix = self.scale = None

    def param_specs(self):
        p, n, names = self.prefix, self.streams, self.names
        # (random weights: sums keep the size of their terms)
        specs = [ParamSpec(p + names["read"], (n,), role="mean_weights", dtype="float32"),
                 ParamSpec(p + names["write"], (n,), role="norm_scale", dtype="float32"),
                 ParamSpec(p + names["mix"], (n, n), role="stream_mix", dtype="float32")]
        if self.scale_name is not None:
            specs.append(ParamSpec(p + self.scale_name, (self.hidden_size,), role="norm_scale", dtype="float32"))
        return specs

    def load(self, get, dtype, device):
        def take(name):
            return get(self.prefix + name).to(torch.float32).to(device).contiguous()

        self.read_weights, self.write_weights, self.mix = (take(self.names[x]) for x in ("read", "write", "mix"))
        if self.scale_name is not None:
            self.scale = take(self.scale_name)

    def read(self, h, delta, norm):
        weight, eps, _ = norm.rms_params()
        return kernels.backend().connect_streams(h, delta, self.read_weights, self.streams, None, weight, eps)

    def written(self, y) -> kernels.StreamUpdate:
        return kernels.StreamUpdate(y, self.scale, self.mix, self.write_weights)


class ConnectedBlock(Block):
    """The pre-norm arrangement on parallel streams: each branch is connected to them by a part of its own."""

    norm_slots = ("mixer", "feed_forward")
    connection_slots = ("mixer", "feed_forward")

    def __init__(self, mixer, feed_forward, norms, connections):
        super().__init__(mixer, feed_forward, norms)
        self.connections = dict(connections)
        for slot in self.norm_slots:
            if not isinstance(self.norms[slot], RMSNorm) or self.norms[slot].weight_offset:
                raise ValueError(f"the connected arrangement's norm '{slot}' must be an RMS norm whose weight is stored as it is")

    def parts(self):
        return super().parts() + [self.connections[s] for s in self.connection_slots]

    def forward(self, h, delta, ctx, cache, state):
        connection = self.connections["mixer"]
        x, h = connection.read(h, delta, self.norms["mixer"])
        delta = connection.written(self.mixer.forward(x, ctx, cache, state))
        if self.feed_forward is None:
            return h, delta
        connection = self.connections["feed_forward"]
        x, h = connection.read(h, delta, self.norms["feed_forward"])
        return h, connection.written(self.feed_forward.forward(x, ctx))


class ConnectedMixerOnlyBlock(ConnectedBlock):
    """The same for a layer that has no feed-forward."""

    norm_slots = ("mixer",)
    connection_slots = ("mixer",)
    uses_feed_forward = False


register_part("stream_connection", "hyper_connection", HyperConnection)
register_part("block", "connected", ConnectedBlock)
register_part("block", "connected_mixer_only", ConnectedMixerOnlyBlock)
