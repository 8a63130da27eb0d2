"""A mixture of experts as a layer's feed-forward.

Every token goes to the `top` experts with the largest router logits z = W_r x + b (float32), weighted by the softmax
over those logits alone; an expert is W_down (silu(W_gate x) * (W_up x)) without biases.  With `routing='softmax_all'`
the scores are s = softmax(z) over all experts, the `top` experts with the largest s + correction (a stored number per
expert that only steers the choice) are chosen, and they weigh s over the sum of the chosen scores (`normalized` False: s
itself), times `weight_scale`; with `groups` the experts form that many equal groups of neighbours, a group's score is the
largest s + correction in it, and only experts of the best `keep_groups` groups can be chosen.  The last `identities` of the
router's outputs are identity experts without tensors, which hand on x itself.  With `expert='relu2'` an expert has no gate product: W_down relu(W_up x)^2.  An optional shared
feed-forward runs for every token and is added.  Where the stream takes additions (fixed point, steps of few tokens) the
weighted sum is added into it.  Routing, grouping of the rows by expert and the experts' products
all happen on the device, so a step with experts is launched like any other and replays from a graph.
"""
from __future__ import annotations

import torch

from .. import kernels
from .base import FeedForward, PendingNorm, make_part, register_part
from .spec import ParamSpec, PartSpec


class ExpertMixture(FeedForward):
    graph_safe = True
    takes_pending_norm = True

    def __init__(self, prefix: str, hidden_size: int, n_experts: int, top: int, intermediate_size: int,
                 shared: PartSpec | None = None, router_bias: bool = True, names: dict | None = None,
                 routing: str = "softmax_top", weight_scale: float = 1.0, expert: str = "swiglu", identities: int = 0,
                 groups: int = 1, keep_groups: int = 1, normalized: bool = True):
        """names: `expert` (the prefix of expert i's tensors, with {i}), `gate`, `up`, `down`, `router`, `router_bias`,
        `correction` behind `prefix`.  shared: a feed-forward part that every token runs through as well.  routing:
        'softmax_top' or 'softmax_all' (with the tensor `correction`, float [experts + identities]); expert: 'swiglu' or
        'relu2'; groups, keep_groups, normalized: with 'softmax_all'."""
        if routing not in ("softmax_top", "softmax_all"):
            raise ValueError(f"routing '{routing}' is not supported (softmax_top, softmax_all)")
        if expert not in ("swiglu", "relu2"):
            raise ValueError(f"expert '{expert}' is not supported (swiglu, relu2)")
        self.routing, self.weight_scale, self.expert = routing, float(weight_scale), expert
        self.identities, self.groups, self.keep_groups, self.normalized = int(identities), int(groups), int(keep_groups), bool(normalized)
        self.outputs = int(n_experts) + self.identities
        if not 0 < int(top) <= self.outputs:
            raise ValueError(f"top ({top}) must be between 1 and the number of experts ({self.outputs})")
        if (self.groups > 1 or not self.normalized) and routing != "softmax_all":
            raise ValueError("groups of experts and weights as they are go with routing 'softmax_all'")
        if (self.groups < 1 or self.outputs % self.groups or not 0 < self.keep_groups <= self.groups
                or self.outputs // self.groups * self.keep_groups < int(top)):
            raise ValueError(f"{self.keep_groups} of {self.groups} groups of {self.outputs} experts cannot hold {top} choices")
        self.prefix, self.hidden_size = prefix, int(hidden_size)
        self.n_experts, self.top, self.intermediate_size = int(n_experts), int(top), int(intermediate_size)
        self.has_router_bias = bool(router_bias)
        self.names = dict(expert="e{i}.", gate="gate", up="up", down="down", router="router", router_bias="router.b",
                          correction="correction")
        self.correction = None
        self.names.update(names or {})
        self.shared = make_part("feed_forward", shared, hidden_size=hidden_size) if shared is not None else None
        if self.shared is not None and not self.shared.graph_safe:
            self.graph_safe = False
        self.w_router = self.b_router = self.w_gate_up = self.w_down = None

    def _expert(self, i: int, which: str) -> str:
        return self.prefix + self.names["expert"].format(i=i) + self.names[which]

    def param_specs(self):
        h, f = self.hidden_size, self.intermediate_size
        specs = []
        for i in range(self.n_experts):
            if self.expert == "swiglu":
                specs.append(ParamSpec(self._expert(i, "gate"), (f, h)))
            specs += [ParamSpec(self._expert(i, "up"), (f, h)), ParamSpec(self._expert(i, "down"), (h, f))]
        specs.append(ParamSpec(self.prefix + self.names["router"], (self.outputs, h)))
        if self.routing == "softmax_all":
            specs.append(ParamSpec(self.prefix + self.names["correction"], (self.outputs,), role="bias", dtype="float32"))
        if self.has_router_bias:
            specs.append(ParamSpec(self.prefix + self.names["router_bias"], (self.outputs,), role="bias"))
        if self.shared is not None:
            specs += self.shared.param_specs()
        return specs

    def load(self, get, dtype, device):
        e, h, f = self.n_experts, self.hidden_size, self.intermediate_size
        gated = self.expert == "swiglu"
        # an expert's gate rows, then its up rows; without a gate its up rows alone
        self.w_gate_up = torch.empty((e, 2 * f if gated else f, h), dtype=dtype, device=device)
        self.w_down = torch.empty((e, h, f), dtype=dtype, device=device)
        for i in range(e):
            if gated:
                self.w_gate_up[i, :f].copy_(get(self._expert(i, "gate")).to(dtype))
            self.w_gate_up[i, f if gated else 0 :].copy_(get(self._expert(i, "up")).to(dtype))
            self.w_down[i].copy_(get(self._expert(i, "down")).to(dtype))
        if self.routing == "softmax_all":
            self.correction = get(self.prefix + self.names["correction"]).to(torch.float32).to(device).contiguous()
        self.w_router = self._to(get(self.prefix + self.names["router"]), "compute", dtype, device)
        if self.has_router_bias:
            self.b_router = self._to(get(self.prefix + self.names["router_bias"]), "compute", dtype, device)
        if self.shared is not None:
            self.shared.load(get, dtype, device)

    def forward(self, x, ctx=None):
        residual = None
        if isinstance(x, PendingNorm):
            pending, x = x, x.materialize()           # router and experts read the normed rows as they are
            residual = pending.residual() if self.shared is None else None
        options = {}
        if self.routing != "softmax_top" or self.expert != "swiglu":
            options = dict(gated=self.expert == "swiglu", score_all=self.routing == "softmax_all", correction=self.correction,
                           weight_scale=self.weight_scale)
        if self.identities or self.groups > 1 or not self.normalized:
            options.update(identities=self.identities, groups=self.groups, keep_groups=self.keep_groups, normalized=self.normalized)
        if residual is not None:
            options.update(residual=residual)
        out = kernels.backend().expert_mixture(x, self.w_router, self.b_router, self.w_gate_up, self.w_down, self.top, **options)
        if residual is not None:
            return None
        out = out[None]
        if self.shared is None:
            return out
        s = self.shared.forward(x, ctx)
        if s.dim() != 3:
            s = s.float()[None]
        return torch.cat([out, s], dim=0)          # float32 partial sums: whoever adds to the stream adds them up


register_part("feed_forward", "expert_mixture", ExpertMixture)
