"""Routed experts: a mixture of small gated feed-forwards (clamped, or with a plain silu gate) of which each
token uses a few, chosen among groups of experts, beside one that every token uses (unweighted, or times a
sigmoid gate per token). Experts may also be plain two-matrix feed-forwards with a squared relu, and the last
outputs of the router identity experts, which have no tensors and hand the input on.

Router logits and everything behind them up to the weights are float32. The tokens of a step are
sorted by expert on the device, the two products run per expert over its run of tokens, and a
token's weighted sum is taken in float32 and handed to the residual sum as it is; nothing waits for
the host, so steps with such a layer can be captured.
"""

from __future__ import annotations

import torch

from ..config.specs import ClampedGLUSpec, ReluSquaredSpec, RoutedExpertsSpec, SwiGLUSpec
from .registry import TensorDecl, build_part, register_part, tensors_of

NO_LIMIT = 3.0e38        # a clamp that never bites: what the products per expert get for a plain silu gate


def _expert_form(expert):
    """((gate, up, down): an expert's local tensor names, (limit, slope, shift) of g sigmoid(slope g) (u + shift))."""
    if isinstance(expert, SwiGLUSpec):
        return expert.names, (NO_LIMIT, 1.0, 0.0)
    if isinstance(expert, ClampedGLUSpec):
        return ("gate", "up", "down"), (expert.limit, expert.slope, 1.0)
    raise TypeError(f"routed experts of {type(expert).__name__}: a clamped or a silu-gated feed-forward")


class RoutedExperts:
    @staticmethod
    def tensors(spec: RoutedExpertsSpec):
        t = {"router": TensorDecl((spec.n_experts, spec.hidden))}
        if spec.logit_bias:
            t["router.b"] = TensorDecl((spec.n_experts,), "vector")
        if spec.corrected:
            t["correction"] = TensorDecl((spec.n_experts,), "vector")
        for e in range(spec.n_experts - spec.n_identity):
            for local, decl in tensors_of(spec.expert).items():
                t[f"e{e}.{local}"] = decl
        if spec.shared is not None:
            for local, decl in tensors_of(spec.shared).items():
                t[f"shared.{local}"] = decl
        if spec.shared_gate:
            t["shared.sg"] = TensorDecl((1, spec.hidden))
        return t

    def __init__(self, spec: RoutedExpertsSpec, tensors, ops):
        self.spec, self.ops = spec, ops
        E = spec.n_experts - spec.n_identity
        # (the shared expert's gate is one more row of the router's product)
        self.w_router = torch.cat([tensors["router"], tensors["shared.sg"]], dim=0).contiguous() if spec.shared_gate else tensors["router"]
        self.correction, self.logit_bias = tensors.get("correction"), tensors.get("router.b")
        self.squared = isinstance(spec.expert, ReluSquaredSpec)
        # [E, gate | up, hidden] (or up alone) and [E, hidden, ff]: one operand each for the products per expert
        if self.squared:
            self.w_up = torch.stack([tensors[f"e{e}.up"] for e in range(E)]).contiguous()
            down = "down"
        else:
            (gate, up, down), self.form = _expert_form(spec.expert)
            self.w_gate_up = torch.stack([torch.cat([tensors[f"e{e}.{gate}"], tensors[f"e{e}.{up}"]], dim=0) for e in range(E)]).contiguous()
        self.w_down = torch.stack([tensors[f"e{e}.{down}"] for e in range(E)]).contiguous()
        self.shared = None
        self.offers_sums = spec.shared is None
        if spec.shared is not None:
            own = {k[len("shared."):]: v for k, v in tensors.items() if k.startswith("shared.") and k != "shared.sg"}
            self.shared = build_part(spec.shared, own, ops)
            if hasattr(self.shared, "rows_as_they_are"):
                self.shared.rows_as_they_are()

    def forward(self, x, ctx=None, whole=True):
        """``whole`` False (where ``offers_sums`` says so): each expert's results by place, their weighted sum left to
        the block's own sum."""
        s, ops = self.spec, self.ops
        E = s.n_experts
        logits = ops.linear(x, self.w_router, out_dtype=torch.float32)
        plain = s.scoring == "softmax" and s.group_top == 1 and s.scale == 1.0 and not s.shared_gate
        how = {} if plain else dict(scoring=s.scoring, group_top=s.group_top, scale=s.scale)
        if not s.renorm:
            how["renorm"] = False
        if self.logit_bias is not None:
            how["bias"] = self.logit_bias
        experts, weights = ops.moe_route(logits[:, :E] if s.shared_gate else logits, self.correction, s.top, s.n_groups,
                                         s.keep_groups, s.renorm_eps, **how)
        extra = None
        if self.shared is not None and getattr(self.shared, "takes_projection", False):
            # (a feed-forward that would hand partial sums to a norm: here its last product is whole)
            extra = self.shared.forward(x, project=lambda act, w: ops.linear(act, w))
        elif self.shared is not None:
            extra = self.shared.forward(x)
        same = {"identity": True} if s.n_identity else {}        # (their choices lie behind the stacked experts)
        if self.squared:
            more = {"extra_gate": logits[:, E]} if s.shared_gate else {}
            more.update(same)
            if not whole:
                return ops.moe_experts_squared(x, experts, weights, self.w_up, self.w_down, whole=False, **same)
            return ops.moe_experts_squared(x, experts, weights, self.w_up, self.w_down, extra, **more).unsqueeze(0)
        limit, slope, shift = self.form
        more = dict(same)
        if shift != 1.0:
            more["shift"] = shift
        if s.shared_gate:
            more["extra_gate"] = logits[:, E]
        if not whole:
            return ops.moe_experts(x, experts, weights, self.w_gate_up, self.w_down, limit, slope, whole=False, **more)
        y = ops.moe_experts(x, experts, weights, self.w_gate_up, self.w_down, limit, slope, extra, **more)
        return y.unsqueeze(0)        # float32 sums: the residual sum takes them as they are


register_part(RoutedExpertsSpec, RoutedExperts)
