"""Mixtures of experts."""
from __future__ import annotations

import torch

from . import hip_op, register_feed_forward, require_size
from .feed_forward import ClampedGLU
from ..mops.hip.mixture_ops import CommonUnit, Weighted


class Mixture:
    """Experts of one size that are gated units of their own, and a router.  Returns the choices' results, `top` rows per token, that
    count as their sum."""

    @staticmethod
    def validate(sizes):
        require_size(sizes["router"], "experts", "top")
        require_size(sizes["expert"], "ff")
        if sizes["router"]["top"] > sizes["router"]["experts"]:
            raise ValueError("top must not exceed the number of experts")

    def __init__(self, sizes, weights, prefix, m):
        self.experts, self.top, ff = sizes["router"]["experts"], sizes["router"]["top"], sizes["expert"]["ff"]
        take = weights.take
        self.router = take(prefix + "router", (self.experts, m.width))
        # hidden sizes are padded with zeros to 16-byte pieces
        pad = -ff % 8
        self.gate_up = torch.zeros((self.experts, 2, ff + pad, m.width), dtype=m.dtype, device=m.device)
        self.down = torch.zeros((self.experts, m.width, ff + pad), dtype=m.dtype, device=m.device)
        for e in range(self.experts):
            for i, n in enumerate(("gate", "up")):
                self.gate_up[e, i, :ff] = take(f"{prefix}e{e}.{n}", (ff, m.width))
            self.down[e, :, :ff] = take(f"{prefix}e{e}.down", (m.width, ff))
        self.route, self.op_gate_up, self.op_down = hip_op("moe_route"), hip_op("moe_gate_up"), hip_op("moe_down")

    def __call__(self, x):
        raise NotImplementedError


@register_feed_forward("scaled_input_mixture")
class ScaledInputMixture(Mixture):
    """The `top` experts with the largest sigmoid scores, each a gated unit W_down (silu(W_gate h) * W_up h) that reads the token
    times its score."""

    def __call__(self, x):
        routing = self.route(x, self.router, self.top)
        return self.op_down(self.op_gate_up(x, self.gate_up, routing), self.down, routing)


@register_feed_forward("grouped_mixture")
class GroupedMixture(Mixture):
    """Experts W_down (g sigmoid(1.702 g) (u + 1)) with limits on g and u.  A token takes the `top` experts with the largest sigmoid
    scores plus a correction among those of its best groups of neighbours; the results count with the chosen ones' sigmoids over their
    sum, times a factor.  A shared unit of the same form, with sizes of its own, sees every token."""

    @staticmethod
    def validate(sizes):
        Mixture.validate(sizes)
        float(sizes["expert"]["limit"]), float(sizes["router"]["scale"])
        groups, experts = sizes["router"].get("groups"), sizes["router"]["experts"]
        if groups is not None:
            require_size(groups, "count", "keep")
            if experts % groups["count"] or groups["keep"] > groups["count"] or sizes["router"]["top"] > experts // groups["count"] * groups["keep"]:
                raise ValueError("the experts must divide into the groups, and the kept groups must hold enough of them")
        if sizes.get("shared") is not None:
            ClampedGLU.validate(sizes["shared"])

    def __init__(self, sizes, weights, prefix, m):
        super().__init__(sizes, weights, prefix, m)
        router = sizes["router"]
        groups = router.get("groups") or {"count": 1, "keep": 1}
        self.weighted = Weighted(weights.take(prefix + "correction", (self.experts,), "vector").float().contiguous(), groups["count"], groups["keep"],
                                 float(router["scale"]))
        self.limit = float(sizes["expert"]["limit"])
        self.shared = ClampedGLU(sizes["shared"], weights, prefix + "shared.", m) if sizes.get("shared") is not None else None
        s = self.shared
        self.common = None if s is None else CommonUnit(s.gate_up, s.down.contiguous(), s.ff, s.half, s.limit)

    def __call__(self, x):
        routing = self.route(x, self.router, self.top, weighted=self.weighted)
        if self.common is not None and routing.takes_common:      # small batches: in the experts' launches
            y, yc = self.op_gate_up(x, self.gate_up, routing, self.limit, ClampedGLU.ALPHA, common=self.common)
            return self.op_down(y, self.down, routing, common=self.common, common_y=yc)
        y = self.op_down(self.op_gate_up(x, self.gate_up, routing, self.limit, ClampedGLU.ALPHA), self.down, routing)
        return y if self.shared is None else (y, self.shared(x))
