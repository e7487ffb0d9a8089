"""Mixtures of experts."""
from __future__ import annotations

import torch

from . import hip_op, register_feed_forward, require_size


@register_feed_forward("scaled_input_mixture")
class ScaledInputMixture:
    """The `top` experts with the largest sigmoid scores, each a gated unit W_down (silu(W_gate h) * W_up h) that reads the token
    times its score.  Returns the choices' results, `top` rows per token, that count as their sum."""

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
        routing = self.route(x, self.router, self.top)
        return self.op_down(self.op_gate_up(x, self.gate_up, routing), self.down, routing)
