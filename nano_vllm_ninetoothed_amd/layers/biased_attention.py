"""Grouped-query attention without rotation: norms over the whole query and key projections, a query factor that grows in steps
with the position, and a linear distance bias per head."""
from __future__ import annotations

import torch

from . import hip_op, pack, register_mixer
from .paged_attention import LONG_PORTION, PagedAttention  # noqa: F401


def distance_slopes(heads: int) -> torch.Tensor:
    """2^(-8 (h + 1) / heads)"""
    return torch.pow(2.0, -8.0 * torch.arange(1, heads + 1, dtype=torch.float64) / heads).float()


@register_mixer("biased_attention")
class BiasedAttention(PagedAttention):

    @staticmethod
    def validate(sizes):
        PagedAttention.validate(sizes)
        if sizes.get("q_temp") is not None and not (float(sizes["q_temp"]["every"]) > 0 and float(sizes["q_temp"]["coef"]) == sizes["q_temp"]["coef"]):
            raise ValueError("q_temp.every must be positive")

    def __init__(self, sizes, weights, prefix, m):
        h, g, d, v = [sizes[n] for n in ("heads", "kv_heads", "dim", "vdim")]
        take = weights.take
        self.qkv = pack([take(prefix + "q", (h * d, m.width)), take(prefix + "k", (g * d, m.width)), take(prefix + "v", (g * v, m.width))])
        self.q_norm, self.k_norm = take(prefix + "q.norm", (h * d,), "norm"), take(prefix + "k.norm", (g * d,), "norm")
        self.o = take(prefix + "o", (m.width, h * v))
        temp = sizes.get("q_temp")
        self.q_factor = m.rotary.steps(temp["coef"], temp["every"]) if temp is not None else None
        self.slopes = distance_slopes(h).to(m.device)
        self.prepare = hip_op("attention_prepare")
        super().__init__(sizes, m)

    def __call__(self, x, ctx):
        q = self.prepare(self.linear(x, self.qkv), self.q_norm, self.k_norm, self.eps, ctx["positions32"], ctx["slot_mapping"], self.k_pages, self.v_pages,
                         self.heads, self.kv_heads, self.dim, self.vdim, q_factor=self.q_factor)
        return self.linear(self.attend(q, ctx), self.o)
