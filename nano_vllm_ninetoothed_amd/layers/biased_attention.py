"""Grouped-query attention without rotation: norms over the whole query and key projections, a query factor that grows in steps
with the position, and a linear distance bias per head."""
from __future__ import annotations

import torch

from . import Mixer, hip_op, pack, register_mixer, require_size
from ..mops.hip.attention_ops import padded


def distance_slopes(heads: int) -> torch.Tensor:
    """2^(-8 (h + 1) / heads)"""
    return torch.pow(2.0, -8.0 * torch.arange(1, heads + 1, dtype=torch.float64) / heads).float()


@register_mixer("biased_attention")
class BiasedAttention(Mixer):
    uses_pages, uses_slots = True, False

    @staticmethod
    def validate(sizes):
        require_size(sizes, "heads", "kv_heads", "dim", "vdim")
        if sizes["heads"] % sizes["kv_heads"]:
            raise ValueError("heads must be a multiple of kv_heads")
        float(sizes["scale"])
        if sizes.get("q_temp") is not None and not (float(sizes["q_temp"]["every"]) > 0 and float(sizes["q_temp"]["coef"]) == sizes["q_temp"]["coef"]):
            raise ValueError("q_temp.every must be positive")

    def __init__(self, sizes, weights, prefix, m):
        self.heads, self.kv_heads, self.dim, self.vdim = h, g, d, v = [sizes[n] for n in ("heads", "kv_heads", "dim", "vdim")]
        self.scale, self.eps, self.dtype = float(sizes["scale"]), m.eps, m.dtype
        take = weights.take
        self.qkv = pack([take(prefix + "q", (h * d, m.width)), take(prefix + "k", (g * d, m.width)), take(prefix + "v", (g * v, m.width))])
        self.q_norm, self.k_norm = take(prefix + "q.norm", (h * d,), "norm"), take(prefix + "k.norm", (g * d,), "norm")
        self.o = take(prefix + "o", (m.width, h * v))
        temp = sizes.get("q_temp")
        self.q_factor = m.rotary.steps(temp["coef"], temp["every"]) if temp is not None else None
        self.slopes = distance_slopes(h).to(m.device)
        self.linear, self.prepare, self.rows = hip_op("linear"), hip_op("attention_prepare"), hip_op("biased_attention_rows")
        self.allocate(m.cache)

    def allocate(self, cache):
        self.k_pages = cache.paged(self.kv_heads, padded(self.dim), dtype=self.dtype)
        self.v_pages = cache.paged(self.kv_heads, padded(self.vdim), dtype=self.dtype)

    def __call__(self, x, ctx):
        q = self.prepare(self.linear(x, self.qkv), self.q_norm, self.k_norm, self.eps, ctx["positions32"], ctx["slot_mapping"], self.k_pages, self.v_pages,
                         self.heads, self.kv_heads, self.dim, self.vdim, q_factor=self.q_factor)
        o = self.rows(q, self.k_pages, self.v_pages, self.dim, self.vdim, ctx["token_context"], ctx["block_tables"], self.scale, slopes=self.slopes,
                      row_seq=ctx["token_seq"])
        return self.linear(o.view(x.shape[0], self.heads * self.vdim), self.o)
