"""Grouped-query attention with biases on its projections, as a sublayer of two products: with rotary positions on neighbouring elements
and keys that count on their own (the sigmoid of their score, no softmax), or with norms per head and a bias that grows with the
logarithm of the distance."""
from __future__ import annotations

import torch

from . import hip_op, register_mixer, require_size
from .joined import TwoProducts
from .paged_attention import PagedAttention
from ..mops.hip.attention_ops import Scores


class ProjectedAttention(TwoProducts, PagedAttention):
    HEAD_NORMS = ROTATION = GATE = OUTPUT_BIAS = False

    def __init__(self, sizes, weights, prefix, m):
        h, g, d, v = [sizes[n] for n in ("heads", "kv_heads", "dim", "vdim")]
        take = weights.take
        rows = {"q": h * d, "k": g * d, "v": g * v}
        into = [torch.cat([take(prefix + n, (k, m.width)) for n, k in rows.items()])]
        self.qkv_bias = torch.cat([take(f"{prefix}{n}.b", (k,), "vector") for n, k in rows.items()]).contiguous()
        if self.GATE:
            into.append(take(prefix + "g", (h * v, m.width)))
        self.q_norm, self.k_norm = (take(prefix + n, (d,), "norm") if self.HEAD_NORMS else None for n in ("q.norm", "k.norm"))
        self.trig = m.rotary.table(sizes["rot"]["base"], sizes["rot"]["dims"]) if self.ROTATION else None
        self.products(into, take(prefix + "o", (m.width, h * v)), take(prefix + "o.b", (m.width,), "vector") if self.OUTPUT_BIAS else None)
        self.prepare = hip_op("rotary_prepare")
        PagedAttention.__init__(self, sizes, m)

    def mix(self, p, ctx, out, scale=1.0):
        qkv, *gate = self.parts_of(p)
        q = self.prepare(qkv, ctx["positions32"], ctx["slot_mapping"], self.k_pages, self.v_pages, self.heads, self.kv_heads, self.dim, self.vdim,
                         cos_sin=self.trig, q_weight=self.q_norm, k_weight=self.k_norm, eps=self.eps, bias=self.qkv_bias, neighbours=True)
        self.attend(q, ctx, gate[0] if gate else None, out, scale)


@register_mixer("sigmoid_attention")
class SigmoidAttention(ProjectedAttention):
    """A key counts with sigmoid(score + a number per head); a gate per element on the heads' results."""
    ROTATION = GATE = OUTPUT_BIAS = True

    @staticmethod
    def validate(sizes):
        PagedAttention.validate(sizes)
        rot = sizes["rot"]
        require_size(rot, "dims")
        if rot["dims"] % 2 or rot["dims"] > sizes["dim"] or not float(rot["base"]) > 0:
            raise ValueError("rot.dims must be even and at most dim, rot.base positive")

    def __init__(self, sizes, weights, prefix, m):
        self.scores = Scores(weight_bias=weights.take(prefix + "pb", (sizes["heads"],), "vector").float().contiguous())
        super().__init__(sizes, weights, prefix, m)


@register_mixer("log_distance_attention")
class LogDistanceAttention(ProjectedAttention):
    """Softmax over the last tokens of score - rate ln(1 + step distance), rate and step per head."""
    HEAD_NORMS = True

    @staticmethod
    def validate(sizes):
        PagedAttention.validate(sizes)
        require_size(sizes["mask"], "size")

    def __init__(self, sizes, weights, prefix, m):
        rate, step = (weights.take(prefix + n, (sizes["heads"],), "norm").float().contiguous() for n in ("r1", "r2"))
        self.scores = Scores(window=sizes["mask"]["size"], log_distance=(rate, step))
        super().__init__(sizes, weights, prefix, m)
