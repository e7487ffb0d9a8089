"""Grouped-query attention with rotary positions on the first elements of every head (pairs of an element and the one half the rotated
part further on), capped scores, and options: an RMS norm per query and key head, a part of the sequence that a token sees, a learned
sink per head in the softmax's denominator, a gate per head on the output."""
from __future__ import annotations

from . import hip_op, pack, register_mixer, require_size
from .paged_attention import PagedAttention
from ..mops.hip.attention_ops import Scores

PACKED_ROWS = 1024      # above, the few columns of the gates cost the packed product more than a product of their own


class RotaryAttention(PagedAttention):
    HEAD_NORMS = SINK = GATE = False

    @staticmethod
    def visible(mask) -> dict:
        """The fields of Scores that say what a token sees."""
        return {}

    @classmethod
    def validate(cls, sizes):
        PagedAttention.validate(sizes)
        rot = sizes["rot"]
        require_size(rot, "dims")
        if rot["dims"] % 2 or rot["dims"] > sizes["dim"] or not float(rot["base"]) > 0:
            raise ValueError("rot.dims must be even and at most dim, rot.base positive")
        if sizes.get("softcap") is not None and not float(sizes["softcap"]) > 0:
            raise ValueError("softcap must be positive")
        cls.visible(sizes.get("mask"))

    def __init__(self, sizes, weights, prefix, m):
        h, g, d, v = [sizes[n] for n in ("heads", "kv_heads", "dim", "vdim")]
        take = weights.take
        projections = [take(prefix + "q", (h * d, m.width)), take(prefix + "k", (g * d, m.width)), take(prefix + "v", (g * v, m.width))]
        if self.GATE:
            projections.append(take(prefix + "g", (h, m.width)))
        self.qkv = pack(projections)
        self.gate_at = (h + g) * d + g * v if self.GATE else None
        self.gate_rows = pack([projections[-1]]) if self.GATE else None
        self.q_norm, self.k_norm = (take(prefix + n, (d,), "norm") if self.HEAD_NORMS else None for n in ("q.norm", "k.norm"))
        self.o = take(prefix + "o", (m.width, h * v))
        self.scores = Scores(softcap=float(sizes.get("softcap") or 0.0), **self.visible(sizes.get("mask")),
                             sinks=take(prefix + "sink", (h,), "vector").float().contiguous() if self.SINK else None)
        self.trig = m.rotary.table(sizes["rot"]["base"], sizes["rot"]["dims"])
        self.prepare = hip_op("rotary_prepare")
        super().__init__(sizes, m)

    def __call__(self, x, ctx):
        packed = x.shape[0] <= PACKED_ROWS or not self.GATE
        qkv = self.linear(x, self.qkv if packed else self.qkv[:self.gate_at])
        q = self.prepare(qkv, ctx["positions32"], ctx["slot_mapping"], self.k_pages, self.v_pages, self.heads, self.kv_heads, self.dim, self.vdim,
                         cos_sin=self.trig, q_weight=self.q_norm, k_weight=self.k_norm, eps=self.eps)
        gate = None
        if self.GATE:
            gate = qkv[:, self.gate_at:self.gate_at + self.heads] if packed else self.linear(x, self.gate_rows)[:, :self.heads]
        return self.linear(self.attend(q, ctx, gate), self.o)


@register_mixer("chunked_attention")
class ChunkedAttention(RotaryAttention):
    """A token sees its chunk of the sequence up to itself."""
    HEAD_NORMS = SINK = True

    @staticmethod
    def visible(mask):
        require_size(mask, "size")
        return {"chunk": mask["size"]}


@register_mixer("windowed_attention")
class WindowedAttention(RotaryAttention):
    """A token sees the last tokens up to itself, and the first ones of its sequence."""
    GATE = True

    @staticmethod
    def visible(mask):
        require_size(mask, "size")
        keep = mask.get("keep_first", 0)
        if not isinstance(keep, int) or isinstance(keep, bool) or keep < 0:
            raise ValueError(f"keep_first must be a non-negative integer, got {keep!r}")
        return {"window": mask["size"], "keep_first": keep}
