"""Matrix memory: a matrix state and a normalizer per head with exponential input and forget gates, kept relative to a running maximum
of their logarithms; a norm per head and a gate per element."""
from __future__ import annotations

import torch

from . import ChunkedRecurrence, Mixer, hip_op, register_mixer, require_size
from .joined import TwoProducts
from ..mops.hip.recurrent_ops import MemoryGates, matrix_memory_copies, recurrence_state_pitch


@register_mixer("matrix_memory")
class MatrixMemory(TwoProducts, Mixer):
    uses_pages, uses_slots = False, True

    @staticmethod
    def validate(sizes):
        require_size(sizes, "heads", "dim", "vdim")
        if not float(sizes["gate_cap"]) > 0:
            raise ValueError("gate_cap must be positive")

    def __init__(self, sizes, weights, prefix, m):
        self.heads, self.dim, self.vdim = h, d, v = sizes["heads"], sizes["dim"], sizes["vdim"]
        self.cap, self.eps = float(sizes["gate_cap"]), m.eps
        take = weights.take
        qkv = torch.cat([take(prefix + n, (h * k, m.width)) for n, k in (("q", d), ("k", d), ("v", v))])
        gate = take(prefix + "g", (h * v, m.width))
        gates = torch.cat([take(prefix + n, (h, m.width)) for n in ("i", "f")])
        self.products([qkv, gate, gates], take(prefix + "o", (m.width, h * v)))
        self.biases = [take(f"{prefix}{n}.b", (h,), "vector").float().contiguous() for n in ("i", "f")]
        self.norm = take(prefix + "norm", (h * v,), "norm")
        self.portions = ChunkedRecurrence(h, h, d, v, m.dtype)
        self.recurrence, self.group_norm = hip_op("decayed_recurrence"), hip_op("gated_group_norm")
        self.allocate(m.cache)

    def allocate(self, cache):
        copies = matrix_memory_copies(self.vdim)
        self.state = cache.per_slot(self.heads, self.vdim + copies, recurrence_state_pitch(self.dim))
        self.top = cache.per_slot(self.heads, copies)

    def mix(self, p, ctx, out, scale=1.0):
        h, d, v = self.heads, self.dim, self.vdim
        qkv, gate, both = self.parts_of(p)
        q, k, vv = qkv[:, :h * d], qkv[:, h * d:2 * h * d], qkv[:, 2 * h * d:]
        o = torch.empty((p.shape[0], h * v), dtype=p.dtype, device=p.device)
        nd, slots, starts = ctx["n_decode"], ctx["state_slots"], ctx["starts"]

        def options(rows):
            return dict(gates=MemoryGates(both[rows, :h], both[rows, h:], *self.biases, self.cap, self.top, d ** -0.5))

        if nd:
            self.recurrence(q[:nd], k[:nd], vv[:nd], o[:nd], self.state, slots[:nd], starts[:nd], h, h, d, v, **options(slice(nd)))
        if nd < slots.numel():
            self.portions(q[nd:], k[nd:], vv[nd:], o[nd:], self.state, ctx, **options(slice(nd, None)))
        self.group_norm(o, gate, h, self.eps, weight=self.norm, activation="sigmoid", scale=scale, out=out)
