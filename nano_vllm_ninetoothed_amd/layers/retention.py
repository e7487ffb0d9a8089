"""Retention: linear attention with a fixed decay per head, rotary positions on q and k, no softmax and no denominator."""
from __future__ import annotations

import math

import torch

from . import ChunkedRecurrence, Mixer, hip_op, pack, register_mixer, require_size
from ..mops.hip.recurrent_ops import recurrence_state_pitch


@register_mixer("retention")
class Retention(Mixer):
    uses_pages, uses_slots = False, True

    @staticmethod
    def validate(sizes):
        require_size(sizes, "heads", "dim", "vdim")
        if len(sizes["decay"]) != sizes["heads"]:
            raise ValueError("decay must list one value per head")
        if any(not 0.0 <= d <= 1.0 for d in sizes["decay"]):
            raise ValueError("decays lie between 0 and 1")
        rot = sizes["rot"]["dims"]
        if rot < 0 or rot % 2 or rot > sizes["dim"]:
            raise ValueError("rot.dims must be even and at most dim")

    def __init__(self, sizes, weights, prefix, m):
        self.heads, self.dim, self.vdim = h, d, v = sizes["heads"], sizes["dim"], sizes["vdim"]
        self.eps = m.eps
        take = weights.take
        self.qkvg = pack([take(prefix + "q", (h * d, m.width)), take(prefix + "k", (h * d, m.width)),
                          take(prefix + "v", (h * v, m.width)), take(prefix + "g", (h * v, m.width))])
        self.o = take(prefix + "o", (m.width, h * v))
        decay = torch.tensor([float(x) for x in sizes["decay"]], dtype=torch.float64)
        self.decay = decay.float().to(m.device)
        # a decay of zero forgets everything: its logarithm is kept finite so that differences of sums stay defined
        self.log_decay = decay.clamp(min=math.exp(-80.0)).log().float().to(m.device)
        self.cos_sin = m.rotary.table(sizes["rot"]["base"], sizes["rot"]["dims"]) if sizes["rot"]["dims"] else None
        self.k_scale = d ** -0.5
        self.allocate(m.cache)
        self.portions = ChunkedRecurrence(h, h, d, v, m.dtype)
        self.linear, self.recurrence, self.group_norm = hip_op("linear"), hip_op("decayed_recurrence"), hip_op("gated_group_norm")

    def allocate(self, cache):
        self.state = cache.per_slot(self.heads, self.vdim, recurrence_state_pitch(self.dim))

    def __call__(self, x, ctx):
        h, d, v = self.heads, self.dim, self.vdim
        p = self.linear(x, self.qkvg)
        q, k, vv, gate = p[:, :h * d], p[:, h * d:2 * h * d], p[:, 2 * h * d:2 * h * d + h * v], p[:, 2 * h * d + h * v:2 * h * (d + v)]
        o = torch.empty((x.shape[0], h * v), dtype=x.dtype, device=x.device)
        nd = ctx["n_decode"]
        slots, starts = ctx["state_slots"], ctx["starts"]
        opts = dict(decay=self.decay, log_decay=self.log_decay, cos_sin=self.cos_sin, k_scale=self.k_scale)
        if nd:
            self.recurrence(q[:nd], k[:nd], vv[:nd], o[:nd], self.state, slots[:nd], starts[:nd], h, h, d, v, **opts)
        if nd < slots.numel():
            self.portions(q[nd:], k[nd:], vv[nd:], o[nd:], self.state, ctx, **opts)
        return self.linear(self.group_norm(o, gate, h, self.eps), self.o)
