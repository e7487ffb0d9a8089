"""Mamba-2 (state-space duality): short convolution, time-step dependent decay per head, gated group norm."""
from __future__ import annotations

import torch

from . import ChunkedRecurrence, Mixer, hip_op, pack, register_mixer, require_size
from ..mops.hip.recurrent_ops import recurrence_state_pitch


@register_mixer("mamba2")
class Mamba2(Mixer):
    uses_pages, uses_slots = False, True

    @staticmethod
    def validate(sizes):
        require_size(sizes, "heads", "vdim", "state", "groups", "conv", "norm_groups")
        if sizes["heads"] % sizes["groups"]:
            raise ValueError("heads must be a multiple of groups")
        if sizes["heads"] * sizes["vdim"] % sizes["norm_groups"]:
            raise ValueError("norm_groups must divide heads * vdim")

    def __init__(self, sizes, weights, prefix, m):
        self.heads, self.vdim, self.n, self.groups = h, v, n, g = sizes["heads"], sizes["vdim"], sizes["state"], sizes["groups"]
        self.taps, self.norm_groups, self.eps = sizes["conv"], sizes["norm_groups"], m.eps
        self.inner = inner = h * v
        self.channels = ch = inner + 2 * g * n
        take = weights.take
        self.w_in = pack([take(prefix + "in", (inner + ch + h, m.width))])
        # per-channel constants in float32, the taps as rows
        self.conv_w = take(prefix + "conv", (ch, self.taps), "vector", 0.3).float().t().contiguous()
        self.conv_b = take(prefix + "conv.b", (ch,), "vector").float().contiguous()
        self.dt_bias = take(prefix + "dt_bias", (h,), "vector").float().contiguous()
        self.neg_a = -torch.exp(take(prefix + "A_log", (h,), "vector").float()).contiguous()
        self.skip = take(prefix + "D", (h,), "norm").float().contiguous()
        self.norm = take(prefix + "norm", (inner,), "norm")
        self.o = take(prefix + "o", (m.width, inner))
        self.dtype = m.dtype
        self.allocate(m.cache)
        self.portions = ChunkedRecurrence(h, g, n, v, m.dtype)
        self.linear, self.recurrence, self.group_norm = hip_op("linear"), hip_op("decayed_recurrence"), hip_op("gated_group_norm")
        self.conv, self.conv_update = hip_op("short_conv"), hip_op("short_conv_update")

    def allocate(self, cache):
        self.state = cache.per_slot(self.heads, self.vdim, recurrence_state_pitch(self.n))
        self.ring = cache.per_slot(self.taps, self.channels, dtype=self.dtype)

    def __call__(self, x, ctx):
        h, v, n, g, inner, ch = self.heads, self.vdim, self.n, self.groups, self.inner, self.channels
        p = self.linear(x, self.w_in)
        z, xbc, dt = p[:, :inner], p[:, inner:inner + ch], p[:, inner + ch:inner + ch + h]
        y = torch.empty((x.shape[0], inner), dtype=x.dtype, device=x.device)
        nd = ctx["n_decode"]
        slots, starts = ctx["state_slots"], ctx["starts"]
        opts = dict(dt_bias=self.dt_bias, neg_a=self.neg_a, skip=self.skip)

        def parts(t):
            return t[:, inner + g * n:inner + 2 * g * n], t[:, inner:inner + g * n], t[:, :inner]

        if nd:   # one token per sequence: the convolution runs inside the recurrence
            q, k, vv = parts(xbc[:nd])
            self.recurrence(q, k, vv, y[:nd], self.state, slots[:nd], starts[:nd], h, g, n, v, dt=dt[:nd],
                            conv=(self.conv_w, self.conv_b, self.ring, (inner + g * n, inner, 0)), **opts)
        if nd < slots.numel():
            c = self.conv(xbc[nd:], self.conv_w, self.conv_b, self.ring, ctx["portion_token_seq"], ctx["portion_cu"], starts[nd:], slots[nd:])
            q, k, vv = parts(c)
            self.portions(q, k, vv, y[nd:], self.state, ctx, dt=dt[nd:], **opts)
            self.conv_update(xbc[nd:], self.ring, ctx["portion_cu"], starts[nd:], slots[nd:])
        y = self.group_norm(y, z, self.norm_groups, self.eps, weight=self.norm, gate_first=True)
        return self.linear(y, self.o)
