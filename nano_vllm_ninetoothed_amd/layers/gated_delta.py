"""The gated delta rule: a matrix state per head decays by a factor per key channel and token, and a write replaces part of what the
state holds under its key; short convolutions in front of queries, keys and values, unit queries and keys, a gated norm per head."""
from __future__ import annotations

import torch

from . import DeltaRecurrence, Mixer, hip_op, register_mixer, require_size
from .joined import TwoProducts
from ..mops.hip.recurrent_ops import recurrence_state_pitch

UNIT_EPS = 1e-6      # under the root of a unit vector's length


@register_mixer("gated_delta")
class GatedDelta(TwoProducts, Mixer):
    uses_pages, uses_slots = False, True

    @staticmethod
    def validate(sizes):
        require_size(sizes, "heads", "kv_heads", "dim", "vdim", "conv")
        if sizes["heads"] % sizes["kv_heads"]:
            raise ValueError("heads must be a multiple of kv_heads")

    def __init__(self, sizes, weights, prefix, m):
        self.heads, self.groups, self.dim, self.vdim, self.taps = h, g, d, v, taps = [sizes[n] for n in ("heads", "kv_heads", "dim", "vdim", "conv")]
        self.eps, self.dtype = m.eps, m.dtype
        take = weights.take
        rows = {"q": g * d, "k": g * d, "v": h * v}
        self.channels = sum(rows.values())
        # the sizes of the two-step projections are the tensors' own
        low = {n: (weights.shape_of(prefix + n) or (max(16, m.width // 32),))[0] for n in ("a1", "g1")}
        into = [torch.cat([take(prefix + n, (k, m.width)) for n, k in rows.items()]), take(prefix + "b", (h, m.width))]
        into += [take(prefix + n, (r, m.width)) for n, r in low.items()]
        self.products(into, take(prefix + "o", (m.width, h * v)))
        # the taps as rows, in float32
        self.conv_w = torch.cat([take(f"{prefix}{n}.conv", (k, taps), "vector", 0.3) for n, k in rows.items()]).float().t().contiguous()
        self.a2, self.g2 = take(prefix + "a2", (h * d, low["a1"])).contiguous(), take(prefix + "g2", (h * v, low["g1"])).contiguous()
        self.dt_bias = take(prefix + "dt_bias", (h * d,), "vector").float().contiguous()
        self.rate = -torch.exp(take(prefix + "A_log", (h,), "vector").float()).contiguous()
        self.norm = take(prefix + "norm", (v,), "norm")
        self.portions = DeltaRecurrence(h, g, d, v, m.dtype)
        self.recurrence, self.conv, self.conv_update = hip_op("delta_rule"), hip_op("short_conv"), hip_op("short_conv_update")
        self.decay, self.group_norm = hip_op("low_rank_decay"), hip_op("gated_group_norm")
        self.allocate(m.cache)

    def allocate(self, cache):
        self.state = cache.per_slot(self.heads, self.vdim, recurrence_state_pitch(self.dim))
        self.ring = cache.per_slot(self.taps, self.channels, dtype=self.dtype)

    def mix(self, p, ctx, out, scale=1.0):
        h, g, d, v = self.heads, self.groups, self.dim, self.vdim
        qkv, beta, a, z = self.parts_of(p)
        log_decay, gate = self.decay(a, self.a2, self.dt_bias, rate=self.rate), self.multiply(z, self.g2)
        o = torch.empty((p.shape[0], h * v), dtype=p.dtype, device=p.device)
        nd, slots, starts = ctx["n_decode"], ctx["state_slots"], ctx["starts"]
        sizes, at = (h, g, d, v), (0, g * d, 2 * g * d)

        def parts(t):
            return t[:, :at[1]], t[:, at[1]:at[2]], t[:, at[2]:]

        def options(rows):
            return dict(log_decay=log_decay[rows], beta=beta[rows], q_scale=d ** -0.5, unit_eps=UNIT_EPS)

        if nd:      # one token per sequence: the convolutions run inside the recurrence
            self.recurrence(*parts(qkv[:nd]), o[:nd], self.state, slots[:nd], starts[:nd], *sizes, conv=(self.conv_w, self.ring, at), **options(slice(nd)))
        if nd < slots.numel():
            cu = ctx["portion_cu"]
            c = self.conv(qkv[nd:], self.conv_w, None, self.ring, ctx["portion_token_seq"], cu, starts[nd:], slots[nd:])
            self.portions(*parts(c), o[nd:], self.state, ctx, **options(slice(nd, None)))
            self.conv_update(qkv[nd:], self.ring, cu, starts[nd:], slots[nd:])
        self.group_norm(o, gate, h, self.eps, weight=self.norm, activation="sigmoid", scale=scale, out=out)
