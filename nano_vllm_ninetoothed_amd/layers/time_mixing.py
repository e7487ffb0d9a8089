"""Time mixing: every projection reads its own blend of a token and the one in front of it; a matrix state per head decays by a
factor per key channel and token, and a bonus weighs the current token."""
from __future__ import annotations

import torch

from . import ChannelRecurrence, Mixer, hip_op, pack, register_mixer, require_size
from ..mops.hip.recurrent_ops import recurrence_state_pitch

GROUPED_ROWS = 256      # 16-bit batches up to this many tokens run all projections as one launch


@register_mixer("time_mixing")
class TimeMixing(Mixer):
    uses_pages, uses_slots = False, True

    @staticmethod
    def validate(sizes):
        require_size(sizes, "heads", "dim")

    def __init__(self, sizes, weights, prefix, m):
        self.heads, self.dim, self.eps = h, d, _ = sizes["heads"], sizes["dim"], m.eps
        self.width, self.dtype, self.inner = m.width, m.dtype, h * d
        take = weights.take
        self.mu = torch.stack([take(prefix + "mu." + n, (m.width,), "vector") for n in "rkvgw"]).float().contiguous()
        self.rkvg = torch.stack([take(prefix + n, (h * d, m.width)) for n in "rkvg"]).contiguous()
        self.each = list(self.rkvg.unbind(0))
        rank = (weights.shape_of(prefix + "w1") or (max(16, m.width // 32),))[0]      # the tensors alone say it
        self.rank = rank
        self.w1 = pack([take(prefix + "w1", (rank, m.width))])
        self.w2 = take(prefix + "w2", (h * d, rank)).contiguous()
        self.w0 = take(prefix + "w0", (h * d,), "vector").float().contiguous()
        self.bonus = take(prefix + "u", (h, d), "vector").float().reshape(-1).contiguous()
        self.norm = take(prefix + "norm", (h * d,), "norm")
        self.o = take(prefix + "o", (m.width, h * d))
        self.portions = ChannelRecurrence(h, h, d, d, m.dtype)
        self.linear, self.grouped_linear, self.mix = hip_op("linear"), hip_op("grouped_linear"), hip_op("token_mix")
        self.grouped_rows = GROUPED_ROWS if m.dtype == torch.bfloat16 and self.w1.shape[0] <= h * d else 0
        self.decay, self.recurrence, self.group_norm = hip_op("low_rank_decay"), hip_op("decayed_recurrence"), hip_op("gated_group_norm")
        self.allocate(m.cache)

    def allocate(self, cache):
        self.state = cache.per_slot(self.heads, self.dim, recurrence_state_pitch(self.dim))
        self.before = cache.per_slot(self.width, dtype=self.dtype)

    def __call__(self, x, ctx):
        h, d = self.heads, self.dim
        t, nd = x.shape[0], ctx["n_decode"]
        slots, starts = ctx["state_slots"], ctx["starts"]
        mixes = self.mix(x, self.mu, self.before, starts, slots, ctx["token_seq"], ctx["cu_seqlens"])
        if t <= self.grouped_rows:
            (r, k, v, gate), z = self.grouped_linear(mixes, self.rkvg, self.w1)
        else:
            r, k, v, gate = (self.linear(mixes[i], self.each[i]) for i in range(4))
            z = self.linear(mixes[4], self.w1)
        log_decay = self.decay(z[:, :self.rank], self.w2, self.w0)
        o = torch.empty((t, self.inner), dtype=x.dtype, device=x.device)
        if nd:
            self.recurrence(r[:nd], k[:nd], v[:nd], o[:nd], self.state, slots[:nd], starts[:nd], h, h, d, d, channel_decay=log_decay[:nd], bonus=self.bonus)
        if nd < slots.numel():
            self.portions(r[nd:], k[nd:], v[nd:], o[nd:], self.state, ctx, channel_decay=log_decay[nd:], bonus=self.bonus)
        return self.linear(self.group_norm(o, gate, h, self.eps, weight=self.norm), self.o)
