"""Latent attention: queries, keys and values go through low-rank latents; the cache holds one latent row and one rotated
key part per token, shared by all heads."""
from __future__ import annotations

import torch

from . import hip_op, pack, register_mixer, require_size


@register_mixer("latent_attention")
class LatentAttention:
    uses_pages, uses_slots = True, False

    @staticmethod
    def validate(sizes):
        require_size(sizes, "heads", "dim", "rot_dim", "vdim", "q_rank", "kv_rank")
        if sizes["rot"]["dims"] != sizes["rot_dim"] or sizes["rot_dim"] % 2:
            raise ValueError("rot.dims must equal rot_dim and be even")
        float(sizes["scale"])

    def __init__(self, sizes, weights, prefix, m):
        self.heads, self.dim, self.rot_dim, self.vdim = h, d, r, v = sizes["heads"], sizes["dim"], sizes["rot_dim"], sizes["vdim"]
        self.q_rank, self.kv_rank, self.scale, self.eps = qr, kr, _, _ = sizes["q_rank"], sizes["kv_rank"], float(sizes["scale"]), m.eps
        take = weights.take
        self.down = pack([take(prefix + "dq", (qr, m.width)), take(prefix + "dkv", (kr + r, m.width))])
        self.q_norm = take(prefix + "dq.norm", (qr,), "norm")
        self.kv_norm = take(prefix + "dkv.norm", (kr,), "norm")
        self.uq = pack([take(prefix + "uq", (h * (d + r), qr))])
        uk, uv = take(prefix + "uk", (h * d, kr)), take(prefix + "uv", (h * v, kr))
        self.q_to_latent = uk.view(h, d, kr).transpose(1, 2).contiguous()     # [H, kv_rank, dim]
        self.latent_to_v = uv.view(h, v, kr)                                  # [H, vdim, kv_rank]
        self.o = take(prefix + "o", (m.width, h * v))
        self.pages = m.cache.paged((kr + r + 7) // 8 * 8, dtype=m.dtype)
        self.cos_sin = m.rotary.table(sizes["rot"]["base"], r)
        self.linear, self.prepare, self.head_linear = hip_op("linear"), hip_op("latent_prepare"), hip_op("head_linear")
        self.rows = hip_op("latent_attention_rows")

    def __call__(self, x, ctx):
        h, d, r, v = self.heads, self.dim, self.rot_dim, self.vdim
        t = x.shape[0]
        down = self.linear(x, self.down)
        cq = self.prepare(down, self.q_norm, self.kv_norm, self.eps, self.cos_sin, ctx["positions32"], ctx["slot_mapping"], self.pages,
                          self.q_rank, self.kv_rank, r)
        q = self.linear(cq, self.uq)[:, :h * (d + r)].unflatten(1, (h, d + r))
        o = self._absorbed(q, ctx["token_context"], ctx["token_seq"], ctx)
        return self.linear(o.reshape(t, h * v), self.o)

    def _absorbed(self, q, context_lens, row_seq, ctx):
        """Query rows against the cache in the latent space: cheap per row, no key or value is ever expanded."""
        q_latent = self.head_linear(q[..., :self.dim], self.q_to_latent)
        o = self.rows(q_latent, q[..., self.dim:], self.pages, self.cos_sin, context_lens, ctx["block_tables"], self.scale, row_seq)
        return self.head_linear(o, self.latent_to_v)
