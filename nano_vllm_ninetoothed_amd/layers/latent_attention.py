"""Latent attention: queries, keys and values go through low-rank latents; the cache holds one latent row and one rotated
key part per token, shared by all heads."""
from __future__ import annotations

import torch

from . import Mixer, hip_op, pack, register_mixer, require_size
from ..mops.hip.recurrent_ops import latent_decode_covers, latent_prefill_covers, latent_prefill_plan

EXPAND_FROM = 64     # portions of at least this many tokens expand keys and values instead of absorbing the projections


def pad_rows(w, rows):
    """w [heads, n, k] with zero rows up to `rows` per head."""
    return torch.nn.functional.pad(w, (0, 0, 0, rows - w.shape[1]))


@register_mixer("latent_attention")
class LatentAttention(Mixer):
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
        # queries leave the projection with both parts of a head padded to multiples of eight: [dim | 0 | rot_dim | 0]
        self.dim_pad, self.rot_pad = dp, rp = (d + 7) // 8 * 8, (r + 7) // 8 * 8
        uq = take(prefix + "uq", (h * (d + r), qr)).view(h, d + r, qr)
        self.uq = torch.cat((pad_rows(uq[:, :d], dp), pad_rows(uq[:, d:], rp)), dim=1).reshape(h * (dp + rp), qr).contiguous()
        uk, uv = take(prefix + "uk", (h * d, kr)), take(prefix + "uv", (h * v, kr))
        self.q_to_latent = uk.view(h, d, kr).transpose(1, 2).contiguous()     # [H, kv_rank, dim]
        self.latent_to_v = uv.view(h, v, kr)                                  # [H, vdim, kv_rank]
        self.o = take(prefix + "o", (m.width, h * v))
        self.dtype = m.dtype
        self.allocate(m.cache)
        self.cos_sin = m.rotary.table(sizes["rot"]["base"], r)
        self.linear, self.prepare, self.head_linear = hip_op("linear"), hip_op("latent_prepare"), hip_op("head_linear")
        self.rows = hip_op("latent_decode" if latent_decode_covers(m.dtype, kr, r, m.cache.block_size) else "latent_attention_rows")
        self.expands = latent_prefill_covers(m.dtype, d, r, v)
        if self.expands:
            # the expansion reads gathered latents whose row length is a multiple of eight, and gives keys in the queries' layout
            pad = -kr % 8
            self.w_k = torch.nn.functional.pad(pad_rows(uk.view(h, d, kr), dp), (0, pad)).reshape(h * dp, kr + pad).contiguous()
            self.w_v = torch.nn.functional.pad(uv, (0, pad)).contiguous()
            self.gather, self.rotate, self.prefill = hip_op("latent_gather"), hip_op("rotate_pairs"), hip_op("latent_prefill")

    def allocate(self, cache):
        self.pages = cache.paged((self.kv_rank + self.rot_dim + 7) // 8 * 8, dtype=self.dtype)

    def __call__(self, x, ctx):
        h, d, r, v = self.heads, self.dim, self.rot_dim, self.vdim
        t = x.shape[0]
        down = self.linear(x, self.down)
        cq = self.prepare(down, self.q_norm, self.kv_norm, self.eps, self.cos_sin, ctx["positions32"], ctx["slot_mapping"], self.pages,
                          self.q_rank, self.kv_rank, r)
        q = self.linear(cq, self.uq).view(t, h, self.dim_pad + self.rot_pad)
        plan = self._plan(ctx, x.device) if self.expands else None
        if plan is None:
            o = self._absorbed(q, ctx["token_context"], ctx["token_seq"], ctx)
        else:
            first = plan[0]
            o = torch.empty((t, h, v), dtype=x.dtype, device=x.device)
            if first:
                o[:first] = self._absorbed(q[:first], ctx["token_context"][:first], ctx["token_seq"][:first], ctx)
            self._expanded(q, plan, ctx, o)
        return self.linear(o.reshape(t, h * v), self.o)

    def _absorbed(self, q, context_lens, row_seq, ctx):
        """Query rows against the cache in the latent space: cheap per row, no key or value is ever expanded."""
        q_latent = self.head_linear(q[..., :self.dim], self.q_to_latent)
        o = self.rows(q_latent, q[..., self.dim_pad:self.dim_pad + self.rot_dim], self.pages, self.cos_sin, context_lens, ctx["block_tables"], self.scale, row_seq)
        return self.head_linear(o, self.latent_to_v)

    def _plan(self, ctx, device):
        """(first token row, row_seq, row_pos, tiles) of the batch's long portions, which come last; None without any.
        Shared by the layers of a step."""
        if not ctx["is_prefill"]:
            return None
        if "latent_plan" not in ctx:
            counts, starts = ctx["seq_counts"], ctx["seq_starts"]
            i = next((i for i, n in enumerate(counts) if n >= EXPAND_FROM), len(counts))
            plan = None
            if i < len(counts):
                first = sum(counts[:i])
                row_seq, row_pos, tiles = latent_prefill_plan(counts[i:], starts[i:], first, i)
                n = len(row_pos)
                flat = torch.tensor(row_seq + row_pos + [x for t in tiles for x in t], dtype=torch.int32).to(device, non_blocking=True)
                plan = (first, flat[:n], flat[n:2 * n], flat[2 * n:].view(-1, 5))
            ctx["latent_plan"] = plan
        return ctx["latent_plan"]

    def _expanded(self, q, plan, ctx, out):
        """Long portions: keys and values of the whole context are expanded once, then ordinary attention."""
        first, row_seq, row_pos, tiles = plan
        c, kr = self.gather(self.pages, ctx["block_tables"], row_seq, row_pos, self.kv_rank, self.rot_dim)
        k = self.linear(c, self.w_k)
        vt = self.linear(self.w_v, c)
        self.rotate(q[first:, :, self.dim_pad:self.dim_pad + self.rot_dim], ctx["positions32"][first:], self.cos_sin)
        self.prefill(q, k, kr, vt, tiles, self.scale, out)
