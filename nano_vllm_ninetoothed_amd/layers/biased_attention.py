"""Grouped-query attention without rotation: norms over the whole query and key projections, a query factor that grows in steps
with the position, and a linear distance bias per head."""
from __future__ import annotations

import torch

from . import Mixer, hip_op, pack, register_mixer, require_size
from ..mops.hip.attention_ops import biased_matrix_covers, biased_prefill_tiles, padded

LONG_PORTION = 32     # portions of at least this many tokens share reads of keys and values among their queries


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
        self.matrix = biased_matrix_covers(m.dtype, d, v, m.cache.block_size)
        self.linear, self.prepare, self.prefill = hip_op("linear"), hip_op("attention_prepare"), hip_op("biased_prefill")
        self.rows = hip_op("biased_decode" if self.matrix else "biased_attention_rows")
        self.allocate(m.cache)

    def allocate(self, cache):
        self.k_pages = cache.paged(self.kv_heads, padded(self.dim), dtype=self.dtype)
        self.v_pages = cache.paged(self.kv_heads, padded(self.vdim), dtype=self.dtype)

    def __call__(self, x, ctx):
        q = self.prepare(self.linear(x, self.qkv), self.q_norm, self.k_norm, self.eps, ctx["positions32"], ctx["slot_mapping"], self.k_pages, self.v_pages,
                         self.heads, self.kv_heads, self.dim, self.vdim, q_factor=self.q_factor)
        lens, seqs = ctx["token_context"], ctx["token_seq"]
        common = (self.k_pages, self.v_pages, self.dim, self.vdim)
        plan = self._plan(ctx, x.device) if self.matrix else None
        if plan is None:
            o = self.rows(q, *common, lens, ctx["block_tables"], self.scale, slopes=self.slopes, row_seq=seqs)
        else:
            first, tiles = plan
            o = torch.empty((x.shape[0], self.heads, self.vdim), dtype=x.dtype, device=x.device)
            if first:
                self.rows(q[:first], *common, lens[:first], ctx["block_tables"], self.scale, slopes=self.slopes, row_seq=seqs[:first], out=o[:first])
            self.prefill(q, *common, tiles, ctx["block_tables"], self.scale, lens, slopes=self.slopes, out=o)
        return self.linear(o.view(x.shape[0], self.heads * self.vdim), self.o)

    @staticmethod
    def _plan(ctx, device):
        """(first token row, tiles) of the batch's long portions, which come last; None without any.  Shared by the layers of a step."""
        if not ctx["is_prefill"]:
            return None
        if "biased_plan" not in ctx:
            counts, starts = ctx["seq_counts"], ctx["seq_starts"]
            i = next((i for i, n in enumerate(counts) if n >= LONG_PORTION), len(counts))
            plan = None
            if i < len(counts):
                first = sum(counts[:i])
                tiles = biased_prefill_tiles(counts[i:], starts[i:], first, i)
                plan = (first, torch.tensor(tiles, dtype=torch.int32).to(device, non_blocking=True))
            ctx["biased_plan"] = plan
        return ctx["biased_plan"]
