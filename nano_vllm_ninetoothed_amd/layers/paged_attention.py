"""What mixers share that attend to keys and values in pages."""
from __future__ import annotations

import torch

from . import Mixer, hip_op, require_size
from ..mops.hip.attention_ops import biased_matrix_covers, biased_prefill_tiles, padded

LONG_PORTION = 32     # portions of at least this many tokens share reads of keys and values among their queries


class PagedAttention(Mixer):
    """Grouped-query attention: query head h reads key/value head h / (heads / kv_heads).  A subclass sets what becomes of its scores
    (`slopes`: a distance bias per head, `scores`: cap, visible tokens and sinks) and calls attend()."""
    uses_pages, uses_slots = True, False
    slopes = scores = None

    @staticmethod
    def validate(sizes):
        require_size(sizes, "heads", "kv_heads", "dim", "vdim")
        if sizes["heads"] % sizes["kv_heads"]:
            raise ValueError("heads must be a multiple of kv_heads")
        float(sizes["scale"])

    def __init__(self, sizes, m):
        self.heads, self.kv_heads, self.dim, self.vdim = [sizes[n] for n in ("heads", "kv_heads", "dim", "vdim")]
        self.scale, self.eps, self.dtype = float(sizes["scale"]), m.eps, m.dtype
        self.matrix = biased_matrix_covers(m.dtype, self.dim, self.vdim, m.cache.block_size)
        self.linear, self.prefill = hip_op("linear"), hip_op("biased_prefill")
        self.rows = hip_op("biased_decode" if self.matrix else "biased_attention_rows")
        self.allocate(m.cache)

    def allocate(self, cache):
        self.k_pages = cache.paged(self.kv_heads, padded(self.dim), dtype=self.dtype)
        self.v_pages = cache.paged(self.kv_heads, padded(self.vdim), dtype=self.dtype)

    def attend(self, q, ctx, gate=None, out=None, scale=1.0):
        """Attention of all rows of the batch [tokens, heads * vdim], into `out` if given; gate [tokens, heads] or [tokens, heads * vdim]:
        times its sigmoid.  Everything times scale."""
        lens, seqs, table = ctx["token_context"], ctx["token_seq"], ctx["block_tables"]
        common, options = (self.k_pages, self.v_pages, self.dim, self.vdim), {"slopes": self.slopes, "scores": self.scores, "out_scale": scale}
        plan = self._plan(ctx, q.device) if self.matrix else None
        o = torch.empty((q.shape[0], self.heads * self.vdim), dtype=q.dtype, device=q.device) if out is None else out
        if plan is None:
            self.rows(q, *common, lens, table, self.scale, row_seq=seqs, gate=gate, out=o, **options)
        else:
            n, tiles = plan
            if n:
                self.rows(q[:n], *common, lens[:n], table, self.scale, row_seq=seqs[:n], gate=None if gate is None else gate[:n], out=o[:n], **options)
            self.prefill(q, *common, tiles, table, self.scale, lens, gate=gate, out=o, **options)
        return o

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
