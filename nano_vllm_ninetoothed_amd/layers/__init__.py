"""Sublayers of models that are put together layer by layer from a configuration.

A mixer is built as cls(sizes, weights, prefix, ModelContext) and called as mixer(x, ctx) with x [tokens, width] in the
activation dtype and the batch description ctx of the engine; it returns [tokens, width] and updates its cache or state.
The first ctx["n_decode"] sequences of a batch bring one token each, the others portions of any length.
A mixer takes its cache or state in allocate(cache); again(cache) gives another mixer on the same weights with a cache or state of
its own, for layers that run several times in a forward pass.
A feed-forward is built the same way and called as ff(x).  Its result may have several rows per token, one behind the other,
that count as their sum; or be a pair of such a result and one more [tokens, width] that is added.
Sublayers of two products (joined.py) can be run as one where they read the same input.
"""
from __future__ import annotations

import copy
from dataclasses import dataclass

import torch

from .. import mops
from ..mops.hip.recurrent_ops import CHUNK_MAX_DIM, channel_segments, delta_cuts, recurrence_segments

MIXERS: dict = {}
FEED_FORWARDS: dict = {}


def register_mixer(name):
    def decorator(cls):
        MIXERS[name] = cls
        return cls
    return decorator


def register_feed_forward(name):
    def decorator(cls):
        FEED_FORWARDS[name] = cls
        return cls
    return decorator


@dataclass
class ModelContext:
    """What every sublayer of one model shares."""
    width: int
    eps: float
    dtype: torch.dtype
    device: torch.device
    cache: object
    rotary: object


class Mixer:
    def allocate(self, cache) -> None:
        raise NotImplementedError

    def again(self, cache) -> "Mixer":
        other = copy.copy(self)
        other.allocate(cache)
        return other


def require_size(sizes: dict, *names):
    for n in names:
        v = sizes.get(n)
        if not isinstance(v, int) or isinstance(v, bool) or v <= 0:
            raise ValueError(f"{n} must be a positive integer, got {v!r}")


def pack(tensors, multiple: int = 8) -> torch.Tensor:
    """Projections of one input as one weight; zero rows round the row count up, so that row strides of the result are
    multiples of 16 bytes and the GEMM library's aligned path applies."""
    rows = sum(t.shape[0] for t in tensors)
    pad = -rows % multiple
    if pad:
        tensors = [*tensors, torch.zeros((pad, tensors[0].shape[1]), dtype=tensors[0].dtype, device=tensors[0].device)]
    return torch.cat(tensors).contiguous()


class Rotary:
    """Tables over positions: cos/sin tables [max_positions, dims] (cosines, then sines; float32, angles taken in float64), one per (base, dims)."""

    def __init__(self, max_positions: int, device):
        self.max_positions, self.device = max_positions, device
        self._tables: dict = {}

    def table(self, base: float, dims: int) -> torch.Tensor:
        key = (float(base), int(dims))
        if key not in self._tables:
            i = torch.arange(dims // 2, dtype=torch.float64)
            a = torch.outer(torch.arange(self.max_positions, dtype=torch.float64), float(base) ** (-2.0 * i / dims))
            self._tables[key] = torch.cat((a.cos(), a.sin()), dim=-1).float().to(self.device).contiguous()
        return self._tables[key]

    def steps(self, coef: float, every: float) -> torch.Tensor:
        """1 + coef ln(floor((p + 1) / every) + 1) for every position p (float32, taken in float64)."""
        key = ("steps", float(coef), float(every))
        if key not in self._tables:
            p = torch.arange(1, self.max_positions + 1, dtype=torch.float64)
            self._tables[key] = (1 + float(coef) * torch.log(torch.floor(p / float(every)) + 1)).float().to(self.device).contiguous()
        return self._tables[key]


class ChunkedRecurrence:
    """Runs a decayed recurrence over the portions of a batch: in chunks on the matrix cores in bf16, token by token for what
    those kernels do not cover (float32, head sizes beyond theirs)."""
    RECURRENCE, CHUNKS = "decayed_recurrence", "decayed_chunks"

    def __init__(self, heads, groups, d, vd, dtype):
        self.sizes = (heads, groups, d, vd)
        self.chunked = dtype == torch.bfloat16 and d <= CHUNK_MAX_DIM
        self.recurrence, self.chunks = hip_op(self.RECURRENCE), hip_op(self.CHUNKS)

    def segments(self, counts):
        """Host lists: tables of rows, then the bounds of every portion's segments."""
        heads, groups, _, vd = self.sizes
        return recurrence_segments(counts, heads, groups, vd)

    def __call__(self, q, k, v, out, state, ctx, **options):
        """q, k, v, out: the rows of the portions.  The cut into segments is shared by the layers of a step."""
        heads, groups, _, vd = self.sizes
        nd = ctx["n_decode"]
        slots, starts, cu = ctx["state_slots"][nd:], ctx["starts"][nd:], ctx["portion_cu"]
        if not self.chunked:
            return self.recurrence(q, k, v, out, state, slots, starts, *self.sizes, cu_seqlens=cu, **options)
        cuts = ctx.setdefault("segment_cuts", {})
        key = (self.CHUNKS, heads, groups, vd)
        if key not in cuts:
            *tables, bounds = self.segments(ctx["seq_counts"][nd:])
            sizes = [len(t) * len(t[0]) for t in tables] + [len(bounds)]
            flat = torch.tensor([x for t in tables for row in t for x in row] + bounds, dtype=torch.int32).to(v.device, non_blocking=True).split(sizes)
            cuts[key] = [f.view(len(t), -1) for f, t in zip(flat, tables)] + [flat[-1]]
        return self.chunks(q, k, v, out, state, slots, starts, *self.sizes, *cuts[key], cu_seqlens=cu, **options)


class ChannelRecurrence(ChunkedRecurrence):
    """The same for a recurrence with a decay per key channel and a bonus for the current token."""
    CHUNKS = "channel_chunks"

    def segments(self, counts):
        return channel_segments(counts, self.sizes[0], self.sizes[3])


class DeltaRecurrence(ChunkedRecurrence):
    """The same for the gated delta rule; a cut also lists the chunks."""
    RECURRENCE, CHUNKS = "delta_rule", "delta_chunks"

    def segments(self, counts):
        return delta_cuts(counts, self.sizes[0], self.sizes[3])


def hip_op(name):
    return mops.get_op(name, "hip")


from . import (biased_attention, feed_forward, gated_delta, latent_attention, mamba2, matrix_memory, mixture, projected_attention, retention,  # noqa: E402,F401
               rotary_attention, side_by_side, time_mixing)  # (register themselves)
