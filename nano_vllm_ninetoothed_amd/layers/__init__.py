"""Sublayers of models that are put together layer by layer from a configuration.

A mixer is built as cls(sizes, weights, prefix, ModelContext) and called as mixer(x, ctx) with x [tokens, width] in the
activation dtype and the batch description ctx of the engine; it returns [tokens, width] and updates its cache or state.
The first ctx["n_decode"] sequences of a batch bring one token each, the others portions of any length.
A feed-forward is built the same way and called as ff(x).
"""
from __future__ import annotations

from dataclasses import dataclass

import torch

from .. import mops

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
    """cos/sin tables [max_positions, dims] (cosines, then sines; float32, angles taken in float64), one per (base, dims)."""

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


def hip_op(name):
    return mops.get_op(name, "hip")


from . import feed_forward, latent_attention, mamba2, retention  # noqa: E402,F401  (register themselves)
