"""Sublayers of the form W_out f(W_in x) + bias, and several of them with one input as one: their input projections are one product, and
so are their output projections, which add up the sublayers' results in the product's own float32 sums."""
from __future__ import annotations

import torch

from . import Mixer, hip_op, pack


def _columns(w, multiple: int = 8):
    """w [n, k] with zero columns up to a multiple."""
    return torch.nn.functional.pad(w, (0, -w.shape[1] % multiple)).contiguous()


class TwoProducts:
    """A sublayer taken apart.  w_in [rows, width]: its input projections, every one from a multiple of eight rows on; w_out [width,
    columns]: its output projection, its `inner` columns padded with zeros to a multiple of eight; bias: the output's, or None.  Between
    the products mix(p, ctx, out, scale) reads p [tokens, rows] and fills out [tokens, inner], everything times scale."""
    bias = None

    def products(self, into, out_of, bias=None):
        self.blocks, at = [], 0
        for w in into:
            self.blocks.append((at, at + w.shape[0]))
            at += (w.shape[0] + 7) // 8 * 8
        self.w_in, self.w_out = torch.cat([pack([w]) for w in into]).contiguous(), _columns(out_of)
        self.inner, self.bias, self.multiply = out_of.shape[1], bias, hip_op("linear")

    def parts_of(self, p):
        return [p[:, a:b] for a, b in self.blocks]

    def mix(self, p, ctx, out, scale: float = 1.0) -> None:
        raise NotImplementedError

    def unbiased(self, x, ctx):
        columns = self.w_out.shape[1]
        out = (torch.empty if columns == self.inner else torch.zeros)((x.shape[0], columns), dtype=x.dtype, device=x.device)
        self.mix(self.multiply(x, self.w_in), ctx, out[:, :self.inner])
        return self.multiply(out, self.w_out)

    def __call__(self, x, ctx=None):
        y = self.unbiased(x, ctx)
        return y if self.bias is None else y + self.bias.to(y.dtype)


class Joined(TwoProducts, Mixer):
    """The sum of several sublayers' results, each times a factor.  The parts hand their weights over."""

    def __init__(self, parts, scales=None):
        self.parts, self.scales = list(parts), [1.0] * len(parts) if scales is None else [float(s) for s in scales]
        self.rows, self.columns, a, c = [], [], 0, 0
        for p in self.parts:
            self.rows.append((a, a + p.w_in.shape[0]))
            self.columns.append((c, c + p.inner))
            a, c = a + p.w_in.shape[0], c + p.w_out.shape[1]
        self.padded = any(p.inner != p.w_out.shape[1] for p in self.parts) or any(getattr(p, "padded", False) for p in self.parts)
        self.w_in, self.w_out = torch.cat([p.w_in for p in self.parts]), torch.cat([p.w_out for p in self.parts], dim=1).contiguous()
        self.inner, self.multiply = self.w_out.shape[1], hip_op("linear")
        biases = [p.bias.float() * s for p, s in zip(self.parts, self.scales) if p.bias is not None]
        self.bias = sum(biases[1:], biases[0]).contiguous() if biases else None
        for p in self.parts:
            p.w_in = p.w_out = None

    def allocate(self, cache):
        self.parts = [p.again(cache) if isinstance(p, Mixer) else p for p in self.parts]

    def mix(self, p, ctx, out, scale: float = 1.0):
        for part, s, (a, b), (c, d) in zip(self.parts, self.scales, self.rows, self.columns):
            part.mix(p[:, a:b], ctx, out[:, c:d], s * scale)

    def unbiased(self, x, ctx):
        out = (torch.zeros if self.padded else torch.empty)((x.shape[0], self.inner), dtype=x.dtype, device=x.device)
        self.mix(self.multiply(x, self.w_in), ctx, out)
        return self.multiply(out, self.w_out)
