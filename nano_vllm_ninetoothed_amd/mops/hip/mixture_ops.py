"""Extension ops of the `hip` backend for mixtures of experts: routing and grouped products (the rules of recurrent_ops.py hold).
Nothing comes back to the host, so that a captured step routes anew at every replay."""
from __future__ import annotations

from ctypes import byref
from dataclasses import dataclass

import torch

from ... import _capi
from .ops import _require, _stream
from .recurrent_ops import _dtype, _flat, _rows
from .registry import register_hip_op

SMALL_BLOCK, LARGE_BLOCK = 32, 128


@dataclass
class Routing:
    """Where every token goes: chosen experts and their scores [tokens, top], the choices ordered by expert, blocks of them."""
    args: object
    chosen: torch.Tensor
    score: torch.Tensor
    rows: torch.Tensor
    tiles: torch.Tensor

    @property
    def takes_common(self) -> bool:
        """Whether the products take a unit that all tokens share along."""
        return self.args.dtype == 0 and self.args.block_rows == SMALL_BLOCK


@dataclass(frozen=True)
class CommonUnit:
    """A unit of clamped_glu's form that every token goes through: gate_up [2 * up_at or more, width] with gate rows from 0 and up rows
    from up_at on, down [width, ff]."""
    gate_up: torch.Tensor
    down: torch.Tensor
    ff: int
    up_at: int
    limit: float


@dataclass(frozen=True)
class Weighted:
    """The weighted form of routing: experts chosen by sigmoid + correction (float32 [experts]) among those of the `keep` best of `groups`
    equal groups of neighbours (by the sum of a group's two best); a choice's weight is its sigmoid over the sum of the chosen ones,
    times factor."""
    correction: torch.Tensor
    groups: int = 1
    keep: int = 1
    factor: float = 1.0


@register_hip_op
def moe_route(h: torch.Tensor, router: torch.Tensor, top: int, block_rows: int = None, weighted: Weighted = None) -> Routing:
    """The `top` experts with the largest logits router @ h (float32) per token, their sigmoids, and the plan of the grouped products.
    weighted: another choice, and weights instead of sigmoids; moe_gate_up then leaves its inputs as they are, and moe_down multiplies
    its results."""
    code = _dtype("h", h)
    tokens, (experts, width) = h.shape[0], router.shape
    stride = _rows("h", h, width, h.dtype)
    _require(0 < top <= experts, "top must lie between 1 and the number of experts")
    if block_rows is None:
        block_rows = LARGE_BLOCK if h.dtype == torch.bfloat16 and tokens * top >= 48 * experts else SMALL_BLOCK
    lib = _capi.load()
    n = tokens * top
    tiles = lib.mops_hip_moe_max_tiles(tokens, experts, top, block_rows)
    sizes = [lib.mops_hip_moe_route_workgroups(tokens) * experts, n, n, n, 1 + 3 * tiles]      # the counts first: their rows are aligned
    counts, chosen, rank, rows, tile_list = torch.empty(sum(sizes), dtype=torch.int32, device=h.device).split(sizes)
    score = torch.empty((tokens, top), dtype=torch.float32, device=h.device)
    m = _capi.Moe()
    m.rows, m.tiles, m.score = rows.data_ptr(), tile_list.data_ptr(), score.data_ptr()
    m.tokens, m.experts, m.top, m.width, m.ff, m.block_rows, m.dtype = tokens, experts, top, width, 1, block_rows, code
    if weighted is not None:
        m.correction = _flat("correction", weighted.correction, experts, torch.float32)
        m.groups, m.keep, m.factor = weighted.groups, weighted.keep, weighted.factor
    st = lib.mops_hip_moe_route(h.data_ptr(), stride, _flat("router", router, experts * width, h.dtype), chosen.data_ptr(), rank.data_ptr(), counts.data_ptr(),
                                byref(m), _stream(h))
    _capi.check("mops_hip_moe_route", st)
    return Routing(m, chosen.view(tokens, top), score, rows, tile_list)


@register_hip_op
def moe_gate_up(h: torch.Tensor, w: torch.Tensor, routing: Routing, limit: float = None, alpha: float = 1.702, common: CommonUnit = None):
    """silu(s W_gate h) * (s W_up h) of every choice, s its score, in the order of routing.rows.  w [experts, 2, ff, width].  With a
    limit the unit of clamped_glu instead, which takes no score; with a common unit (routing.takes_common) a pair, the second what
    that unit makes of every token."""
    code = _dtype("h", h)
    m = routing.args
    experts, two, ff, width = w.shape
    _require(m.tokens == h.shape[0] and m.experts == experts and m.width == width and m.dtype == code and two == 2, "the routing was made for another problem")
    m.ff, m.unit = ff, 0 if limit is None else 1
    m.limit, m.alpha = limit or 0.0, alpha
    y = torch.empty((m.tokens * m.top, ff), dtype=h.dtype, device=h.device)
    yc = None if common is None else torch.empty((m.tokens, common.ff), dtype=h.dtype, device=h.device)
    if common is not None:
        _require(limit is not None and common.gate_up.shape[0] >= common.up_at + common.ff, "a common unit comes with limits, and with all its rows")
        _set_common(m, h, _rows("h", h, width, h.dtype), _flat("gate_up", common.gate_up, common.gate_up.shape[0] * width, h.dtype), yc, common)
    st = _capi.load().mops_hip_moe_gate_up(h.data_ptr(), _rows("h", h, width, h.dtype), _flat("w", w, w.numel(), h.dtype), ff, y.data_ptr(), ff, byref(m), _stream(h))
    m.common_w = None
    _capi.check("mops_hip_moe_gate_up", st)
    return y if common is None else (y, yc)


def _set_common(m, x, x_stride, w, out, common):
    m.common_x, m.common_x_stride, m.common_w = x.data_ptr(), x_stride, w
    m.common_out, m.common_out_stride = out.data_ptr(), out.shape[1]
    m.common_ff, m.common_up_at, m.common_limit = common.ff, common.up_at, common.limit


@register_hip_op
def moe_down(y: torch.Tensor, w: torch.Tensor, routing: Routing, common: CommonUnit = None, common_y: torch.Tensor = None):
    """W_down y of every choice, times its weight if the routing has weights: [tokens * top, width], a token's choices one behind the
    other.  w [experts, width, ff].  common, common_y: the unit and its result of moe_gate_up; then a pair, the second what the unit
    adds per token."""
    code = _dtype("y", y)
    m = routing.args
    experts, width, ff = w.shape
    _require(y.shape == (m.tokens * m.top, ff) and y.is_contiguous() and m.experts == experts and m.width == width and m.dtype == code,
             "the routing was made for another problem")
    m.ff = ff
    z = torch.empty((m.tokens * m.top, width), dtype=y.dtype, device=y.device)
    zc = None if common is None else torch.empty((m.tokens, width), dtype=y.dtype, device=y.device)
    if common is not None:
        _require(common_y.shape[0] == m.tokens, "common_y must have a row per token")
        _set_common(m, common_y, _rows("common_y", common_y, common.ff, y.dtype), _flat("down", common.down, width * common.ff, y.dtype), zc, common)
    st = _capi.load().mops_hip_moe_down(y.data_ptr(), ff, _flat("w", w, w.numel(), y.dtype), ff, z.data_ptr(), width, byref(m), _stream(y))
    m.common_w = None
    _capi.check("mops_hip_moe_down", st)
    return z if common is None else (z, zc)


@register_hip_op
def grouped_linear(x: torch.Tensor, w: torch.Tensor, w_last: torch.Tensor = None):
    """y[g] = x[g] @ w[g].T for x [groups, tokens, k] and w [groups, n, k] (bf16, contiguous) in one launch, for small batches.  w_last
    [at most n, k]: weights of one more group of rows behind them; then (y, y_last)."""
    groups, n, k = w.shape
    tokens = x.shape[1]
    _require(x.dim() == 3 and x.shape[0] == groups + (w_last is not None) and x.shape[2] == k, "x must be [groups, tokens, k]")
    y = torch.empty((groups, tokens, n), dtype=x.dtype, device=x.device)
    last = None if w_last is None else torch.empty((tokens, w_last.shape[0]), dtype=x.dtype, device=x.device)
    st = _capi.load().mops_hip_grouped_linear(_flat("x", x, x.numel(), torch.bfloat16), _flat("w", w, w.numel(), torch.bfloat16), y.data_ptr(),
                                              None if last is None else _flat("w_last", w_last, w_last.shape[0] * k, torch.bfloat16),
                                              None if last is None else last.data_ptr(), 0 if last is None else w_last.shape[0], groups, tokens, n, k, _stream(x))
    _capi.check("mops_hip_grouped_linear", st)
    return y if last is None else (y, last)
