"""Extension ops of the `hip` backend for models with recurrent layers, latent attention and a float32 residual stream.
They run in bfloat16 and in float32 (the tensors' dtype decides); the rules of ops.py hold: layouts are checked here with
exceptions, outputs come from the torch allocator, everything runs on the current stream and nothing synchronises.
"""
from __future__ import annotations

from ctypes import byref
from dataclasses import dataclass

import torch

from ... import _capi
from .ops import _require, _stream
from .registry import register_hip_op

_DTYPES = {torch.bfloat16: 0, torch.float32: 1}


def _dtype(name: str, t: torch.Tensor) -> int:
    if not t.is_cuda:
        raise ValueError(f"{name} must live on the GPU")
    code = _DTYPES.get(t.dtype)
    if code is None:
        raise ValueError(f"{name} must be bfloat16 or float32, got {t.dtype}")
    return code


def _rows(name: str, t: torch.Tensor, cols: int, dtype: torch.dtype) -> int:
    """Checks a 2-D tensor with contiguous rows of `cols` elements; returns its row stride."""
    if not (t.is_cuda and t.dim() == 2 and t.shape[1] == cols and t.dtype == dtype and (t.stride(1) == 1 or cols == 1)):
        raise ValueError(f"{name} must be a GPU tensor [rows, {cols}] of {dtype} with contiguous rows, got {tuple(t.shape)} {t.dtype}")
    return t.stride(0) if t.shape[0] > 1 else max(t.stride(0), cols)


def _flat(name: str, t: torch.Tensor, n: int, dtype: torch.dtype) -> int:
    """Checks a contiguous tensor of n elements; returns its address."""
    if not (t.is_cuda and t.numel() == n and t.dtype == dtype and t.is_contiguous()):
        raise ValueError(f"{name} must be a contiguous GPU tensor of {n} x {dtype}, got {tuple(t.shape)} {t.dtype}")
    return t.data_ptr()


@register_hip_op
def embed_residual(ids: torch.Tensor, table: torch.Tensor, scale: float = 1.0, need_act: bool = True, act=None):
    """Scaled embedding rows as (float32 residual, activation copy in the table's dtype or None); act: rows for the copy."""
    code = _dtype("table", table)
    _require(table.dim() == 2 and table.stride(1) == 1, "table must be [vocab, width] with contiguous rows")
    _require(ids.is_cuda and ids.dtype == torch.int64 and ids.dim() == 1 and ids.is_contiguous(), "ids must be a contiguous int64 GPU vector")
    n, (vocab, width) = ids.numel(), table.shape
    residual = torch.empty((n, width), dtype=torch.float32, device=table.device)
    if act is None and need_act:
        act = torch.empty((n, width), dtype=table.dtype, device=table.device)
    act_stride = width if act is None else _rows("act", act, width, table.dtype)
    _require(act is None or act.shape[0] == n, "act must have one row per id")
    st = _capi.load().mops_hip_embed_residual(ids.data_ptr(), table.data_ptr(), table.stride(0), code, float(scale), residual.data_ptr(),
                                              None if act is None else act.data_ptr(), act_stride, n, vocab, width, _stream(table))
    _capi.check("mops_hip_embed_residual", st)
    return residual, act


@register_hip_op
def embed_pairs(ids, table, pairs, mul_prev: int, mul_cur: int, before, starts, state_slots, token_seq=None, cu_seqlens=None, scale: float = 1.0):
    """float32 residual: scaled embedding rows plus a row of `pairs` [buckets + 1, width], picked by a hash of the token and the one in
    front of it (the last row for a sequence's first token).  `before` [slots] int32 holds each sequence's last token of earlier steps
    and receives the new one.  Without cu_seqlens every sequence brings one token."""
    _require(table.dim() == 2 and pairs.dim() == 2 and table.shape[1] == pairs.shape[1] and pairs.shape[0] > 1, "table and pairs must be [rows, width]")
    n, (vocab, width), batch = ids.numel(), table.shape, state_slots.numel()
    _require((token_seq is None) == (cu_seqlens is None) and (cu_seqlens is not None or n == batch), "packed portions need token_seq and cu_seqlens")
    a = _capi.EmbedPairs()
    a.dtype, a.scale = _dtype("table", table), float(scale)
    a.ids = _flat("ids", ids, n, torch.int64)
    a.table, a.table_stride, a.pairs, a.pairs_stride = table.data_ptr(), _rows("table", table, width, table.dtype), pairs.data_ptr(), _rows("pairs", pairs, width, table.dtype)
    a.buckets, a.mul_prev, a.mul_cur = pairs.shape[0] - 1, mul_prev, mul_cur
    a.before, a.num_slots = _flat("before", before, before.numel(), torch.int32), before.numel()
    if cu_seqlens is not None:
        a.token_seq, a.cu_seqlens = _flat("token_seq", token_seq, n, torch.int32), _flat("cu_seqlens", cu_seqlens, batch + 1, torch.int32)
    a.starts, a.state_slots = _flat("starts", starts, batch, torch.int32), _flat("state_slots", state_slots, batch, torch.int32)
    residual = torch.empty((n, width), dtype=torch.float32, device=table.device)
    a.residual, a.tokens, a.vocab, a.width = residual.data_ptr(), n, vocab, width
    st = _capi.load().mops_hip_embed_pairs(byref(a), _stream(table))
    _capi.check("mops_hip_embed_pairs", st)
    return residual


@register_hip_op
def norm_residual_add(residual: torch.Tensor, y: torch.Tensor, weight: torch.Tensor, eps: float, weight_offset: float = 0.0):
    """residual += rms(y) * (weight_offset + weight), in place; returns the new residual in y's dtype."""
    code = _dtype("y", y)
    rows, n = residual.shape
    _flat("residual", residual, rows * n, torch.float32)
    stride = _rows("y", y, n, y.dtype)
    _require(y.shape[0] == rows, "y must have as many rows as the residual")
    act = torch.empty((rows, n), dtype=y.dtype, device=y.device)
    st = _capi.load().mops_hip_norm_residual_add(residual.data_ptr(), y.data_ptr(), stride, _flat("weight", weight, n, y.dtype),
                                                 float(weight_offset), float(eps), act.data_ptr(), code, rows, n, _stream(y))
    _capi.check("mops_hip_norm_residual_add", st)
    return act


@register_hip_op
def add_norm_norm(residual: torch.Tensor, y: torch.Tensor, w_out: torch.Tensor, w_in: torch.Tensor, eps: float, center: bool = False, extra=None):
    """residual += rms(y) * w_out in place; returns rms(residual) * w_in in y's dtype.  y [rows * parts, n]: `parts` consecutive
    rows are summed first (the outputs of several experts), and those of extra [rows, n] with them.  center: layer norms instead
    of RMS norms."""
    code = _dtype("y", y)
    rows, n = residual.shape
    parts = y.shape[0] // rows if rows else 1
    _flat("residual", residual, rows * n, torch.float32)
    stride = _rows("y", y, n, y.dtype)
    _require(parts > 0 and y.shape[0] == rows * parts, "y must have a whole number of rows per residual row")
    out = torch.empty((rows, n), dtype=y.dtype, device=y.device)
    st = _capi.load().mops_hip_add_norm_norm(residual.data_ptr(), y.data_ptr(), stride, parts, None if extra is None else _flat("extra", extra, rows * n, y.dtype),
                                             _flat("w_out", w_out, n, y.dtype), _flat("w_in", w_in, n, y.dtype), float(eps), 1 if center else 0,
                                             out.data_ptr(), code, rows, n, _stream(y))
    _capi.check("mops_hip_add_norm_norm", st)
    return out


@register_hip_op
def add_norm(residual: torch.Tensor, y=None, shift=None, replace: bool = False, weight=None, bias=None, eps: float = 0.0, center: bool = False, out=None,
             dtype=None):
    """residual += y + shift in place (replace: = y + shift; shift: float32 vector); returns norm(residual) * weight + bias, or the residual
    without weight, in the dtype of `out` (rows to fill), of weight or `dtype`.  center: layer norms instead of RMS norms."""
    rows, n = residual.shape
    dtype = out.dtype if out is not None else (weight.dtype if weight is not None else dtype)
    if out is None:
        out = torch.empty((rows, n), dtype=dtype, device=residual.device)
    a = _capi.AddNorm()
    a.residual, a.rows, a.n = _flat("residual", residual, rows * n, torch.float32), rows, n
    if y is not None:
        a.y, a.y_stride = y.data_ptr(), _rows("y", y, n, dtype)
        _require(y.shape[0] == rows, "y must have as many rows as the residual")
    if shift is not None:
        a.shift = _flat("shift", shift, n, torch.float32)
    if weight is not None:
        a.w = _flat("weight", weight, n, dtype)
    if bias is not None:
        a.b = _flat("bias", bias, n, dtype)
    a.out, a.out_stride = out.data_ptr(), _rows("out", out, n, dtype)
    _require(out.shape[0] == rows, "out must have as many rows as the residual")
    a.eps, a.replace, a.center, a.dtype = float(eps), 1 if replace else 0, 1 if center else 0, _dtype("out", out)
    st = _capi.load().mops_hip_add_norm(byref(a), _stream(residual))
    _capi.check("mops_hip_add_norm", st)
    return out


@register_hip_op
def layer_norm_f32(x: torch.Tensor, weight: torch.Tensor, eps: float):
    """(x - mean) / sqrt(variance + eps) * weight of float32 rows, in the weight's dtype."""
    code = _dtype("weight", weight)
    rows, n = x.shape
    out = torch.empty((rows, n), dtype=weight.dtype, device=x.device)
    st = _capi.load().mops_hip_layer_norm_f32(_flat("x", x, rows * n, torch.float32), _flat("weight", weight, n, weight.dtype), float(eps), out.data_ptr(),
                                              code, rows, n, _stream(x))
    _capi.check("mops_hip_layer_norm_f32", st)
    return out


@register_hip_op
def rms_norm_f32(x: torch.Tensor, weight: torch.Tensor, eps: float, weight_offset: float = 0.0):
    """rms(x) * (weight_offset + weight) of float32 rows, in the weight's dtype."""
    code = _dtype("weight", weight)
    rows, n = x.shape
    out = torch.empty((rows, n), dtype=weight.dtype, device=x.device)
    st = _capi.load().mops_hip_rms_norm_f32(_flat("x", x, rows * n, torch.float32), _flat("weight", weight, n, weight.dtype),
                                            float(weight_offset), float(eps), out.data_ptr(), code, rows, n, _stream(x))
    _capi.check("mops_hip_rms_norm_f32", st)
    return out


@register_hip_op
def gated_group_norm(y: torch.Tensor, gate: torch.Tensor, groups: int, eps: float, weight=None, gate_first: bool = False, activation: str = "silu",
                     scale: float = 1.0, out=None):
    """rms over `groups` equal parts of every row, multiplied by silu(gate), or its sigmoid, before (gate_first) or after the division.
    weight: for the whole row, or for one part and shared by all.  Everything times scale."""
    code = _dtype("y", y)
    rows, n = y.shape
    _require(groups > 0 and n % groups == 0, "the row must divide into the groups")
    ys, gs = _rows("y", y, n, y.dtype), _rows("gate", gate, n, y.dtype)
    _require(gate.shape[0] == rows, "gate must have as many rows as y")
    _require(activation in ("silu", "sigmoid"), "activation must be silu or sigmoid")
    if out is None:
        out = torch.empty((rows, n), dtype=y.dtype, device=y.device)
    _require(out.shape[0] == rows, "out must have as many rows as y")
    shared = weight is not None and weight.numel() != n
    st = _capi.load().mops_hip_gated_group_norm(y.data_ptr(), ys, gate.data_ptr(), gs,
                                                None if weight is None else _flat("weight", weight, n // groups if shared else n, y.dtype), 1 if shared else 0,
                                                float(eps), 1 if gate_first else 0, 1 if activation == "sigmoid" else 0, float(scale), out.data_ptr(),
                                                _rows("out", out, n, y.dtype), code, rows, groups, n // groups, _stream(y))
    _capi.check("mops_hip_gated_group_norm", st)
    return out


def _glu(name, gate, up, out, *constants):
    code = _dtype("gate", gate)
    rows, n = gate.shape
    gs, us = _rows("gate", gate, n, gate.dtype), _rows("up", up, n, gate.dtype)
    _require(up.shape[0] == rows, "gate and up must have the same shape")
    if out is None:
        out = torch.empty((rows, n), dtype=gate.dtype, device=gate.device)
    _require(out.shape[0] == rows, "out must have as many rows as gate")
    st = getattr(_capi.load(), name)(gate.data_ptr(), gs, up.data_ptr(), us, out.data_ptr(), _rows("out", out, n, gate.dtype), code, rows, n, *constants,
                                     _stream(gate))
    _capi.check(name, st)
    return out


@register_hip_op
def clamped_glu(gate: torch.Tensor, up: torch.Tensor, limit: float, alpha: float = 1.702, out=None):
    """g * sigmoid(alpha g) * (u + 1) with g = min(gate, limit) and u = clamp(up, -limit, limit)."""
    return _glu("mops_hip_clamped_glu", gate, up, out, float(alpha), float(limit))


@register_hip_op
def gelu_glu(gate: torch.Tensor, up: torch.Tensor, out=None):
    """gelu(gate) * up, gelu in its tanh form."""
    return _glu("mops_hip_gelu_glu", gate, up, out)


@register_hip_op
def relu_glu(gate: torch.Tensor, up: torch.Tensor, out=None):
    """max(gate, 0) * up"""
    return _glu("mops_hip_relu_glu", gate, up, out)


@register_hip_op
def squared_relu(x: torch.Tensor):
    """max(x, 0)^2"""
    code = _dtype("x", x)
    rows, n = x.shape
    out = torch.empty((rows, n), dtype=x.dtype, device=x.device)
    st = _capi.load().mops_hip_squared_relu(x.data_ptr(), _rows("x", x, n, x.dtype), out.data_ptr(), code, rows, n, _stream(x))
    _capi.check("mops_hip_squared_relu", st)
    return out


def matrix_memory_copies(vd: int) -> int:
    """Rows behind the vd value rows of a head's state that hold a matrix memory's normalizer, and copies of its running maximum."""
    return _capi.load().mops_hip_matrix_memory_copies(vd)


@dataclass(frozen=True)
class MemoryGates:
    """A matrix memory's gates: projections [tokens, heads] in front of bias and cap, biases (float32 [heads]), the cap, the running maximum
    of every slot (float32 [slots, heads, copies]), and a factor on the queries."""
    input: torch.Tensor
    forget: torch.Tensor
    input_bias: torch.Tensor
    forget_bias: torch.Tensor
    cap: float
    top: torch.Tensor
    q_scale: float = 1.0


def recurrence_state_pitch(d: int) -> int:
    """Row pitch (elements) of the recurrent state [slots, heads, vd, pitch]."""
    return _capi.load().mops_hip_recurrence_state_pitch(d)


def _recurrence_args(q, k, v, out, state, state_slots, starts, heads, groups, d, vd, *, cu_seqlens=None, decay=None, log_decay=None, dt=None,
                     dt_bias=None, neg_a=None, skip=None, cos_sin=None, k_scale=1.0, conv=None, channel_decay=None, bonus=None, gates=None):
    code = _dtype("v", v)
    tokens = v.shape[0]
    batch = state_slots.numel()
    r = _capi.Recurrence()
    _require(heads > 0 and groups > 0 and heads % groups == 0, "heads must be a multiple of groups")
    copies = 0 if gates is None else matrix_memory_copies(vd)
    _require(state.is_cuda and state.dtype == torch.float32 and state.is_contiguous() and state.dim() == 4
             and tuple(state.shape[1:]) == (heads, vd + copies, recurrence_state_pitch(d)), "state must be float32 [slots, heads, vd (+ copies), pitch]")
    r.q_stride, r.k_stride = _rows("q", q, groups * d, v.dtype), _rows("k", k, groups * d, v.dtype)
    r.v_stride, r.out_stride = _rows("v", v, heads * vd, v.dtype), _rows("out", out, heads * vd, v.dtype)
    r.q, r.k, r.v, r.out = q.data_ptr(), k.data_ptr(), v.data_ptr(), out.data_ptr()
    _require(q.shape[0] == k.shape[0] == out.shape[0] == tokens, "q, k, v and out must have the same number of tokens")
    r.state, r.num_slots = state.data_ptr(), state.shape[0]
    r.state_slots, r.starts = _flat("state_slots", state_slots, batch, torch.int32), _flat("starts", starts, batch, torch.int32)
    if cu_seqlens is None:
        _require(tokens == batch, "without cu_seqlens every sequence brings one token")
    else:
        r.cu_seqlens = _flat("cu_seqlens", cu_seqlens, batch + 1, torch.int32)
    _require(sum(x is not None for x in (decay, dt, channel_decay, gates)) == 1, "give a constant decay, time steps, a decay per channel or gates")
    if gates is not None:
        r.input_gate, r.forget_gate, r.gate_stride = gates.input.data_ptr(), gates.forget.data_ptr(), _rows("input gate", gates.input, heads, v.dtype)
        _require(_rows("forget gate", gates.forget, heads, v.dtype) == r.gate_stride and gates.input.shape[0] == gates.forget.shape[0] == tokens,
                 "the gates must have one row per token and the same stride")
        r.input_bias, r.forget_bias = _flat("input bias", gates.input_bias, heads, torch.float32), _flat("forget bias", gates.forget_bias, heads, torch.float32)
        r.top, r.gate_cap = _flat("top", gates.top, state.shape[0] * heads * copies, torch.float32), float(gates.cap)
    elif channel_decay is not None:
        r.channel_decay, r.channel_decay_stride = channel_decay.data_ptr(), _rows("channel_decay", channel_decay, heads * d, torch.float32)
        _require(channel_decay.shape[0] == tokens, "channel_decay must have one row per token")
        r.bonus = _flat("bonus", bonus, heads * d, torch.float32)
    elif decay is not None:
        r.decay = _flat("decay", decay, heads, torch.float32)
        if log_decay is not None:
            r.log_decay = _flat("log_decay", log_decay, heads, torch.float32)
    else:
        r.dt, r.dt_stride = dt.data_ptr(), _rows("dt", dt, heads, v.dtype)
        _require(dt.shape[0] == tokens, "dt must have one row per token")
        r.dt_bias, r.neg_a = _flat("dt_bias", dt_bias, heads, torch.float32), _flat("neg_a", neg_a, heads, torch.float32)
    if skip is not None:
        r.skip = _flat("skip", skip, heads, torch.float32)
    if cos_sin is not None:
        r.rot, r.max_positions = cos_sin.shape[1], cos_sin.shape[0]
        r.cos_sin = _flat("cos_sin", cos_sin, cos_sin.numel(), torch.float32)
    if conv is not None:
        weight, bias, ring, (r.q_channel, r.k_channel, r.v_channel) = conv
        r.taps, r.channels = weight.shape
        r.conv_weight = _flat("conv weight", weight, weight.numel(), torch.float32)
        r.conv_bias = _flat("conv bias", bias, weight.shape[1], torch.float32)
        r.conv_ring = _flat("conv ring", ring, state.shape[0] * weight.numel(), v.dtype)
    r.batch, r.heads, r.groups, r.d, r.vd = batch, heads, groups, d, vd
    r.k_scale, r.dtype = float(k_scale if gates is None else gates.q_scale), code
    return r


@register_hip_op
def decayed_recurrence(q, k, v, out, state, state_slots, starts, heads, groups, d, vd, **options):
    """S <- a S + k (s v)^T, o = S^T q + skip v, token by token with the state of state_slots[b] in float32 (layout and options:
    mops_hip_recurrence in include/mops_hip.h).  Options: cu_seqlens (None: one token per sequence), decay | dt + dt_bias +
    neg_a | channel_decay + bonus | gates (a matrix memory), skip, cos_sin (rotates q and k), k_scale, conv = (weight [taps, channels] float32, bias, ring, (q, k, v channel
    offsets)).  Writes `out` and the state in place."""
    r = _recurrence_args(q, k, v, out, state, state_slots, starts, heads, groups, d, vd, **options)
    st = _capi.load().mops_hip_decayed_recurrence(byref(r), _stream(v))
    _capi.check("mops_hip_decayed_recurrence", st)
    return out


def _delta_args(q, k, v, out, state, state_slots, starts, heads, groups, d, vd, log_decay, beta, q_scale, unit_eps, cu_seqlens=None, conv=None):
    a = _capi.Delta()
    a.dtype = _dtype("v", v)
    tokens, batch = v.shape[0], state_slots.numel()
    _require(heads > 0 and groups > 0 and heads % groups == 0, "heads must be a multiple of groups")
    _require(state.is_cuda and state.dtype == torch.float32 and state.is_contiguous() and state.dim() == 4
             and tuple(state.shape[1:]) == (heads, vd, recurrence_state_pitch(d)), "state must be float32 [slots, heads, vd, pitch]")
    a.q_stride, a.k_stride = _rows("q", q, groups * d, v.dtype), _rows("k", k, groups * d, v.dtype)
    a.v_stride, a.out_stride = _rows("v", v, heads * vd, v.dtype), _rows("out", out, heads * vd, v.dtype)
    a.q, a.k, a.v, a.out = q.data_ptr(), k.data_ptr(), v.data_ptr(), out.data_ptr()
    a.log_decay, a.log_decay_stride = log_decay.data_ptr(), _rows("log_decay", log_decay, heads * d, torch.float32)
    a.beta, a.beta_stride = beta.data_ptr(), _rows("beta", beta, heads, v.dtype)
    _require(all(x.shape[0] == tokens for x in (q, k, out, log_decay, beta)), "all inputs must have the same number of tokens")
    a.state, a.num_slots = state.data_ptr(), state.shape[0]
    a.state_slots, a.starts = _flat("state_slots", state_slots, batch, torch.int32), _flat("starts", starts, batch, torch.int32)
    if cu_seqlens is None:
        _require(tokens == batch, "without cu_seqlens every sequence brings one token")
    else:
        a.cu_seqlens = _flat("cu_seqlens", cu_seqlens, batch + 1, torch.int32)
    if conv is not None:
        weight, ring, (a.q_channel, a.k_channel, a.v_channel) = conv
        a.taps, a.channels = weight.shape
        a.conv_weight = _flat("conv weight", weight, weight.numel(), torch.float32)
        a.conv_ring = _flat("conv ring", ring, state.shape[0] * weight.numel(), v.dtype)
    a.batch, a.heads, a.groups, a.d, a.vd = batch, heads, groups, d, vd
    a.q_scale, a.unit_eps = float(q_scale), float(unit_eps)
    return a


@register_hip_op
def delta_rule(q, k, v, out, state, state_slots, starts, heads, groups, d, vd, **options):
    """The gated delta rule token by token, S <- exp(log_decay) S, S <- S + k (sigmoid(beta) (v - S^T k))^T, o = S^T q, with q and k as unit
    vectors and the state of state_slots[b] in float32 (mops_hip_delta in include/mops_hip.h).  Options: log_decay (float32 [tokens, heads *
    d]), beta [tokens, heads], q_scale, unit_eps, cu_seqlens (None: one token per sequence), conv = (weight [taps, channels] float32, ring,
    (q, k, v channel offsets)).  Writes `out` and the state in place."""
    a = _delta_args(q, k, v, out, state, state_slots, starts, heads, groups, d, vd, **options)
    st = _capi.load().mops_hip_delta_rule(byref(a), _stream(v))
    _capi.check("mops_hip_delta_rule", st)
    return out


DELTA_CHUNK = 16      # tokens


def delta_cuts(counts, heads: int, vd: int, wanted: int = 256, enough: int = 128):
    """Cuts portions of counts[i] tokens (packed one behind the other) for delta_chunks: host lists (chunks, segments, bounds of the
    segments per portion).  One segment per portion if those give enough workgroups, else about `wanted` workgroups in all."""
    per_segment, length = _capi.load().mops_hip_delta_chunks_workgroups(heads, vd), max(counts)
    if len(counts) * per_segment < enough and length > 256:
        length = max(128, -(-sum(counts) * per_segment // wanted // DELTA_CHUNK) * DELTA_CHUNK)
    length = -(-length // DELTA_CHUNK) * DELTA_CHUNK
    chunks, segments, bounds, at = [], [], [0], 0
    for i, n in enumerate(counts):
        for begin in range(0, n, length):
            segments.append((i, at + begin, at + min(n, begin + length), len(chunks) + begin // DELTA_CHUNK))
        bounds.append(len(segments))
        chunks += [(at + begin, min(DELTA_CHUNK, n - begin)) for begin in range(0, n, DELTA_CHUNK)]
        at += n
    return chunks, segments, bounds


@register_hip_op
def delta_chunks(q, k, v, out, state, state_slots, starts, heads, groups, d, vd, chunks, segments, seq_segments, **options):
    """delta_rule for packed portions of many tokens, on the matrix cores (bf16, d up to CHUNK_MAX_DIM).  chunks [n, 2], segments [m, 4]
    and seq_segments [sequences + 1] are the int32 device copies of what delta_cuts returns; cu_seqlens is required."""
    a = _delta_args(q, k, v, out, state, state_slots, starts, heads, groups, d, vd, **options)
    n, m, lib = chunks.shape[0], segments.shape[0], _capi.load()
    _require(a.batch == seq_segments.numel() - 1, "seq_segments must bound the segments of every sequence")
    ws = torch.empty(max(16, lib.mops_hip_delta_chunks_workspace_bytes(n, m, a.batch, heads, d, vd)), dtype=torch.uint8, device=v.device)
    st = lib.mops_hip_delta_chunks(byref(a), _flat("chunks", chunks, 2 * n, torch.int32), n, _flat("segments", segments, 4 * m, torch.int32), m,
                                   _flat("seq_segments", seq_segments, a.batch + 1, torch.int32), ws.data_ptr(), ws.numel(), _stream(v))
    _capi.check("mops_hip_delta_chunks", st)
    return out


CHUNK_MAX_DIM = 256       # head sizes (d) the chunked kernels cover


def recurrence_segments(counts, heads: int, groups: int, vd: int, wanted: int = 512):
    """Cuts portions of counts[i] tokens (packed one behind the other) into segments for decayed_chunks: one per portion if
    those give enough workgroups, else about `wanted` workgroups in all.  Returns host lists (segments, bounds per portion)."""
    return _segments(counts, _capi.load().mops_hip_decayed_chunks_workgroups(heads, groups, vd), wanted, wanted // 2)


def channel_segments(counts, heads: int, vd: int, wanted: int = 1024, enough: int = 192):
    """The same for channel_chunks."""
    return _segments(counts, _capi.load().mops_hip_channel_chunks_workgroups(heads, vd), wanted, enough)


def _segments(counts, per_segment: int, wanted: int, enough: int):
    length = max(counts)
    if len(counts) * per_segment < enough and length > 256:
        length = max(128, -(-sum(counts) * per_segment // wanted // 64) * 64)
    segments, bounds, at = [], [0], 0
    for i, n in enumerate(counts):
        for begin in range(0, n, length):
            segments.append((i, at + begin, at + min(n, begin + length)))
        bounds.append(len(segments))
        at += n
    return segments, bounds


def _chunks(name, seg_decay_shape, q, k, v, out, state, state_slots, starts, heads, groups, d, vd, segments, seq_segments, **options):
    r = _recurrence_args(q, k, v, out, state, state_slots, starts, heads, groups, d, vd, **options)
    if options.get("gates") is not None:      # token by token, but numbers per head only
        per_token = torch.empty((3, v.shape[0], heads), dtype=torch.float32, device=v.device)
        r.log_keep, r.input_scale, r.least = (x.data_ptr() for x in per_token)
        st = _capi.load().mops_hip_matrix_memory_gates(byref(r), r.log_keep, r.input_scale, r.least, _stream(v))
        _capi.check("mops_hip_matrix_memory_gates", st)
    n = segments.shape[0]
    _require(r.batch == seq_segments.numel() - 1, "seq_segments must bound the segments of every sequence")
    seg_state = seg_decay = None
    if n > r.batch:
        seg_state = torch.empty((n, *state.shape[1:]), dtype=torch.float32, device=v.device)
        seg_decay = torch.empty((n, *seg_decay_shape), dtype=torch.float32, device=v.device)
    st = getattr(_capi.load(), name)(byref(r), _flat("segments", segments, 3 * n, torch.int32), n,
                                     _flat("seq_segments", seq_segments, r.batch + 1, torch.int32),
                                     None if seg_state is None else seg_state.data_ptr(),
                                     None if seg_decay is None else seg_decay.data_ptr(), _stream(v))
    _capi.check(name, st)
    return out


@register_hip_op
def decayed_chunks(q, k, v, out, state, state_slots, starts, heads, groups, d, vd, segments, seq_segments, **options):
    """decayed_recurrence for packed portions of many tokens, on the matrix cores (bf16).  segments [n, 3] and seq_segments
    [sequences + 1] are the int32 device copies of what recurrence_segments returns; cu_seqlens is required."""
    return _chunks("mops_hip_decayed_chunks", (heads,), q, k, v, out, state, state_slots, starts, heads, groups, d, vd, segments, seq_segments, **options)


@register_hip_op
def channel_chunks(q, k, v, out, state, state_slots, starts, heads, groups, d, vd, segments, seq_segments, **options):
    """The same for channel_decay and bonus; segments from channel_segments."""
    return _chunks("mops_hip_channel_chunks", (heads, state.shape[3]), q, k, v, out, state, state_slots, starts, heads, groups, d, vd, segments,
                   seq_segments, **options)


@register_hip_op
def short_conv(x, weight, bias, ring, token_seq, cu_seqlens, starts, state_slots):
    """silu(causal convolution per channel + bias) of packed portions; inputs before a portion come from the ring."""
    code = _dtype("x", x)
    tokens, channels = x.shape
    taps = weight.shape[0]
    batch = state_slots.numel()
    stride = _rows("x", x, channels, x.dtype)
    _require(ring.dim() == 3 and ring.shape[1:] == (taps, channels), "ring must be [slots, taps, channels]")
    out = torch.empty((tokens, channels), dtype=x.dtype, device=x.device)
    st = _capi.load().mops_hip_short_conv(x.data_ptr(), stride, _flat("weight", weight, taps * channels, torch.float32),
                                          None if bias is None else _flat("bias", bias, channels, torch.float32), _flat("ring", ring, ring.numel(), x.dtype), ring.shape[0],
                                          _flat("token_seq", token_seq, tokens, torch.int32), _flat("cu_seqlens", cu_seqlens, batch + 1, torch.int32),
                                          _flat("starts", starts, batch, torch.int32), _flat("state_slots", state_slots, batch, torch.int32),
                                          out.data_ptr(), code, tokens, channels, taps, _stream(x))
    _capi.check("mops_hip_short_conv", st)
    return out


@register_hip_op
def short_conv_update(x, ring, cu_seqlens, starts, state_slots):
    """Files the last taps-1 rows of every portion in the ring."""
    code = _dtype("x", x)
    channels = x.shape[1]
    batch = state_slots.numel()
    stride = _rows("x", x, channels, x.dtype)
    _require(ring.dim() == 3 and ring.shape[2] == channels, "ring must be [slots, taps, channels]")
    st = _capi.load().mops_hip_short_conv_update(x.data_ptr(), stride, _flat("ring", ring, ring.numel(), x.dtype), ring.shape[0],
                                                 _flat("cu_seqlens", cu_seqlens, batch + 1, torch.int32),
                                                 _flat("starts", starts, batch, torch.int32), _flat("state_slots", state_slots, batch, torch.int32),
                                                 code, batch, channels, ring.shape[1], _stream(x))
    _capi.check("mops_hip_short_conv_update", st)


@register_hip_op
def token_mix(x, mu, before, starts, state_slots, token_seq=None, cu_seqlens=None):
    """[parts, tokens, width]: every row of x moved by mu[p] (float32) towards the row in front of it; `before` [slots, width] holds the
    last row of each sequence's earlier tokens and receives the new last row.  Without cu_seqlens every sequence brings one token."""
    code = _dtype("x", x)
    tokens, width = x.shape
    parts, batch = mu.shape[0], state_slots.numel()
    stride = _rows("x", x, width, x.dtype)
    _require(before.dim() == 2 and before.shape[1] == width, "before must be [slots, width]")
    _require((token_seq is None) == (cu_seqlens is None) and (cu_seqlens is not None or tokens == batch), "packed portions need token_seq and cu_seqlens")
    out = torch.empty((parts, tokens, width), dtype=x.dtype, device=x.device)
    st = _capi.load().mops_hip_token_mix(x.data_ptr(), stride, _flat("mu", mu, parts * width, torch.float32), parts,
                                         _flat("before", before, before.numel(), x.dtype), before.shape[0],
                                         None if token_seq is None else _flat("token_seq", token_seq, tokens, torch.int32),
                                         None if cu_seqlens is None else _flat("cu_seqlens", cu_seqlens, batch + 1, torch.int32),
                                         _flat("starts", starts, batch, torch.int32), _flat("state_slots", state_slots, batch, torch.int32),
                                         out.data_ptr(), code, tokens, width, _stream(x))
    _capi.check("mops_hip_token_mix", st)
    return out


@register_hip_op
def low_rank_decay(z, w2, w0, rate=None):
    """-exp(w2 tanh(z) + w0), or with a rate per head (float32) rate softplus(w2 z + w0); float32: the logarithm of a decay per channel.  w2
    in z's dtype, w0 float32."""
    code = _dtype("z", z)
    tokens, (channels, rank) = z.shape[0], w2.shape
    out = torch.empty((tokens, channels), dtype=torch.float32, device=z.device)
    st = _capi.load().mops_hip_low_rank_decay(z.data_ptr(), _rows("z", z, rank, z.dtype), _flat("w2", w2, channels * rank, z.dtype),
                                              _flat("w0", w0, channels, torch.float32), None if rate is None else _flat("rate", rate, rate.numel(), torch.float32),
                                              0 if rate is None else channels // rate.numel(), out.data_ptr(), code, tokens, channels, rank, _stream(z))
    _capi.check("mops_hip_low_rank_decay", st)
    return out


def _latent_cache(cache, width, dtype):
    _require(cache.dim() == 3 and cache.dtype == dtype and cache.is_cuda and cache.is_contiguous() and cache.shape[2] >= width,
             "the latent cache must be a contiguous [blocks, block_size, pitch] tensor of the activation dtype")
    return cache.shape


@register_hip_op
def latent_prepare(down, q_weight, kv_weight, eps, cos_sin, positions, slot_mapping, cache, q_rank, kv_rank, rot_dim):
    """Norms of the query and kv latents, rotation of the shared key part, scatter of the cache rows; returns the query latent."""
    code = _dtype("down", down)
    tokens = down.shape[0]
    _require(down.dim() == 2 and down.shape[1] >= q_rank + kv_rank + rot_dim and down.stride(1) == 1, "down must be [tokens, q_rank + kv_rank + rot_dim]")
    nblk, bs, pitch = _latent_cache(cache, kv_rank + rot_dim, down.dtype)
    _require(cos_sin.dim() == 2 and cos_sin.shape[1] == rot_dim, "cos_sin must be [positions, rot_dim]")
    cq = torch.empty((tokens, q_rank), dtype=down.dtype, device=down.device)
    st = _capi.load().mops_hip_latent_prepare(down.data_ptr(), down.stride(0) if tokens > 1 else down.shape[1],
                                              _flat("q_weight", q_weight, q_rank, down.dtype), _flat("kv_weight", kv_weight, kv_rank, down.dtype),
                                              float(eps), _flat("cos_sin", cos_sin, cos_sin.numel(), torch.float32), cos_sin.shape[0],
                                              _flat("positions", positions, tokens, torch.int32), _flat("slot_mapping", slot_mapping, tokens, torch.int32),
                                              cq.data_ptr(), cache.data_ptr(), nblk * bs, pitch, code, tokens, q_rank, kv_rank, rot_dim, _stream(down))
    _capi.check("mops_hip_latent_prepare", st)
    return cq


@register_hip_op
def head_linear(x, weight):
    """y[t, h, :] = weight[h] @ x[t, h, :]; x [tokens, heads, k] (last dimension contiguous), weight [heads, n, k]."""
    code = _dtype("x", x)
    tokens, heads, k = x.shape
    _require(x.stride(2) == 1 or k == 1, "x must have a contiguous last dimension")
    _require(weight.dim() == 3 and weight.shape[0] == heads and weight.shape[2] == k and weight.is_contiguous() and weight.dtype == x.dtype,
             "weight must be a contiguous [heads, n, k] tensor of x's dtype")
    n = weight.shape[1]
    y = torch.empty((tokens, heads, n), dtype=x.dtype, device=x.device)
    st = _capi.load().mops_hip_head_linear(x.data_ptr(), x.stride(0), x.stride(1), weight.data_ptr(), y.data_ptr(), heads * n, n, code, tokens,
                                           heads, n, k, _stream(x))
    _capi.check("mops_hip_head_linear", st)
    return y


def _latent_rows(q_latent, q_rot, cache, cos_sin, context_lens, block_table, scale, row_seq, out):
    code = _dtype("q_latent", q_latent)
    rows, heads, kv_rank = q_latent.shape
    rot_dim = q_rot.shape[2]
    _require(q_latent.is_contiguous() and q_rot.shape[:2] == (rows, heads) and q_rot.dtype == q_latent.dtype and q_rot.stride(2) == 1,
             "q_latent must be contiguous [rows, heads, kv_rank], q_rot [rows, heads, rot_dim]")
    nblk, bs, pitch = _latent_cache(cache, kv_rank + rot_dim, q_latent.dtype)
    _require(cos_sin.dim() == 2 and cos_sin.shape[1] == rot_dim, "cos_sin must be [positions, rot_dim]")
    _require(block_table.dtype == torch.int32 and block_table.is_cuda and block_table.dim() == 2 and block_table.stride(1) == 1
             and (row_seq is not None or block_table.shape[0] >= rows), "block_table must be an int32 GPU tensor [sequences, blocks]")
    a = _capi.LatentRows()
    a.q_latent, a.q_rot, a.q_rot_token_stride, a.q_rot_head_stride = q_latent.data_ptr(), q_rot.data_ptr(), q_rot.stride(0), q_rot.stride(1)
    a.cache, a.pitch = cache.data_ptr(), pitch
    a.cos_sin, a.max_positions = _flat("cos_sin", cos_sin, cos_sin.numel(), torch.float32), cos_sin.shape[0]
    a.row_seq = None if row_seq is None else _flat("row_seq", row_seq, rows, torch.int32)
    a.context_lens = _flat("context_lens", context_lens, rows, torch.int32)
    a.block_table, a.max_blocks = block_table.data_ptr(), block_table.shape[1]
    a.block_table_stride = block_table.stride(0) if block_table.shape[0] > 1 else block_table.shape[1]
    a.block_size, a.num_blocks = bs, nblk
    a.out, a.rows, a.heads, a.kv_rank, a.rot_dim = out.data_ptr(), rows, heads, kv_rank, rot_dim
    a.scale, a.dtype = float(scale), code
    return a


@register_hip_op
def latent_attention_rows(q_latent, q_rot, cache, cos_sin, context_lens, block_table, scale, row_seq=None):
    """Attention of single query rows against the paged latent cache, in the latent space; returns [rows, heads, kv_rank].
    Row r sees the first context_lens[r] tokens of block table row row_seq[r] (r itself without row_seq).  The plain form:
    any size, bf16 or float32; latent_decode is the one on the matrix cores."""
    out = torch.empty_like(q_latent)
    a = _latent_rows(q_latent, q_rot, cache, cos_sin, context_lens, block_table, scale, row_seq, out)
    st = _capi.load().mops_hip_latent_attention_rows(byref(a), _stream(q_latent))
    _capi.check("mops_hip_latent_attention_rows", st)
    return out


def latent_decode_covers(dtype, kv_rank: int, rot_dim: int, block_size: int) -> bool:
    return dtype == torch.bfloat16 and kv_rank <= 512 and kv_rank + rot_dim <= 576 and block_size % 32 == 0


@register_hip_op
def latent_decode(q_latent, q_rot, cache, cos_sin, context_lens, block_table, scale, row_seq=None):
    """latent_attention_rows on the matrix cores (sizes: latent_decode_covers)."""
    out = torch.empty_like(q_latent)
    a = _latent_rows(q_latent, q_rot, cache, cos_sin, context_lens, block_table, scale, row_seq, out)
    lib = _capi.load()
    nbytes = lib.mops_hip_latent_decode_workspace_bytes(a.rows, a.heads, a.kv_rank, a.rot_dim)
    ws = torch.empty(max(nbytes, 16), dtype=torch.uint8, device=out.device)
    st = lib.mops_hip_latent_decode(byref(a), ws.data_ptr(), ws.numel(), _stream(q_latent))
    _capi.check("mops_hip_latent_decode", st)
    return out


def latent_prefill_covers(dtype, dim: int, rot_dim: int, vdim: int) -> bool:
    return dtype == torch.bfloat16 and (dim + 7) // 8 * 8 + (rot_dim + 7) // 8 * 8 <= 256 and vdim <= 256


PREFILL_QUERIES, PREFILL_KEYS = 128, 64


def latent_prefill_plan(counts, starts, first_token: int, first_seq: int):
    """Host lists for latent_gather and latent_prefill: portions of counts[i] tokens at positions starts[i].., packed from token
    row first_token on; sequence i of the list is block table row first_seq + i.  Returns (row_seq, row_pos, tiles)."""
    row_seq, row_pos, tiles = [], [], []
    at = first_token
    for i, (n, start) in enumerate(zip(counts, starts)):
        keys, base = start + n, len(row_pos)
        pad = -keys % PREFILL_KEYS
        row_seq += [first_seq + i] * (keys + pad)
        row_pos += list(range(keys)) + [-1] * pad
        for q in range(0, n, PREFILL_QUERIES):
            tiles.append((at + q, min(PREFILL_QUERIES, n - q), start + q, base, keys))
        at += n
    tiles.sort(key=lambda t: -(t[1] + t[2]))      # the longest first: they bound the launch
    return row_seq, row_pos, tiles


@register_hip_op
def latent_gather(cache, block_table, row_seq, row_pos, kv_rank, rot_dim):
    """Latent rows and key parts of whole contexts out of the pages: (c [rows, kv_rank], kr [rows, rot_dim]), row strides
    multiples of eight."""
    nblk, bs, pitch = _latent_cache(cache, kv_rank + rot_dim, torch.bfloat16)
    rows = row_pos.numel()
    _require(block_table.dtype == torch.int32 and block_table.is_cuda and block_table.dim() == 2 and block_table.stride(1) == 1,
             "block_table must be an int32 GPU tensor [sequences, blocks]")
    c = torch.empty((rows, (kv_rank + 7) // 8 * 8), dtype=cache.dtype, device=cache.device)
    kr = torch.empty((rows, (rot_dim + 7) // 8 * 8), dtype=cache.dtype, device=cache.device)
    st = _capi.load().mops_hip_latent_gather(cache.data_ptr(), pitch, block_table.data_ptr(),
                                             block_table.stride(0) if block_table.shape[0] > 1 else block_table.shape[1], bs, nblk,
                                             block_table.shape[1], _flat("row_seq", row_seq, rows, torch.int32),
                                             _flat("row_pos", row_pos, rows, torch.int32), c.data_ptr(), c.shape[1], kr.data_ptr(), kr.shape[1],
                                             rows, kv_rank, rot_dim, _stream(cache))
    _capi.check("mops_hip_latent_gather", st)
    return c, kr


@register_hip_op
def rotate_pairs(x, positions, cos_sin):
    """Rotates the pairs (2i, 2i+1) of x [tokens, heads, rot] (bf16, any token and head strides) in place."""
    _require(x.dim() == 3 and x.is_cuda and x.dtype == torch.bfloat16 and x.stride(2) == 1 and cos_sin.dim() == 2 and cos_sin.shape[1] == x.shape[2],
             "x must be [tokens, heads, rot] in bfloat16 and cos_sin [positions, rot]")
    tokens, heads, rot = x.shape
    st = _capi.load().mops_hip_rotate_pairs(x.data_ptr(), x.stride(0), x.stride(1) if heads > 1 else max(rot, x.stride(1)),
                                            _flat("positions", positions, tokens, torch.int32), _flat("cos_sin", cos_sin, cos_sin.numel(), torch.float32),
                                            cos_sin.shape[0], tokens, heads, rot, _stream(x))
    _capi.check("mops_hip_rotate_pairs", st)
    return x


@register_hip_op
def latent_prefill(q, k, kr, vt, tiles, scale, out):
    """Causal attention of long portions over expanded keys and values: q [tokens, heads, dim + rot] (rotated), k [rows,
    heads * dim], kr [rows, rot], vt [heads * vdim, rows]; writes the portions' rows of out [tokens, heads, vdim].  dim, rot and
    the strides are multiples of eight."""
    _require(q.dim() == 3 and q.dtype == torch.bfloat16 and q.is_cuda and q.stride(2) == 1, "q must be [tokens, heads, dim + rot] in bfloat16")
    heads, rot, rows = q.shape[1], kr.shape[1], k.shape[0]
    dim, vdim = q.shape[2] - rot, out.shape[2]
    _require(out.shape == (q.shape[0], heads, vdim) and out.is_contiguous() and out.dtype == q.dtype, "out must be contiguous [tokens, heads, vdim]")
    _require(dim > 0 and k.shape[1] == heads * dim and k.stride(1) == 1 and kr.shape[0] == rows and kr.stride(1) == 1
             and vt.shape == (heads * vdim, rows) and vt.stride(1) == 1 and k.dtype == kr.dtype == vt.dtype == q.dtype
             and rows % PREFILL_KEYS == 0, "k [rows, heads * dim], kr [rows, rot], vt [heads * vdim, rows], rows a multiple of 64")
    n = tiles.shape[0]
    st = _capi.load().mops_hip_latent_prefill(q.data_ptr(), q.stride(0), q.stride(1), k.data_ptr(), k.stride(0), kr.data_ptr(), kr.stride(0),
                                              vt.data_ptr(), vt.stride(0), _flat("tiles", tiles, 5 * n, torch.int32), n, out.data_ptr(), heads, dim, rot,
                                              vdim, float(scale), _stream(q))
    _capi.check("mops_hip_latent_prefill", st)
    return out
