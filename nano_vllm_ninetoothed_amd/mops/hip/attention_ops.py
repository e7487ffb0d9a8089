"""Extension ops of the `hip` backend for grouped-query attention over paged keys and values of any two sizes, with a linear distance
bias or capped scores, over all of a sequence or a part of it (the rules of recurrent_ops.py hold)."""
from __future__ import annotations

from ctypes import byref
from dataclasses import dataclass

import torch

from ... import _capi
from .ops import _require, _stream
from .recurrent_ops import _dtype, _flat, _rows
from .registry import register_hip_op


def padded(n: int) -> int:
    """Head sizes in queries and pages: rounded up to 16-byte pieces of bf16."""
    return (n + 7) // 8 * 8


def _pages(name, pages, heads, size, dtype):
    _require(pages.is_cuda and pages.dtype == dtype and pages.is_contiguous() and pages.dim() == 4 and pages.shape[2:] == (heads, padded(size)),
             f"{name} must be contiguous [blocks, block_size, {heads}, {padded(size)}] of {dtype}")
    return pages.data_ptr()


@register_hip_op
def attention_prepare(qkv, q_weight, k_weight, eps, positions, slot_mapping, k_pages, v_pages, heads, kv_heads, dim, vdim, q_factor=None):
    """qkv rows [q | k | v]: RMS norms over the whole of q and of k, a factor per position on q, k and v into their pages.
    Returns q [tokens, heads, padded dim]."""
    code = _dtype("qkv", qkv)
    tokens = qkv.shape[0]
    a = _capi.AttentionPrepare()
    _require(qkv.dim() == 2 and qkv.stride(1) == 1 and qkv.shape[1] >= (heads + kv_heads) * dim + kv_heads * vdim, "qkv must be [tokens, q | k | v]")
    a.qkv, a.qkv_stride = qkv.data_ptr(), qkv.stride(0) if tokens > 1 else qkv.shape[1]
    a.q_weight, a.k_weight = _flat("q_weight", q_weight, heads * dim, qkv.dtype), _flat("k_weight", k_weight, kv_heads * dim, qkv.dtype)
    a.max_positions = 1
    if q_factor is not None:
        a.q_factor, a.max_positions = _flat("q_factor", q_factor, q_factor.numel(), torch.float32), q_factor.numel()
    a.positions, a.slot_mapping = _flat("positions", positions, tokens, torch.int32), _flat("slot_mapping", slot_mapping, tokens, torch.int32)
    q = torch.empty((tokens, heads, padded(dim)), dtype=qkv.dtype, device=qkv.device)
    a.q, a.k_pages, a.v_pages = q.data_ptr(), _pages("k_pages", k_pages, kv_heads, dim, qkv.dtype), _pages("v_pages", v_pages, kv_heads, vdim, qkv.dtype)
    _require(k_pages.shape[:2] == v_pages.shape[:2], "k_pages and v_pages must have the same blocks")
    a.num_slots, a.tokens, a.heads, a.kv_heads, a.dim, a.vdim = k_pages.shape[0] * k_pages.shape[1], tokens, heads, kv_heads, dim, vdim
    a.eps, a.dtype = float(eps), code
    st = _capi.load().mops_hip_attention_prepare(byref(a), _stream(qkv))
    _capi.check("mops_hip_attention_prepare", st)
    return q


@register_hip_op
def rotary_prepare(qkv, positions, slot_mapping, k_pages, v_pages, heads, kv_heads, dim, vdim, cos_sin=None, q_weight=None, k_weight=None, eps=0.0,
                   bias=None, neighbours=False):
    """qkv rows [q | k | v | anything], plus bias over [q | k | v]: an RMS norm per head on q and k where there are weights [dim], their
    first cos_sin.shape[1] elements turned by the token's position (pairs half of that apart, or neighbours), k and v into their pages.
    Returns q [tokens, heads, padded dim]."""
    a = _capi.RotaryPrepare()
    a.dtype = _dtype("qkv", qkv)
    tokens = qkv.shape[0]
    _require(qkv.dim() == 2 and qkv.stride(1) == 1 and qkv.shape[1] >= (heads + kv_heads) * dim + kv_heads * vdim, "qkv must be [tokens, q | k | v]")
    a.qkv, a.qkv_stride = qkv.data_ptr(), qkv.stride(0) if tokens > 1 else qkv.shape[1]
    if q_weight is not None:
        a.q_weight = _flat("q_weight", q_weight, dim, qkv.dtype)
    if k_weight is not None:
        a.k_weight = _flat("k_weight", k_weight, dim, qkv.dtype)
    a.max_positions = 1
    if cos_sin is not None:
        a.max_positions, a.rot = cos_sin.shape
        a.cos_sin = _flat("cos_sin", cos_sin, a.max_positions * a.rot, torch.float32)
    a.positions, a.slot_mapping = _flat("positions", positions, tokens, torch.int32), _flat("slot_mapping", slot_mapping, tokens, torch.int32)
    q = torch.empty((tokens, heads, padded(dim)), dtype=qkv.dtype, device=qkv.device)
    a.q, a.k_pages, a.v_pages = q.data_ptr(), _pages("k_pages", k_pages, kv_heads, dim, qkv.dtype), _pages("v_pages", v_pages, kv_heads, vdim, qkv.dtype)
    _require(k_pages.shape[:2] == v_pages.shape[:2], "k_pages and v_pages must have the same blocks")
    a.num_slots, a.tokens, a.heads, a.kv_heads, a.dim, a.vdim = k_pages.shape[0] * k_pages.shape[1], tokens, heads, kv_heads, dim, vdim
    a.eps, a.neighbours = float(eps), 1 if neighbours else 0
    if bias is not None:
        a.bias = _flat("bias", bias, (heads + kv_heads) * dim + kv_heads * vdim, qkv.dtype)
    st = _capi.load().mops_hip_rotary_prepare(byref(a), _stream(qkv))
    _capi.check("mops_hip_rotary_prepare", st)
    return q


@dataclass(frozen=True)
class Scores:
    """What a design does to the scores of attention beside scaling them, and what a token sees.  Zeros and None leave it out.
    softcap: softcap tanh(score / softcap).  window: the last `window` tokens; chunk: the token's chunk of a sequence cut from its start;
    both up to the token itself, and the first keep_first tokens with them.  sinks (float32 [heads]): logarithms of one more term of
    the denominator.  log_distance (two of float32 [heads]): rate ln(1 + step distance) is taken off.  weight_bias (float32 [heads]): no
    softmax, a key counts with sigmoid(score + weight_bias)."""
    softcap: float = 0.0
    window: int = 0
    chunk: int = 0
    keep_first: int = 0
    sinks: torch.Tensor = None
    log_distance: tuple = None
    weight_bias: torch.Tensor = None


WIDEST = 1 << 30      # more than any sequence holds: a window or chunk without effect


def _biased_args(q, k_pages, v_pages, dim, vdim, context_lens, block_table, scale, slopes, row_seq, out, own_rows=True, scores=None, gate=None,
                 out_scale=1.0):
    code = _dtype("q", q)
    rows, heads, dp = q.shape
    kv_heads = k_pages.shape[2]
    _require(q.is_contiguous() and dp == padded(dim), "q must be contiguous [rows, heads, padded dim]")
    _require(heads % kv_heads == 0, "query heads must be a multiple of kv heads")
    out = out.view(rows, heads * vdim) if out.dim() == 3 else out
    a = _capi.BiasedAttention()
    a.out_stride, a.out_scale = _rows("out", out, heads * vdim, q.dtype), float(out_scale)
    _require(out.shape[0] == rows, "out must have as many rows as q")
    a.q, a.k_pages, a.v_pages = q.data_ptr(), _pages("k_pages", k_pages, kv_heads, dim, q.dtype), _pages("v_pages", v_pages, kv_heads, vdim, q.dtype)
    _require(k_pages.shape[:2] == v_pages.shape[:2], "k_pages and v_pages must have the same blocks")
    if slopes is not None:
        a.slopes = _flat("slopes", slopes, heads, torch.float32)
    if row_seq is not None:
        a.row_seq = _flat("row_seq", row_seq, rows, torch.int32)
    a.context_lens = _flat("context_lens", context_lens, rows, torch.int32)
    _require(block_table.dtype == torch.int32 and block_table.is_cuda and block_table.dim() == 2 and block_table.stride(1) == 1
             and (row_seq is not None or not own_rows or block_table.shape[0] >= rows), "block_table must be an int32 GPU tensor [sequences, blocks]")
    a.block_table, a.max_blocks = block_table.data_ptr(), block_table.shape[1]
    a.block_table_stride = block_table.stride(0) if block_table.shape[0] > 1 else block_table.shape[1]
    a.num_blocks, a.block_size = k_pages.shape[:2]
    a.out, a.rows, a.heads, a.kv_heads, a.dim, a.vdim = out.data_ptr(), rows, heads, kv_heads, dim, vdim
    a.scale, a.dtype = float(scale), code
    if scores is not None:
        a.softcap = float(scores.softcap)
        a.window, a.chunk, a.keep_first = (min(int(n), WIDEST) for n in (scores.window, scores.chunk, scores.keep_first))
        if scores.sinks is not None:
            a.sinks = _flat("sinks", scores.sinks, heads, torch.float32)
        if scores.log_distance is not None:
            a.log_rate, a.log_step = (_flat("log_distance", x, heads, torch.float32) for x in scores.log_distance)
        if scores.weight_bias is not None:
            a.weight_bias = _flat("weight_bias", scores.weight_bias, heads, torch.float32)
    if gate is not None:
        a.gate_each = 1 if gate.shape[1] != heads else 0      # values of one element: the two are the same
        a.gate, a.gate_stride = gate.data_ptr(), _rows("gate", gate, heads * vdim if a.gate_each else heads, q.dtype)
        _require(gate.shape[0] == rows, "gate must be [rows, heads] or [rows, heads * vdim]")
    return a


@register_hip_op
def biased_attention_rows(q, k_pages, v_pages, dim, vdim, context_lens, block_table, scale, slopes=None, row_seq=None, scores=None, gate=None, out=None,
                          out_scale=1.0):
    """Attention of single query rows against the pages: row r sees the first context_lens[r] tokens of block table row row_seq[r]
    (r itself without row_seq), or of these what scores lets it see; score = q.k scale - slope (distance), or capped.  gate [rows,
    heads] or [rows, heads * vdim]: the result is multiplied by its sigmoid, and by out_scale.  out: [rows, heads, vdim], or rows [rows,
    heads * vdim] with a stride.  Returns [rows, heads, vdim].  The plain form: any size, bf16 or float32."""
    if out is None:
        out = torch.empty((q.shape[0], q.shape[1], vdim), dtype=q.dtype, device=q.device)
    a = _biased_args(q, k_pages, v_pages, dim, vdim, context_lens, block_table, scale, slopes, row_seq, out, scores=scores, gate=gate, out_scale=out_scale)
    st = _capi.load().mops_hip_biased_attention_rows(byref(a), _stream(q))
    _capi.check("mops_hip_biased_attention_rows", st)
    return out


def biased_matrix_covers(dtype, dim: int, vdim: int, block_size: int) -> bool:
    """Whether biased_decode and biased_prefill cover these sizes."""
    return dtype == torch.bfloat16 and dim <= 256 and vdim <= 256 and block_size % 32 == 0


@register_hip_op
def biased_decode(q, k_pages, v_pages, dim, vdim, context_lens, block_table, scale, slopes=None, row_seq=None, out=None, scores=None, gate=None,
                  out_scale=1.0):
    """biased_attention_rows on the matrix cores (sizes: biased_matrix_covers)."""
    if out is None:
        out = torch.empty((q.shape[0], q.shape[1], vdim), dtype=q.dtype, device=q.device)
    a = _biased_args(q, k_pages, v_pages, dim, vdim, context_lens, block_table, scale, slopes, row_seq, out, scores=scores, gate=gate, out_scale=out_scale)
    lib = _capi.load()
    ws = torch.empty(max(16, lib.mops_hip_biased_decode_workspace_bytes(a.rows, a.heads, a.kv_heads, dim, vdim)), dtype=torch.uint8, device=q.device)
    st = lib.mops_hip_biased_decode(byref(a), ws.data_ptr(), ws.numel(), _stream(q))
    _capi.check("mops_hip_biased_decode", st)
    return out


BIASED_QUERIES = 128


def biased_prefill_tiles(counts, starts, first_token: int, first_seq: int):
    """Host list for biased_prefill: portions of counts[i] tokens at positions starts[i].., packed from row first_token on; sequence i
    of the list is block table row first_seq + i.  The tiles that see most come first: they bound the launch."""
    tiles, at = [], first_token
    for i, (n, start) in enumerate(zip(counts, starts)):
        tiles += [(at + q, min(BIASED_QUERIES, n - q), start + q, first_seq + i, start + n) for q in range(0, n, BIASED_QUERIES)]
        at += n
    return sorted(tiles, key=lambda t: -(t[1] + t[2]))


@register_hip_op
def biased_prefill(q, k_pages, v_pages, dim, vdim, tiles, block_table, scale, context_lens, slopes=None, out=None, scores=None, gate=None,
                   out_scale=1.0):
    """Causal attention of long portions, whose keys and values are in the pages already: tiles [n, 5] is the int32 device copy of
    biased_prefill_tiles.  context_lens: of every row.  Writes the portions' rows of out [rows, heads, vdim]."""
    if out is None:
        out = torch.empty((q.shape[0], q.shape[1], vdim), dtype=q.dtype, device=q.device)
    a = _biased_args(q, k_pages, v_pages, dim, vdim, context_lens, block_table, scale, slopes, None, out, own_rows=False, scores=scores, gate=gate, out_scale=out_scale)
    n = tiles.shape[0]
    st = _capi.load().mops_hip_biased_prefill(byref(a), _flat("tiles", tiles, 5 * n, torch.int32), n, _stream(q))
    _capi.check("mops_hip_biased_prefill", st)
    return out
