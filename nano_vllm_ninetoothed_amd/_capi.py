"""ctypes binding of libmops_hip.so — the only way the Python host code reaches the HIP kernels.

The library is loaded lazily on first use and the load fails loudly: there is no CPU or torch
fallback behind these functions.  Signatures mirror include/mops_hip.h one to one.
"""
from __future__ import annotations

import ctypes
import os
from ctypes import POINTER, Structure, c_char_p, c_float, c_int, c_int64, c_void_p
from pathlib import Path

# MOPS_HIP_LIB points at another build of the same ABI (kernel tuning experiments)
LIB_PATH = Path(os.environ.get("MOPS_HIP_LIB") or Path(__file__).resolve().parent / "lib" / "libmops_hip.so")

class Recurrence(Structure):
    """mops_hip_recurrence of the header, field by field."""
    _fields_ = ([(n, c_void_p) for n in ("q", "k", "v")] + [(n, c_int64) for n in ("q_stride", "k_stride", "v_stride")]
                + [("out", c_void_p), ("out_stride", c_int64), ("state", c_void_p), ("num_slots", c_int64)]
                + [(n, c_void_p) for n in ("state_slots", "cu_seqlens", "starts", "decay", "log_decay", "neg_a", "dt_bias", "skip", "cos_sin", "dt")]
                + [(n, c_int64) for n in ("dt_stride", "batch", "heads", "groups", "d", "vd", "rot", "max_positions")]
                + [(n, c_void_p) for n in ("conv_weight", "conv_bias", "conv_ring")]
                + [(n, c_int64) for n in ("taps", "channels", "q_channel", "k_channel", "v_channel")]
                + [("channel_decay", c_void_p), ("bonus", c_void_p), ("channel_decay_stride", c_int64)]
                + [("k_scale", c_float), ("dtype", c_int)]
                + [("input_gate", c_void_p), ("forget_gate", c_void_p), ("gate_stride", c_int64)]
                + [(n, c_void_p) for n in ("input_bias", "forget_bias", "top", "log_keep", "input_scale", "least")] + [("gate_cap", c_float)])


class Delta(Structure):
    """mops_hip_delta of the header, field by field."""
    _fields_ = ([(n, c_void_p) for n in ("q", "k", "v")] + [(n, c_int64) for n in ("q_stride", "k_stride", "v_stride")]
                + [("out", c_void_p), ("out_stride", c_int64), ("state", c_void_p), ("num_slots", c_int64)]
                + [(n, c_void_p) for n in ("state_slots", "cu_seqlens", "starts", "log_decay", "beta")]
                + [(n, c_int64) for n in ("log_decay_stride", "beta_stride", "batch", "heads", "groups", "d", "vd")]
                + [("conv_weight", c_void_p), ("conv_ring", c_void_p)] + [(n, c_int64) for n in ("taps", "channels", "q_channel", "k_channel", "v_channel")]
                + [("q_scale", c_float), ("unit_eps", c_float), ("dtype", c_int)])


class AddNorm(Structure):
    """mops_hip_add_norm_args of the header, field by field."""
    _fields_ = ([("residual", c_void_p), ("y", c_void_p), ("y_stride", c_int64)] + [(n, c_void_p) for n in ("shift", "w", "b", "out")]
                + [(n, c_int64) for n in ("out_stride", "rows", "n")] + [("eps", c_float)] + [(n, c_int) for n in ("replace", "center", "dtype")])


class LatentRows(Structure):
    """mops_hip_latent_rows of the header, field by field."""
    _fields_ = ([(n, c_void_p) for n in ("q_latent", "q_rot")] + [(n, c_int64) for n in ("q_rot_token_stride", "q_rot_head_stride")]
                + [("cache", c_void_p), ("pitch", c_int64), ("cos_sin", c_void_p), ("max_positions", c_int64)]
                + [(n, c_void_p) for n in ("row_seq", "context_lens", "block_table")]
                + [(n, c_int64) for n in ("block_table_stride", "block_size", "num_blocks", "max_blocks")]
                + [("out", c_void_p)] + [(n, c_int64) for n in ("rows", "heads", "kv_rank", "rot_dim")]
                + [("scale", c_float), ("dtype", c_int)])


class AttentionPrepare(Structure):
    """mops_hip_attention_prepare_args of the header, field by field."""
    _fields_ = ([("qkv", c_void_p), ("qkv_stride", c_int64)] + [(n, c_void_p) for n in ("q_weight", "k_weight", "q_factor")]
                + [("max_positions", c_int64)] + [(n, c_void_p) for n in ("positions", "slot_mapping", "q", "k_pages", "v_pages")]
                + [(n, c_int64) for n in ("num_slots", "tokens", "heads", "kv_heads", "dim", "vdim")] + [("eps", c_float), ("dtype", c_int)])


class BiasedAttention(Structure):
    """mops_hip_biased_attention of the header, field by field."""
    _fields_ = ([(n, c_void_p) for n in ("q", "k_pages", "v_pages", "slopes", "row_seq", "context_lens", "block_table")]
                + [(n, c_int64) for n in ("block_table_stride", "block_size", "num_blocks", "max_blocks")]
                + [("out", c_void_p)] + [(n, c_int64) for n in ("rows", "heads", "kv_heads", "dim", "vdim")]
                + [("scale", c_float), ("dtype", c_int), ("softcap", c_float)] + [(n, c_int64) for n in ("window", "chunk", "keep_first")]
                + [("sinks", c_void_p), ("gate", c_void_p), ("gate_stride", c_int64)]
                + [(n, c_void_p) for n in ("log_rate", "log_step", "weight_bias")] + [("gate_each", c_int64), ("out_stride", c_int64), ("out_scale", c_float)])


class RotaryPrepare(Structure):
    """mops_hip_rotary_prepare_args of the header, field by field."""
    _fields_ = ([("qkv", c_void_p), ("qkv_stride", c_int64)] + [(n, c_void_p) for n in ("q_weight", "k_weight", "cos_sin")]
                + [("max_positions", c_int64), ("rot", c_int64)] + [(n, c_void_p) for n in ("positions", "slot_mapping", "q", "k_pages", "v_pages")]
                + [(n, c_int64) for n in ("num_slots", "tokens", "heads", "kv_heads", "dim", "vdim")] + [("eps", c_float), ("dtype", c_int)]
                + [("bias", c_void_p), ("neighbours", c_int64)])


class EmbedPairs(Structure):
    """mops_hip_embed_pairs_args of the header, field by field."""
    _fields_ = ([(n, c_void_p) for n in ("ids", "table", "pairs")]
                + [(n, c_int64) for n in ("table_stride", "pairs_stride", "buckets", "mul_prev", "mul_cur")] + [("before", c_void_p), ("num_slots", c_int64)]
                + [(n, c_void_p) for n in ("token_seq", "cu_seqlens", "starts", "state_slots", "residual")]
                + [(n, c_int64) for n in ("tokens", "vocab", "width")] + [("scale", c_float), ("dtype", c_int)])


class Moe(Structure):
    """mops_hip_moe of the header, field by field."""
    _fields_ = ([(n, c_void_p) for n in ("rows", "tiles", "score")]
                + [(n, c_int64) for n in ("tokens", "experts", "top", "width", "ff", "block_rows")] + [("dtype", c_int), ("unit", c_int)]
                + [("limit", c_float), ("alpha", c_float), ("correction", c_void_p), ("groups", c_int64), ("keep", c_int64), ("factor", c_float)]
                + [("common_limit", c_float)] + [(n, c_void_p) for n in ("common_x", "common_w", "common_out")]
                + [(n, c_int64) for n in ("common_x_stride", "common_out_stride", "common_ff", "common_up_at")])


# name -> (restype, argtypes); the exported surface declared in include/mops_hip.h
SIGNATURES = {
    "mops_hip_abi_version": (c_int, []),
    "mops_hip_status_string": (c_char_p, [c_int]),
    "mops_hip_last_hip_error": (c_int, []),
    "mops_hip_store_kvcache": (c_int, [c_void_p, c_int64, c_void_p, c_int64, c_void_p, c_void_p, c_void_p,
                                       c_int64, c_int64, c_int64, c_void_p]),
    "mops_hip_embedding": (c_int, [c_void_p, c_int, c_void_p, c_int64, c_void_p, c_int64, c_int64, c_int64,
                                   c_void_p]),
    "mops_hip_rms_forward": (c_int, [c_void_p, c_void_p, c_void_p, c_int64, c_int64, c_int64, c_int64, c_int64,
                                     c_float, c_void_p]),
    "mops_hip_add_rms_forward": (c_int, [c_void_p, c_int64, c_void_p, c_int64, c_void_p, c_void_p, c_void_p,
                                         c_int64, c_int64, c_float, c_void_p]),
    "mops_hip_paged_decode_workspace_bytes": (c_int64, [c_int64, c_int64, c_int64, c_int64, c_int64]),
    "mops_hip_attn_paged_decode_bf16": (c_int, [c_void_p, c_int64, c_void_p, c_void_p, c_void_p, c_void_p,
                                                c_int64, c_void_p, c_int64, c_int64, c_int64, c_int64,
                                                c_int64, c_int64, c_int64, c_float, c_void_p, c_int64,
                                                c_void_p]),
    "mops_hip_attn_paged_decode_planned_bf16": (c_int, [c_void_p, c_int64, c_void_p, c_void_p, c_void_p, c_void_p,
                                                c_int64, c_void_p, c_int64, c_int64, c_int64, c_int64,
                                                c_int64, c_int64, c_int64, c_float, c_void_p, c_int64,
                                                c_int, c_void_p]),
    "mops_hip_attn_paged_decode_noalloc_bf16": (c_int, [c_void_p, c_int64, c_void_p, c_void_p, c_void_p, c_void_p,
                                                        c_int64, c_void_p, c_int64, c_int64, c_int64, c_int64,
                                                        c_int64, c_int64, c_int64, c_float, c_void_p]),
    "mops_hip_attn_varlen_causal_bf16": (c_int, [c_void_p, c_int64, c_void_p, c_int64, c_void_p, c_int64,
                                                 c_void_p, c_int64, c_void_p, c_void_p, c_void_p, c_int64,
                                                 c_int64, c_int64, c_int64, c_int64, c_int64, c_int64, c_int64,
                                                 c_int64, c_int64, c_int64, c_float, c_void_p]),
    "mops_hip_silu_and_mul": (c_int, [c_void_p, c_int64, c_void_p, c_int64, c_void_p, c_int64, c_int64, c_void_p]),
    "mops_hip_apply_rotary_emb": (c_int, [c_void_p, c_int64, c_int64, c_void_p, c_int64, c_void_p, c_int64, c_void_p,
                                          c_int64, c_int64, c_int64, c_void_p]),
    "mops_hip_sampler_argmax": (c_int, [c_void_p, c_int64, c_void_p, c_int64, c_int64, c_void_p]),
    "mops_hip_launch_floor": (c_int, [c_void_p]),
    "mops_hip_qk_norm_rope_store": (c_int, [c_void_p, c_int64, c_void_p, c_void_p, c_void_p, c_int64, c_void_p, c_int64,
                                            c_void_p, c_void_p, c_void_p, c_void_p, c_void_p, c_int64, c_int64, c_int64,
                                            c_int64, c_int64, c_float, c_void_p]),
    "mops_hip_linear_bf16": (c_int, [c_void_p, c_int64, c_void_p, c_int64, c_void_p, c_void_p, c_int64, c_int64, c_int64,
                                     c_int64, c_void_p, c_int64, c_void_p]),
    "mops_hip_embed_residual": (c_int, [c_void_p, c_void_p, c_int64, c_int, c_float, c_void_p, c_void_p, c_int64, c_int64, c_int64, c_int64, c_void_p]),
    "mops_hip_add_norm": (c_int, [POINTER(AddNorm), c_void_p]),
    "mops_hip_norm_residual_add": (c_int, [c_void_p, c_void_p, c_int64, c_void_p, c_float, c_float, c_void_p, c_int, c_int64, c_int64,
                                           c_void_p]),
    "mops_hip_add_norm_norm": (c_int, [c_void_p, c_void_p, c_int64, c_int64, c_void_p, c_void_p, c_void_p, c_float, c_int, c_void_p, c_int, c_int64,
                                       c_int64, c_void_p]),
    "mops_hip_layer_norm_f32": (c_int, [c_void_p, c_void_p, c_float, c_void_p, c_int, c_int64, c_int64, c_void_p]),
    "mops_hip_embed_pairs": (c_int, [POINTER(EmbedPairs), c_void_p]),
    "mops_hip_rms_norm_f32": (c_int, [c_void_p, c_void_p, c_float, c_float, c_void_p, c_int, c_int64, c_int64, c_void_p]),
    "mops_hip_gated_group_norm": (c_int, [c_void_p, c_int64, c_void_p, c_int64, c_void_p, c_int, c_float, c_int, c_int, c_float, c_void_p, c_int64,
                                          c_int, c_int64, c_int64, c_int64, c_void_p]),
    "mops_hip_clamped_glu": (c_int, [c_void_p, c_int64, c_void_p, c_int64, c_void_p, c_int64, c_int, c_int64, c_int64, c_float, c_float, c_void_p]),
    "mops_hip_gelu_glu": (c_int, [c_void_p, c_int64, c_void_p, c_int64, c_void_p, c_int64, c_int, c_int64, c_int64, c_void_p]),
    "mops_hip_relu_glu": (c_int, [c_void_p, c_int64, c_void_p, c_int64, c_void_p, c_int64, c_int, c_int64, c_int64, c_void_p]),
    "mops_hip_matrix_memory_copies": (c_int64, [c_int64]),
    "mops_hip_delta_rule": (c_int, [POINTER(Delta), c_void_p]),
    "mops_hip_delta_chunks_workgroups": (c_int64, [c_int64] * 2),
    "mops_hip_delta_chunks_workspace_bytes": (c_int64, [c_int64] * 6),
    "mops_hip_delta_chunks": (c_int, [POINTER(Delta), c_void_p, c_int64, c_void_p, c_int64, c_void_p, c_void_p, c_int64, c_void_p]),
    "mops_hip_matrix_memory_gates": (c_int, [POINTER(Recurrence)] + [c_void_p] * 4),
    "mops_hip_recurrence_state_pitch": (c_int64, [c_int64]),
    "mops_hip_decayed_recurrence": (c_int, [POINTER(Recurrence), c_void_p]),
    "mops_hip_decayed_chunks_workgroups": (c_int64, [c_int64] * 3),
    "mops_hip_decayed_chunks": (c_int, [POINTER(Recurrence), c_void_p, c_int64, c_void_p, c_void_p, c_void_p, c_void_p]),
    "mops_hip_channel_chunks_workgroups": (c_int64, [c_int64] * 2),
    "mops_hip_channel_chunks": (c_int, [POINTER(Recurrence), c_void_p, c_int64, c_void_p, c_void_p, c_void_p, c_void_p]),
    "mops_hip_short_conv": (c_int, [c_void_p, c_int64, c_void_p, c_void_p, c_void_p, c_int64, c_void_p, c_void_p, c_void_p, c_void_p,
                                    c_void_p, c_int, c_int64, c_int64, c_int64, c_void_p]),
    "mops_hip_short_conv_update": (c_int, [c_void_p, c_int64, c_void_p, c_int64, c_void_p, c_void_p, c_void_p, c_int, c_int64, c_int64,
                                           c_int64, c_void_p]),
    "mops_hip_latent_prepare": (c_int, [c_void_p, c_int64, c_void_p, c_void_p, c_float, c_void_p, c_int64, c_void_p, c_void_p, c_void_p,
                                        c_void_p, c_int64, c_int64, c_int, c_int64, c_int64, c_int64, c_int64, c_void_p]),
    "mops_hip_head_linear": (c_int, [c_void_p, c_int64, c_int64, c_void_p, c_void_p, c_int64, c_int64, c_int, c_int64, c_int64, c_int64,
                                     c_int64, c_void_p]),
    "mops_hip_latent_attention_rows": (c_int, [POINTER(LatentRows), c_void_p]),
    "mops_hip_latent_decode_workspace_bytes": (c_int64, [c_int64] * 4),
    "mops_hip_latent_decode": (c_int, [POINTER(LatentRows), c_void_p, c_int64, c_void_p]),
    "mops_hip_latent_gather": (c_int, [c_void_p, c_int64, c_void_p, c_int64, c_int64, c_int64, c_int64, c_void_p, c_void_p, c_void_p,
                                       c_int64, c_void_p, c_int64, c_int64, c_int64, c_int64, c_void_p]),
    "mops_hip_latent_prefill": (c_int, [c_void_p, c_int64, c_int64, c_void_p, c_int64, c_void_p, c_int64, c_void_p, c_int64, c_void_p,
                                        c_int64, c_void_p, c_int64, c_int64, c_int64, c_int64, c_float, c_void_p]),
    "mops_hip_rotate_pairs": (c_int, [c_void_p, c_int64, c_int64, c_void_p, c_void_p, c_int64, c_int64, c_int64, c_int64, c_void_p]),
    "mops_hip_token_mix": (c_int, [c_void_p, c_int64, c_void_p, c_int64, c_void_p, c_int64, c_void_p, c_void_p, c_void_p, c_void_p, c_void_p,
                                   c_int, c_int64, c_int64, c_void_p]),
    "mops_hip_low_rank_decay": (c_int, [c_void_p, c_int64, c_void_p, c_void_p, c_void_p, c_int64, c_void_p, c_int, c_int64, c_int64, c_int64, c_void_p]),
    "mops_hip_squared_relu": (c_int, [c_void_p, c_int64, c_void_p, c_int, c_int64, c_int64, c_void_p]),
    "mops_hip_attention_prepare": (c_int, [POINTER(AttentionPrepare), c_void_p]),
    "mops_hip_rotary_prepare": (c_int, [POINTER(RotaryPrepare), c_void_p]),
    "mops_hip_biased_attention_rows": (c_int, [POINTER(BiasedAttention), c_void_p]),
    "mops_hip_biased_decode_workspace_bytes": (c_int64, [c_int64] * 5),
    "mops_hip_biased_decode": (c_int, [POINTER(BiasedAttention), c_void_p, c_int64, c_void_p]),
    "mops_hip_biased_prefill": (c_int, [POINTER(BiasedAttention), c_void_p, c_int64, c_void_p]),
    "mops_hip_moe_max_tiles": (c_int64, [c_int64] * 4),
    "mops_hip_moe_route_workgroups": (c_int64, [c_int64]),
    "mops_hip_moe_route": (c_int, [c_void_p, c_int64, c_void_p, c_void_p, c_void_p, c_void_p, POINTER(Moe), c_void_p]),
    "mops_hip_moe_gate_up": (c_int, [c_void_p, c_int64, c_void_p, c_int64, c_void_p, c_int64, POINTER(Moe), c_void_p]),
    "mops_hip_grouped_linear": (c_int, [c_void_p] * 5 + [c_int64] * 5 + [c_void_p]),
    "mops_hip_moe_down": (c_int, [c_void_p, c_int64, c_void_p, c_int64, c_void_p, c_int64, POINTER(Moe), c_void_p]),
    "mops_hip_linear_pin_solution": (c_int, [c_int64, c_int64, c_int64, c_int]),
    "mops_hip_linear_tune": (c_int, [c_int64, c_int64, c_int64, c_int64, c_int, c_void_p, c_int64, c_void_p, c_void_p, c_void_p]),
}

ABI_VERSION = 13

_lib = None


class MopsHipError(RuntimeError):
    """A launcher of libmops_hip.so returned a negative status."""

    def __init__(self, func: str, status: int, text: str):
        super().__init__(f"{func} failed with status {status}: {text}")
        self.func = func
        self.status = status


def load() -> ctypes.CDLL:
    """Loads the library (once) and fixes the prototypes.  Raises if it is missing or stale."""
    global _lib
    if _lib is not None:
        return _lib
    if not LIB_PATH.exists():
        raise ImportError(
            f"{LIB_PATH} is missing: the hip backend has no fallback. Build it with "
            "`python -m nano_vllm_ninetoothed_amd.build` (needs hipcc, no GPU required)."
        )
    try:
        # torch wheels carry their own HIP runtime and hipBLASLt under the sonames this library links
        # against; importing torch first keeps one copy of each in the process, whichever order the caller
        # imports things in (and the GEMM solution table was measured against that copy)
        import torch  # noqa: F401
    except ImportError:
        pass
    lib = ctypes.CDLL(str(LIB_PATH))
    for name, (restype, argtypes) in SIGNATURES.items():
        fn = getattr(lib, name)  # AttributeError here means header and library disagree
        fn.restype = restype
        fn.argtypes = argtypes
    if lib.mops_hip_abi_version() != ABI_VERSION:
        raise ImportError(f"{LIB_PATH} has ABI {lib.mops_hip_abi_version()}, binding expects {ABI_VERSION}; rebuild")
    _lib = lib
    return lib


def check(func: str, status: int) -> None:
    if status != 0:
        lib = load()
        text = lib.mops_hip_status_string(status).decode()
        if status == -5:  # MOPS_HIP_ELAUNCH
            text += f" (hipError {lib.mops_hip_last_hip_error()})"
        raise MopsHipError(func, status, text)
