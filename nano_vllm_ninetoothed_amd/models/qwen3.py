"""Qwen3 decoder: configuration, weights and forward pass over the mops operators.

Op order of a decoder layer and of the model as in the reference (nanovllm/models/qwen3.py:69-82, 140-153, 167-177,
199-210): embedding -> [rms/add_rms -> qkv linear -> q_norm/k_norm on strided views -> rotary -> store_kvcache + varlen
prefill | paged decode -> o_proj -> add_rms -> gate_up linear -> siluAndMul -> down linear] x L -> add_rms -> lm head (tied)
on the wanted rows.  The per-layer k/v caches are slabs of one contiguous [2, L, blocks, block_size, Hkv, D] tensor
(nanovllm/engine/model_runner.py:100-118).
"""
from __future__ import annotations

from dataclasses import dataclass

import torch

from . import register_model
from .. import mops


@dataclass
class Qwen3Shape:
    """Qwen3-0.6B architecture numbers."""
    num_layers: int = 28
    hidden: int = 1024
    num_heads: int = 16
    num_kv_heads: int = 8
    head_dim: int = 128
    intermediate: int = 3072
    vocab: int = 151936
    rms_eps: float = 1e-6
    rope_theta: float = 1000000.0
    max_position: int = 40960

    @classmethod
    def from_dict(cls, raw: dict) -> "Qwen3Shape":
        if not raw.get("tie_word_embeddings", False) or raw.get("attention_bias", False):
            raise ValueError("only Qwen3 models with tied embeddings and without attention biases are supported")
        return cls(num_layers=raw["num_hidden_layers"], hidden=raw["hidden_size"], num_heads=raw["num_attention_heads"],
                   num_kv_heads=raw["num_key_value_heads"], head_dim=raw.get("head_dim", 128), intermediate=raw["intermediate_size"],
                   vocab=raw["vocab_size"], rms_eps=raw["rms_norm_eps"], rope_theta=raw["rope_theta"],
                   max_position=raw.get("max_position_embeddings", 40960))


@register_model("Qwen3ForCausalLM")
class Qwen3Model:
    config_class = Qwen3Shape
    dtypes = (torch.bfloat16,)
    uses_pages, uses_slots = True, False

    @classmethod
    def needs(cls, config):
        """(pages, state slots)"""
        return True, False

    def __init__(self, config: Qwen3Shape, weights, cache, backend: str = "hip", max_model_len: int = None):
        self.shape = s = config
        self.backend, self.cache = backend, cache
        self.dtype, self.hidden, self.vocab = torch.bfloat16, s.hidden, s.vocab
        self.max_positions = s.max_position
        for name in mops.OP_NAMES:
            op = mops.get_op(name, backend)
            if op is None and name != "softmax":
                raise RuntimeError(f"backend {backend} does not provide {name}")
            setattr(self, "op_" + name, op)
        # the fused q_norm + k_norm + rotary + store_kvcache launch, where the backend has it
        self.op_qk_norm_rope_store = mops.get_op("qk_norm_rope_store", backend) if mops.has_op("qk_norm_rope_store", backend) else None
        self.use_fused_qk = True
        self.share_decode_plan = True   # layers 2..N of a decode step reuse layer 1's split of the KV stream

        q_size, kv_size = s.num_heads * s.head_dim, s.num_kv_heads * s.head_dim
        self.q_size, self.kv_size = q_size, kv_size
        take = weights.take
        self.embed = take("model.embed_tokens.weight", (s.vocab, s.hidden), "embed")          # tied: also the lm head
        self.layers = []
        for i in range(s.num_layers):
            p = f"model.layers.{i}."
            L = dict(input_norm=take(p + "input_layernorm.weight", (s.hidden,), "norm"),
                     post_norm=take(p + "post_attention_layernorm.weight", (s.hidden,), "norm"),
                     q_norm=take(p + "self_attn.q_norm.weight", (s.head_dim,), "norm"),
                     k_norm=take(p + "self_attn.k_norm.weight", (s.head_dim,), "norm"))
            L["qkv"] = torch.cat([take(p + f"self_attn.{n}_proj.weight", (rows, s.hidden))
                                  for n, rows in (("q", q_size), ("k", kv_size), ("v", kv_size))])
            L["o"] = take(p + "self_attn.o_proj.weight", (s.hidden, q_size))
            L["gate_up"] = torch.cat([take(p + f"mlp.{n}_proj.weight", (s.intermediate, s.hidden)) for n in ("gate", "up")])
            L["down"] = take(p + "mlp.down_proj.weight", (s.hidden, s.intermediate))
            self.layers.append(L)
        self.final_norm = take("model.norm.weight", (s.hidden,), "norm")
        weights.finish()

        inv_freq = 1.0 / (s.rope_theta ** (torch.arange(0, s.head_dim, 2, dtype=torch.float32) / s.head_dim))
        freqs = torch.outer(torch.arange(s.max_position, dtype=torch.float32), inv_freq)
        self.cos_sin = torch.cat((freqs.cos(), freqs.sin()), dim=-1).unsqueeze(1).to(self.embed.device)   # [P, 1, D]
        self.kv_cache = cache.paged(s.num_kv_heads, s.head_dim, lead=(2, s.num_layers))
        self.scale = s.head_dim ** -0.5

    def reserve_graph_scratch(self, max_bs: int, max_blocks: int) -> None:
        """Sizes the scratch of the current stream for captured decode steps of up to max_bs sequences."""
        if self.backend == "hip":
            from ..mops.hip.ops import reserve_decode_workspace
            reserve_decode_workspace(max_bs, self.shape.num_heads, self.shape.num_kv_heads, max_blocks, self.cache.block_size, self.embed.device)

    def _attention(self, layer_id, q, k, v, ctx, stored=False):
        k_cache, v_cache = self.kv_cache[0, layer_id], self.kv_cache[1, layer_id]
        if not stored:
            self.op_store_kvcache(k, v, k_cache, v_cache, ctx["slot_mapping"])
        if ctx["is_prefill"]:
            if ctx.get("has_prefix"):     # portions behind tokens of earlier steps: keys and values come from the pages
                return self.op_flash_attn_varlen_func(q, k_cache, v_cache, max_seqlen_q=ctx["max_seqlen"], cu_seqlens_q=ctx["cu_seqlens"],
                                                      max_seqlen_k=ctx["max_context"], cu_seqlens_k=ctx["cu_context"],
                                                      softmax_scale=self.scale, causal=True, block_table=ctx["block_tables"])
            return self.op_flash_attn_varlen_func(q, k, v, max_seqlen_q=ctx["max_seqlen"], cu_seqlens_q=ctx["cu_seqlens"],
                                                  max_seqlen_k=ctx["max_seqlen"], cu_seqlens_k=ctx["cu_seqlens"],
                                                  softmax_scale=self.scale, causal=True, block_table=None)
        extra = {"reuse_plan": True} if (self.backend == "hip" and self.share_decode_plan and layer_id > 0) else {}
        return self.op_flash_attn_with_kvcache(q.unsqueeze(1), k_cache, v_cache, cache_seqlens=ctx["context_lens"],
                                               block_table=ctx["block_tables"], softmax_scale=self.scale, causal=True, **extra)

    @torch.inference_mode()
    def forward(self, input_ids, positions, ctx):
        s = self.shape
        h = self.op_embedding(input_ids, self.embed)
        residual = None
        cos, sin = self.cos_sin[positions].chunk(2, dim=-1)
        for i, L in enumerate(self.layers):
            if residual is None:
                h, residual = self.op_rms_forward(h, L["input_norm"], s.rms_eps), h
            else:
                h, residual = self.op_add_rms_forward(h, residual, L["input_norm"], s.rms_eps)
            qkv = self.op_linear(h, L["qkv"])
            if self.op_qk_norm_rope_store is not None and self.use_fused_qk:
                q, k, v = self.op_qk_norm_rope_store(qkv, L["q_norm"], L["k_norm"], s.rms_eps, cos, sin, self.kv_cache[0, i],
                                                     self.kv_cache[1, i], ctx["slot_mapping"], s.num_heads, s.num_kv_heads,
                                                     need_k=ctx["is_prefill"])
                o = self._attention(i, q, k, v, ctx, stored=True)
            else:
                q, k, v = qkv.split([self.q_size, self.kv_size, self.kv_size], dim=-1)
                q = self.op_rms_forward(q.view(-1, s.num_heads, s.head_dim), L["q_norm"], s.rms_eps)
                k = self.op_rms_forward(k.view(-1, s.num_kv_heads, s.head_dim), L["k_norm"], s.rms_eps)
                v = v.view(-1, s.num_kv_heads, s.head_dim)
                q = self.op_apply_rotary_emb(q, cos, sin)
                k = self.op_apply_rotary_emb(k, cos, sin)
                o = self._attention(i, q, k, v, ctx)
            h = self.op_linear(o.flatten(1, -1), L["o"])
            h, residual = self.op_add_rms_forward(h, residual, L["post_norm"], s.rms_eps)
            gate, up = self.op_linear(h, L["gate_up"]).chunk(2, -1)
            h = self.op_linear(self.op_siluAndMul(gate, up), L["down"])
        h, _ = self.op_add_rms_forward(h, residual, self.final_norm, s.rms_eps)
        if ctx.get("hidden_only"):
            return h
        if ctx.get("logit_rows") is not None:
            h = h[ctx["logit_rows"]]
        elif ctx["is_prefill"]:
            h = h[ctx["cu_seqlens"][1:].long() - 1].contiguous()
        return self.logits(h)

    def logits(self, hidden):
        return self.op_linear(hidden, self.embed)
