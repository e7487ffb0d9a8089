"""Nepulix: a decoder whose layers are listed one by one in the configuration, each with a mixer of its own kind and an
optional feed-forward.

The residual stream is float32.  A sublayer reads the stream itself; its output goes through an RMS norm (weight stored
around zero) and is then added: x <- x + norm1(mixer(x)), x <- x + norm2(ff(x)).  A final norm of the same kind, then the
embedding table as the output projection.  Runs in bfloat16 and in float32.
"""
from __future__ import annotations

from dataclasses import dataclass

import torch

from . import register_model
from ..layers import FEED_FORWARDS, MIXERS, ModelContext, Rotary, hip_op


TYPES = ("retention", "mamba2", "latent_attention")
KINDS = {"dense": "clamped_glu"}      # the configuration's feed-forwards


@dataclass
class NepulixConfig:
    vocab: int
    width: int
    eps: float
    layers: list          # dicts with "type", "mixer" (sizes) and "mlp" (sizes with "kind", or None)

    @classmethod
    def from_dict(cls, raw: dict) -> "NepulixConfig":
        for layer in raw["layers"]:
            if layer["type"] not in TYPES:
                raise ValueError(f"unknown mixer {layer['type']!r}")
            MIXERS[layer["type"]].validate(layer["mixer"])
            mlp = layer.get("mlp")
            if mlp is not None:
                if mlp["kind"] not in KINDS:
                    raise ValueError(f"unknown feed-forward {mlp['kind']!r}")
                FEED_FORWARDS[KINDS[mlp["kind"]]].validate(mlp)
        return cls(vocab=int(raw["vocab"]), width=int(raw["width"]), eps=float(raw["norm"]["eps"]), layers=list(raw["layers"]))


@register_model("Nepulix")
class NepulixModel:
    config_class = NepulixConfig
    dtypes = (torch.bfloat16, torch.float32)
    NORM_OFFSET = 1.0        # norm weights are stored around zero

    @classmethod
    def needs(cls, config):
        """(pages, state slots)"""
        kinds = [MIXERS[layer["type"]] for layer in config.layers]
        return any(k.uses_pages for k in kinds), any(k.uses_slots for k in kinds)

    def __init__(self, config: NepulixConfig, weights, cache, backend: str = "hip", max_model_len: int = 32768):
        if backend != "hip":
            raise ValueError("Nepulix runs on the hip backend only")
        self.shape, self.cache, self.backend = config, cache, backend
        self.dtype, self.hidden, self.vocab, self.max_positions = weights.dtype, config.width, config.vocab, max_model_len
        take = weights.take
        m = ModelContext(config.width, config.eps, weights.dtype, weights.device, cache, Rotary(max_model_len, weights.device))
        self.embed = take("embed", (config.vocab, config.width), "embed", 1.0)
        self.layers = []
        for i, spec in enumerate(config.layers):
            p = f"l{i}."
            norm1 = take(p + "norm1", (config.width,), "norm_offset")
            mixer = MIXERS[spec["type"]](spec["mixer"], weights, p + "mix.", m)
            norm2 = ff = None
            if spec.get("mlp") is not None:
                norm2 = take(p + "norm2", (config.width,), "norm_offset")
                ff = FEED_FORWARDS[KINDS[spec["mlp"]["kind"]]](spec["mlp"], weights, p + "mlp.", m)
            self.layers.append((mixer, norm1, ff, norm2))
        self.final_norm = take("final.norm", (config.width,), "norm_offset")
        weights.finish()
        self.op_embed, self.op_norm_add, self.op_norm = hip_op("embed_residual"), hip_op("norm_residual_add"), hip_op("rms_norm_f32")
        self.op_linear, self.op_sampler_forward = hip_op("linear"), hip_op("sampler_forward")
        self.layer_hook = None   # called as hook(layer index, float32 residual) after every layer

    def reserve_graph_scratch(self, max_bs: int, max_blocks: int) -> None:
        """Makes the scratch of the current stream exist before a capture."""
        from ..mops.hip.ops import _linear_workspace
        _linear_workspace(self.embed.device)

    @torch.inference_mode()
    def forward(self, input_ids, positions, ctx):
        eps, off = self.shape.eps, self.NORM_OFFSET
        residual, x = self.op_embed(input_ids, self.embed)
        for i, (mixer, norm1, ff, norm2) in enumerate(self.layers):
            x = self.op_norm_add(residual, mixer(x, ctx), norm1, eps, off)
            if ff is not None:
                x = self.op_norm_add(residual, ff(x), norm2, eps, off)
            if self.layer_hook is not None:
                self.layer_hook(i, residual)
        if not ctx.get("hidden_only"):
            rows = ctx.get("logit_rows")
            if rows is None and ctx["is_prefill"]:
                rows = ctx["cu_seqlens"][1:].long() - 1
            if rows is not None:
                residual = residual[rows]
        h = self.op_norm(residual, self.final_norm, eps, off)
        return h if ctx.get("hidden_only") else self.logits(h)

    def logits(self, hidden):
        return self.op_linear(hidden, self.embed)
