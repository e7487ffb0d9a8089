"""Sozarax: a decoder whose layers are listed one by one in the configuration, with time mixing or attention with a distance bias,
and a dense or a routed feed-forward; a run of layers may be passed several times.

The residual stream is float32, with an RMS norm in front of and behind every sublayer: x <- x + norm1b(mixer(norm1(x))), x <- x +
norm2b(ff(norm2(x))).  The norm behind a sublayer, the sum and the norm in front of the next sublayer are one pass.  The embedding
is scaled; the output projection is a matrix of its own.  Runs in bfloat16 and in float32.
"""
from __future__ import annotations

from dataclasses import dataclass

import torch

from . import register_model
from ..layers import FEED_FORWARDS, MIXERS, ModelContext, Rotary, hip_op

TYPES = {"wkv": "time_mixing", "attention": "biased_attention"}              # the configuration's mixers
KINDS = {"dense": "squared_relu", "moe": "scaled_input_mixture"}             # and feed-forwards


@dataclass
class SozaraxConfig:
    vocab: int
    width: int
    eps: float
    embedding_scale: float
    layers: list          # dicts with "type", "mixer" (sizes) and "mlp" (sizes with "kind", or None)
    loop: tuple           # (start, stop, times): layers start .. stop-1 run `times` times in a row

    @classmethod
    def from_dict(cls, raw: dict) -> "SozaraxConfig":
        layers = list(raw["layers"])
        for layer in layers:
            if layer["type"] not in TYPES:
                raise ValueError(f"unknown mixer {layer['type']!r}")
            MIXERS[TYPES[layer["type"]]].validate(layer["mixer"])
            mlp = layer.get("mlp")
            if mlp is not None:
                if mlp["kind"] not in KINDS:
                    raise ValueError(f"unknown feed-forward {mlp['kind']!r}")
                FEED_FORWARDS[KINDS[mlp["kind"]]].validate(mlp)
        loop = raw.get("loop") or {"start": 0, "stop": 0, "times": 1}
        start, stop, times = (int(loop[n]) for n in ("start", "stop", "times"))
        if not 0 <= start <= stop <= len(layers) or times < 1:
            raise ValueError(f"a loop over the layers {start} .. {stop - 1} of {len(layers)}, {times} times")
        return cls(vocab=int(raw["vocab"]), width=int(raw["width"]), eps=float(raw["norm"]["eps"]), embedding_scale=float(raw["embedding"]["scale"]),
                   layers=layers, loop=(start, stop, times))

    def order(self) -> list:
        """Layer numbers in the order in which they run."""
        start, stop, times = self.loop
        return [*range(start), *list(range(start, stop)) * times, *range(stop, len(self.layers))]


@register_model("Sozarax")
class SozaraxModel:
    config_class = SozaraxConfig
    dtypes = (torch.bfloat16, torch.float32)

    @classmethod
    def needs(cls, config):
        """(pages, state slots)"""
        kinds = [MIXERS[TYPES[layer["type"]]] for layer in config.layers]
        return any(k.uses_pages for k in kinds), any(k.uses_slots for k in kinds)

    def __init__(self, config: SozaraxConfig, weights, cache, backend: str = "hip", max_model_len: int = 32768):
        if backend != "hip":
            raise ValueError("Sozarax runs on the hip backend only")
        self.shape, self.cache, self.backend = config, cache, backend
        self.dtype, self.hidden, self.vocab, self.max_positions = weights.dtype, config.width, config.vocab, max_model_len
        take = weights.take
        m = ModelContext(config.width, config.eps, weights.dtype, weights.device, cache, Rotary(max_model_len, weights.device))
        self.embed = take("embed", (config.vocab, config.width), "embed", 1.0)
        layers = []
        for i, spec in enumerate(config.layers):
            p = f"l{i}."
            norm = lambda n: take(p + n, (config.width,), "norm")      # noqa: E731
            n1, n1b = norm("norm1"), norm("norm1b")
            mixer = MIXERS[TYPES[spec["type"]]](spec["mixer"], weights, p + "mix.", m)
            n2 = n2b = ff = None
            if spec.get("mlp") is not None:
                n2, n2b = norm("norm2"), norm("norm2b")
                ff = FEED_FORWARDS[KINDS[spec["mlp"]["kind"]]](spec["mlp"], weights, p + "mlp.", m)
            layers.append((n1, mixer, n1b, n2, ff, n2b))
        self.final_norm = take("final.norm", (config.width,), "norm")
        self.head = take("head", (config.vocab, config.width))
        weights.finish()
        # every run of a layer: the same weights, a cache or state of its own
        self.runs, seen = [], set()
        for i in config.order():
            n1, mixer, *rest = layers[i]
            self.runs.append((n1, mixer.again(cache) if i in seen else mixer, *rest))
            seen.add(i)
        self.op_embed, self.op_norm, self.op_add_norm_norm = hip_op("embed_residual"), hip_op("rms_norm_f32"), hip_op("add_norm_norm")
        self.op_linear, self.op_sampler_forward = hip_op("linear"), hip_op("sampler_forward")
        self.layer_hook = None   # called as hook(number of the layer run, float32 residual) after every layer run

    def reserve_graph_scratch(self, max_bs: int, max_blocks: int) -> None:
        """Makes the scratch of the current stream exist before a capture."""
        from ..mops.hip.ops import _linear_workspace
        _linear_workspace(self.embed.device)

    @torch.inference_mode()
    def forward(self, input_ids, positions, ctx):
        eps, runs = self.shape.eps, self.runs
        residual, _ = self.op_embed(input_ids, self.embed, self.shape.embedding_scale, need_act=False)
        x = self.op_norm(residual, runs[0][0] if runs else self.final_norm, eps)
        for i, (_, mixer, norm1b, norm2, ff, norm2b) in enumerate(runs):
            following = runs[i + 1][0] if i + 1 < len(runs) else self.final_norm
            x = self.op_add_norm_norm(residual, mixer(x, ctx), norm1b, norm2 if ff is not None else following, eps)
            if ff is not None:
                x = self.op_add_norm_norm(residual, ff(x), norm2b, following, eps)
            if self.layer_hook is not None:
                self.layer_hook(i, residual)
        if ctx.get("hidden_only"):
            return x
        rows = ctx.get("logit_rows")
        if rows is None and ctx["is_prefill"]:
            rows = ctx["cu_seqlens"][1:].long() - 1
        return self.logits(x if rows is None else x[rows])

    def logits(self, hidden):
        return self.op_linear(hidden, self.head)
