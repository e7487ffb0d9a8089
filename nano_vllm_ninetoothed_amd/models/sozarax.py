"""Sozarax: a decoder whose layers are listed one by one in the configuration, with time mixing or attention with a distance bias,
and a dense or a routed feed-forward; a run of layers may be passed several times.  RMS norms; the embedding is scaled."""
from __future__ import annotations

from dataclasses import dataclass

from . import register_model
from .listed import looped, parse_loop
from .sandwich import SandwichDecoder
from ..layers import hip_op


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
            SozaraxModel.validate_layer(layer)
        return cls(vocab=int(raw["vocab"]), width=int(raw["width"]), eps=float(raw["norm"]["eps"]), embedding_scale=float(raw["embedding"]["scale"]),
                   layers=layers, loop=parse_loop(raw, len(layers)))

    def order(self) -> list:
        """Layer numbers in the order in which they run."""
        return looped(self.loop, len(self.layers))


@register_model("Sozarax")
class SozaraxModel(SandwichDecoder):
    config_class = SozaraxConfig
    TYPES = {"wkv": "time_mixing", "attention": "biased_attention"}
    KINDS = {"dense": "squared_relu", "moe": "scaled_input_mixture"}

    def take_embedding(self, config, weights, cache):
        self.embed = weights.take("embed", (config.vocab, config.width), "embed", 1.0)
        self.op_embed = hip_op("embed_residual")

    def embedding(self, input_ids, ctx):
        return self.op_embed(input_ids, self.embed, self.shape.embedding_scale, need_act=False)[0]
