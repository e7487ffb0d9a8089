"""Lulizen: a decoder whose layers are listed one by one in the configuration, with rotary attention over chunks (norms per head, a sink)
or over a window and the first tokens (a gate per head), and a dense or a routed feed-forward; a layer may run with another one's
weights.  Layer norms; the embedding adds a row for the pair of a token and the one in front of it."""
from __future__ import annotations

from dataclasses import dataclass

import torch

from . import register_model
from .sandwich import SandwichDecoder
from ..layers import hip_op


@dataclass
class LulizenConfig:
    vocab: int
    width: int
    eps: float
    bigram: tuple         # (buckets, mul_prev, mul_cur)
    layers: list          # dicts with "type", "mixer" (sizes) and "mlp" (sizes with "kind", or None), or also "weights_of"

    @classmethod
    def from_dict(cls, raw: dict) -> "LulizenConfig":
        layers = list(raw["layers"])
        for layer in layers:
            LulizenModel.validate_layer(layer)
        bigram = raw["embedding"]["bigram"]
        buckets, mul_prev, mul_cur = (int(bigram[n]) for n in ("buckets", "mul_prev", "mul_cur"))
        if buckets <= 0:
            raise ValueError("embedding.bigram.buckets must be positive")
        config = cls(vocab=int(raw["vocab"]), width=int(raw["width"]), eps=float(raw["norm"]["eps"]), bigram=(buckets, mul_prev, mul_cur), layers=layers)
        config.order()
        return config

    def order(self) -> list:
        """Numbers of the layers whose tensors run, in their order."""
        def owner(i):
            seen = {i}
            while self.layers[i].get("weights_of") is not None:
                j = self.layers[i]["weights_of"]
                if not isinstance(j, int) or not 0 <= j < len(self.layers) or j in seen:
                    raise ValueError(f"layer {i} has the weights of {j!r}")
                if any(self.layers[i].get(n) != self.layers[j].get(n) for n in ("type", "mixer", "mlp")):
                    raise ValueError(f"layer {i} has the weights of layer {j}, which is another kind of layer")
                seen.add(j)
                i = j
            return i
        return [owner(i) for i in range(len(self.layers))]


@register_model("Lulizen")
class LulizenModel(SandwichDecoder):
    config_class = LulizenConfig
    TYPES = {"attention": "chunked_attention", "attention_2": "windowed_attention"}
    KINDS = {"dense": "gelu_glu", "moe": "grouped_mixture"}
    CENTER = True
    EMBEDDING_SLOTS = True      # a sequence's last token

    def take_embedding(self, config, weights, cache):
        buckets, self.mul_prev, self.mul_cur = config.bigram
        self.embed = weights.take("embed", (config.vocab, config.width), "embed", 1.0)
        self.pairs = weights.take("bigram", (buckets + 1, config.width), "embed", 1.0)
        self.before = cache.per_slot(dtype=torch.int32)
        self.op_embed = hip_op("embed_pairs")

    def embedding(self, input_ids, ctx):
        return self.op_embed(input_ids, self.embed, self.pairs, self.mul_prev, self.mul_cur, self.before, ctx["starts"], ctx["state_slots"],
                             ctx["token_seq"], ctx["cu_seqlens"])
