"""Fedovik: a decoder whose layers are listed one by one in the configuration, with a matrix memory, attention without a softmax, or
attention over a window beside a gated delta rule, and a gated feed-forward.  A layer has one layer norm; mixer and feed-forward both
read its output, and their results are added to the stream together.  A run of layers may be passed several times: in front of every
pass the stream is mixed with the embedding by a projection and moved by a vector of that pass.

The residual stream is float32.  The projections into both sublayers are one product and those out of them another; the sum with the
stream and the norm in front of the next layer are one pass.  The embedding table is the output projection.  Runs in bfloat16 and in
float32.
"""
from __future__ import annotations

from dataclasses import dataclass

import torch

from . import register_model
from .listed import ListedDecoder, looped, parse_loop
from ..layers import FEED_FORWARDS, MIXERS, ModelContext, Rotary, hip_op
from ..layers.joined import Joined


@dataclass
class FedovikConfig:
    vocab: int
    width: int
    eps: float
    embedding_scale: float
    layers: list          # dicts with "type", "mixer" (sizes) and "mlp" (sizes with "kind", or None)
    loop: tuple           # (start, stop, times): layers start .. stop-1 run `times` times in a row

    @classmethod
    def from_dict(cls, raw: dict) -> "FedovikConfig":
        layers = list(raw["layers"])
        for layer in layers:
            FedovikModel.validate_layer(layer)
        return cls(vocab=int(raw["vocab"]), width=int(raw["width"]), eps=float(raw["norm"]["eps"]), embedding_scale=float(raw["embedding"]["scale"]),
                   layers=layers, loop=parse_loop(raw, len(layers)))

    def order(self) -> list:
        """Layer numbers in the order in which they run."""
        return looped(self.loop, len(self.layers))

    def passes(self) -> dict:
        """Place in order() where a pass of the loop begins -> number of the pass."""
        start, stop, times = self.loop
        return {start + t * (stop - start): t for t in range(times)} if stop > start else {}


@register_model("Fedovik")
class FedovikModel(ListedDecoder):
    config_class = FedovikConfig
    TYPES = {"mlstm": "matrix_memory", "attention": "sigmoid_attention", "parallel": "attention_beside_delta"}
    KINDS = {"dense": "relu_glu"}

    def __init__(self, config: FedovikConfig, weights, cache, backend: str = "hip", max_model_len: int = 32768):
        if backend != "hip":
            raise ValueError("Fedovik runs on the hip backend only")
        self.shape, self.cache, self.backend = config, cache, backend
        self.dtype, self.hidden, self.vocab, self.max_positions = weights.dtype, config.width, config.vocab, max_model_len
        take, w = weights.take, config.width
        m = ModelContext(w, config.eps, weights.dtype, weights.device, cache, Rotary(max_model_len, weights.device))
        norm = lambda n: (take(n, (w,), "norm"), take(n + ".b", (w,), "vector"))      # noqa: E731
        self.embed = self.head = take("embed", (config.vocab, w), "embed", 1.0)
        passes = config.passes()
        if passes:
            self.loop_in, self.loop_step = take("loop.in", (w, 2 * w)), take("loop.step", (len(passes), w), "vector").float().contiguous()
        order, layers = config.order(), {}
        for i in sorted(set(order)):
            spec, p = config.layers[i], f"l{i}."
            parts = [MIXERS[self.TYPES[spec["type"]]](spec["mixer"], weights, p + "mix.", m)]
            if spec.get("mlp") is not None:
                parts.append(FEED_FORWARDS[self.KINDS[spec["mlp"]["kind"]]](spec["mlp"], weights, p + "mlp.", m))
            layers[i] = (norm(p + "norm1"), Joined(parts))
        self.final_norm = norm("final.norm")
        weights.finish()
        # every run of a layer: the same weights, a cache or state of its own
        self.runs, seen = [], set()
        for at, i in enumerate(order):
            n, sublayers = layers[i]
            self.runs.append((n, sublayers.again(cache) if i in seen else sublayers, passes.get(at)))
            seen.add(i)
        self.op_embed, self.op_add_norm = hip_op("embed_residual"), hip_op("add_norm")
        self.op_linear, self.op_sampler_forward = hip_op("linear"), hip_op("sampler_forward")
        self.layer_hook = None   # called as hook(number of the layer run, float32 residual) after every layer run

    @torch.inference_mode()
    def forward(self, input_ids, positions, ctx):
        t, w, eps = input_ids.numel(), self.hidden, self.shape.eps
        looping = any(begins is not None for *_, begins in self.runs)
        pair = torch.empty((t, 2 * w), dtype=self.dtype, device=self.embed.device) if looping else None      # the stream, the embedding
        residual, _ = self.op_embed(input_ids, self.embed, self.shape.embedding_scale, need_act=False, act=pair[:, w:] if looping else None)
        y = shift = None

        def add(run, replace=False, norm=(None, None), out=None):
            """The stream takes what waits for it; run: the layer run whose result that is, or None."""
            h = self.op_add_norm(residual, y, shift, replace, *norm, eps, center=True, out=out)
            if self.layer_hook is not None and run is not None:
                self.layer_hook(run, residual)
            return h

        for i, (norm, sublayers, begins) in enumerate(self.runs):
            before = i - 1 if i else None
            if begins is None:
                h = add(before, norm=norm)
            else:
                add(before, out=pair[:, :w])
                y, shift = self.op_linear(pair, self.loop_in), self.loop_step[begins]
                h = add(None, True, norm)
            y, shift = sublayers.unbiased(h, ctx), sublayers.bias
        return self.result(add(len(self.runs) - 1 if self.runs else None, norm=self.final_norm), ctx)
