"""What decoders share whose sublayers stand between two norms: x <- x + norm1b(mixer(norm1(x))), x <- x + norm2b(ff(norm2(x))).

Layers are listed one by one in the configuration, each with a mixer and a feed-forward of its own kind (or none).  The residual
stream is float32.  The norm behind a sublayer, the sum and the norm in front of the next sublayer are one pass.  The output
projection is a matrix of its own.  Runs in bfloat16 and in float32.
"""
from __future__ import annotations

import torch

from .listed import ListedDecoder
from ..layers import FEED_FORWARDS, MIXERS, ModelContext, Rotary, hip_op


class SandwichDecoder(ListedDecoder):
    """A subclass also says which norms it has, takes the tensors of its embedding and computes it.  The configuration offers vocab, width,
    eps, layers and order(): the numbers of the layers in the order in which they run."""
    CENTER = False      # layer norms instead of RMS norms

    def __init__(self, config, weights, cache, backend: str = "hip", max_model_len: int = 32768):
        if backend != "hip":
            raise ValueError(f"{type(self).__name__} runs on the hip backend only")
        self.shape, self.cache, self.backend = config, cache, backend
        self.dtype, self.hidden, self.vocab, self.max_positions = weights.dtype, config.width, config.vocab, max_model_len
        take = weights.take
        m = ModelContext(config.width, config.eps, weights.dtype, weights.device, cache, Rotary(max_model_len, weights.device))
        self.take_embedding(config, weights, cache)
        order, layers = config.order(), {}
        for i in sorted(set(order)):
            spec, p = config.layers[i], f"l{i}."
            norm = lambda n: take(p + n, (config.width,), "norm")      # noqa: E731
            n1, n1b = norm("norm1"), norm("norm1b")
            mixer = MIXERS[self.TYPES[spec["type"]]](spec["mixer"], weights, p + "mix.", m)
            n2 = n2b = ff = None
            if spec.get("mlp") is not None:
                n2, n2b = norm("norm2"), norm("norm2b")
                ff = FEED_FORWARDS[self.KINDS[spec["mlp"]["kind"]]](spec["mlp"], weights, p + "mlp.", m)
            layers[i] = (n1, mixer, n1b, n2, ff, n2b)
        self.final_norm = take("final.norm", (config.width,), "norm")
        self.head = take("head", (config.vocab, config.width))
        weights.finish()
        # every run of a layer: the same weights, a cache or state of its own
        self.runs, seen = [], set()
        for i in order:
            n1, mixer, *rest = layers[i]
            self.runs.append((n1, mixer.again(cache) if i in seen else mixer, *rest))
            seen.add(i)
        self.op_norm, self.op_add_norm_norm = hip_op("layer_norm_f32" if self.CENTER else "rms_norm_f32"), hip_op("add_norm_norm")
        self.op_linear, self.op_sampler_forward = hip_op("linear"), hip_op("sampler_forward")
        self.layer_hook = None   # called as hook(number of the layer run, float32 residual) after every layer run

    def take_embedding(self, config, weights, cache) -> None:
        raise NotImplementedError

    def embedding(self, input_ids, ctx) -> torch.Tensor:
        """The float32 residual stream [tokens, width]."""
        raise NotImplementedError

    def _add(self, residual, y, norm_behind, norm_in_front):
        y, extra = y if isinstance(y, tuple) else (y, None)
        return self.op_add_norm_norm(residual, y, norm_behind, norm_in_front, self.shape.eps, center=self.CENTER, extra=extra)

    @torch.inference_mode()
    def forward(self, input_ids, positions, ctx):
        runs = self.runs
        residual = self.embedding(input_ids, ctx)
        x = self.op_norm(residual, runs[0][0] if runs else self.final_norm, self.shape.eps)
        for i, (_, mixer, norm1b, norm2, ff, norm2b) in enumerate(runs):
            following = runs[i + 1][0] if i + 1 < len(runs) else self.final_norm
            x = self._add(residual, mixer(x, ctx), norm1b, norm2 if ff is not None else following)
            if ff is not None:
                x = self._add(residual, ff(x), norm2b, following)
            if self.layer_hook is not None:
                self.layer_hook(i, residual)
        return self.result(x, ctx)
