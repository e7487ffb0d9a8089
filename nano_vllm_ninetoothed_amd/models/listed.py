"""What decoders share whose layers are listed one by one in the configuration, each with a mixer and a feed-forward of its own kind (or
none); a run of layers may be passed several times in a row."""
from __future__ import annotations

import torch

from ..layers import FEED_FORWARDS, MIXERS


def parse_loop(raw: dict, layers: int) -> tuple:
    """(start, stop, times) of a configuration's "loop": layers start .. stop-1 run `times` times in a row."""
    loop = raw.get("loop") or {"start": 0, "stop": 0, "times": 1}
    start, stop, times = (int(loop[n]) for n in ("start", "stop", "times"))
    if not 0 <= start <= stop <= layers or times < 1:
        raise ValueError(f"a loop over the layers {start} .. {stop - 1} of {layers}, {times} times")
    return start, stop, times


def looped(loop: tuple, layers: int) -> list:
    """Layer numbers in the order in which they run."""
    start, stop, times = loop
    return [*range(start), *list(range(start, stop)) * times, *range(stop, layers)]


class ListedDecoder:
    """A subclass names its mixers and feed-forwards (the configuration's names and those they are registered under) and builds
    self.embed, self.head, the operators linear and sampler_forward and its layers."""
    TYPES: dict = {}
    KINDS: dict = {}
    EMBEDDING_SLOTS = False      # whether the embedding keeps something per sequence
    dtypes = (torch.bfloat16, torch.float32)

    @classmethod
    def validate_layer(cls, layer) -> None:
        if layer["type"] not in cls.TYPES:
            raise ValueError(f"unknown mixer {layer['type']!r}")
        MIXERS[cls.TYPES[layer["type"]]].validate(layer["mixer"])
        mlp = layer.get("mlp")
        if mlp is not None:
            if mlp["kind"] not in cls.KINDS:
                raise ValueError(f"unknown feed-forward {mlp['kind']!r}")
            FEED_FORWARDS[cls.KINDS[mlp["kind"]]].validate(mlp)

    @classmethod
    def needs(cls, config):
        """(pages, state slots)"""
        kinds = [MIXERS[cls.TYPES[layer["type"]]] for layer in config.layers]
        return any(k.uses_pages for k in kinds), cls.EMBEDDING_SLOTS or any(k.uses_slots for k in kinds)

    def reserve_graph_scratch(self, max_bs: int, max_blocks: int) -> None:
        """Makes the scratch of the current stream exist before a capture."""
        from ..mops.hip.ops import _linear_workspace
        _linear_workspace(self.embed.device)

    def result(self, x, ctx):
        """The final hidden rows, or the logits of the wanted ones."""
        if ctx.get("hidden_only"):
            return x
        rows = ctx.get("logit_rows")
        if rows is None and ctx["is_prefill"]:
            rows = ctx["cu_seqlens"][1:].long() - 1
        return self.logits(x if rows is None else x[rows])

    def logits(self, hidden):
        return self.op_linear(hidden, self.head)
