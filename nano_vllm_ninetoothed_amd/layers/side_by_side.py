"""Two mixers that read the same input; their results, each times a factor, are added."""
from __future__ import annotations

from . import MIXERS, register_mixer
from .joined import Joined


class SideBySide(Joined):
    LEFT = RIGHT = None      # registered mixers of two products

    @classmethod
    def validate(cls, sizes):
        MIXERS[cls.LEFT].validate(sizes["left"])
        MIXERS[cls.RIGHT].validate(sizes["right"])
        float(sizes["left_scale"]), float(sizes["right_scale"])

    def __init__(self, sizes, weights, prefix, m):
        super().__init__([MIXERS[self.LEFT](sizes["left"], weights, prefix + "left.", m), MIXERS[self.RIGHT](sizes["right"], weights, prefix + "right.", m)],
                         (sizes["left_scale"], sizes["right_scale"]))


@register_mixer("attention_beside_delta")
class AttentionBesideDelta(SideBySide):
    LEFT, RIGHT = "log_distance_attention", "gated_delta"
    uses_pages, uses_slots = True, True
