"""Feed-forward sublayers."""
from __future__ import annotations

from . import hip_op, pack, register_feed_forward, require_size
from .joined import TwoProducts


class GatedLinearUnit(TwoProducts):
    """W_down f(W_gate x, W_up x); a subclass says what f is."""

    @staticmethod
    def validate(sizes):
        require_size(sizes, "ff")

    def __init__(self, sizes, weights, prefix, m):
        self.ff = sizes["ff"]
        # the halves start at multiples of eight columns
        self.half = (self.ff + 7) // 8 * 8
        gate, up = (weights.take(prefix + n, (self.ff, m.width)) for n in ("gate", "up"))
        self.down = weights.take(prefix + "down", (m.width, self.ff))
        self.products([gate, up], self.down)
        self.gate_up, self.linear = self.w_in, hip_op("linear")

    def unit(self, gate, up, out=None):
        raise NotImplementedError

    def mix(self, p, ctx, out, scale=1.0):
        if scale != 1.0:
            raise ValueError("a gated unit takes no factor")
        self.unit(*self.parts_of(p), out=out)

    def __call__(self, x, ctx=None):
        return self.linear(self.unit(*self.parts_of(self.linear(x, self.gate_up))), self.down)


@register_feed_forward("clamped_glu")
class ClampedGLU(GatedLinearUnit):
    """f = g * sigmoid(1.702 g) * (u + 1) with g = min(W_gate x, limit) and u = clamp(W_up x, -limit, limit)."""
    ALPHA = 1.702

    @staticmethod
    def validate(sizes):
        GatedLinearUnit.validate(sizes)
        float(sizes["limit"])

    def __init__(self, sizes, weights, prefix, m):
        super().__init__(sizes, weights, prefix, m)
        self.limit, self.glu = float(sizes["limit"]), hip_op("clamped_glu")

    def unit(self, gate, up, out=None):
        return self.glu(gate, up, self.limit, self.ALPHA, out=out)


@register_feed_forward("gelu_glu")
class GeluGLU(GatedLinearUnit):
    """f = gelu(W_gate x) * W_up x, gelu in its tanh form."""

    def __init__(self, sizes, weights, prefix, m):
        super().__init__(sizes, weights, prefix, m)
        self.glu = hip_op("gelu_glu")

    def unit(self, gate, up, out=None):
        return self.glu(gate, up, out=out)


@register_feed_forward("relu_glu")
class ReluGLU(GatedLinearUnit):
    """f = max(W_gate x, 0) * W_up x."""

    def __init__(self, sizes, weights, prefix, m):
        super().__init__(sizes, weights, prefix, m)
        self.glu = hip_op("relu_glu")

    def unit(self, gate, up, out=None):
        return self.glu(gate, up, out=out)


@register_feed_forward("squared_relu")
class SquaredReLU:
    """W_down max(W_up x, 0)^2."""

    @staticmethod
    def validate(sizes):
        require_size(sizes, "ff")

    def __init__(self, sizes, weights, prefix, m):
        self.ff = sizes["ff"]
        self.up = pack([weights.take(prefix + "up", (self.ff, m.width))])
        self.down = weights.take(prefix + "down", (m.width, self.ff))
        self.linear, self.act = hip_op("linear"), hip_op("squared_relu")

    def __call__(self, x):
        return self.linear(self.act(self.linear(x, self.up)[:, :self.ff]), self.down)
