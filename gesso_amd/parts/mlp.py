"""An ungated feed-forward: ``W_down act(W_up x)``, no biases; ``act`` is the error-function or tanh form of gelu, silu or
the square of relu, applied in float32 to the product's rows."""
from __future__ import annotations

from .base import MATRIX, Part, TensorSpec
from .registry import register


class MLP(Part):
    graph_safe = True
    stage, out_stage = "dense_ffn", "ffn_down"

    def __init__(self, spec, rt):
        super().__init__(spec, rt)
        if spec.activation not in rt.ops.GATED_ACTS:
            raise ValueError(f"activation {spec.activation!r}; the kernel has {sorted(rt.ops.GATED_ACTS)}")

    @staticmethod
    def tensor_specs(spec):
        H, F = spec.hidden, spec.intermediate
        return {"up.weight": TensorSpec((F, H), MATRIX), "down.weight": TensorSpec((H, F), MATRIX)}

    def bind(self, tensors):
        self.w_up = self.rt.prepare(tensors["up.weight"])
        self.w_down = self.rt.prepare(tensors["down.weight"])

    def forward(self, x, ctx):
        rt = self.rt
        with rt.stage("ffn_up"):
            a = rt.ops.activate(rt.linear(rt.dense(x), self.w_up), self.spec.activation, rt.dtype)
        return rt.linear(a, self.w_down)


register("ffn", "mlp", MLP)
