"""What a token brings to a layer by itself: a part of its row in a second table, gated by the stream.

``y = W_proj (gelu_tanh(W_gate h) * table[token, offset : offset + dim])``, then an RMS norm with a weight that the block's
pass over the stream applies (:meth:`TokenSide.out_seam`).  The table is one tensor whose columns the layers share out
between them.  The bottleneck's weights are held with rows and columns of zeros up to whole steps of the matrix cores.
"""
from __future__ import annotations

import torch

from .base import MATRIX, TABLE, VECTOR, Part, TensorSpec
from .registry import register


class TokenSide(Part):
    graph_safe = True
    UNIT = 32               # the bottleneck's width as the products hold it is a multiple of this

    def __init__(self, spec, rt):
        super().__init__(spec, rt)
        if not 0 <= spec.offset <= spec.columns - spec.dim:
            raise ValueError(f"columns {spec.offset} to {spec.offset + spec.dim} lie outside a table of {spec.columns}")
        self.width = -(-spec.dim // self.UNIT) * self.UNIT

    @staticmethod
    def tensor_specs(spec):
        return {"table": TensorSpec((spec.vocab, spec.columns), TABLE), "gate.weight": TensorSpec((spec.dim, spec.hidden), MATRIX),
                "proj.weight": TensorSpec((spec.hidden, spec.dim), MATRIX),
                "norm.weight": TensorSpec((spec.hidden,), VECTOR, "one_plus_normal")}

    def bind(self, tensors):
        rt, s = self.rt, self.spec
        self.table = tensors["table"]
        gate, proj = tensors["gate.weight"], tensors["proj.weight"]
        spare = self.width - s.dim
        if spare:
            gate = torch.cat([gate, torch.zeros((spare, s.hidden), dtype=gate.dtype, device=gate.device)], 0)
            proj = torch.cat([proj, torch.zeros((s.hidden, spare), dtype=proj.dtype, device=proj.device)], 1)
        self.w_gate, self.w_proj = rt.prepare(gate.contiguous()), rt.prepare(proj.contiguous())
        self._seam = rt.ops.SeamNorm("rms", tensors["norm.weight"], eps=s.eps)

    def out_seam(self):
        return self._seam

    def forward(self, x, ctx):
        rt, ops, s = self.rt, self.rt.ops, self.spec
        # (a wide bottleneck is an ordinary product, its rows in the activation type)
        z = rt.narrow_linear(x, self.w_gate) if self.width <= ops.NARROW_MAX_OUT else rt.linear(x, self.w_gate)
        g = ops.side_gate(z, self.table, ctx.token_ids, s.offset, s.dim, self.width, rt.dtype)
        return rt.linear(g, self.w_proj)


register("side", "token_side", TokenSide)
