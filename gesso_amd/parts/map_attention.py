"""Attention as the difference of two softmax maps over one value row, over the paged cache.

    [q | k | v | g] = W_in x         one product; q: ``n_heads`` heads of two queries, k: ``n_kv_heads`` heads of two keys,
                                     v: ``n_kv_heads`` values, g: a gate's logit a head
    q, k turned by the position, each map's features for themselves
    o_m = softmax(q_m k_m^T scale) v      m = 1, 2, within the window
    lam = exp(q1 . k1) - exp(q2 . k2) + share        four stored vectors: one number for the layer, formed when they are bound
    o   = o_1 - lam o_2;   y_h = o / sqrt(mean(o^2) + eps) * (1 - share) * sigmoid(g_h);   out = W_o y

A token's cache row per key head is its two keys side by side and its value.  Scores, softmax weights, both maps' sums,
their difference, its norm and the gate are float32 in both precisions.
"""
from __future__ import annotations

import torch

from .base import MATRIX, VECTOR, PagedKV, Part, TensorSpec
from .gated_state import stacked
from .registry import build, register


class MapAttention(Part):
    graph_safe = True
    stage, out_stage = "map_mixer", "map_out"

    def __init__(self, spec, rt):
        super().__init__(spec, rt)
        if spec.n_heads % spec.n_kv_heads:
            raise ValueError("query heads must be a multiple of key heads")
        self.position = build("position", spec.position, rt)
        if self.position.rotary_dim > spec.map_dim:
            raise ValueError("more turned features than a map has")
        G = spec.n_kv_heads
        # columns of a row of the input product: where k, v and the gate's logits begin (q is first)
        self.ok = 2 * spec.n_heads * spec.map_dim
        self.ov = self.ok + 2 * G * spec.map_dim
        self.og = self.ov + G * spec.value_dim

    @staticmethod
    def tensor_specs(spec):
        W, H, G, d, vd = spec.hidden, spec.n_heads, spec.n_kv_heads, spec.map_dim, spec.value_dim
        out = {"q_proj.weight": TensorSpec((2 * H * d, W), MATRIX), "k_proj.weight": TensorSpec((2 * G * d, W), MATRIX),
               "v_proj.weight": TensorSpec((G * vd, W), MATRIX), "out_proj.weight": TensorSpec((W, H * vd), MATRIX)}
        if spec.head_gate:
            out["gate_proj.weight"] = TensorSpec((H, W), MATRIX)
        out.update({f"share.{n}": TensorSpec((d,), VECTOR) for n in ("q1", "k1", "q2", "k2")})
        return out

    @staticmethod
    def cache_need(spec):
        vd = spec.value_dim
        return PagedKV(spec.n_kv_heads, 2 * spec.map_dim, spec.window, value_dim=None if vd == 2 * spec.map_dim else vd)

    def bind(self, tensors):
        rt, s = self.rt, self.spec
        self.w_in = rt.prepare(stacked([tensors[k + "_proj.weight"] for k in ("q", "k", "v") + (("gate",) if s.head_gate else ())]))
        self.w_out = rt.prepare(tensors["out_proj.weight"])
        dot = [float((tensors[f"share.q{m}"].double() * tensors[f"share.k{m}"].double()).sum().exp()) for m in (1, 2)]
        self.lam = dot[0] - dot[1] + s.share

    def forward(self, x, ctx, cache):
        s, rt, ops, pos = self.spec, self.rt, self.rt.ops, self.position
        H, G, d, vd = s.n_heads, s.n_kv_heads, s.map_dim, s.value_dim
        with rt.stage("map_in"):
            rows = rt.linear(rt.dense(x), self.w_in)                   # q | k | v | g (| spare columns)
        with rt.stage("map_turn"):
            ops.qknorm_rope_kv(rows, None, None, 1.0, pos.cos, pos.sin, pos.rotary_dim, ctx.positions, ctx.seq_of_token,
                               cache.block_table, cache.page_size, cache.k, cache.v, 2 * H, G, d, write_kv=cache.write,
                               layout=pos.layout, vd=vd, maps=2)
        with rt.stage("map_core"):
            o = self.attend(rows, ctx, cache)
        return rt.linear(o, self.w_out)

    def attend(self, rows, ctx, cache) -> torch.Tensor:
        """The heads' outputs, normed and gated: ``(T, n_heads * value_dim)``."""
        s, ops = self.spec, self.rt.ops
        return ops.attention_maps(rows, cache.k, cache.v, ctx.positions, ctx.seq_of_token, cache.block_table, cache.page_size,
                                  s.window, s.scale, self.lam, s.eps, 1.0 - s.share, self.og if s.head_gate else -1,
                                  s.n_heads, s.n_kv_heads, s.map_dim, s.value_dim)


register("mixer", "map_attention", MapAttention)
