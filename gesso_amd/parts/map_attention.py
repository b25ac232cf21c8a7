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

    def _single(self, rows, ctx, cache, nseq: int, out):
        """The first ``nseq`` sequences, one query each (their rows are the first ``nseq`` rows)."""
        s, ops = self.spec, self.rt.ops
        longest = ctx.max_kv_len if ctx.max_kv_len is not None else cache.block_table.shape[1] * cache.page_size
        if s.window:
            longest = min(longest, s.window)
        # keys are split over blocks only where the batch alone does not fill the chip, 1,024 keys a split and more
        blocks = ops.attention_decode_maps_blocks(s.n_heads, s.n_kv_heads)
        nsplit = max(1, min(-(-longest // 64) // 16, 64, 256 // max(1, nseq * blocks)))
        return ops.attention_decode_maps(rows, cache.k, cache.v, ctx.positions, cache.block_table, cache.page_size, *self._rule(),
                                         nseq, nsplit, out=out)

    def _rule(self):
        """Window, scale, share, norm, gate and sizes, in the order in which the kernels' faces take them."""
        s = self.spec
        return (s.window, s.scale, self.lam, s.eps, 1.0 - s.share, self.og if s.head_gate else -1, s.n_heads, s.n_kv_heads,
                s.map_dim, s.value_dim)

    def attend(self, rows, ctx, cache) -> torch.Tensor:
        """The heads' outputs, normed and gated: ``(T, n_heads * value_dim)``.  The general kernel takes every size and
        both precisions; the kernels for prompt portions and for single queries take over where they take the sizes."""
        s, ops = self.spec, self.rt.ops
        sizes = (s.n_heads, s.n_kv_heads, s.map_dim, s.value_dim)
        fast = rows.dtype == torch.bfloat16 and cache.page_size >= 2 and rows.shape[1] % 8 == 0
        single = fast and ops.attention_decode_maps_supports(*sizes)
        if single and ctx.all_single:
            return self._single(rows, ctx, cache, ctx.nseq, None)
        if fast and not ctx.all_single and ops.attention_prefill_maps_supports(*sizes):
            # decoded tokens at the batch's head go to the kernel for single queries, portions in tiles of queries
            out = torch.empty((ctx.T, s.n_heads * s.value_dim), dtype=rows.dtype, device=rows.device)
            lead = ctx.lead_single if single else 0
            if lead:
                self._single(rows, ctx, cache, lead, out[:lead])
            # tiles of 32 share every key and value fragment between two products (maps of 128 have no registers for them)
            tile = 32 if ctx.max_q_len >= 64 and s.map_dim <= 64 else 16
            return ops.attention_prefill_maps(rows, cache.k, cache.v, ctx.positions, ctx.query_tiles(tile, lead),
                                              cache.block_table, cache.page_size, *self._rule(), out=out, tile_rows=tile)
        return ops.attention_maps(rows, cache.k, cache.v, ctx.positions, ctx.seq_of_token, cache.block_table, cache.page_size,
                                  *self._rule())


register("mixer", "map_attention", MapAttention)
