"""RMSNorm: ``y = x / sqrt(mean(x^2) + eps) * w`` over the last axis, eps inside the root.  A spec with an ``offset``
stores its weight around zero: ``w = offset + stored`` is formed once, in float32, when the weight is bound.

Reference: ``src/Operators/cpu.jl:293-312``.  The kernel folds the residual add that precedes
the norm into the same pass, as the reference's seam does (``src/Inference/Inference.jl:1936-1939``).
"""
from __future__ import annotations

import torch

from .base import VECTOR, Part, TensorSpec
from .registry import register


class ResidualStream:
    """The float32 hidden state ``res (T, H)`` and a sub-layer output not yet added to it.

    ``push`` takes a sub-layer's output: a tensor becomes ``pending`` (the next norm adds it), a
    deferred product (:class:`~gesso_amd.parts.runtime.DeferredLinear`) is computed straight into
    ``res``, which leaves the new rows' sums of squares in ``ssq`` for a lazy norm.

    Whoever knows which norm reads the stream next may say so (``next_norm`` of ``push``; ``following``, set
    by the model, names the norm after the current block).  If that norm offers ``row_weight`` (a float32
    vector ``w`` with ``norm(x) = inv_rms(x) * (x * w)``), the deferred product also leaves ``xs = res * w``
    in bfloat16, and the norm's consumer needs no norm pass at all.  ``xs_for`` is the norm ``xs`` was made for.
    """

    __slots__ = ("res", "pending", "ssq", "xs", "xs_for", "following", "normed", "rows", "bias")

    def __init__(self, res, pending=None, ssq=None, xs=None, xs_for=None):
        self.res = res
        self.pending = pending
        self.ssq = ssq
        self.xs, self.xs_for = xs, xs_for
        self.following = None
        self.normed = None            # the rows normed for ``xs_for``, where the last push made them
        self.rows = None              # the stream itself in the activation type, where the last writer left it
        self.bias = None              # a float32 vector still to be added to every row (a last product's bias, left
                                      # for the pass that adds the product itself)

    def push(self, out, rt, next_norm=None) -> None:
        from .runtime import DeferredLinear
        self.flush(rt)
        self.xs = self.xs_for = self.normed = self.rows = None
        if isinstance(out, DeferredLinear) and self.res.shape[0] > rt.weighted_rows_max:
            # many rows: K is shared out over many blocks, and the pass that adds their partial sums to the stream
            # norms the rows for the next norm on its way (it sees whole rows)
            w = getattr(next_norm, "row_weight", None)
            eps = getattr(getattr(next_norm, "spec", None), "eps", None)
            if w is not None and (w.shape != (self.res.shape[1],) or eps is None):
                w = None
            eps = eps if w is not None else 0.0
            self.ssq, self.normed = rt.ops.gemm_skinny_residual_parts(
                out.x, out.w, self.res, rt.split_parts(out.w), wt=rt.tiles_of(out.w), next_weight=w, eps=eps, out_dtype=rt.dtype,
                tiled=w is not None and rt.rows_tiled(self.res.shape[1]))
            self.xs_for = next_norm if self.normed is not None else None
        elif isinstance(out, DeferredLinear):
            w = row_weight_of(next_norm, self.res, rt)
            if w is not None:
                self.xs = rt.new_rows(*self.res.shape)
                self.xs_for = next_norm
            self.ssq = rt.ops.gemm_skinny_residual(out.x, out.w, self.res, wt=rt.tiles_of(out.w), next_weight=w, xs=self.xs)
        else:
            self.pending, self.ssq = out, None

    def flush(self, rt) -> None:
        """Add what is pending, if a norm has not done so."""
        if self.pending is not None:
            for delta in (self.pending if isinstance(self.pending, tuple) else (self.pending,)):
                if delta is not None:
                    rt.ops.residual_add(self.res, delta)      # (a parallel block leaves two results)
            self.pending, self.ssq = None, None
            self.xs = self.xs_for = self.normed = self.rows = None
        if self.bias is not None:
            rt.ops.add_bias(self.res, self.bias, torch.float32, out=self.res)
            self.bias, self.ssq = None, None
            self.xs = self.xs_for = self.normed = self.rows = None


def row_weight_of(norm, res, rt):
    """``norm.row_weight`` if the norm offers one that fits the stream's width and the rows are few enough, else None."""
    w = getattr(norm, "row_weight", None)
    if w is None or w.dtype != res.dtype or w.shape != (res.shape[1],) or res.shape[0] > rt.weighted_rows_max:
        return None
    return w


class RMSNorm(Part):
    graph_safe = True
    portions_recordable = True

    @staticmethod
    def tensor_specs(spec):
        around_zero = getattr(spec, "offset", 0.0) != 0.0
        return {"weight": TensorSpec((spec.size,), VECTOR, "normal" if around_zero else "one_plus_normal")}

    def bind(self, tensors):
        offset = float(getattr(self.spec, "offset", 0.0))
        self.weight = tensors["weight"] if offset == 0.0 else (tensors["weight"].float() + offset).contiguous()

    @property
    def row_weight(self):
        """``norm(x) = inv_rms(x) * (x * row_weight)``: what lets a producer pre-weight the rows for this norm."""
        return self.weight if self.rt.dtype == torch.bfloat16 else None

    def add_norm(self, stream: ResidualStream, rows=None, out=None, out_dtype=None):
        """Add what is pending to the stream, then norm it (only ``rows`` of it when given).

        While a decode step is recorded with fused kernels, and the stream's sums of squares are at
        hand, the norm is not run: a :class:`~gesso_amd.kernels.ops.LazyNorm` goes to the product that
        follows, which norms on the fly.
        """
        if isinstance(stream.pending, tuple) or stream.bias is not None:
            held = stream.pending if isinstance(stream.pending, tuple) else (stream.pending, None)
            if rows is None and out is None and len(held) == 2 and len({d.dtype for d in held if d is not None}) <= 1:
                # what a block with two results left, and a vector for every row: added in the norm's own pass
                y, _ = self.rt.ops.add_rmsnorm_pair(stream.res, held[0], held[1], self.weight, None, self.spec.eps,
                                                    out_dtype or self.rt.dtype, bias=stream.bias)
                stream.pending = stream.ssq = stream.xs = stream.xs_for = stream.normed = stream.rows = stream.bias = None
                return y
            stream.flush(self.rt)
        if self.rt.fused and rows is None and stream.pending is None and stream.ssq is not None:
            mine = stream.xs_for is self
            return self.rt.ops.LazyNorm(stream.res, stream.ssq, self.weight, self.spec.eps, self.rt.dtype,
                                        xs=stream.xs if mine else None, ready=stream.normed if mine else None)
        y = self.rt.ops.add_rmsnorm(stream.res, stream.pending, self.weight, self.spec.eps, out_dtype or self.rt.dtype,
                                    rows=rows, out=out)
        if rows is None:
            stream.pending = None
            stream.ssq = None
        return y


    def seam(self):
        return self.rt.ops.SeamNorm("rms", self.weight, eps=self.spec.eps)


class GroupRMSNorm(Part):
    """RMS norm in parts: the row is cut into ``groups`` equal consecutive parts, each divided by its own
    ``sqrt(mean(part^2) + eps)``; then the weight.  One part: the plain norm.  float32 arithmetic."""

    graph_safe = True

    @staticmethod
    def tensor_specs(spec):
        return {"weight": TensorSpec((spec.size,), VECTOR, "one_plus_normal")}

    def bind(self, tensors):
        self.weight = tensors["weight"]

    def add_norm(self, stream: ResidualStream, rows=None, out=None, out_dtype=None):
        """Add what is pending to the stream (both results of a block that left two), then norm it (only ``rows`` of
        it when given)."""
        rt = self.rt
        if stream.bias is not None or (rows is not None and stream.pending is not None):
            stream.flush(rt)
        held = stream.pending if isinstance(stream.pending, tuple) else (stream.pending, None)
        if len(held) > 2 or len({d.dtype for d in held if d is not None}) > 1:
            stream.flush(rt)
            held = (None, None)
        y = rt.ops.add_group_rmsnorm(stream.res, held[0], held[1], self.weight, self.spec.eps, self.spec.groups,
                                     out_dtype or rt.dtype, rows=rows)
        if rows is None or stream.pending is None:
            stream.pending = None
        stream.ssq = stream.xs = stream.xs_for = stream.normed = stream.rows = None
        return y


class LayerNorm(Part):
    """``(x - mean) / sqrt(var + eps) * w + b`` over the last axis, the variance the mean of the squared deviations;
    float32 arithmetic.  The pass adds what the sub-layer before left beside the stream, as the other norms' do."""

    graph_safe = True

    @staticmethod
    def tensor_specs(spec):
        out = {"weight": TensorSpec((spec.size,), VECTOR, "one_plus_normal")}
        if getattr(spec, "bias", True):
            out["bias"] = TensorSpec((spec.size,), VECTOR)
        return out

    def bind(self, tensors):
        self.weight = tensors["weight"]
        self.bias = tensors.get("bias")

    def add_norm(self, stream: ResidualStream, rows=None, out=None, out_dtype=None):
        """Add what is pending to the stream, then norm it (only ``rows`` of it when given)."""
        rt = self.rt
        if isinstance(stream.pending, tuple) or stream.bias is not None:
            stream.flush(rt)
        y = rt.ops.add_layernorm(stream.res, stream.pending, self.weight, self.bias, self.spec.eps, out_dtype or rt.dtype,
                                 rows=rows, out=out)
        if rows is None:
            stream.pending = None
        stream.ssq = stream.xs = stream.xs_for = stream.normed = stream.rows = None
        return y


class DynTanh(Part):
    """``tanh(alpha x) w + b``: no mean, no variance, so the pass is elementwise.  float32 arithmetic.  Between two
    sub-layers a block asks for :meth:`seam` and lets one kernel do this norm and the add before it."""

    graph_safe = True

    @staticmethod
    def tensor_specs(spec):
        return {"weight": TensorSpec((spec.size,), VECTOR, "one_plus_normal"), "bias": TensorSpec((spec.size,), VECTOR),
                "alpha": TensorSpec((), VECTOR, "one_plus_normal")}

    def bind(self, tensors):
        self.weight, self.bias = tensors["weight"], tensors["bias"]
        self.alpha = tensors["alpha"].reshape(1).contiguous()
        self._seam = self.rt.ops.SeamNorm("dyn_tanh", self.weight, self.bias, self.alpha)

    def seam(self):
        return self._seam

    def add_norm(self, stream: ResidualStream, rows=None, out=None, out_dtype=None):
        """Add what is pending to the stream, then norm it (only ``rows`` of it when given); rows that the last writer
        of the stream made for this norm are taken as they are."""
        rt = self.rt
        dtype = out_dtype or rt.dtype
        if rows is None and out is None and stream.xs_for is self and stream.normed is not None and stream.normed.dtype == dtype:
            return stream.normed
        if isinstance(stream.pending, tuple) or stream.bias is not None or rows is not None:
            stream.flush(rt)
        y = rt.ops.norm_seam(stream.res, stream.pending, None, 1.0, self._seam, dtype, rows=rows, out=out)
        if stream.pending is not None:
            stream.pending = None
            stream.ssq = stream.xs = stream.xs_for = stream.normed = stream.rows = None
        return y


register("norm", "rmsnorm", RMSNorm)
register("norm", "dyn_tanh", DynTanh)
register("norm", "layernorm", LayerNorm)
register("norm", "group_rmsnorm", GroupRMSNorm)
