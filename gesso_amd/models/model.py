"""The model: an embedding table, blocks run in the order the schedule gives, a final norm, a head.

Built from a :class:`~gesso_amd.config.spec.ModelSpec` alone; which architecture the spec came
from plays no part here.  ``tensor_table`` lists every tensor the model reads, by its name in
the weight file, with the shape the spec implies (the reference's shape law,
``src/Inference/materialize_architecture.jl:31-121``).
"""
from __future__ import annotations

from typing import Dict, List, Optional

import torch

from ..config.spec import ModelSpec
from ..errors import ConfigError
from ..parts.base import MATRIX, TABLE, VECTOR, PagedKV, TensorSpec
from ..parts.registry import build, part_class
from ..parts.rmsnorm import ResidualStream, row_weight_of


def tensor_table(spec: ModelSpec) -> Dict[str, TensorSpec]:
    """``file name -> TensorSpec`` of every tensor the model must find."""
    out: Dict[str, TensorSpec] = {}

    def put(name, ts):
        if name in out and out[name] != ts:
            raise ConfigError(f"tensor {name!r} is claimed twice with different shapes")
        out[name] = ts

    put(spec.names["embed"], TensorSpec((spec.vocab, spec.hidden), TABLE))
    for local, ts in part_class("norm", spec.final_norm).tensor_specs(spec.final_norm).items():
        put(spec.names["final_norm." + local], ts)
    if spec.embed_norm is not None:
        for local, ts in part_class("norm", spec.embed_norm).tensor_specs(spec.embed_norm).items():
            put(spec.names["embed_norm." + local], ts)
    if not spec.tie_embeddings:
        put(spec.names["head"], TensorSpec((spec.vocab, spec.hidden), MATRIX))
    if spec.reentry is not None:
        if spec.reentry.mix:
            put(spec.names["reentry.weight"], TensorSpec((spec.hidden, 2 * spec.hidden), MATRIX))
        put(spec.names["reentry.step"], TensorSpec((len(spec.reentry.at), spec.hidden), VECTOR))
    for i, b in enumerate(spec.blocks):
        for local, ts in part_class("block", b).tensor_specs(b).items():
            if local not in b.names:
                raise ConfigError(f"block {i} has no file name for its tensor {local!r}")
            put(b.names[local], ts)
    return out


def tied_aliases(spec: ModelSpec) -> Dict[str, str]:
    """Tensors a file may hold though nobody reads them, if they equal another: a tied head."""
    if spec.tie_embeddings and "head" in spec.names:
        return {spec.names["head"]: spec.names["embed"]}
    return {}


def schedule_cache_needs(spec: ModelSpec) -> List[Optional[object]]:
    """See :meth:`Model.cache_needs`."""
    out: List[Optional[object]] = []
    for call in spec.schedule:
        b = spec.blocks[call.layer]
        need = part_class("block", b).cache_need(b)
        if call.cache is None:
            out.append(need)
            continue
        src = call.cache
        while spec.schedule[src].cache is not None:
            src = spec.schedule[src].cache
        if isinstance(need, PagedKV) and isinstance(out[src], PagedKV):
            out[src] = out[src].reaching(need)
        out.append(None)
    return out


class Model:
    def __init__(self, spec: ModelSpec, rt):
        self.spec = spec
        self.rt = rt
        self.blocks = [build("block", b, rt) for b in spec.blocks]
        self.final_norm = build("norm", spec.final_norm, rt)
        self.embed_norm = build("norm", spec.embed_norm, rt) if spec.embed_norm is not None else None
        self.embed = None
        self.head = None
        self.reentry_weight = self.reentry_step = None

    def cache_needs(self) -> List[Optional[object]]:
        """For each entry of the schedule: what its own cache must hold (None: none, or it reads another's).  A cache that
        later calls read keeps the rows that any of its readers may still see."""
        return schedule_cache_needs(self.spec)

    def bind(self, tensors: Dict[str, torch.Tensor]) -> None:
        s = self.spec
        self.embed = tensors[s.names["embed"]]
        self.head = self.rt.prepare(self.embed if s.tie_embeddings else tensors[s.names["head"]])
        self.final_norm.bind({k: tensors[s.names["final_norm." + k]]
                              for k in part_class("norm", s.final_norm).tensor_specs(s.final_norm)})
        if self.embed_norm is not None:
            self.embed_norm.bind({k: tensors[s.names["embed_norm." + k]]
                                  for k in part_class("norm", s.embed_norm).tensor_specs(s.embed_norm)})
        if s.reentry is not None:
            if s.reentry.mix:
                self.reentry_weight = self.rt.prepare(tensors[s.names["reentry.weight"]])
            self.reentry_step = tensors[s.names["reentry.step"]].contiguous()
        for b, block in zip(s.blocks, self.blocks):
            local = {k: tensors[b.names[k]] for k in part_class("block", b).tensor_specs(b)}
            block.bind(local)

    @property
    def graph_safe(self) -> bool:
        norms = [self.final_norm] + ([self.embed_norm] if self.embed_norm is not None else [])
        return all(getattr(b, "graph_safe", False) for b in self.blocks) and all(getattr(n, "graph_safe", False) for n in norms)

    def forward(self, ctx) -> Optional[torch.Tensor]:
        """Run the tokens of ``ctx`` through every scheduled block; float32 logits at ``ctx.want_rows``."""
        stream = self.run_blocks(ctx)
        if ctx.n_want == 0:
            return None
        # every row wanted, in order (a decode step): no gather, and the norm may stay lazy
        return self.logits(stream, None if ctx.decode_only else ctx.want_rows)

    def run_blocks(self, ctx) -> ResidualStream:
        """The embedding and every scheduled block: the residual stream as the last block leaves it (what is still
        pending is added by the norm that follows)."""
        rt = self.rt
        ctx.shared = {}          # what a part of this step leaves for a later one (a context may serve several runs)
        # the norm that reads the stream after the i-th scheduled block: the next block's first, then the final one
        # (``first_norm`` and ``row_weight`` are the optional hints of blocks and norms, see parts/base.py)
        order = [self.blocks[call.layer] for call in self.spec.schedule]
        readers = [getattr(b, "first_norm", None) for b in order[1:]] + [self.final_norm if ctx.decode_only else None]
        scale = 1.0 if self.spec.embed_scale is None else float(self.spec.embed_scale)
        with rt.stage("embed"):
            stream = self._embed(ctx, order, scale)
        reentries = {} if self.spec.reentry is None else {at: t for t, at in enumerate(self.spec.reentry.at)}
        # the embedding output, kept for every re-entry of this step (in the activation type: it is a product's operand
        # from here on)
        x0 = stream.res.to(rt.dtype, copy=True) if reentries and self.spec.reentry.mix else None
        for i, call in enumerate(self.spec.schedule):
            if i in reentries:
                with rt.stage("reentry"):
                    stream = self._reenter(stream, x0, reentries[i])
            stream.following = readers[i]
            order[i].forward(stream, ctx, ctx.cache_view(i))
        return stream

    def _reenter(self, stream: ResidualStream, x0, t: int) -> ResidualStream:
        """``x <- W [x; x0] + step[t]``: the stream and the embedding output side by side through one product, float32
        sums, the pass's vector added in float32; the result is the new stream.  Without the product the vector is left
        beside the stream, for the norm that reads it next to add."""
        rt = self.rt
        if not self.spec.reentry.mix:
            if stream.bias is not None:
                stream.flush(rt)
            stream.bias = self.reentry_step[t]
            return stream
        stream.flush(rt)
        T, W = stream.res.shape
        rows = torch.empty((T, 2 * W), dtype=rt.dtype, device=stream.res.device)
        rows[:, :W].copy_(stream.res)
        rows[:, W:].copy_(x0)
        y = rt.linear(rows, self.reentry_weight, out_dtype=torch.float32)
        return ResidualStream(rt.ops.add_bias(y, self.reentry_step[t], torch.float32, out=y))

    def logits(self, stream: ResidualStream, rows) -> torch.Tensor:
        """The final norm of the stream's ``rows`` (int32 on the device; None: all, in order) and the head: float32."""
        ops, rt = self.rt.ops, self.rt
        with rt.stage("norm"):
            normed = self.final_norm.add_norm(stream, rows=rows)
        with rt.stage("lm_head"):
            logits = self.rt.linear(normed, self.head, out_dtype=torch.float32)
            if self.spec.logit_softcap is not None:
                ops.softcap(logits, float(self.spec.logit_softcap))
        return logits

    @property
    def portions_recordable(self) -> bool:
        """Whether steps of prompt portions through this model may be recorded for replay (every part says so: what it
        launches then depends on the step's token count and on device buffers alone, or it tells the recorder)."""
        return all(getattr(b, "portions_recordable", False) for b in self.blocks) and \
            getattr(self.final_norm, "portions_recordable", False)

    def replay_key(self, q_lens, max_kv_len):
        """What a recording of a step of prompt portions must share with the step that replays it, beside the token
        count: each block's own answer (None: nothing; False from any block: such a step is not to be recorded, and
        the answer is None)."""
        key = tuple(b.replay_key(q_lens, max_kv_len) if hasattr(b, "replay_key") else None for b in self.blocks)
        return None if any(k is False for k in key) else key

    def _embed(self, ctx, order, scale):
        ops, rt = self.rt.ops, self.rt
        if self.embed_norm is not None:
            # the embedding rows are normed before the first block: the stream starts from the normed rows (float32)
            raw = ops.embed(ctx.token_ids, self.embed, scale=scale)
            return ResidualStream(self.embed_norm.add_norm(ResidualStream(raw), out_dtype=torch.float32))
        if rt.fused:
            ssq = torch.empty((ctx.T, 1), dtype=torch.float32, device=rt.device)
            first = getattr(order[0], "first_norm", None) if order else None
            res = torch.empty((ctx.T, self.embed.shape[1]), dtype=torch.float32, device=rt.device)
            w = row_weight_of(first, res, rt)
            xs = rt.new_rows(*res.shape) if w is not None else None
            ops.embed(ctx.token_ids, self.embed, out=res, ssq=ssq, next_weight=w, xs=xs, scale=scale)
            stream = ResidualStream(res, ssq=ssq, xs=xs, xs_for=first if xs is not None else None)
        else:
            stream = ResidualStream(ops.embed(ctx.token_ids, self.embed, scale=scale))
        return stream

