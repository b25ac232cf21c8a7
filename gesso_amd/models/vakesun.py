"""Vakesun as a composition of parts: configuration -> model as data.

A decoder whose blocks have a norm before and after every sub-layer (``SandwichBlockSpec``; the norm is an elementwise
``tanh(alpha x) w + b``, ``DynTanhSpec``) and end with what the token brings to the layer by itself (``TokenSideSpec``), each
addition scaled by one constant.  A block's mixer is grouped-query softmax attention over all positions with normed heads and
a partial rotation with slowed pairs (``AttentionSpec``, ``ScaledRopeSpec``); a matrix memory with exponential gates
(``MatrixMemorySpec``); or latent attention without positions, within a window, with a sink and a gate a head
(``LatentAttentionSpec``), over its own latent rows or over those an earlier layer has cached (``LayerCall.cache``).  The
feed-forward is ungated with the square of relu (``MLPSpec``).  The embedding rows are scaled; the head is the embedding
table itself.

This file holds what is Vakesun's own: the tensor names and the way the typed configuration fills the parts' sizes.
Layers may differ from one another in every size.
"""
from __future__ import annotations

from ..config.registry import register_architecture
from ..config.spec import (AttentionSpec, DynTanhSpec, LatentAttentionSpec, LayerCall, MatrixMemorySpec, MLPSpec, ModelSpec,
                           NoPositionSpec, RMSNormSpec, SandwichBlockSpec, ScaledRopeSpec, TokenSideSpec)
from ..config.vakesun import ARCHITECTURE, ATTENTION, MLSTM, VakesunConfig, complete


def _named(p, pairs):
    return {local: p + stored for local, stored in pairs}


def _norm_names(role: str, stored: str) -> dict:
    return {role + ".weight": stored, role + ".bias": stored + ".b", role + ".alpha": stored + ".alpha"}


def _attention(mx, W, eps, p, max_position):
    position = NoPositionSpec()
    if mx.rot is not None:
        sc = mx.rot.scaling
        scaling = {} if sc is None else dict(factor=sc.factor, original=sc.original, fast=sc.fast, slow=sc.slow)
        position = ScaledRopeSpec(head_dim=mx.dim, rotary_dim=mx.rot.dims, theta=mx.rot.base, max_position=max_position,
                                  layout="half", **scaling)
    spec = AttentionSpec(hidden=W, n_heads=mx.heads, n_kv_heads=mx.kv_heads, head_dim=mx.dim, value_dim=mx.vdim,
                         position=position, qk_norm=RMSNormSpec(size=mx.dim, eps=eps), scale=mx.scale)
    return spec, _named(p, (("q_proj.weight", "q"), ("k_proj.weight", "k"), ("v_proj.weight", "v"), ("q_norm.weight", "q.norm"),
                            ("k_norm.weight", "k.norm"), ("out_proj.weight", "o")))


def _memory(mx, W, eps, p):
    spec = MatrixMemorySpec(hidden=W, n_heads=mx.heads, key_dim=mx.dim, value_dim=mx.vdim, gate_cap=mx.gate_cap, eps=eps)
    return spec, _named(p, (("q_proj.weight", "q"), ("k_proj.weight", "k"), ("v_proj.weight", "v"), ("gate_proj.weight", "g"),
                            ("input_gate.weight", "i"), ("input_gate.bias", "i.b"), ("forget_gate.weight", "f"),
                            ("forget_gate.bias", "f.b"), ("out_norm.weight", "norm"), ("out_proj.weight", "o")))


def _latent(mx, W, eps, p):
    own = mx.kv_from is None
    spec = LatentAttentionSpec(hidden=W, n_heads=mx.heads, plain_dim=mx.dim, rot_dim=0, value_dim=mx.vdim, q_rank=mx.q_rank,
                               kv_rank=mx.kv_rank, scale=mx.scale, eps=eps, position=NoPositionSpec(), window=mx.window,
                               gated=True, sinks=True, own_rows=own)
    return spec, _named(p, (("q_down.weight", "dq"), ("q_norm.weight", "dq.norm"), ("q_up.weight", "uq"), ("k_up.weight", "uk"),
                            ("v_up.weight", "uv"), ("sinks", "sink"), ("gate.weight", "g"), ("out.weight", "o"))
                        + ((("kv_down.weight", "dkv"), ("kv_norm.weight", "dkv.norm")) if own else ()))


def vakesun_spec(cfg: VakesunConfig) -> ModelSpec:
    W, eps = cfg.width, cfg.norm_eps
    norm = DynTanhSpec(size=W)
    blocks, schedule = [], []
    for i, layer in enumerate(cfg.layers):
        p, mx = f"l{i}.", layer.mixer
        if layer.type == ATTENTION:
            mixer, local = _attention(mx, W, eps, p + "mix.", cfg.max_position)
        elif layer.type == MLSTM:
            mixer, local = _memory(mx, W, eps, p + "mix.")
        else:
            mixer, local = _latent(mx, W, eps, p + "mix.")
        names = {"mixer." + k: v for k, v in local.items()}
        names.update(_norm_names("mixer_norm", p + "norm1"))
        names.update(_norm_names("mixer_out_norm", p + "norm1b"))
        ffn = side = None
        if layer.mlp is not None:
            ffn = MLPSpec(hidden=W, intermediate=layer.mlp.ff, activation="relu_squared")
            names.update({"ffn.up.weight": p + "mlp.up", "ffn.down.weight": p + "mlp.down"})
            names.update(_norm_names("ffn_norm", p + "norm2"))
            names.update(_norm_names("ffn_out_norm", p + "norm2b"))
        if cfg.side_dim is not None:
            side = TokenSideSpec(hidden=W, vocab=cfg.vocab, dim=cfg.side_dim, columns=cfg.side_dim * len(cfg.layers),
                                 offset=cfg.side_dim * i, eps=eps)
            names.update({"side.table": "side.embed", "side.gate.weight": p + "side.gate", "side.proj.weight": p + "side.proj",
                          "side.norm.weight": p + "side.norm"})
        ffn_norm = norm if ffn is not None else None
        blocks.append(SandwichBlockSpec(mixer=mixer, mixer_norm=norm, mixer_out_norm=norm, ffn=ffn, ffn_norm=ffn_norm,
                                        ffn_out_norm=ffn_norm, side=side, mult=cfg.residual_mult, names=names))
        schedule.append(LayerCall(i, cache=getattr(mx, "kv_from", None)))
    names = {"embed": "embed"}
    names.update(_norm_names("final_norm", "final.norm"))
    return ModelSpec(architecture=ARCHITECTURE, hidden=W, vocab=cfg.vocab, blocks=tuple(blocks), schedule=tuple(schedule),
                     final_norm=norm, tie_embeddings=True, max_position=cfg.max_position, names=names,
                     embed_scale=cfg.embedding_scale)


register_architecture(ARCHITECTURE, VakesunConfig.from_dict, vakesun_spec, VakesunConfig.to_json, complete=complete)
