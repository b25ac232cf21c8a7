"""Bilolix as a composition of parts: configuration -> model as data.

A decoder whose blocks have one norm (an RMS norm whose weight is stored around zero) that both sub-layers read, and add
both results to the stream (``SharedNormBlockSpec``).  A block's mixer is attention as the difference of two softmax maps
over one value row within a window, with neighbouring rotation pairs and a gate per head (``MapAttentionSpec``); linear
attention with a decay per key channel (``GatedLinearSpec``); or the gated delta rule with a decay per key channel and a
gate through a bottleneck (``GatedDeltaSpec``).  The feed-forward is an ungated one with the error-function gelu
(``MLPSpec``) or a mixture of gated units chosen by a softmax router with a bias (``RoutedMoESpec``).  A run of layers may
be passed through several times with the same weights, each pass with its own cache; a vector of the pass's own is added
to the stream before it (``ReentrySpec`` without a product).  The head is untied.

This file holds what is Bilolix's own: the tensor names and the way the typed configuration fills the parts' sizes.
Layers may differ from one another in every size.
"""
from __future__ import annotations

from ..config.bilolix import ARCHITECTURE, ATTENTION, GLA, BilolixConfig, GeluFFConfig, complete
from ..config.registry import register_architecture
from ..config.spec import (GatedDeltaSpec, GatedLinearSpec, LayerCall, MapAttentionSpec, MLPSpec, ModelSpec, NoPositionSpec,
                           ReentrySpec, RMSNormSpec, RopeSpec, RoutedMoESpec, SharedNormBlockSpec)
from .togalorn import run_order

UNIT_EPS = 1e-6              # under the root where the delta rule makes q and k unit vectors


def _named(p, pairs):
    return {local: p + stored for local, stored in pairs}


def _attention(mx, W, eps, p, max_position):
    position = NoPositionSpec() if mx.rot is None else RopeSpec(
        head_dim=mx.dim, rotary_dim=mx.rot.dims, theta=mx.rot.base, max_position=max_position, layout="interleaved")
    spec = MapAttentionSpec(hidden=W, n_heads=mx.heads, n_kv_heads=mx.kv_heads, map_dim=mx.dim, value_dim=mx.vdim,
                            position=position, scale=mx.scale, share=mx.diff, eps=eps, window=mx.window, head_gate=True)
    return spec, _named(p, (("q_proj.weight", "q"), ("k_proj.weight", "k"), ("v_proj.weight", "v"), ("gate_proj.weight", "g"),
                            ("share.q1", "lq1"), ("share.k1", "lk1"), ("share.q2", "lq2"), ("share.k2", "lk2"),
                            ("out_proj.weight", "o")))


def _fading(mx, W, eps, p):
    spec = GatedLinearSpec(hidden=W, n_heads=mx.heads, key_dim=mx.dim, value_dim=mx.vdim, decay_rank=mx.rank, tau=mx.tau,
                           eps=eps)
    return spec, _named(p, (("q_proj.weight", "q"), ("k_proj.weight", "k"), ("v_proj.weight", "v"), ("gate_proj.weight", "g"),
                            ("decay_down.weight", "a1"), ("decay_up.weight", "a2"), ("decay_up.bias", "a2.b"),
                            ("out_norm.weight", "norm"), ("out_proj.weight", "o")))


def _delta(mx, W, eps, p):
    spec = GatedDeltaSpec(hidden=W, n_heads=mx.heads, qk_heads=mx.kv_heads, key_dim=mx.dim, value_dim=mx.vdim,
                          conv_taps=mx.conv, eps=eps, unit_eps=UNIT_EPS, decay_rank=mx.rank, gate_rank=mx.gate_rank,
                          gate="sigmoid")
    return spec, _named(p, (("q_proj.weight", "q"), ("k_proj.weight", "k"), ("v_proj.weight", "v"), ("q_conv.weight", "q.conv"),
                            ("k_conv.weight", "k.conv"), ("v_conv.weight", "v.conv"), ("beta_proj.weight", "b"),
                            ("A_log", "A_log"), ("dt_bias", "dt_bias"), ("decay_down.weight", "a1"), ("decay_up.weight", "a2"),
                            ("gate_down.weight", "g1"), ("gate_up.weight", "g2"), ("out_norm.weight", "norm"),
                            ("out_proj.weight", "o")))


def _feed_forward(m, W, p):
    if isinstance(m, GeluFFConfig):
        return MLPSpec(hidden=W, intermediate=m.ff, activation="gelu"), {"up.weight": p + "up", "down.weight": p + "down"}
    spec = RoutedMoESpec(hidden=W, n_experts=m.experts, top=m.top, expert_ff=m.ff, limit=None, alpha=1.0, shift=0.0,
                         correction=False, router_bias=True)
    names = {"router.weight": p + "router", "router.bias": p + "router.b"}
    for e in range(m.experts):
        for w in ("gate", "up", "down"):
            names[f"experts.{e}.{w}.weight"] = p + f"e{e}.{w}"
    return spec, names


def bilolix_spec(cfg: BilolixConfig) -> ModelSpec:
    W, eps = cfg.width, cfg.norm_eps
    norm = RMSNormSpec(size=W, eps=eps, offset=1.0)
    blocks = []
    for i, layer in enumerate(cfg.layers):
        p = f"l{i}."
        if layer.type == ATTENTION:
            mixer, local = _attention(layer.mixer, W, eps, p + "mix.", cfg.max_position)
        else:
            mixer, local = (_fading if layer.type == GLA else _delta)(layer.mixer, W, eps, p + "mix.")
        names = {"norm.weight": p + "norm1"}
        names.update({"mixer." + k: v for k, v in local.items()})
        ffn = None
        if layer.mlp is not None:
            ffn, local = _feed_forward(layer.mlp, W, p + "mlp.")
            names.update({"ffn." + k: v for k, v in local.items()})
        blocks.append(SharedNormBlockSpec(mixer=mixer, norm=norm, ffn=ffn, names=names))
    order, starts = run_order(cfg)
    names = {"embed": "embed", "final_norm.weight": "final.norm", "head": "head"}
    reentry = None
    if starts:
        reentry = ReentrySpec(at=tuple(starts), mix=False)
        names["reentry.step"] = "loop.step"
    return ModelSpec(architecture=ARCHITECTURE, hidden=W, vocab=cfg.vocab, blocks=tuple(blocks),
                     schedule=tuple(LayerCall(i) for i in order), final_norm=norm, tie_embeddings=False,
                     max_position=cfg.max_position, names=names, reentry=reentry)


register_architecture(ARCHITECTURE, BilolixConfig.from_dict, bilolix_spec, BilolixConfig.to_json, complete=complete)
