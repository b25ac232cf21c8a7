"""Tiny Bilolix configurations of the tests.

A: every mixer, both feed-forwards, a run of layers in the middle passed twice; query heads sharing key heads in groups of
   two and three, a turn over part of a map, windows of 40 and 7.
B: values that are often equal made different and values that are often one made otherwise: no loop, as many key heads as
   query heads in one layer and one key head in another, no window, no turn, a constant share of zero, one and five taps,
   bottlenecks of three and five features, tau of one, one expert used of three and all of four used, a layer without a
   feed-forward, keys wider than values.
C: sizes in whole tiles of the matrix cores (maps of 32 and 64, values of 64 and 128, states of 64 and 128 rows), sequences
   of a few hundred tokens, windows of 64 and 96, all layers passed twice.
D: sizes that are multiples of nothing (width 100, vocabulary 97, maps of 10 and 6, values of 6 and 22, an expert width of
   12), a window of one, a loop of one pass over the last layers.

``write_tiny`` draws the weights and then sets those whose scale matters to values that make the mechanisms show: decays
from almost none to fast (``A_log`` from -6 to 1 over the heads, biases of the channels' decays spread), the four vectors of
the maps' share so that the second map counts for a third to more than the first, and routers sharp enough to choose.
"""
import os

import torch

from gesso_amd.config import (BilolixConfig, BilolixLayer, ChannelDeltaConfig, FadingConfig, GeluFFConfig, LoopConfig,
                              MapAttentionConfig, PairTurn, SoftmaxMoEConfig)
from gesso_amd.weights import write_model_folder

STD = 0.12


def attention(heads, kv_heads, dim, vdim, scale, diff, mlp, rot=None, window=None):
    return BilolixLayer("attention", MapAttentionConfig(heads, kv_heads, dim, vdim, scale, diff, rot, window), mlp)


def fading(heads, dim, vdim, tau, rank, mlp):
    return BilolixLayer("gla", FadingConfig(heads, dim, vdim, tau, rank), mlp)


def delta(heads, kv_heads, dim, vdim, conv, rank, gate_rank, mlp):
    return BilolixLayer("channel_delta", ChannelDeltaConfig(heads, kv_heads, dim, vdim, conv, rank, gate_rank), mlp)


def dense(ff):
    return GeluFFConfig(ff)


def moe(experts, top, ff):
    return SoftmaxMoEConfig(experts, top, ff)


BX_A = BilolixConfig(vocab=211, width=96, norm_eps=1e-6, max_position=1024, loop=LoopConfig(1, 3, 2), layers=(
    delta(4, 2, 16, 24, 4, 8, 12, dense(80)),
    attention(4, 2, 24, 40, 0.2, 0.3, moe(6, 2, 40), PairTurn(1e5, 16), 40),
    fading(3, 16, 24, 8.0, 8, moe(5, 2, 24)),
    attention(6, 2, 16, 32, 0.25, 0.55, dense(48), PairTurn(2e4, 16), 7),
    delta(6, 3, 12, 20, 3, 16, 8, moe(6, 3, 24))))

BX_B = BilolixConfig(vocab=150, width=64, norm_eps=1e-5, max_position=512, layers=(
    fading(2, 24, 8, 1.0, 3, None),
    attention(3, 3, 24, 12, 0.3, 0.0, moe(3, 1, 16)),
    delta(6, 1, 8, 12, 1, 5, 3, moe(4, 4, 24)),
    attention(4, 1, 8, 40, 0.35, 0.8, dense(40), PairTurn(100.0, 4), 33),
    delta(2, 2, 20, 12, 5, 3, 40, dense(24)),
    attention(2, 1, 16, 8, 0.3, 0.2, None, PairTurn(1e4, 16), 500)))

BX_C = BilolixConfig(vocab=320, width=128, norm_eps=1e-6, max_position=1024, loop=LoopConfig(0, 4, 2), layers=(
    delta(2, 2, 64, 64, 4, 32, 16, dense(256)),
    attention(4, 1, 32, 64, 0.18, 0.35, moe(8, 2, 64), PairTurn(5e5, 32), 96),
    fading(2, 128, 128, 16.0, 16, moe(8, 4, 32)),
    attention(2, 1, 64, 128, 0.125, 0.6, dense(192), PairTurn(1e4, 32), 64)))

BX_D = BilolixConfig(vocab=97, width=100, norm_eps=1e-4, max_position=384, loop=LoopConfig(2, 4, 1), layers=(
    attention(5, 5, 10, 6, 0.3, 0.1, moe(3, 2, 12), PairTurn(3e4, 6), 1),
    fading(5, 6, 14, 2.0, 7, dense(36)),
    delta(5, 1, 10, 6, 3, 9, 11, None),
    attention(3, 1, 6, 22, 0.4, 0.45, moe(7, 3, 12), PairTurn(500.0, 2), 19)))

CONFIGS = {"A": (BX_A, 90), "B": (BX_B, 91), "C": (BX_C, 92), "D": (BX_D, 93)}


def sharpen(tensors: dict, seed: int) -> dict:
    """The drawn tensors with those whose scale matters set (see the module's text); keeps every type."""
    g = torch.Generator().manual_seed(seed)
    out = dict(tensors)
    for name, t in tensors.items():
        n = t.numel()
        last = name.rsplit(".", 1)[-1]
        if last == "A_log":
            v = torch.linspace(-6.0, 1.0, n) if n > 1 else torch.tensor([-2.0])
        elif last == "dt_bias":
            v = torch.rand(n, generator=g) * 4.0 - 3.0
        elif last in ("lq1", "lk1", "lq2", "lk2"):
            v = torch.randn(n, generator=g) * 0.7 / n ** 0.25
        elif name.endswith(".a2.b"):
            v = torch.rand(n, generator=g) * 6.0
        elif name.endswith(".router.b"):
            v = 0.5 * torch.randn(n, generator=g)
        elif last in ("router", "conv"):
            v = t.float() * 4.0
        elif name == "loop.step":
            v = t.float() * 8.0
        else:
            continue
        out[name] = v.reshape(t.shape).to(t.dtype)
    return out


def write_folder(out_dir: str, cfg, seed: int, dtype=torch.float32, std: float = STD) -> str:
    """A model folder with drawn and sharpened weights."""
    from safetensors.torch import load_file

    from gesso_amd.weights import write_safetensors
    write_model_folder(out_dir, cfg, seed, dtype, std=std)
    path = os.path.join(out_dir, "model.safetensors")
    write_safetensors(path, sharpen(load_file(path), seed), metadata={"format": "pt", "seed": str(seed)})
    return out_dir


def write_tiny(root: str, name: str, dtype=torch.float32) -> str:
    cfg, seed = CONFIGS[name]
    d = os.path.join(root, f"bilolix_{name}_{str(dtype).split('.')[-1]}")
    if not os.path.exists(os.path.join(d, "model.safetensors")):
        write_folder(d, cfg, seed, dtype)
    return d
