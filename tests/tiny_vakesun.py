"""Tiny Vakesun configurations of the tests.

A: every mixer, with and without a feed-forward; query heads sharing key heads in groups of two and three, values narrower
   and wider than keys, slowed pairs over part of a head, a second latent layer over the first one's rows whose window
   reaches further back than the first one's own.
B: values that are often equal made different and values that are often one made otherwise: no slowed pairs in one layer
   and no turn in another, as many key heads as query heads and one key head, no window in one latent layer, two readers of
   one layer's rows (one of them seeing less, one more), a gate cap below two, embedding scale and residual factor of one.
C: sizes in whole tiles of the matrix cores (heads of 32, 64 and 96 turned whole and in part, latents of 64 and 128, keys of
   the memories 32 to 128 wide, a side input of 80), sequences of a few hundred tokens, windows of 64 and 96.
D: sizes that are multiples of nothing (width 100, vocabulary 97, heads of 10, 6 and 14, latents of 18, keys of 10), a window
   of one, a side input of 7.

``write_tiny`` draws the weights and then sets those whose scale matters to values that make the mechanisms show: the norms'
slopes from flat to nearly saturated, sinks from ones that hardly count to ones that take most of a head's weight, forget
gates from almost nothing kept to almost all, input gates spread over both signs, and a token's own input as large as the
stream's.
"""
import os

import torch

from gesso_amd.config import (GroupedAttentionConfig, MatrixMemoryConfig, SinkLatentConfig, SquaredReluConfig, VakesunConfig,
                              VakesunLayer, YarnScaling, YarnTurn)
from gesso_amd.weights import write_model_folder

STD = 0.12


def dense(ff):
    return None if ff is None else SquaredReluConfig(ff)


def attention(heads, kv_heads, dim, vdim, scale, ff, base=1e4, dims=0, scaling=None):
    turn = YarnTurn(base, dims, None if scaling is None else YarnScaling(*scaling)) if dims else None
    return VakesunLayer("attention", GroupedAttentionConfig(heads, kv_heads, dim, vdim, scale, turn), dense(ff))


def memory(heads, dim, vdim, cap, ff=None):
    return VakesunLayer("mlstm", MatrixMemoryConfig(heads, dim, vdim, cap), dense(ff))


def latent(heads, dim, vdim, scale, q_rank, kv_rank, ff, window=None, kv_from=None):
    return VakesunLayer("latent_attention", SinkLatentConfig(heads, dim, vdim, scale, q_rank, kv_rank, window, kv_from), dense(ff))


VK_A = VakesunConfig(vocab=211, width=96, embedding_scale=5.0, norm_eps=1e-6, residual_mult=0.6, side_dim=12, max_position=1024, layers=(
    attention(4, 2, 24, 16, 0.25, 80, 1e4, 16, (4.0, 64.0, 8.0, 1.0)),
    memory(4, 16, 24, 15.0),
    latent(4, 16, 20, 0.4, 24, 32, 48, window=21),
    attention(6, 2, 16, 32, 0.3, None, 5e4, 16, (2.5, 128.0, 32.0, 1.0)),
    memory(3, 12, 20, 4.0, 40),
    latent(3, 24, 12, 0.3, 40, 32, None, window=40, kv_from=2)))

VK_B = VakesunConfig(vocab=150, width=64, embedding_scale=1.0, norm_eps=1e-5, residual_mult=1.0, side_dim=5, max_position=512, layers=(
    memory(2, 24, 8, 1.5, 24),
    latent(3, 12, 20, 0.5, 16, 48, 40, window=9),
    attention(3, 3, 24, 12, 0.3, 16),
    latent(5, 8, 8, 0.6, 40, 48, None, window=4, kv_from=1),
    attention(4, 1, 8, 8, 0.5, None, 100.0, 4),
    latent(2, 20, 4, 0.3, 8, 48, 24, window=33, kv_from=1),
    latent(1, 16, 16, 0.3, 12, 20, 24)))

VK_C = VakesunConfig(vocab=320, width=128, embedding_scale=8.0, norm_eps=1e-6, residual_mult=0.8, side_dim=80, max_position=1024, layers=(
    attention(4, 1, 32, 32, 0.18, 256, 5e5, 16, (8.0, 128.0, 16.0, 1.0)),
    memory(2, 64, 128, 10.0),
    attention(2, 1, 96, 96, 0.1, 192, 1e4, 48, (4.0, 256.0, 32.0, 1.0)),
    latent(4, 32, 32, 0.18, 64, 128, 256, window=96),
    attention(4, 2, 64, 64, 0.125, None, 2e4, 64, (4.0, 100.0, 32.0, 2.0)),
    memory(2, 128, 64, 15.0, 128),
    memory(3, 32, 136, 6.0),
    latent(8, 16, 64, 0.25, 32, 128, 64, window=64, kv_from=3)))

VK_D = VakesunConfig(vocab=97, width=100, embedding_scale=3.0, norm_eps=1e-4, residual_mult=0.35, side_dim=7, max_position=384, layers=(
    latent(3, 14, 6, 0.5, 18, 18, 36, window=1),
    attention(5, 5, 10, 6, 0.35, 12, 3e4, 6, (3.0, 40.0, 4.0, 0.5)),
    memory(5, 10, 6, 8.0),
    latent(5, 6, 10, 0.5, 22, 18, None, window=19, kv_from=0),
    memory(1, 30, 50, 2.5, 20),
    attention(3, 1, 6, 22, 0.4, 28, 500.0, 2)))

CONFIGS = {"A": (VK_A, 120), "B": (VK_B, 121), "C": (VK_C, 122), "D": (VK_D, 123)}


def sharpen(tensors: dict, seed: int) -> dict:
    """The drawn tensors with those whose scale matters set (see the module's text); keeps every type."""
    g = torch.Generator().manual_seed(seed)
    out = dict(tensors)
    for name in sorted(tensors):
        t = tensors[name]
        n, last = t.numel(), name.rsplit(".", 1)[-1]
        if last == "alpha":
            v = torch.exp(torch.rand(1, generator=g) * 3.0 - 2.3)                # 0.1 to 2
        elif last == "sink":
            v = torch.linspace(-2.0, 3.0, n) if n > 1 else torch.tensor([1.0])
        elif name.endswith(".f.b"):
            v = torch.linspace(-2.0, 6.0, n) if n > 1 else torch.tensor([3.0])
        elif name.endswith(".i.b"):
            v = torch.rand(n, generator=g) * 6.0 - 3.0
        elif last in ("i", "f"):
            v = t.float() * 4.0
        elif name == "side.embed":
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
    d = os.path.join(root, f"vakesun_{name}_{str(dtype).split('.')[-1]}")
    if not os.path.exists(os.path.join(d, "model.safetensors")):
        write_folder(d, cfg, seed, dtype)
    return d
