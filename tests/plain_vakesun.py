"""Plain Vakesun: a slow, whole-sequence, cache-free implementation used as the oracle.

Nothing is imported from ``gesso_amd``: a model folder is read with ``json`` and the ``safetensors`` package, the
arithmetic is explicit torch on the CPU in float64 (or another type on request).  One function per mechanism:

    embedding  dyt  rms  gelu_tanh  yarn  rotate_half  visible  softmax_head  attention  gates  matrix_memory  mlstm
    latent  latent_attention  dense  side_input  layer  forward

Notation.  Rows are tokens: activations are ``(T, features)``, a linear weight ``W`` is ``(out, in)`` and acts as
``y = x @ W.T``; positions count from 0.  ``rms(x) = x / sqrt(mean(x^2) + eps)``, eps under the root;
``dyt(x) = tanh(alpha x) w + b`` with one number ``alpha`` and vectors ``w``, ``b`` a norm (no statistics of the row).

The model.  ``x = s E[token]``.  A layer norms a sub-layer's input and its output:
``x <- x + m dyt_1b(mixer(dyt_1(x)))``, then, where it has a feed-forward, ``x <- x + m dyt_2b(ff(dyt_2(x)))``; at its end
comes the token's own input: with ``e`` the layer's part of the token's row of a second table,
``y = W_proj (gelu_tanh(W_gate x) * e)`` and ``x <- x + m rms(y) w_side``.  Logits are ``E dyt_final(x)``.

Mixer ``attention``.  Grouped-query softmax attention over all earlier positions; q and k are normed per head
(``rms`` with a weight the heads share), then turned over their first ``rot.dims`` features, feature ``i`` with
``i + dims/2``, with slow pairs slowed and an amplitude (``yarn``).

Mixer ``mlstm``.  A matrix memory a head with exponential gates.  ``i = cap tanh((W_i h + b_i) / cap)``,
``f = log sigmoid(cap tanh((W_f h + b_f) / cap))``; with a running maximum ``p`` from 0 on,
``p_t = max(f + p_(t-1), i)``, ``S_t = exp(f + p_(t-1) - p_t) S_(t-1) + exp(i - p_t) k v^T``, ``n_t`` likewise with ``k`` in
``k v^T``'s place, and ``o = S^T q / (max(|n . q|, exp(-p)) + 1e-6)`` with ``q`` times ``dim^-0.5``; each head's ``o`` becomes
``rms(o)``, all heads are multiplied by a weight and by ``sigmoid(W_g h)``.

Mixer ``latent_attention``.  ``q = W_uq (rms(W_dq h) w_q)``; ``c = rms(W_dkv h) w_kv`` is a token's latent; a head has keys
``W_uk c`` and values ``W_uv c``, no positions, a window, and one more term ``exp(sink_h)`` in its softmax's denominator;
its output is multiplied by ``sigmoid(W_g h)_h``.  A layer with ``kv_from`` has no ``W_dkv``: ``c`` is that layer's.

Feed-forward: ``W_down relu(W_up h)^2``.
"""
from __future__ import annotations

import json
import math
import os

import torch

DEN_EPS = 1e-6


def _keep(x):
    return x


def to_bfloat16(x: torch.Tensor) -> torch.Tensor:
    """Round to bfloat16 and widen back: what a pipeline with bfloat16 activations does where it stores one."""
    return x.to(torch.bfloat16).to(x.dtype)


def linear(x, W, b=None):
    y = x @ W.T
    return y if b is None else y + b


# --------------------------------------------------------------------------- small mechanisms

def embedding(table, ids, scale: float):
    rows = []
    for tok in ids:
        tok = int(tok)
        if not 0 <= tok < table.shape[0]:
            raise ValueError(f"token id {tok} outside the vocabulary of {table.shape[0]}")
        rows.append(table[tok] * scale)
    return torch.stack(rows, 0)


def rms(x, eps: float):
    return x / torch.sqrt((x * x).mean(dim=-1, keepdim=True) + eps)


def dyt(x, W, name: str):
    return torch.tanh(W[name + ".alpha"].reshape(()) * x) * W[name] + W[name + ".b"]


def gelu_tanh(z):
    return 0.5 * z * (1.0 + torch.tanh(math.sqrt(2.0 / math.pi) * (z + 0.044715 * z ** 3)))


def log_sigmoid(z):
    return -torch.log1p(torch.exp(-z.abs())) + torch.clamp(z, max=0.0)


def yarn(dims: int, base: float, scaling):
    """``(angles a position of the dims/2 pairs, factor on cos and sin)``; ``scaling`` None: as they are."""
    f = [float(base) ** (-2.0 * i / dims) for i in range(dims // 2)]
    if scaling is None:
        return f, 1.0
    factor, original = float(scaling["factor"]), float(scaling["original"])

    def pair_of(turns):
        return dims * math.log(original / (2.0 * math.pi * turns)) / (2.0 * math.log(base))

    lo = max(math.floor(pair_of(float(scaling["fast"]))), 0)
    hi = min(math.ceil(pair_of(float(scaling["slow"]))), dims - 1)
    out = []
    for i, fi in enumerate(f):
        ramp = min(1.0, max(0.0, (i - lo) / max(hi - lo, 0.001)))
        out.append(fi / factor * ramp + fi * (1.0 - ramp))
    return out, 0.1 * math.log(factor) + 1.0


def rotate_half(x, positions, freqs, amplitude: float = 1.0):
    """``x (T, heads, d)``: the first ``2 len(freqs)`` features turned, feature ``i`` with ``i + len(freqs)``; the rest as
    they are."""
    n = len(freqs)
    y = x.clone()
    for t, p in enumerate(positions):
        for i in range(n):
            a = float(p) * float(freqs[i])
            c, s = math.cos(a) * amplitude, math.sin(a) * amplitude
            u, v = x[t, ..., i], x[t, ..., i + n]
            y[t, ..., i] = u * c - v * s
            y[t, ..., i + n] = v * c + u * s
    return y


def visible(i: int, j: int, window=None) -> bool:
    """Whether the query at position ``i`` sees the key at position ``j``."""
    return j <= i and (window is None or i - j < window)


def softmax_head(q, k, v, scale: float, window=None, sink=None):
    """One head over a whole sequence: ``q, k (T, d)``, ``v (T, vd)`` -> ``(T, vd)``.  ``sink``: one more term
    ``exp(sink)`` in the denominator."""
    T = q.shape[0]
    gap = torch.arange(T)[:, None] - torch.arange(T)[None, :]
    seen = (gap >= 0) if window is None else (gap >= 0) & (gap < window)
    s = ((q @ k.T) * scale).masked_fill(~seen, -math.inf)
    top = s.max(dim=-1, keepdim=True).values
    if sink is not None:
        top = torch.maximum(top, sink.reshape(1, 1).expand_as(top))
    e = torch.exp(s - top)
    den = e.sum(dim=-1, keepdim=True)
    if sink is not None:
        den = den + torch.exp(sink - top)
    return (e / den) @ v


def gates(zi, zf, cap: float):
    """Log input and log forget gates from their products (biases added)."""
    return cap * torch.tanh(zi / cap), log_sigmoid(cap * torch.tanh(zf / cap))


def matrix_memory(q, k, v, i, f):
    """One head: ``q, k (T, n)``, ``v (T, m)``, log gates ``i, f (T,)`` -> ``(T, m)``."""
    S = torch.zeros((q.shape[1], v.shape[1]), dtype=q.dtype)
    n = torch.zeros(q.shape[1], dtype=q.dtype)
    p = torch.zeros((), dtype=q.dtype)
    out = []
    for t in range(q.shape[0]):
        new = torch.maximum(f[t] + p, i[t])
        keep, write = torch.exp(f[t] + p - new), torch.exp(i[t] - new)
        S = keep * S + write * torch.outer(k[t], v[t])
        n = keep * n + write * k[t]
        p = new
        out.append((S.T @ q[t]) / (torch.maximum((n @ q[t]).abs(), torch.exp(-p)) + DEN_EPS))
    return torch.stack(out, 0)


# --------------------------------------------------------------------------- mixers

def attention(h, W, p, m, positions, eps, store=_keep):
    """``store``: applied wherever a pipeline with activations of another type would store one (here and below)."""
    T = h.shape[0]
    H, G, d, vd = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    rot = m.get("rot")
    freqs, amplitude = yarn(int(rot["dims"]), float(rot["base"]), rot.get("scaling")) if rot else ([], 1.0)
    q = rms(store(linear(h, W[p + "q"])).reshape(T, H, d), eps) * W[p + "q.norm"]
    k = rms(store(linear(h, W[p + "k"])).reshape(T, G, d), eps) * W[p + "k.norm"]
    q, k = (store(rotate_half(z, positions, freqs, amplitude)) for z in (q, k))
    v = store(linear(h, W[p + "v"])).reshape(T, G, vd)
    o = torch.stack([softmax_head(q[:, j], k[:, j // (H // G)], v[:, j // (H // G)], m["scale"]) for j in range(H)], 1)
    return store(linear(store(o).reshape(T, H * vd), W[p + "o"]))


def mlstm(h, W, p, m, eps, store=_keep):
    T = h.shape[0]
    H, n, vd = m["heads"], m["dim"], m["vdim"]
    q = store(linear(h, W[p + "q"])).reshape(T, H, n) * n ** -0.5
    k = store(linear(h, W[p + "k"])).reshape(T, H, n)
    v = store(linear(h, W[p + "v"])).reshape(T, H, vd)
    i, f = gates(linear(h, W[p + "i"], W[p + "i.b"]), linear(h, W[p + "f"], W[p + "f.b"]), float(m["gate_cap"]))
    o = torch.stack([rms(matrix_memory(q[:, j], k[:, j], v[:, j], i[:, j], f[:, j]), eps) for j in range(H)], 1)
    o = o.reshape(T, H * vd) * W[p + "norm"] * torch.sigmoid(store(linear(h, W[p + "g"])))
    return store(linear(store(o), W[p + "o"]))


def latent(h, W, p, eps, store=_keep):
    """A layer's latent rows ``(T, kv_rank)``, as its cache holds them."""
    return store(rms(store(linear(h, W[p + "dkv"])), eps) * W[p + "dkv.norm"])


def latent_attention(h, W, p, m, eps, c, store=_keep):
    """``c``: the latent rows attended to, this layer's or another's."""
    T = h.shape[0]
    H, n, vd = m["heads"], m["dim"], m["vdim"]
    q = store(linear(store(rms(store(linear(h, W[p + "dq"])), eps) * W[p + "dq.norm"]), W[p + "uq"])).reshape(T, H, n)
    k = store(linear(c, W[p + "uk"])).reshape(T, H, n)
    v = store(linear(c, W[p + "uv"])).reshape(T, H, vd)
    window = (m.get("mask") or {}).get("size")
    o = torch.stack([softmax_head(q[:, j], k[:, j], v[:, j], m["scale"], window, W[p + "sink"][j]) for j in range(H)], 1)
    o = o * torch.sigmoid(store(linear(h, W[p + "g"])))[:, :, None]
    return store(linear(store(o).reshape(T, H * vd), W[p + "o"]))


# --------------------------------------------------------------------------- feed-forward, the token's own input

def dense(h, W, p, store=_keep):
    u = torch.clamp(store(linear(h, W[p + "up"])), min=0.0)
    return store(linear(store(u * u), W[p + "down"]))


def side_input(x, W, p, e, eps, store=_keep):
    """What the stream gains from the token's own row ``e (T, dim)`` of this layer."""
    g = store(gelu_tanh(store(linear(store(x), W[p + "side.gate"]))) * e)
    return rms(store(linear(g, W[p + "side.proj"])), eps) * W[p + "side.norm"]


# --------------------------------------------------------------------------- the model

def layer(x, W, i: int, entry, ids, eps, mult: float, side_dim, latents: dict, store=_keep):
    """``latents``: layer index -> latent rows of the layers that make their own; this layer's are put there."""
    p, m = f"l{i}.", entry["mixer"]
    positions = range(len(ids))
    h = store(dyt(x, W, p + "norm1"))
    if entry["type"] == "attention":
        y = attention(h, W, p + "mix.", m, positions, eps, store)
    elif entry["type"] == "mlstm":
        y = mlstm(h, W, p + "mix.", m, eps, store)
    elif entry["type"] == "latent_attention":
        if m.get("kv_from") is None:
            latents[i] = latent(h, W, p + "mix.", eps, store)
        y = latent_attention(h, W, p + "mix.", m, eps, latents[i if m.get("kv_from") is None else m["kv_from"]], store)
    else:
        raise ValueError(f"unknown layer type {entry['type']!r}")
    x = x + mult * dyt(y, W, p + "norm1b")
    if entry.get("mlp") is not None:
        x = x + mult * dyt(dense(store(dyt(x, W, p + "norm2")), W, p + "mlp.", store), W, p + "norm2b")
    if side_dim:
        e = torch.stack([W["side.embed"][int(t), i * side_dim:(i + 1) * side_dim] for t in ids], 0)
        x = x + mult * side_input(x, W, p, e, eps, store)
    return x


def forward(cfg: dict, W: dict, ids, store=_keep, layers_out=None):
    """Logits ``(T, vocab)`` of one whole sequence from position 0, in the tensors' type.  ``layers_out``: a list that
    receives the stream after every layer run."""
    eps = float(cfg["norm"]["eps"])
    x = embedding(W["embed"], ids, float(cfg["embedding"]["scale"]))
    side = cfg.get("token_side")
    latents: dict = {}
    for i, entry in enumerate(cfg["layers"]):
        x = layer(x, W, i, entry, ids, eps, float(cfg["residual_mult"]), None if side is None else int(side["dim"]), latents, store)
        if layers_out is not None:
            layers_out.append(x.clone())
    return linear(store(dyt(x, W, "final.norm")), W["embed"])


def greedy(cfg: dict, W: dict, prompt, n_new: int):
    """The prompt and ``n_new`` tokens after it, each the largest logit's (the lowest id among equals), every step from
    the whole sequence anew."""
    ids = list(prompt)
    for _ in range(n_new):
        ids.append(int(torch.argmax(forward(cfg, W, ids)[-1])))
    return ids


def read_config(folder: str) -> dict:
    with open(os.path.join(folder, "config.json"), encoding="utf-8") as f:
        return json.load(f)


def read_weights(folder: str, dtype=torch.float64) -> dict:
    from safetensors.torch import load_file
    return {k: (v.to(dtype) if v.is_floating_point() else v)
            for k, v in load_file(os.path.join(folder, "model.safetensors")).items()}
