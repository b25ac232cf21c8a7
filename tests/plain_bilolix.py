"""Plain Bilolix: a slow, whole-sequence, cache-free implementation used as the oracle.

Nothing is imported from ``gesso_amd``: a model folder is read with ``json`` and the ``safetensors`` package, the
arithmetic is explicit torch on the CPU in float64 (or another type on request).  One function per mechanism:

    embedding  rms  frequencies  rotate_pairs  visible  softmax_map  share  two_maps  attention  channel_decays
    fading_state  gla  causal_conv  unit  delta_rule  channel_delta  gelu  silu_glu  dense  route  moe  run_order  layer
    forward

Notation.  Rows are tokens: activations are ``(T, features)``, a linear weight ``W`` is ``(out, in)`` and acts as
``y = x @ W.T``; positions count from 0.  ``rms(x) = x / sqrt(mean(x^2) + eps)``, eps under the root.

The model.  ``x = E[token]``.  A layer: ``a = rms(x) (1 + w)``, ``x <- x + mixer(a) + ff(a)``.  A run of layers may be
passed through several times with the same weights; pass ``t`` begins with ``x <- x + step[t]``.  Logits are
``W_head (rms(x) (1 + w_final))``.

Mixer ``attention`` (two maps).  A head has two queries and its key head two keys of ``dim`` features each, turned by the
position over their first ``rot.dims`` features (neighbouring features are a pair), and one value of ``vdim``.  Each pair of
query and key gives an attention of its own over the last ``mask.size`` positions, ``o1`` and ``o2``; with
``lam = exp(lq1 . lk1) - exp(lq2 . lk2) + diff`` the head's output is ``rms(o1 - lam o2) (1 - diff) sigmoid(W_g a)_h``.

Mixer ``gla``.  ``alpha = sigmoid(W_a2 W_a1 a + b)^(1/tau)`` per head and key channel, ``S_t = diag(alpha_t) S_(t-1) +
k_t v_t^T``, ``o_t = S_t^T (q_t dim^-0.5)``; each head's ``o`` is normed with a weight, times ``silu(W_g a)``.

Mixer ``channel_delta``.  q, k, v pass a causal convolution per channel and silu; q and k become unit vectors per head (q
also times ``dim^-0.5``); ``beta = sigmoid(W_b a)`` per head and ``g = exp(-exp(A_log) softplus(W_a2 W_a1 a + dt_bias))``
per head and key channel; ``S <- diag(g) S; u = beta (v - S^T k); S <- S + k u^T; o = S^T q``; each head's ``o`` is normed
with a weight, times ``sigmoid(W_g2 W_g1 a)``.

Feed-forward.  ``dense``: ``W_down gelu(W_up a)`` with the error-function gelu.  ``moe``: the ``top`` experts with the largest
``W_router a + b``, weighted by the softmax over the chosen ones' logits; an expert is
``W_down (silu(W_gate a) * W_up a)``.
"""
from __future__ import annotations

import json
import math
import os

import torch

UNIT_EPS = 1e-6


def _keep(x):
    return x


def to_bfloat16(x: torch.Tensor) -> torch.Tensor:
    """Round to bfloat16 and widen back: what a pipeline with bfloat16 activations does where it stores one."""
    return x.to(torch.bfloat16).to(x.dtype)


def linear(x, W, b=None):
    y = x @ W.T
    return y if b is None else y + b


def silu(z):
    return z * torch.sigmoid(z)


def softplus(z):
    return torch.where(z > 30, z, torch.log1p(torch.exp(torch.clamp(z, max=30.0))))


def gelu(z):
    return 0.5 * z * (1 + torch.erf(z / math.sqrt(2.0)))


# --------------------------------------------------------------------------- small mechanisms

def embedding(table, ids):
    rows = []
    for tok in ids:
        tok = int(tok)
        if not 0 <= tok < table.shape[0]:
            raise ValueError(f"token id {tok} outside the vocabulary of {table.shape[0]}")
        rows.append(table[tok])
    return torch.stack(rows, 0)


def rms(x, eps: float):
    return x / torch.sqrt((x * x).mean(dim=-1, keepdim=True) + eps)


def frequencies(dims: int, base: float):
    """``f_i = base^(-2i/dims)`` for ``i`` below ``dims / 2``."""
    return torch.tensor([base ** (-2.0 * i / dims) for i in range(dims // 2)], dtype=torch.float64)


def rotate_pairs(x, positions, freqs):
    """``x (T, ..., d)``: the first ``2 len(freqs)`` features turned, feature ``2i`` with ``2i + 1``; the rest as they are."""
    n = len(freqs)
    y = x.clone()
    for t, p in enumerate(positions):
        for i in range(n):
            c, s = math.cos(float(p) * float(freqs[i])), math.sin(float(p) * float(freqs[i]))
            u, v = x[t, ..., 2 * i], x[t, ..., 2 * i + 1]
            y[t, ..., 2 * i] = u * c - v * s
            y[t, ..., 2 * i + 1] = v * c + u * s
    return y


def visible(i: int, j: int, window=None) -> bool:
    """Whether the query at position ``i`` sees the key at position ``j``."""
    return j <= i and (window is None or i - j < window)


def softmax_map(q, k, v, positions, scale, window=None):
    """One head of one map: ``q, k (T, d)``, ``v (T, vd)`` -> the weighted sums ``(T, vd)``."""
    T = q.shape[0]
    pos = torch.tensor(list(positions))
    gap = pos[:, None] - pos[None, :]
    seen = (gap >= 0) if window is None else (gap >= 0) & (gap < window)
    s = (q @ k.T) * scale
    s = s.masked_fill(~seen, -math.inf)
    e = torch.exp(s - s.max(dim=-1, keepdim=True).values)
    return (e / e.sum(dim=-1, keepdim=True)) @ v


def share(lq1, lk1, lq2, lk2, diff: float):
    """The second map's share ``lam``."""
    return torch.exp((lq1 * lk1).sum()) - torch.exp((lq2 * lk2).sum()) + diff


def two_maps(q, k, v, positions, scale, lam, diff: float, eps: float, window=None):
    """``q (T, H, 2, d)``, ``k (T, G, 2, d)``, ``v (T, G, vd)`` -> ``rms(o1 - lam o2) (1 - diff)`` per head ``(T, H, vd)``."""
    H, G = q.shape[1], k.shape[1]
    out = []
    for h in range(H):
        g = h // (H // G)
        o1, o2 = (softmax_map(q[:, h, m], k[:, g, m], v[:, g], positions, scale, window) for m in (0, 1))
        out.append(rms(o1 - lam * o2, eps) * (1.0 - diff))
    return torch.stack(out, 1)


def fading_state(q, k, v, alpha):
    """One head: ``q, k, alpha (T, n)``, ``v (T, m)``.  ``S_t = diag(alpha_t) S_(t-1) + k_t v_t^T``, ``o_t = S_t^T q_t``."""
    S = torch.zeros((q.shape[1], v.shape[1]), dtype=q.dtype)
    out = []
    for t in range(q.shape[0]):
        S = alpha[t][:, None] * S + torch.outer(k[t], v[t])
        out.append(S.T @ q[t])
    return torch.stack(out, 0)


def causal_conv(x, taps):
    """``x (T, C)``, ``taps (C, n)``: ``y_t = sum_j taps[:, j] x_(t - n + 1 + j)``, zeros before the start."""
    T, C = x.shape
    n = taps.shape[1]
    padded = torch.cat([torch.zeros((n - 1, C), dtype=x.dtype), x], 0)
    y = torch.zeros_like(x)
    for j in range(n):
        y = y + padded[j:j + T] * taps[:, j]
    return y


def unit(x):
    return x / torch.sqrt((x * x).sum(dim=-1, keepdim=True) + UNIT_EPS)


def delta_rule(q, k, v, beta, g):
    """One head: ``q, k, g (T, n)``, ``v (T, m)``, ``beta (T,)``.  ``S <- diag(g) S; u = beta (v - S^T k); S <- S + k u^T;
    o = S^T q``."""
    S = torch.zeros((q.shape[1], v.shape[1]), dtype=q.dtype)
    out = []
    for t in range(q.shape[0]):
        S = g[t][:, None] * S
        u = beta[t] * (v[t] - S.T @ k[t])
        S = S + torch.outer(k[t], u)
        out.append(S.T @ q[t])
    return torch.stack(out, 0)


def channel_decays(z, a_log, dt_bias, heads: int):
    """``z (T, heads n)`` -> ``exp(-exp(A_log_h) softplus(z + dt_bias))`` as ``(T, heads, n)``."""
    T = z.shape[0]
    s = softplus(z + dt_bias).reshape(T, heads, -1)
    return torch.exp(-torch.exp(a_log)[None, :, None] * s)


# --------------------------------------------------------------------------- mixers

def attention(h, W, p, m, positions, eps, store=_keep):
    """``store``: applied wherever a pipeline with activations of another type would store one (here and below)."""
    T = h.shape[0]
    H, G, d, vd = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    rot = m.get("rot")
    f = frequencies(int(rot["dims"]), float(rot["base"])) if rot else frequencies(0, 1.0)
    q = store(rotate_pairs(store(linear(h, W[p + "q"])).reshape(T, H, 2, d), positions, f))
    k = store(rotate_pairs(store(linear(h, W[p + "k"])).reshape(T, G, 2, d), positions, f))
    v = store(linear(h, W[p + "v"])).reshape(T, G, vd)
    lam = share(W[p + "lq1"], W[p + "lk1"], W[p + "lq2"], W[p + "lk2"], m["diff"])
    o = two_maps(q, k, v, positions, m["scale"], lam, m["diff"], eps, (m.get("mask") or {}).get("size"))
    o = o * torch.sigmoid(store(linear(h, W[p + "g"])))[:, :, None]
    return store(linear(store(o).reshape(T, H * vd), W[p + "o"]))


def gla(h, W, p, m, eps, store=_keep):
    T = h.shape[0]
    H, n, vd = m["heads"], m["dim"], m["vdim"]
    q = (store(linear(h, W[p + "q"])) * n ** -0.5).reshape(T, H, n)
    k = store(linear(h, W[p + "k"])).reshape(T, H, n)
    v = store(linear(h, W[p + "v"])).reshape(T, H, vd)
    z = linear(store(linear(h, W[p + "a1"])), W[p + "a2"], W[p + "a2.b"])
    alpha = (torch.sigmoid(z) ** (1.0 / m["tau"])).reshape(T, H, n)
    o = torch.stack([rms(fading_state(q[:, j], k[:, j], v[:, j], alpha[:, j]), eps) * W[p + "norm"] for j in range(H)], 1)
    o = store(o.reshape(T, H * vd) * silu(store(linear(h, W[p + "g"]))))
    return store(linear(o, W[p + "o"]))


def channel_delta(h, W, p, m, eps, store=_keep):
    T = h.shape[0]
    H, G, n, vd = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q = silu(causal_conv(store(linear(h, W[p + "q"])), W[p + "q.conv"])).reshape(T, G, n)
    k = silu(causal_conv(store(linear(h, W[p + "k"])), W[p + "k.conv"])).reshape(T, G, n)
    v = silu(causal_conv(store(linear(h, W[p + "v"])), W[p + "v.conv"])).reshape(T, H, vd)
    q, k = unit(q) * n ** -0.5, unit(k)
    beta = torch.sigmoid(store(linear(h, W[p + "b"])))
    g = channel_decays(linear(store(linear(h, W[p + "a1"])), W[p + "a2"]), W[p + "A_log"], W[p + "dt_bias"], H)
    heads = []
    for hd in range(H):
        j = hd // (H // G)
        heads.append(rms(delta_rule(q[:, j], k[:, j], v[:, hd], beta[:, hd], g[:, hd]), eps) * W[p + "norm"])
    gate = torch.sigmoid(store(linear(store(linear(h, W[p + "g1"])), W[p + "g2"])))
    return store(linear(store(torch.stack(heads, 1).reshape(T, H * vd) * gate), W[p + "o"]))


# --------------------------------------------------------------------------- feed-forward

def dense(h, W, p, store=_keep):
    return store(linear(store(gelu(store(linear(h, W[p + "up"])))), W[p + "down"]))


def silu_glu(h, W, p, store=_keep):
    return linear(store(silu(store(linear(h, W[p + "gate"]))) * store(linear(h, W[p + "up"]))), W[p + "down"])


def route(h, W, p, top: int):
    """``(chosen experts (T, top), their weights (T, top))``; ties go to the lower index."""
    z = linear(h, W[p + "router"], W[p + "router.b"])
    chosen = torch.sort(z, dim=-1, descending=True, stable=True).indices[:, :top]
    e = torch.gather(z, 1, chosen)
    e = torch.exp(e - e.max(dim=-1, keepdim=True).values)
    return chosen, e / e.sum(dim=-1, keepdim=True)


def moe(h, W, p, mlp, store=_keep):
    chosen, weights = route(h, W, p, mlp["router"]["top"])
    out = torch.zeros_like(h)
    for e in range(mlp["router"]["experts"]):
        for t, k in (chosen == e).nonzero().tolist():
            out[t] = out[t] + weights[t, k] * silu_glu(h[t:t + 1], W, f"{p}e{e}.", store)[0]
    return store(out)


# --------------------------------------------------------------------------- the model

def run_order(cfg: dict):
    """``[(layer, pass that begins before it or None)]`` in the order in which the layers run."""
    n, loop = len(cfg["layers"]), cfg.get("loop")
    if not loop:
        return [(i, None) for i in range(n)]
    a, b, times = loop["start"], loop["stop"], loop["times"]
    out = [(i, None) for i in range(a)]
    for t in range(times):
        out += [(i, t if i == a else None) for i in range(a, b)]
    return out + [(i, None) for i in range(b, n)]


def layer(x, W, i: int, entry, positions, eps, store=_keep):
    p, m = f"l{i}.", entry["mixer"]
    h = store(rms(x, eps) * (1 + W[p + "norm1"]))
    if entry["type"] == "attention":
        y = attention(h, W, p + "mix.", m, positions, eps, store)
    elif entry["type"] == "gla":
        y = gla(h, W, p + "mix.", m, eps, store)
    elif entry["type"] == "channel_delta":
        y = channel_delta(h, W, p + "mix.", m, eps, store)
    else:
        raise ValueError(f"unknown layer type {entry['type']!r}")
    mlp = entry.get("mlp")
    if mlp is not None:
        y = y + (dense(h, W, p + "mlp.", store) if mlp["kind"] == "dense" else moe(h, W, p + "mlp.", mlp, store))
    return x + y


def forward(cfg: dict, W: dict, ids, store=_keep, layers_out=None):
    """Logits ``(T, vocab)`` of one whole sequence from position 0, in the tensors' type.  ``layers_out``: a list that
    receives the stream after every layer run."""
    eps = float(cfg["norm"]["eps"])
    positions = list(range(len(ids)))
    x = embedding(W["embed"], ids)
    for i, t in run_order(cfg):
        if t is not None:
            x = x + W["loop.step"][t]
        x = layer(x, W, i, cfg["layers"][i], positions, eps, store)
        if layers_out is not None:
            layers_out.append(x.clone())
    return linear(store(rms(x, eps) * (1 + W["final.norm"])), W["head"])


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
