"""Vakesun without a GPU: the configuration through its file and back, ranks read from stored tensors' shapes, errors that
name the key, the model as data (names, shapes, what each call caches, how far a shared cache reaches back), and the plain
implementation's own mechanisms."""
import json
import math

import pytest
import torch

import plain_vakesun as P
from tiny_vakesun import CONFIGS, VK_A, VK_B, write_tiny

from gesso_amd.config import VakesunConfig, load_config
from gesso_amd.errors import ConfigError


def rand(*shape, seed=0, scale=1.0):
    return torch.randn(*shape, generator=torch.Generator().manual_seed(seed), dtype=torch.float64) * scale


# ------------------------------------------------------------------ configuration

@pytest.mark.parametrize("name", sorted(CONFIGS))
def test_configuration_through_its_file_and_back(name, tmp_path):
    cfg, _ = CONFIGS[name]
    raw = cfg.to_json()
    assert VakesunConfig.from_dict(json.loads(json.dumps(raw))) == cfg
    (tmp_path / "config.json").write_text(json.dumps(raw))
    arch, back = load_config(str(tmp_path))
    assert arch.name == "Vakesun" and back == cfg


def test_ranks_that_only_stored_tensors_tell(tmp_path):
    d = write_tiny(str(tmp_path), "A")
    raw = json.loads(open(d + "/config.json").read())
    for L in raw["layers"]:
        if L["type"] == "latent_attention":
            del L["mixer"]["q_rank"], L["mixer"]["kv_rank"]
    open(d + "/config.json", "w").write(json.dumps(raw))
    assert load_config(d)[1] == VK_A
    with pytest.raises(ConfigError) as err:
        VakesunConfig.from_dict(raw)
    assert "q_rank" in str(err.value)


def test_keys_left_out_take_their_defaults_and_unknown_keys_name_themselves():
    raw = VK_A.to_json()
    del raw["embedding"], raw["residual_mult"], raw["token_side"]
    raw["layers"][2]["mixer"]["mask"] = None
    raw["layers"][0]["mixer"].pop("rot")
    raw["layers"][3]["mixer"]["rot"]["scaling"] = None
    raw["layers"][4]["mlp"] = None
    raw["layers"][5]["mixer"]["kv_from"] = None
    cfg = VakesunConfig.from_dict(raw)
    assert cfg.embedding_scale == cfg.residual_mult == 1.0 and cfg.side_dim is None and cfg.layers[2].mixer.window is None
    assert cfg.layers[0].mixer.rot is None and cfg.layers[3].mixer.rot.scaling is None and cfg.layers[4].mlp is None
    assert cfg.layers[5].mixer.kv_from is None
    for path, where in ((("loop",), "config.json"), (("layers", 0, "mixer", "softcap"), "layers[0].mixer"),
                        (("layers", 0, "mixer", "rot", "layout"), "layers[0].mixer.rot"), (("layers", 0, "mixer", "mask"), "layers[0].mixer"),
                        (("layers", 2, "mixer", "mask", "keep_first"), "layers[2].mixer.mask"), (("layers", 2, "mixer", "rot_dim"), "layers[2].mixer"),
                        (("layers", 1, "mixer", "conv"), "layers[1].mixer"), (("layers", 0, "mlp", "limit"), "layers[0].mlp"),
                        (("norm", "groups"), "norm"), (("token_side", "scale"), "token_side"),
                        (("layers", 0, "mixer", "rot", "scaling", "slope"), "layers[0].mixer.rot.scaling")):
        raw = VK_A.to_json()
        at = raw
        for k in path[:-1]:
            at = at[k]
        at[path[-1]] = 3
        with pytest.raises(ConfigError) as err:
            VakesunConfig.from_dict(raw)
        assert path[-1] in str(err.value) and where in str(err.value)


@pytest.mark.parametrize("change,word", [
    (lambda r: r["layers"][0].__setitem__("type", "mamba2"), "type"),
    (lambda r: r["layers"][0]["mixer"]["rot"].__setitem__("dims", 26), "rot.dims"),
    (lambda r: r["layers"][0]["mixer"]["rot"].__setitem__("dims", 7), "rot.dims"),
    (lambda r: r["layers"][0]["mixer"].__setitem__("kv_heads", 3), "kv_heads"),
    (lambda r: r["layers"][1]["mixer"].__setitem__("gate_cap", 0), "gate_cap"),
    (lambda r: r["layers"][1]["mixer"].pop("gate_cap"), "gate_cap"),
    (lambda r: r["layers"][0]["mlp"].__setitem__("kind", "moe"), "kind"),
    (lambda r: r["layers"][5]["mixer"].__setitem__("kv_from", 1), "kv_from"),          # no latent layer
    (lambda r: r["layers"][5]["mixer"].__setitem__("kv_from", 5), "kv_from"),          # not an earlier one
    (lambda r: r["layers"][5]["mixer"].__setitem__("kv_rank", 16), "kv_from"),         # other rows than it makes
    (lambda r: r["layers"].append(dict(r["layers"][5], mixer=dict(r["layers"][5]["mixer"], kv_from=5))), "kv_from"),
    (lambda r: r["norm"].__setitem__("eps", 0.0), "eps")])
def test_contradictions_are_errors(change, word):
    raw = VK_A.to_json()
    change(raw)
    with pytest.raises(ConfigError) as err:
        VakesunConfig.from_dict(raw)
    assert word in str(err.value)


# ------------------------------------------------------------------ the model as data

def test_names_shapes_and_caches():
    from gesso_amd.cache.manager import CacheLayout
    from gesso_amd.config.registry import architecture_of
    from gesso_amd.models.model import schedule_cache_needs, tensor_table
    from gesso_amd.parts import PagedKV
    spec = architecture_of(VK_A.to_json()).to_spec(VK_A)
    assert [c.layer for c in spec.schedule] == list(range(6)) and [c.cache for c in spec.schedule] == [None] * 5 + [2]
    assert spec.tie_embeddings and spec.embed_scale == 5.0 and spec.final_norm.kind == "dyn_tanh"
    t = {k: v.shape for k, v in tensor_table(spec).items()}
    assert t["embed"] == (211, 96) and t["side.embed"] == (211, 72) and "head" not in t
    for i, L in enumerate(VK_A.layers):
        for norm, there in (("norm1", True), ("norm1b", True), ("norm2", L.mlp is not None), ("norm2b", L.mlp is not None)):
            assert (f"l{i}.{norm}" in t) == there
            if there:
                assert t[f"l{i}.{norm}"] == t[f"l{i}.{norm}.b"] == (96,) and t[f"l{i}.{norm}.alpha"] == ()
        assert t[f"l{i}.side.gate"] == (12, 96) and t[f"l{i}.side.proj"] == (96, 12) and t[f"l{i}.side.norm"] == (96,)
    assert t["final.norm"] == t["final.norm.b"] == (96,) and t["final.norm.alpha"] == ()
    assert t["l0.mix.q"] == (96, 96) and t["l0.mix.k"] == (48, 96) and t["l0.mix.v"] == (32, 96) and t["l0.mix.o"] == (96, 64)
    assert t["l0.mix.q.norm"] == t["l0.mix.k.norm"] == (24,) and t["l0.mlp.up"] == (80, 96) and t["l0.mlp.down"] == (96, 80)
    assert t["l1.mix.q"] == t["l1.mix.k"] == (64, 96) and t["l1.mix.v"] == t["l1.mix.g"] == (96, 96) and t["l1.mix.norm"] == (96,)
    assert t["l1.mix.i"] == t["l1.mix.f"] == (4, 96) and t["l1.mix.i.b"] == t["l1.mix.f.b"] == (4,) and "l1.mlp.up" not in t
    assert t["l2.mix.dq"] == (24, 96) and t["l2.mix.uq"] == (64, 24) and t["l2.mix.dkv"] == (32, 96) and t["l2.mix.dkv.norm"] == (32,)
    assert t["l2.mix.uk"] == (64, 32) and t["l2.mix.uv"] == (80, 32) and t["l2.mix.sink"] == (4,) and t["l2.mix.g"] == (4, 96)
    assert "l5.mix.dkv" not in t and "l5.mix.dkv.norm" not in t and t["l5.mix.uk"] == (72, 32) and t["l5.mix.dq"] == (40, 96)
    needs = schedule_cache_needs(spec)
    assert needs[0] == PagedKV(2, 24, None, value_dim=16) and needs[3] == PagedKV(2, 16, None, value_dim=32)
    assert [(e[0], e[1], e[2], e[3]) for e in needs[1].entries()] == [("state", (4, 16, 25), "float32", 0.0), ("peak", (4,), "float32", 0.0)]
    # the rows of layer 2 stay while layer 5, whose window is wider, may still see them
    assert needs[2] == PagedKV(1, 32, 40, value_dim=0) and needs[5] is None
    layout = CacheLayout.plan(needs, [c.cache for c in spec.schedule])
    assert layout.source_of_call[5] == 2 and len(layout.paged) == 3 and len(layout.slots) == 2
    b = architecture_of(VK_B.to_json()).to_spec(VK_B)
    needs = schedule_cache_needs(b)
    assert needs[1].window == 33 and needs[3] is None and needs[5] is None and needs[6].window is None
    assert tensor_table(b)["side.embed"].shape == (150, 35)


def test_a_shared_cache_reaches_as_far_back_as_its_widest_reader():
    from gesso_amd.parts import PagedKV
    a = PagedKV(1, 32, 20, value_dim=0)
    assert a.reaching(PagedKV(1, 32, 7, value_dim=0)) == a
    assert a.reaching(PagedKV(1, 32, 30, value_dim=0)).window == 30
    assert a.reaching(PagedKV(1, 32, None, value_dim=0)).window is None
    assert PagedKV(2, 8, 5, keep_first=3).reaching(PagedKV(2, 8, 9, keep_first=1)) == PagedKV(2, 8, 9, keep_first=3)
    with pytest.raises(ValueError):
        a.reaching(PagedKV(1, 16, 20, value_dim=0))
    with pytest.raises(ValueError):
        a.reaching(PagedKV(1, 32, 20, value_dim=0, chunk=8))


def test_a_block_needs_norms_that_the_pass_between_sub_layers_knows():
    """Every sub-layer's tensors stand under its role, and a feed-forward that is not there names none."""
    from gesso_amd.config import DynTanhSpec, MLPSpec, SandwichBlockSpec
    from gesso_amd.parts import part_class
    n = DynTanhSpec(16)
    mlp = MLPSpec(16, 24, "relu_squared")
    from gesso_amd.config import MatrixMemorySpec
    mixer = MatrixMemorySpec(16, 2, 8, 8, 4.0, 1e-6)
    full = SandwichBlockSpec(mixer=mixer, mixer_norm=n, mixer_out_norm=n, ffn=mlp, ffn_norm=n, ffn_out_norm=n)
    less = SandwichBlockSpec(mixer=mixer, mixer_norm=n, mixer_out_norm=n, ffn=None, ffn_norm=None, ffn_out_norm=None)
    a, b = (part_class("block", s).tensor_specs(s) for s in (full, less))
    assert {"ffn_out_norm.alpha", "ffn.up.weight", "mixer_out_norm.bias"} <= set(a)
    assert not any(k.startswith("ffn") or k.startswith("side") for k in b) and "mixer_out_norm.bias" in b


# ------------------------------------------------------------------ the plain implementation's own mechanisms

def test_the_norm_is_elementwise():
    W = {"n": torch.tensor([2.0, 3.0], dtype=torch.float64), "n.b": torch.tensor([0.5, -1.0], dtype=torch.float64), "n.alpha": torch.tensor(0.25)}
    x = torch.tensor([[4.0, -8.0], [0.0, 100.0]], dtype=torch.float64)
    want = torch.tensor([[2 * math.tanh(1.0) + 0.5, 3 * math.tanh(-2.0) - 1.0], [0.5, 2.0]], dtype=torch.float64)
    assert torch.allclose(P.dyt(x, W, "n"), want)


def test_slow_pairs_are_slowed_and_the_amplitude_is_applied():
    f, amp = P.yarn(8, 1e4, {"factor": 4.0, "original": 64.0, "fast": 8.0, "slow": 1.0})
    plain, one = P.yarn(8, 1e4, None)
    assert one == 1.0 and amp == pytest.approx(0.1 * math.log(4.0) + 1.0)
    pair = lambda turns: 8 * math.log(64.0 / (2 * math.pi * turns)) / (2 * math.log(1e4))
    lo, hi = max(math.floor(pair(8.0)), 0), min(math.ceil(pair(1.0)), 7)
    assert (lo, hi) == (0, 2)
    assert f == pytest.approx([plain[0], plain[1] / 4 * 0.5 + plain[1] * 0.5, plain[2] / 4, plain[3] / 4])
    x = rand(1, 1, 6, seed=1)
    y = P.rotate_half(x, [3], [1.0, 0.1], 1.5)[0, 0]
    for i, a in ((0, 3.0), (1, 0.3)):
        u, v = x[0, 0, i], x[0, 0, i + 2]
        assert torch.isclose(y[i], 1.5 * (u * math.cos(a) - v * math.sin(a))) and torch.isclose(y[i + 2], 1.5 * (v * math.cos(a) + u * math.sin(a)))
    assert torch.equal(y[4:], x[0, 0, 4:])


def test_a_window_shows_itself_and_the_tokens_before_it_and_a_sink_takes_its_share():
    for window in (1, 3, None):
        for i in range(6):
            assert [P.visible(i, j, window) for j in range(6)] == [j <= i and (window is None or j > i - window) for j in range(6)]
    v, z = torch.eye(5, dtype=torch.float64), torch.zeros(5, 2, dtype=torch.float64)
    w = P.softmax_head(z, z, v, 1.0, 2)
    assert torch.allclose(w[4], torch.tensor([0, 0, 0, 0.5, 0.5], dtype=torch.float64)) and torch.allclose(w[0], v[0])
    w = P.softmax_head(z, z, v, 1.0, 3, torch.tensor(math.log(2.0), dtype=torch.float64))
    assert torch.allclose(w.sum(1), torch.tensor([1 / 3, 2 / 4, 3 / 5, 3 / 5, 3 / 5], dtype=torch.float64))
    q, k = rand(5, 3, seed=2), rand(5, 3, seed=3)
    far = P.softmax_head(q, k, v, 0.7, None, torch.tensor(-80.0, dtype=torch.float64))
    assert torch.allclose(far, P.softmax_head(q, k, v, 0.7))
    assert float(P.softmax_head(q, k, v, 0.7, None, torch.tensor(90.0, dtype=torch.float64)).max()) < 1e-30


def test_the_memory_against_the_sum_over_the_past_and_its_running_maximum():
    T, n, m = 7, 3, 2
    q, k, v = rand(T, n, seed=4), rand(T, n, seed=5), rand(T, m, seed=6)
    i, f = rand(T, seed=7, scale=4.0), P.log_sigmoid(rand(T, seed=8, scale=3.0))
    out = P.matrix_memory(q, k, v, i, f)
    for t in range(T):
        # unscaled: C = sum_s e^(i_s + f_(s+1) + ... + f_t) k_s v_s^T; the maximum counts the start (0) as well
        logs = [float(i[s] + f[s + 1:t + 1].sum()) for s in range(t + 1)]
        p = max(logs + [float(f[:t + 1].sum())])
        C = sum(math.exp(l) * torch.outer(k[s], v[s]) for s, l in enumerate(logs))
        nn = sum(math.exp(l) * k[s] for s, l in enumerate(logs))
        want = (C.T @ q[t]) / (max(abs(float(nn @ q[t])), 1.0) + 1e-6 * math.exp(p))
        assert torch.allclose(out[t], want, rtol=1e-9)
    # a small first gate: the maximum stays with the start, so the write is faded and the divisor is at least one
    one = P.matrix_memory(q[:1], k[:1], v[:1], torch.tensor([-5.0], dtype=torch.float64), torch.tensor([0.0], dtype=torch.float64))
    qk = float(q[0] @ k[0]) * math.exp(-5.0)
    assert torch.allclose(one[0], v[0] * qk / (max(abs(qk), 1.0) + 1e-6))


def test_gates_are_capped_and_forgetting_is_at_most_all():
    z = torch.tensor([-1e3, -2.0, 0.0, 3.0, 1e3], dtype=torch.float64)
    i, f = P.gates(z, z, 5.0)
    assert torch.allclose(i, torch.tensor([-5.0, 5 * math.tanh(-0.4), 0.0, 5 * math.tanh(0.6), 5.0], dtype=torch.float64))
    assert (f <= 0).all() and f[4] == pytest.approx(-math.log1p(math.exp(-5.0))) and f[0] == pytest.approx(-5.0 - math.log1p(math.exp(-5.0)))


def test_a_layer_reads_another_layers_rows_and_adds_the_tokens_own_input(tmp_path):
    d = write_tiny(str(tmp_path), "A")
    cfg, W = P.read_config(d), P.read_weights(d)
    ids = [3, 77, 140, 77]
    xs = []
    logits = P.forward(cfg, W, ids, layers_out=xs)
    c = P.latent(P.dyt(xs[1], W, "l2.norm1"), W, "l2.mix.", 1e-6)
    y = P.latent_attention(P.dyt(xs[4], W, "l5.norm1"), W, "l5.mix.", cfg["layers"][5]["mixer"], 1e-6, c)
    x = xs[4] + 0.6 * P.dyt(y, W, "l5.norm1b")
    e = torch.stack([W["side.embed"][t, 60:72] for t in ids])
    g = P.gelu_tanh(x @ W["l5.side.gate"].T) * e
    s = g @ W["l5.side.proj"].T
    x = x + 0.6 * s / torch.sqrt((s * s).mean(-1, keepdim=True) + 1e-6) * W["l5.side.norm"]
    assert torch.allclose(xs[5], x)
    assert torch.allclose(logits, P.dyt(x, W, "final.norm") @ W["embed"].T)
    assert torch.allclose(P.embedding(W["embed"], ids, 5.0), 5.0 * W["embed"][ids])
    assert torch.allclose(P.dense(torch.ones(1, 96, dtype=torch.float64), W, "l0.mlp."),
                          torch.relu(W["l0.mlp.up"].sum(1))[None].square() @ W["l0.mlp.down"].T)
