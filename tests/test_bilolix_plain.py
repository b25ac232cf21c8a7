"""Bilolix without a GPU: the configuration through its file and back, sizes read from stored tensors' shapes, errors that
name the key, the model as data (names, shapes, run order, what each call caches), and the plain implementation's own
mechanisms."""
import json
import math

import pytest
import torch

import plain_bilolix as P
from tiny_bilolix import BX_A, BX_B, BX_D, CONFIGS, write_tiny

from gesso_amd.config import BilolixConfig, load_config
from gesso_amd.errors import ConfigError


def rand(*shape, seed=0, scale=1.0):
    return torch.randn(*shape, generator=torch.Generator().manual_seed(seed), dtype=torch.float64) * scale


# ------------------------------------------------------------------ configuration

@pytest.mark.parametrize("name", sorted(CONFIGS))
def test_configuration_through_its_file_and_back(name, tmp_path):
    cfg, _ = CONFIGS[name]
    raw = cfg.to_json()
    assert BilolixConfig.from_dict(json.loads(json.dumps(raw))) == cfg
    (tmp_path / "config.json").write_text(json.dumps(raw))
    arch, back = load_config(str(tmp_path))
    assert arch.name == "Bilolix" and back == cfg


def test_sizes_that_only_stored_tensors_tell(tmp_path):
    """A file written elsewhere gives the bottlenecks no keys: they are the stored tensors' row counts; without the tensors
    the reader says which key it lacks."""
    d = write_tiny(str(tmp_path), "A")
    raw = json.loads(open(d + "/config.json").read())
    told = [(L["type"], L["mixer"].pop("rank", None), L["mixer"].pop("gate_rank", None)) for L in raw["layers"]]
    assert told[0] == ("channel_delta", 8, 12) and told[2] == ("gla", 8, None) and told[4] == ("channel_delta", 16, 8)
    open(d + "/config.json", "w").write(json.dumps(raw))
    assert load_config(d)[1] == BX_A
    with pytest.raises(ConfigError) as err:
        BilolixConfig.from_dict(raw)
    assert "rank" in str(err.value)


def test_keys_left_out_take_their_defaults_and_unknown_keys_name_themselves():
    raw = BX_A.to_json()
    del raw["loop"]
    raw["layers"][1]["mixer"]["mask"] = None
    raw["layers"][3]["mixer"].pop("rot")
    raw["layers"][2]["mlp"] = None
    cfg = BilolixConfig.from_dict(raw)
    assert cfg.loop is None and cfg.layers[1].mixer.window is None and cfg.layers[3].mixer.rot is None and cfg.layers[2].mlp is None
    for path, where in ((("embedding",), "config.json"), (("layers", 1, "mixer", "softcap"), "layers[1].mixer"),
                        (("layers", 1, "mixer", "rot", "scaling"), "layers[1].mixer.rot"),
                        (("layers", 1, "mixer", "mask", "keep_first"), "layers[1].mixer.mask"),
                        (("layers", 1, "mlp", "router", "scale"), "layers[1].mlp.router"), (("loop", "stride"), "loop"),
                        (("layers", 0, "mlp", "limit"), "layers[0].mlp")):
        raw = BX_A.to_json()
        at = raw
        for k in path[:-1]:
            at = at[k]
        at[path[-1]] = 3
        with pytest.raises(ConfigError) as err:
            BilolixConfig.from_dict(raw)
        assert path[-1] in str(err.value) and where in str(err.value)


@pytest.mark.parametrize("change,word", [
    (lambda r: r["layers"][0].__setitem__("type", "mamba2"), "type"),
    (lambda r: r["layers"][1]["mixer"]["rot"].__setitem__("dims", 26), "rot.dims"),
    (lambda r: r["layers"][1]["mixer"]["rot"].__setitem__("dims", 7), "rot.dims"),
    (lambda r: r["layers"][1]["mixer"].__setitem__("kv_heads", 3), "kv_heads"),
    (lambda r: r["layers"][4]["mixer"].__setitem__("kv_heads", 4), "kv_heads"),
    (lambda r: r["layers"][1]["mlp"]["router"].__setitem__("top", 9), "top"),
    (lambda r: r["layers"][0]["mlp"].__setitem__("kind", "swiglu"), "kind"),
    (lambda r: r["loop"].__setitem__("stop", 6), "loop"), (lambda r: r["loop"].__setitem__("times", 0), "times"),
    (lambda r: r["layers"][1]["mixer"].pop("diff"), "diff"), (lambda r: r["layers"][2]["mixer"].pop("tau"), "tau")])
def test_contradictions_are_errors(change, word):
    raw = BX_A.to_json()
    change(raw)
    with pytest.raises(ConfigError) as err:
        BilolixConfig.from_dict(raw)
    assert word in str(err.value)


# ------------------------------------------------------------------ the model as data

def test_names_shapes_order_and_caches():
    from gesso_amd.cache.manager import CacheLayout
    from gesso_amd.config.registry import architecture_of
    from gesso_amd.models.model import tensor_table
    from gesso_amd.parts import PagedKV, part_class
    spec = architecture_of(BX_A.to_json()).to_spec(BX_A)
    assert [c.layer for c in spec.schedule] == [0, 1, 2, 1, 2, 3, 4] and all(c.cache is None for c in spec.schedule)
    assert spec.reentry.at == (1, 3) and not spec.reentry.mix and not spec.tie_embeddings and spec.final_norm.offset == 1.0
    t = {k: v.shape for k, v in tensor_table(spec).items()}
    assert t["embed"] == t["head"] == (211, 96) and t["final.norm"] == t["l3.norm1"] == (96,) and t["loop.step"] == (2, 96)
    assert not any("norm2" in k or k.endswith(".norm1.b") or k == "loop.in" for k in t)
    assert t["l1.mix.q"] == (4 * 2 * 24, 96) and t["l1.mix.k"] == (2 * 2 * 24, 96) and t["l1.mix.v"] == (2 * 40, 96)
    assert t["l1.mix.g"] == (4, 96) and t["l1.mix.lq1"] == t["l1.mix.lk2"] == (24,) and t["l1.mix.o"] == (96, 4 * 40)
    assert t["l2.mix.a1"] == (8, 96) and t["l2.mix.a2"] == (48, 8) and t["l2.mix.a2.b"] == (48,) and t["l2.mix.g"] == (72, 96)
    assert t["l0.mix.q"] == (2 * 16, 96) and t["l0.mix.v.conv"] == (4 * 24, 4) and t["l0.mix.b"] == (4, 96)
    assert t["l0.mix.A_log"] == (4,) and t["l0.mix.a1"] == (8, 96) and t["l0.mix.a2"] == t["l0.mix.dt_bias"] + (8,) == (64, 8)
    assert t["l0.mix.g1"] == (12, 96) and t["l0.mix.g2"] == (96, 12) and t["l0.mix.norm"] == (24,) and "l0.mix.g" not in t
    assert t["l0.mlp.up"] == (80, 96) and t["l0.mlp.down"] == (96, 80) and "l0.mlp.gate" not in t
    assert t["l1.mlp.router"] == (6, 96) and t["l1.mlp.router.b"] == (6,) and t["l1.mlp.e5.gate"] == (40, 96)
    needs = [part_class("block", b).cache_need(b) for b in spec.blocks]
    assert needs[1] == PagedKV(2, 48, 40, value_dim=40) and needs[3] == PagedKV(2, 32, 7, value_dim=None)
    assert [(e[0], e[1], e[2]) for e in needs[0].entries()] == [("conv_history", (3, 2 * 2 * 16 + 4 * 24), "float32"), ("state", (4, 16, 24), "float32")]
    assert needs[2].entries() == [("state", (3, 16, 24), "float32", 0.0)]
    # every pass of the loop keeps its own: three attention runs on two page groups, four states
    per_call = [needs[c.layer] for c in spec.schedule]
    layout = CacheLayout.plan(per_call, [None] * len(per_call))
    assert sorted(len(g.members) for g in layout.paged) == [1, 2] and len(layout.slots) == 4
    d = architecture_of(BX_D.to_json()).to_spec(BX_D)
    assert [c.layer for c in d.schedule] == [0, 1, 2, 3] and d.reentry.at == (2,) and tensor_table(d)["loop.step"].shape == (1, 100)
    b = architecture_of(BX_B.to_json()).to_spec(BX_B)
    assert b.reentry is None and "loop.step" not in tensor_table(b) and "l0.mlp.up" not in tensor_table(b)


# ------------------------------------------------------------------ the plain implementation's own mechanisms

def test_norm_weights_lie_around_zero_and_eps_is_inside_the_root():
    x = torch.tensor([[3.0, 4.0]], dtype=torch.float64)
    assert torch.allclose(P.rms(x, 0.0), x / math.sqrt(12.5)) and torch.allclose(P.rms(x, 3.5), x / 4.0)


def test_neighbouring_features_turn_together_and_scores_depend_on_distance_alone():
    f = P.frequencies(4, 100.0)
    assert torch.allclose(f, torch.tensor([1.0, 0.1], dtype=torch.float64))
    x = rand(1, 6, seed=1)
    y = P.rotate_pairs(x, [3], f)[0]
    for i, a in ((0, 3.0), (1, 0.3)):
        u, v = x[0, 2 * i], x[0, 2 * i + 1]
        assert torch.isclose(y[2 * i], u * math.cos(a) - v * math.sin(a)) and torch.isclose(y[2 * i + 1], v * math.cos(a) + u * math.sin(a))
    assert torch.equal(y[4:], x[0, 4:])
    q, k = rand(1, 6, seed=2), rand(1, 6, seed=3)
    near = P.rotate_pairs(q, [7], f)[0] @ P.rotate_pairs(k, [5], f)[0]
    far = P.rotate_pairs(q, [107], f)[0] @ P.rotate_pairs(k, [105], f)[0]
    assert torch.isclose(near, far)


def test_a_window_shows_itself_and_the_tokens_before_it():
    for window in (1, 3, None):
        for i in range(6):
            assert [P.visible(i, j, window) for j in range(6)] == [j <= i and (window is None or j > i - window) for j in range(6)]
    v = torch.eye(5, dtype=torch.float64)
    w = P.softmax_map(torch.zeros(5, 2, dtype=torch.float64), torch.zeros(5, 2, dtype=torch.float64), v, range(5), 1.0, 2)
    assert torch.allclose(w[4], torch.tensor([0, 0, 0, 0.5, 0.5], dtype=torch.float64)) and torch.allclose(w[0], v[0])


def test_the_second_map_is_taken_off_the_first():
    T, d, vd = 4, 3, 5
    q, k, v = rand(T, 2, 2, d, seed=4), rand(T, 1, 2, d, seed=5), rand(T, 1, vd, seed=6)
    lam = P.share(*(rand(d, seed=7 + i, scale=0.3) for i in range(4)), 0.25)
    out = P.two_maps(q, k, v, range(T), 0.4, lam, 0.25, 1e-6)
    for h in (0, 1):
        o = [P.softmax_map(q[:, h, m], k[:, 0, m], v[:, 0], range(T), 0.4) for m in (0, 1)]
        want = P.rms(o[0] - lam * o[1], 1e-6) * 0.75
        assert torch.allclose(out[:, h], want)
    one = torch.zeros(d, dtype=torch.float64)
    assert float(P.share(one, one, one, one, 0.25)) == 0.25                    # exp(0) - exp(0) + share
    # the first token sees itself alone: (1 - lam) v, normed, whatever the scores
    assert torch.allclose(out[0, 0], P.rms((1 - lam) * v[0, 0], 1e-6) * 0.75)


def test_the_delta_rule_fades_rows_overwrites_and_reads_its_own_write():
    k = torch.tensor([[1.0, 0.0], [0.0, 1.0], [1.0, 0.0]], dtype=torch.float64)
    v, q = rand(3, 4, seed=8), torch.tensor([[1.0, 0.0]] * 3, dtype=torch.float64)
    ones = torch.ones(3, 2, dtype=torch.float64)
    o = P.delta_rule(q, k, v, torch.ones(3, dtype=torch.float64), ones)
    assert torch.allclose(o, torch.stack([v[0], v[0], v[2]]))                  # the third write replaces the first
    g = ones.clone()
    g[1] = torch.tensor([0.5, 0.25])
    o = P.delta_rule(q, k, v, torch.tensor([1.0, 0.0, 0.0], dtype=torch.float64), g)
    assert torch.allclose(o, torch.stack([v[0], 0.5 * v[0], 0.5 * v[0]]))      # row 0 fades by its own decay


def test_channel_decays_against_the_explicit_sum_over_the_past():
    T, n, m = 6, 3, 2
    q, k, v, a = rand(T, n, seed=9), rand(T, n, seed=10), rand(T, m, seed=11), torch.sigmoid(rand(T, n, seed=12))
    o = P.fading_state(q, k, v, a)
    for t in range(T):
        want = sum(v[s] * (q[t] * k[s] * torch.prod(a[s + 1:t + 1], 0)).sum() for s in range(t + 1))
        assert torch.allclose(o[t], want)
    g = P.channel_decays(rand(2, 6, seed=13), torch.tensor([-1.0, 0.5], dtype=torch.float64), rand(6, seed=14), 2)
    z = rand(2, 6, seed=13) + rand(6, seed=14)
    assert torch.allclose(g[1, 1, 2], torch.exp(-math.exp(0.5) * torch.log1p(torch.exp(z[1, 5]))))


def test_a_convolution_ends_on_the_current_token():
    x, taps = rand(5, 2, seed=15), torch.tensor([[0.0, 0.0, 1.0], [0.0, 1.0, 0.0]], dtype=torch.float64)
    y = P.causal_conv(x, taps)
    assert torch.equal(y[:, 0], x[:, 0]) and torch.equal(y[1:, 1], x[:-1, 1]) and float(y[0, 1]) == 0.0


def test_the_router_weighs_the_chosen_experts_among_themselves():
    W = {"r.router": rand(5, 4, seed=16), "r.router.b": torch.tensor([0.0, 9.0, 0.0, 0.0, -9.0], dtype=torch.float64)}
    x = rand(6, 4, seed=17)
    chosen, w = P.route(x, W, "r.", 2)
    z = x @ W["r.router"].T + W["r.router.b"]
    assert (chosen[:, 0] == 1).all() and not (chosen == 4).any()               # a bias of 9 is chosen first
    for t in range(6):
        e = torch.exp(z[t, chosen[t]])
        assert torch.allclose(w[t], e / e.sum())
    same = {"r.router": torch.zeros(4, 4, dtype=torch.float64), "r.router.b": torch.zeros(4, dtype=torch.float64)}
    chosen, w = P.route(x, same, "r.", 3)
    assert chosen.tolist() == [[0, 1, 2]] * 6 and torch.allclose(w, torch.full((6, 3), 1 / 3, dtype=torch.float64))


def test_gelu_is_the_error_function_form():
    z = torch.tensor([-2.0, 0.0, 1.0], dtype=torch.float64)
    assert torch.allclose(P.gelu(z), z * torch.tensor([0.02275013194817921, 0.5, 0.8413447460685429], dtype=torch.float64))


def test_a_run_of_layers_begins_every_pass_with_its_own_vector(tmp_path):
    d = write_tiny(str(tmp_path), "A")
    cfg, W = P.read_config(d), P.read_weights(d)
    assert P.run_order(cfg) == [(0, None), (1, 0), (2, None), (1, 1), (2, None), (3, None), (4, None)]
    ids = [3, 77, 140]
    layers = []
    P.forward(cfg, W, ids, layers_out=layers)
    x = layers[2] + W["loop.step"][1]
    assert torch.allclose(layers[3], P.layer(x, W, 1, cfg["layers"][1], [0, 1, 2], 1e-6))
    # both sub-layers read the one norm
    p, m = "l0.", cfg["layers"][0]
    x = P.embedding(W["embed"], ids)
    a = P.rms(x, 1e-6) * (1 + W[p + "norm1"])
    assert torch.allclose(layers[0], x + P.channel_delta(a, W, p + "mix.", m["mixer"], 1e-6) + P.dense(a, W, p + "mlp."))
