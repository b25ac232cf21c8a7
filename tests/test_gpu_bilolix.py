"""Bilolix on the GPU against the plain implementation: each kernel alone, each mixer and feed-forward alone (mixers with
their own cache: whole, token by token, in portions, in unequal batches, with pages and slots used again), the residual
stream after every layer run, whole models replayed in the four ways of cutting, long decoding, and greedy generation
through the session, its scheduler and the command line.

Where random weights would hide a fault, the inputs are made so that it shows: one key of one map is made to point along
one query of that map (far back, on a page's first and last row, just inside and just outside a window); two maps that
nearly cancel are given shares that leave a hundredth of either; a state that hardly fades is given one key and, hundreds of
tokens later, the query that meets it.
"""
import random

import pytest
import torch

import plain_bilolix as P
import replay as R
from test_gpu_kuditar import (DEV, DTYPES, Pages, check_rows, four_ways, gen, i32, renamed, scan_case, tiles_of, tol)
from tiny import random_ids
from tiny_bilolix import CONFIGS, write_folder, write_tiny

pytestmark = pytest.mark.gpu


@pytest.fixture(scope="module")
def ops():
    from gesso_amd.kernels import ops
    ops.lib()
    return ops


@pytest.fixture(scope="module")
def folders(tmp_path_factory):
    return str(tmp_path_factory.mktemp("bilolix"))


# ------------------------------------------------------------------ kernels alone

@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("F", [96, 36, 7, 4096])
def test_activations_alone_and_gated(ops, dtype, F):
    x = (torch.randn(5, F, generator=gen(0)) * 3).to(dtype)
    f = {"gelu": P.gelu, "silu": P.silu, "gelu_tanh": lambda z: torch.nn.functional.gelu(z, approximate="tanh")}
    for name, act in f.items():
        got = ops.activate(x.to(DEV), name, dtype).cpu().double()
        want = act(x.double())
        assert float((got - want).abs().max()) <= tol(dtype, want, 2e-6)
    y = (torch.randn(5, 2 * F, generator=gen(1)) * 2).to(dtype)
    got = ops.gated_act(y.to(DEV), None, "gelu", dtype).cpu().double()
    want = P.gelu(y[:, :F].double()) * y[:, F:].double()
    assert float((got - want).abs().max()) <= tol(dtype, want)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("H,G,d,vd,rd", [(3, 3, 10, 6, 4), (4, 2, 32, 64, 16), (4, 1, 64, 128, 64), (2, 2, 16, 20, 0)])
def test_cache_write_of_two_keys_a_head(ops, dtype, H, G, d, vd, rd):
    from gesso_amd.parts.rope import rope_tables
    ps, T = 4, 23
    width = 2 * (H + G) * d + G * vd
    x = (torch.randn(T, width + 8, generator=gen(2)) * 2).to(dtype)
    cos, sin = rope_tables(rd, 1e4, 64) if rd else (None, None)
    pos = [17 + i for i in range(T)]
    pg = Pages(dtype, G, 2 * d, vd, ps, [17 + T], seed=1)
    xd = x.clone().to(DEV)
    ops.qknorm_rope_kv(xd, None, None, 1.0, None if cos is None else cos.to(DEV), None if sin is None else sin.to(DEV), rd, i32(pos),
                       i32([0] * T), pg.table, ps, pg.k, pg.v, 2 * H, G, d, layout="interleaved", vd=vd, maps=2)
    f = P.frequencies(rd, 1e4)
    r = x.double()
    q = P.rotate_pairs(r[:, :2 * H * d].reshape(T, H, 2, d), pos, f)
    k = P.rotate_pairs(r[:, 2 * H * d:2 * (H + G) * d].reshape(T, G, 2, d), pos, f)
    v = r[:, 2 * (H + G) * d:width].reshape(T, G, vd)
    out = xd.cpu().double()
    assert float((out[:, :2 * H * d].reshape(T, H, 2, d) - q).abs().max()) <= tol(dtype, q)
    assert torch.equal(out[:, 2 * H * d:], r[:, 2 * H * d:])
    table = pg.table[0].cpu().tolist()
    for t, p in enumerate(pos):
        page, row = table[p // ps], p % ps
        assert float((pg.k[page, :, row].double().cpu() - k[t].reshape(G, 2 * d)).abs().max()) <= tol(dtype, k)
        assert torch.equal(pg.v[page, :, row].double().cpu(), v[t])


LAM, DIFF, EPS = 0.7, 0.35, 1e-5


def maps_case(ops, route, dtype, H, G, d, vd, lens, cuts, ps=8, window=None, scale=0.3, seed=0, lam=LAM, gated=True, plant=None,
              like=None, rows_of=16, splits=None):
    """Sequences of ``lens`` tokens fed in the pieces ``cuts[s]`` through the cache write and attention over two maps.
    ``route``: "general", or "fast": the kernel for prompt portions, and for steps of single tokens the kernel for single
    queries, with ``splits`` splits of the keys.  ``plant``: ``(map, key position, query position, size)``: in the first
    sequence, that map's key of the first key head points along the first head's query of that map, ``size`` times as long.
    ``like``: the second map's queries and keys are the first's plus that much noise.  Returns the kernel's rows and the plain
    attention's, per sequence."""
    g = gen(seed)
    nq, nk = 2 * H * d, 2 * G * d
    width = nq + nk + G * vd
    ld = -(-(width + H) // 16) * 16
    rows = [torch.randn(n, ld, generator=g) for n in lens]
    if like is not None:
        for r in rows:
            for a, n in ((0, H), (nq, G)):
                z = r[:, a:a + 2 * n * d].reshape(-1, n, 2, d)
                z[:, :, 1] = z[:, :, 0] + like * z[:, :, 1]
    if plant is not None:
        m, kp, qp, size = plant
        qv = rows[0][qp, m * d:(m + 1) * d]
        rows[0][kp, nq + m * d:nq + (m + 1) * d] = qv / qv.norm() * size
    rows = [r.to(dtype) for r in rows]
    pg = Pages(dtype, G, 2 * d, vd, ps, lens, seed)
    done, got = [0] * len(lens), [[] for _ in lens]
    rule = (window, scale, lam, EPS, 1.0 - DIFF, width if gated else -1, H, G, d, vd)
    for step in range(max(len(c) for c in cuts)):
        live = [s for s in range(len(lens)) if step < len(cuts[s])]
        sizes = [cuts[s][step] for s in live]
        x = torch.cat([rows[s][done[s]:done[s] + n] for s, n in zip(live, sizes)]).to(DEV)
        pos = i32([done[s] + i for s, n in zip(live, sizes) for i in range(n)])
        seq_of = i32([i for i, n in enumerate(sizes) for _ in range(n)])
        table = pg.table[live].contiguous()
        ops.qknorm_rope_kv(x, None, None, 1.0, None, None, 0, pos, seq_of, table, ps, pg.k, pg.v, 2 * H, G, d, vd=vd, maps=2)
        if route == "fast" and all(n == 1 for n in sizes):
            ns = splits or (2 if max(done) >= 128 else 1)
            y = ops.attention_decode_maps(x, pg.k, pg.v, pos, table, ps, *rule, len(live), ns)
        elif route == "fast":
            y = ops.attention_prefill_maps(x, pg.k, pg.v, pos, tiles_of(sizes, rows_of), table, ps, *rule, tile_rows=rows_of)
        else:
            y = ops.attention_maps(x, pg.k, pg.v, pos, seq_of, table, ps, *rule)
        at = 0
        for s, n in zip(live, sizes):
            got[s].append(y[at:at + n].double().cpu())
            at += n
            done[s] += n
    assert done == list(lens)
    want = []
    for s, n in enumerate(lens):
        r = rows[s].double()
        o = P.two_maps(r[:, :nq].reshape(n, H, 2, d), r[:, nq:nq + nk].reshape(n, G, 2, d), r[:, nq + nk:width].reshape(n, G, vd),
                       range(n), scale, lam, DIFF, EPS, window)
        if gated:
            o = o * torch.sigmoid(r[:, width:width + H])[:, :, None]
        want.append(o.reshape(n, H * vd))
    return [torch.cat(x) for x in got], want


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("window", [None, 1, 7, 24, 64, 65])
def test_two_maps_through_the_general_kernel(ops, dtype, window):
    for H, G, d, vd, ps, gated in ((4, 2, 24, 40, 8, True), (3, 3, 10, 6, 4, True), (5, 1, 6, 22, 16, False), (2, 1, 64, 300, 16, True)):
        lens = [110, 1, 33, 9]
        cuts = [[30, 1, 1, 60, 2, 16], [1], [33], [2, 2, 1, 1, 3]]
        got, want = maps_case(ops, "general", dtype, H, G, d, vd, lens, cuts, ps=ps, window=window, seed=H + d, gated=gated)
        for s in range(len(lens)):
            assert float((got[s] - want[s]).abs().max()) <= tol(dtype, want[s], 3e-5, 2e-2), (s, H, window)


PREFILL = [(2, 2, 32, 32, 8), (4, 2, 32, 64, 16), (4, 1, 64, 64, 4), (3, 1, 64, 128, 16), (8, 1, 32, 128, 8), (6, 1, 64, 128, 16),
           (2, 1, 128, 128, 16), (8, 2, 128, 128, 8)]


@pytest.mark.parametrize("window", [None, 1, 7, 33, 64, 100])
@pytest.mark.parametrize("rows_of", [16, 32])
def test_two_maps_through_the_prompt_kernel(ops, window, rows_of):
    """Sequences long enough for several steps of keys, fed whole, in long portions and in short ones beside single tokens;
    groups of one to eight query heads a key head, some cut into blocks of their own."""
    for H, G, d, vd, ps in PREFILL:
        lens = [230, 1, 97, 40]
        cuts = [[100, 64, 1, 33, 30, 1, 1], [1], [97], [2, 17, 1, 1, 17, 1, 1]]
        got, want = maps_case(ops, "fast", torch.bfloat16, H, G, d, vd, lens, cuts, ps=ps, window=window, seed=H + d, rows_of=rows_of)
        for s in range(len(lens)):
            assert float((got[s] - want[s]).abs().max()) <= tol(torch.bfloat16, want[s], 3e-5, 2e-2), (s, H, G, d, vd, window)


DECODE = [(2, 2, 16, 32, 8), (4, 1, 16, 64, 16), (2, 1, 32, 32, 8), (4, 2, 32, 64, 16), (8, 1, 32, 128, 4), (3, 3, 64, 64, 16),
          (6, 1, 64, 128, 16), (4, 1, 64, 128, 8), (5, 1, 128, 128, 16), (4, 1, 128, 128, 16), (16, 2, 64, 128, 16)]


@pytest.mark.parametrize("window", [None, 1, 7, 64, 100])
@pytest.mark.parametrize("splits", [1, 3])
def test_two_maps_through_the_kernel_for_single_queries(ops, window, splits):
    for H, G, d, vd, ps in DECODE:
        if ops.attention_prefill_maps_supports(H, G, d, vd):      # single tokens behind a long portion
            lens, cuts = [201, 1, 64, 9], [[190] + [1] * 11, [1], [60, 1, 1, 1, 1], [1] * 9]
            got, want = maps_case(ops, "fast", torch.bfloat16, H, G, d, vd, lens, cuts, ps=ps, window=window, seed=H + d, splits=splits)
            for s in range(len(lens)):
                assert float((got[s] - want[s]).abs().max()) <= tol(torch.bfloat16, want[s], 3e-5, 2e-2), (s, H, G, d, vd, window)
        alone, ref = maps_case(ops, "fast", torch.bfloat16, H, G, d, vd, [130, 70], [[1] * 130, [1] * 70], ps=ps, window=window,
                               seed=H + d + 1, splits=splits)
        for s in range(2):
            assert float((alone[s] - ref[s]).abs().max()) <= tol(torch.bfloat16, ref[s], 3e-5, 2e-2), ("alone", s, H, G, d, vd, window)


@pytest.mark.parametrize("route,dtype", [("general", torch.float32), ("general", torch.bfloat16), ("fast", torch.bfloat16)])
@pytest.mark.parametrize("ps", [8, 16])
def test_a_key_of_one_map_that_stands_out_is_seen_or_not_at_every_edge(ops, route, dtype, ps):
    """One key of one map points along the last query's same map: that map's weight goes there if and only if the window
    lets the query see it, whichever map it is."""
    T, H, G, d, vd = 340, 2, 1, 32, 64
    query, window = T - 1, 50
    first = query - window + 1
    for w, places in ((window, [first, first - 1, first + 1, (query // ps) * ps, (query // ps) * ps - 1, query - 1, 0]),
                      (None, [query - 300, 0, ps - 1, ps, (query // ps) * ps - 1])):
        quiet, _ = maps_case(ops, route, dtype, H, G, d, vd, [T], [[T]], ps=ps, window=w, scale=1.0, seed=3)
        for place in places:
            for m in (0, 1):
                for cuts in ([[T]], [[query, 1]], [[query - 60] + [1] * 61], [[query - 70, 71]]):
                    got, want = maps_case(ops, route, dtype, H, G, d, vd, [T], cuts, ps=ps, window=w, scale=1.0, seed=3,
                                          plant=(m, place, query, 12.0))
                    assert float((got[0] - want[0]).abs().max()) <= tol(dtype, want[0], 1e-4, 3e-2), (w, place, m, cuts[0][:2])
                moved = float((got[0][query, :vd] - quiet[0][query, :vd]).abs().max())
                assert (moved > 0.05) == P.visible(query, place, w), (w, place, m, moved)


@pytest.mark.parametrize("d,vd", [(32, 64), (64, 128)])
def test_two_maps_that_nearly_cancel_keep_what_is_left(ops, d, vd):
    """The second map is the first with two hundredths of noise and counts 0.97: what is left is a few hundredths of either
    map's sum, and softmax weights cut to eight bits would show in it many times over."""
    lens, cuts = [150, 140], [[150], [100] + [1] * 40]
    got, want = maps_case(ops, "fast", torch.bfloat16, 4, 2, d, vd, lens, cuts, scale=0.3, seed=5, like=0.02, lam=0.97, gated=False)
    for s in range(2):
        e = (got[s] - want[s]).reshape(lens[s], 4, vd)[2:]
        rms = ((e * e).mean(-1) / (want[s].reshape(lens[s], 4, vd)[2:] ** 2).mean(-1)).sqrt()
        assert float(rms.max()) <= 6e-3, (s, float(rms.max()))


SCANS = [(4, 2, 16, 24), (6, 1, 32, 64), (2, 2, 64, 128), (2, 1, 128, 128), (5, 5, 6, 14), (1, 1, 200, 40)]


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("H,G,n,m", SCANS)
def test_delta_rule_with_a_decay_a_channel_over_unequal_sequences_and_any_cut(ops, dtype, H, G, n, m):
    lens = [1, 23, 2, 41]
    pieces = [[1], [5, 1, 1, 2, 7, 3, 1, 3], [1, 1], [12, 9, 1, 17, 2]]
    a, want, sa, slots_a = scan_case(ops, dtype, H, G, n, m, lens, [[1], [23], [2], [41]], True, True, seed=n + m)
    b, _, sb, slots_b = scan_case(ops, dtype, H, G, n, m, lens, pieces, True, True, seed=n + m)
    for s in range(len(lens)):
        assert float((a[s] - want[s]).abs().max()) <= tol(torch.float32, want[s], 3e-5), s
        assert torch.equal(a[s], b[s]) and torch.equal(sa[slots_a[s]], sb[slots_b[s]])


@pytest.mark.parametrize("H,G,n,m,seg", [(2, 1, 64, 128, 128), (4, 2, 16, 24, 64), (1, 1, 40, 10, 32)])
def test_delta_rule_with_a_decay_a_channel_in_segments_side_by_side(ops, H, G, n, m, seg):
    lens = [300, 1, 130, 64]
    pieces = [[150, 150], [1], [1, 128, 1], [64]]
    for cuts in ([[300], [1], [130], [64]], pieces):
        got, want, _, _ = scan_case(ops, torch.float32, H, G, n, m, lens, cuts, True, True, seed=n, segment=seg)
        for s in range(len(lens)):
            assert float((got[s] - want[s]).abs().max()) <= tol(torch.float32, want[s], 5e-5), s


@pytest.mark.parametrize("cuts,seg", [([[420]], 0), ([[420]], 128), ([[40] + [1] * 380], 0), ([[200, 220]], 64)])
def test_a_state_of_many_decays_keeps_what_it_was_given_hundreds_of_tokens_before(ops, cuts, seg):
    got, want, _, _ = scan_case(ops, torch.float32, 2, 2, 16, 24, [420], cuts, True, True, seed=7, slow=True, meet=(20, 400), segment=seg)
    assert float(want[0][400].abs().max()) > 10 * float(want[0][399].abs().max())     # the meeting stands out
    assert float((got[0] - want[0]).abs().max()) <= tol(torch.float32, want[0], 3e-5)


@pytest.mark.parametrize("dtype", DTYPES)
def test_what_the_delta_rule_computes_before_its_recurrence_with_a_decay_a_channel(ops, dtype):
    T, G, n, H = 9, 2, 12, 6
    c = torch.randn(T, 2 * G * n + 7, generator=gen(30)) * 3
    rows = (torch.randn(T, 40, generator=gen(31)) * 4).to(dtype)
    z = torch.randn(T, H * n + 9, generator=gen(32)) * 4
    a_log, dt_bias = torch.linspace(-6, 1, H), torch.linspace(-3, 1, H * n)
    cd, zd = c.clone().to(DEV), z.clone().to(DEV)
    beta = ops.delta_rule_prep(cd, G, n, n ** -0.5, 1e-6, rows.to(DEV), 0, 3, a_log.to(DEV), dt_bias.to(DEV), H, channels=zd, oz=4)
    q = P.unit(c[:, :G * n].double().reshape(T, G, n)) * n ** -0.5
    k = P.unit(c[:, G * n:2 * G * n].double().reshape(T, G, n))
    assert float((cd.cpu().double()[:, :2 * G * n] - torch.cat([q, k], 1).reshape(T, -1)).abs().max()) <= 1e-6
    want = P.channel_decays(z[:, 4:4 + H * n].double(), a_log.double(), dt_bias.double(), H).reshape(T, -1)
    assert float((zd.cpu()[:, 4:4 + H * n].double() - want).abs().max()) <= 1e-6
    assert torch.equal(zd.cpu()[:, :4], z[:, :4]) and torch.equal(zd.cpu()[:, 4 + H * n:], z[:, 4 + H * n:])
    assert beta.shape == (T, H) and float((beta.cpu().double() - torch.sigmoid(rows[:, 3:3 + H].double())).abs().max()) <= 1e-6


@pytest.mark.parametrize("H,m", [(3, 24), (4, 128), (5, 6)])
def test_normed_heads_with_a_float32_gate(ops, H, m):
    o, rows, w = torch.randn(7, H * m, generator=gen(33)) * 3, torch.randn(7, H * m + 10, generator=gen(34)), 1 + 0.2 * torch.randn(m, generator=gen(35))
    for out in DTYPES:
        got = ops.gated_outnorm(o.to(DEV), rows.to(DEV), 10, w.repeat(H).to(DEV), 1e-6, H, m, False, "sigmoid", out).cpu().double()
        want = (P.rms(o.double().reshape(7, H, m), 1e-6) * w.double()).reshape(7, -1) * torch.sigmoid(rows[:, 10:].double())
        assert float((got - want).abs().max()) <= tol(out, want)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("E,top,H,F", [(6, 2, 96, 40), (3, 1, 64, 16), (4, 4, 100, 12), (16, 3, 256, 64), (1, 1, 64, 24)])
def test_experts_chosen_by_biased_logits_and_weighed_among_themselves(ops, dtype, E, top, H, F):
    T = 40
    x = torch.randn(T, H, generator=gen(36)).to(dtype)
    W = {"m.router": (torch.randn(E, H, generator=gen(37)) * 0.3).to(dtype), "m.router.b": torch.randn(E, generator=gen(38))}
    for e in range(E):
        for k, shape in (("gate", (F, H)), ("up", (F, H)), ("down", (H, F))):
            W[f"m.e{e}.{k}"] = (torch.randn(*shape, generator=gen(40 + 3 * e + len(k))) * 0.2).to(dtype)
    d = {k: v.double() for k, v in W.items()}
    choice, weight = ops.moe_router(x.to(DEV), W["m.router"].to(DEV), None, top, bias=W["m.router.b"].to(DEV))
    chosen, weights = P.route(x.double(), d, "m.", top)
    z = torch.sort(x.double() @ d["m.router"].T + d["m.router.b"], -1, descending=True).values
    clear = [t for t in range(T) if top == E or float(z[t, top - 1] - z[t, top]) > 1e-4]
    assert len(clear) > T // 2
    for t in clear:
        ref = dict(zip(chosen[t].tolist(), weights[t].tolist()))
        assert sorted(choice[t].tolist()) == sorted(ref)
        assert all(abs(float(w) - ref[int(e)]) <= 1e-5 for e, w in zip(choice[t], weight[t]))
    want = P.moe(x.double(), d, "m.", {"router": {"experts": E, "top": top}})
    gu = torch.stack([torch.cat([W[f"m.e{e}.gate"], W[f"m.e{e}.up"]]) for e in range(E)]).to(DEV)
    down = torch.stack([W[f"m.e{e}.down"] for e in range(E)]).to(DEV)
    runs = [ops.moe_routed]
    if dtype == torch.bfloat16 and ops.moe_routed_grouped_ok(x.to(DEV), gu, down):
        runs.append(ops.moe_routed_grouped)
    for f in runs:
        got = f(x.to(DEV), choice, weight, gu, down, float("inf"), 1.0, shift=0.0).cpu().double()
        assert float((got - want)[clear].abs().max()) <= tol(dtype, want, 2e-5, 2e-2), f.__name__


def test_a_norm_adds_two_results_and_a_vector_for_every_row():
    from gesso_amd.config import RMSNormSpec
    from gesso_amd.parts import ResidualStream, Runtime, build
    rt = Runtime(DEV, torch.float32)
    norm = build("norm", RMSNormSpec(96, 1e-6, offset=1.0), rt)
    w = torch.randn(96, generator=gen(50)) * 0.2
    norm.bind({"weight": w.to(DEV)})
    x, a, b = (torch.randn(5, 96, generator=gen(51 + i)).to(DEV) for i in range(3))
    v = torch.randn(96, generator=gen(54)).to(DEV)
    for pend, bias in (((a, b), None), ((a, None), v), ((a, b), v), (None, v)):
        s = ResidualStream(x.clone(), pending=pend)
        s.bias = bias
        y = norm.add_norm(s)
        want = x + (0 if pend is None else sum(t for t in pend if t is not None)) + (0 if bias is None else bias)
        assert float((s.res - want).abs().max()) <= 1e-6 and s.pending is None and s.bias is None
        ref = P.rms(want.double().cpu(), 1e-6) * (1 + w.double())
        assert float((y.cpu().double() - ref).abs().max()) <= 1e-5


# ------------------------------------------------------------------ mixers and feed-forwards alone

MAPS = {"q_proj.weight": "q", "k_proj.weight": "k", "v_proj.weight": "v", "gate_proj.weight": "g", "out_proj.weight": "o",
        "share.q1": "lq1", "share.k1": "lk1", "share.q2": "lq2", "share.k2": "lk2"}
FADING = {"q_proj.weight": "q", "k_proj.weight": "k", "v_proj.weight": "v", "gate_proj.weight": "g", "decay_down.weight": "a1",
          "decay_up.weight": "a2", "decay_up.bias": "a2.b", "out_norm.weight": "norm", "out_proj.weight": "o"}
DELTA = {"q_proj.weight": "q", "k_proj.weight": "k", "v_proj.weight": "v", "beta_proj.weight": "b", "q_conv.weight": "q.conv",
         "k_conv.weight": "k.conv", "v_conv.weight": "v.conv", "A_log": "A_log", "dt_bias": "dt_bias", "decay_down.weight": "a1",
         "decay_up.weight": "a2", "gate_down.weight": "g1", "gate_up.weight": "g2", "out_norm.weight": "norm", "out_proj.weight": "o"}


def mixer_harness(kind, dtype, W=96, page_size=8, num_pages=64, seed=11, **kw):
    """A mixer of the design with its cache, and the plain function of the same tensors."""
    from test_gpu_kuditar import _harness
    from gesso_amd.config import GatedDeltaSpec, GatedLinearSpec, MapAttentionSpec, NoPositionSpec, RopeSpec
    eps, g = 1e-6, gen(seed)
    if kind == "maps":
        H, G, d, vd = kw.get("H", 4), kw.get("G", 2), kw.get("d", 24), kw.get("vd", 40)
        rd, window, diff = kw.get("rd", 16), kw.get("window", 21), kw.get("diff", 0.3)
        pos = RopeSpec(head_dim=d, rotary_dim=rd, theta=2e4, max_position=1024, layout="interleaved") if rd else NoPositionSpec()
        spec = MapAttentionSpec(hidden=W, n_heads=H, n_kv_heads=G, map_dim=d, value_dim=vd, position=pos, scale=0.2, share=diff,
                                eps=eps, window=window)
        sharp = {f"share.{n}": torch.randn(d, generator=g) * 0.7 / d ** 0.25 for n in ("q1", "k1", "q2", "k2")}
        h = _harness(spec, dtype, seed, page_size, num_pages, sharp)
        w = renamed(h.tensors, MAPS, "m.")
        m = {"heads": H, "kv_heads": G, "dim": d, "vdim": vd, "scale": 0.2, "diff": diff,
             "rot": {"base": 2e4, "dims": rd} if rd else None, "mask": {"size": window} if window else None}
        return h, lambda x: P.attention(x.double(), w, "m.", m, list(range(x.shape[0])), eps)
    if kind == "fading":
        H, n, m_, r, tau = kw.get("H", 3), kw.get("n", 16), kw.get("m", 24), kw.get("r", 8), kw.get("tau", 8.0)
        spec = GatedLinearSpec(hidden=W, n_heads=H, key_dim=n, value_dim=m_, decay_rank=r, tau=tau, eps=eps)
        h = _harness(spec, dtype, seed, page_size, num_pages, {"decay_up.bias": torch.rand(H * n, generator=g) * 6.0})
        w = renamed(h.tensors, FADING, "m.")
        return h, lambda x: P.gla(x.double(), w, "m.", {"heads": H, "dim": n, "vdim": m_, "tau": tau}, eps)
    H, G, n, m_, K = kw.get("H", 4), kw.get("G", 2), kw.get("n", 16), kw.get("m", 24), kw.get("taps", 4)
    spec = GatedDeltaSpec(hidden=W, n_heads=H, qk_heads=G, key_dim=n, value_dim=m_, conv_taps=K, eps=eps, decay_rank=kw.get("r", 8),
                          gate_rank=kw.get("gr", 12), gate="sigmoid")
    sharp = {"A_log": torch.linspace(-6.0, 1.0, H), "dt_bias": torch.rand(H * n, generator=g) * 4 - 3}
    h = _harness(spec, dtype, seed, page_size, num_pages, sharp)
    for k_ in ("q_conv.weight", "k_conv.weight", "v_conv.weight"):
        sharp[k_] = h.tensors[k_] * 4.0
    h = _harness(spec, dtype, seed, page_size, num_pages, sharp)
    w = renamed(h.tensors, DELTA, "m.")
    return h, lambda x: P.channel_delta(x.double(), w, "m.", {"heads": H, "kv_heads": G, "dim": n, "vdim": m_, "conv": K}, eps)


CASES = [("maps", dict()), ("maps", dict(W=64, H=3, G=3, d=10, vd=22, rd=0, window=None)), ("maps", dict(W=64, H=2, G=1, d=12, vd=8, rd=6, window=1)),
         ("maps", dict(W=128, H=4, G=1, d=64, vd=128, rd=64, window=32, page_size=16)), ("maps", dict(W=128, H=4, G=2, d=32, vd=64, rd=8, window=7, diff=0.0)),
         ("maps", dict(W=96, H=6, G=1, d=16, vd=32, rd=16, window=40)),
         ("fading", dict()), ("fading", dict(W=64, H=2, n=24, m=8, r=3, tau=1.0)), ("fading", dict(W=128, H=2, n=128, m=128, r=16, tau=16.0)),
         ("delta", dict()), ("delta", dict(W=64, H=6, G=1, n=8, m=12, taps=1, r=3, gr=40)), ("delta", dict(W=64, H=2, G=2, n=12, m=20, taps=5, r=33, gr=1)),
         ("delta", dict(W=128, H=2, G=2, n=64, m=128, taps=4, r=32, gr=64)), ("delta", dict(W=100, H=5, G=5, n=10, m=6, taps=2, r=7, gr=9))]


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("kind,kw", CASES)
def test_mixers_whole_token_by_token_in_portions_and_in_batches(dtype, kind, kw):
    h, plain = mixer_harness(kind, dtype, **kw)
    W, T = kw.get("W", 96), 90
    x = torch.randn(T, W, generator=gen(60)).to(dtype)
    want = plain(x)
    bound = tol(dtype, want, 5e-5, 3e-2)
    assert float((h.mixer(x, [("whole", T)]) - want).abs().max()) <= bound
    # most of it at once, the rest token by token across the window's edge; the first tokens one by one
    got = [h.mixer(x[:40], [("tail", 40)])] + [h.mixer(x[i:i + 1], [("tail", 1)]) for i in range(40, T)]
    assert float((torch.cat(got) - want).abs().max()) <= bound
    got = [h.mixer(x[i:i + 1], [("first", 1)]) for i in range(6)]
    assert float((torch.cat(got) - want[:6]).abs().max()) <= bound
    at, got = 0, []
    for size in (2, 7, 2, 13, 3, 16, 5, 2, 31, 9):
        got.append(h.mixer(x[at:at + size], [("cut", size)]))
        at += size
    assert at == T and float((torch.cat(got) - want).abs().max()) <= bound
    for rid in ("whole", "tail", "first", "cut"):
        h.manager.release(rid)
    # unequal requests side by side: a single token of one, a portion of another, a whole short one
    y, u = torch.randn(30, W, generator=gen(61)).to(dtype), torch.randn(5, W, generator=gen(62)).to(dtype)
    h.mixer(y[:29], [("b", 29)])
    h.mixer(x[:50], [("a", 50)])
    out = h.mixer(torch.cat([y[29:30], x[50:70], u]), [("b", 1), ("a", 20), ("c", 5)])
    assert float((out[0] - plain(y)[29]).abs().max()) <= bound
    assert float((out[1:21] - want[50:70]).abs().max()) <= bound
    assert float((out[21:] - plain(u)).abs().max()) <= bound


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("kind,kw", [("delta", dict()), ("delta", dict(W=128, H=2, G=1, n=64, m=128, r=32, gr=64)), ("fading", dict()),
                                     ("maps", dict(W=128, H=4, G=2, d=32, vd=64, rd=8, window=200, page_size=16))])
def test_mixers_with_long_portions(dtype, kind, kw):
    """A prompt of several segments whole; the same in two long portions and single tokens; a long portion of one request
    beside a single token of another."""
    h, plain = mixer_harness(kind, dtype, num_pages=256, **kw)
    W, T = kw.get("W", 96), 640
    x = torch.randn(T, W, generator=gen(63)).to(dtype)
    want = plain(x)
    bound = tol(dtype, want, 5e-5, 3e-2)
    assert float((h.mixer(x, [("whole", T)]) - want).abs().max()) <= bound
    got = [h.mixer(x[:300], [("cut", 300)]), h.mixer(x[300:301], [("cut", 1)]), h.mixer(x[301:630], [("cut", 329)])]
    got += [h.mixer(x[i:i + 1], [("cut", 1)]) for i in range(630, T)]
    assert float((torch.cat(got) - want).abs().max()) <= bound
    h.manager.release("whole")
    h.manager.release("cut")
    y = torch.randn(30, W, generator=gen(64)).to(dtype)
    h.mixer(y[:29], [("b", 29)])
    h.mixer(x[:130], [("a", 130)])
    out = h.mixer(torch.cat([y[29:30], x[130:500]]), [("b", 1), ("a", 370)])
    assert float((out[0] - plain(y)[29]).abs().max()) <= bound
    assert float((out[1:] - want[130:500]).abs().max()) <= bound


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("kind,kw", [("maps", dict()), ("maps", dict(W=96, H=4, G=2, d=32, vd=64, rd=32, window=None)), ("fading", dict()), ("delta", dict())])
def test_mixers_with_pages_and_slots_freed_and_used_again(dtype, kind, kw):
    """A pool that holds little more than one request's rows, and four slots: every later request writes pages and a slot
    that an earlier one gave back (filled with NaN in between)."""
    h, plain = mixer_harness(kind, dtype, page_size=8, num_pages=9, **kw)
    for i, T in enumerate((60, 35, 64, 9, 50, 20)):
        x = torch.randn(T, 96, generator=gen(70 + i)).to(dtype)
        want = plain(x)
        at, got = 0, []
        while at < T:
            size = min((11, 2, 1, 16)[(at + i) % 4], T - at)
            got.append(h.mixer(x[at:at + size], [(i, size)]))
            at += size
        assert float((torch.cat(got) - want).abs().max()) <= tol(dtype, want, 5e-5, 3e-2), i
        h.manager.release(i)
        for pool in h.storage.keys + h.storage.values:
            pool[:, :-1].fill_(float("nan"))
        for pool, _ in h.storage.state_pools:
            pool[:, :-1].fill_(float("nan"))


# ------------------------------------------------------------------ whole models

LENGTHS = {"A": (1, 23, 70, 130), "B": (2, 40, 77), "C": (5, 64, 150, 300), "D": (3, 52, 110)}


def sequences(name):
    cfg, seed = CONFIGS[name]
    return {f"s{i}": random_ids(n, cfg.vocab, 100 * seed + i) for i, n in enumerate(LENGTHS[name])}


@pytest.mark.parametrize("name", ["A", "B", "D"])
def test_the_residual_stream_after_every_layer_run(name, folders):
    from gesso_amd.engine.batch import StepEntry
    from gesso_amd.engine.engine import Engine
    cfg, seed = CONFIGS[name]
    model_dir = write_tiny(folders, name, torch.float32)
    ids = random_ids(47, cfg.vocab, 5 * seed)
    want = []
    P.forward(P.read_config(model_dir), P.read_weights(model_dir), ids, layers_out=want)
    eng = Engine.from_folder(model_dir, dtype="float32", device=DEV, page_size=16, max_tokens=256, num_slots=4)
    got = []
    for b in eng.model.blocks:
        def wrapped(stream, ctx, cache, orig=b.forward):
            orig(stream, ctx, cache)
            pend = stream.pending if isinstance(stream.pending, tuple) else (stream.pending,)
            got.append(stream.res.double().cpu() + sum(d.double().cpu() for d in pend if d is not None))
        b.forward = wrapped
    eng.add_request("r")
    eng.step([StepEntry("r", ids[:29], [])])
    first = list(got)
    got.clear()
    eng.step([StepEntry("r", ids[29:], [])])
    assert len(first) == len(got) == len(want) == len(P.run_order(P.read_config(model_dir)))
    for i, w in enumerate(want):
        mine = torch.cat([first[i], got[i]])
        assert float((mine - w).abs().max()) <= 3e-5 * max(1.0, float(w.abs().max())), f"layer run {i}"


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", ["A", "B", "C", "D"])
def test_replay_four_ways(name, dtype, folders, tmp_path):
    cfg, _ = CONFIGS[name]
    model_dir = write_tiny(folders, name, torch.float32 if dtype == "float32" else torch.bfloat16)
    seqs = sequences(name)
    plain = R.Plain(model_dir, seqs, dtype)
    ways, big = four_ways(seqs, 5)
    got, rc = R.run_trace(model_dir, dtype, str(tmp_path / "out"), big, cfg.vocab)
    assert rc == 0
    for way in ways:
        mine = {k.split(".", 1)[1]: v for k, v in got.items() if k.startswith(way + ".")}
        assert {k: len(v) for k, v in mine.items()} == {k: len(v) for k, v in seqs.items()}, way
        check_rows(plain, mine, dtype, f"Bilolix {name} {way}")


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", ["A", "D"])
def test_long_decoding_token_by_token(name, dtype, folders, tmp_path):
    """A short prompt, then two hundred tokens one by one: states carried, histories moved on, windows passed and pages
    begun and given back many times over."""
    cfg, seed = CONFIGS[name]
    model_dir = write_tiny(folders, name, torch.float32 if dtype == "float32" else torch.bfloat16)
    seqs = {"long": random_ids(230, cfg.vocab, 7000 + seed), "other": random_ids(201, cfg.vocab, 7100 + seed)}
    plain = R.Plain(model_dir, seqs, dtype)
    got, rc = R.run_trace(model_dir, dtype, str(tmp_path / "out"), R.trace_tail(seqs, tail=200), cfg.vocab)
    assert rc == 0 and {k: len(v) for k, v in got.items()} == {"long": 230, "other": 201}
    check_rows(plain, got, dtype, f"Bilolix {name}, 200 tokens one by one")


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", ["A", "B"])
def test_replay_with_pages_of_eight_given_back_poisoned(name, dtype, folders, tmp_path):
    cfg, _ = CONFIGS[name]
    model_dir = write_tiny(folders, name, torch.float32 if dtype == "float32" else torch.bfloat16)
    seqs = sequences(name)
    plain = R.Plain(model_dir, seqs, dtype)
    for way, make in (("portions", lambda s: R.trace_portions(s, sizes=(13, 2, 8, 3))), ("mixed", lambda s: R.trace_mixed(s, seed=9))):
        got, rc = R.run_trace(model_dir, dtype, str(tmp_path / way), make(seqs), cfg.vocab, page_size=8, extra=["--poison"])
        assert rc == 0
        check_rows(plain, got, dtype, f"Bilolix {name}, pages of 8, poisoned, {way}")


@pytest.mark.parametrize("name", ["A", "B"])
def test_greedy_generation_through_the_session(name, folders):
    """Prompts of unequal length generated together through the scheduler (prefill in portions, then the decode loop);
    float32 must give the plain model's tokens."""
    from gesso_amd import Session
    from noise import supported
    cfg, _ = CONFIGS[name]
    model_dir = write_tiny(folders, name, torch.float32)
    pc, pw = P.read_config(model_dir), P.read_weights(model_dir)
    prompts = [random_ids(n, cfg.vocab, 900 + n) for n in (3, 41, 18)]
    new = 24
    want = [P.greedy(pc, pw, p, new) for p in prompts]
    session = Session(model_dir, dtype="float32", device=DEV, context_length=256, chunk_size=16)
    try:
        assert session.generate(prompts, max_new_tokens=new) == want
        assert session.generate([prompts[1]], max_new_tokens=new)[0] == want[1]
    finally:
        session.close()
    session = Session(write_tiny(folders, name, torch.bfloat16), dtype="bfloat16", device=DEV, context_length=256)
    try:
        got = session.generate(prompts, max_new_tokens=new)
    finally:
        session.close()
    assert [len(x) for x in got] == [len(w) for w in want]
    pw16 = P.read_weights(write_tiny(folders, name, torch.bfloat16))
    for ids, p in zip(got, prompts):
        lg = P.forward(pc, pw16, ids).numpy()
        assert all(supported(lg[i - 1], ids[i], 0.5) for i in range(len(p), len(ids)))


def test_the_command_line_serves_a_bilolix_folder(folders):
    import json
    import os
    import subprocess
    import sys
    cfg, _ = CONFIGS["D"]
    model_dir = write_tiny(folders, "D", torch.float32)
    prompt = random_ids(19, cfg.vocab, 77)
    want = P.greedy(P.read_config(model_dir), P.read_weights(model_dir), prompt, 24)
    root = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
    r = subprocess.run([sys.executable, "-m", "gesso_amd", "--model", model_dir, "--dtype", "float32", "--prompt-ids",
                        ",".join(str(t) for t in prompt), "--max-new-tokens", "24", "--n-ctx", "128"],
                       capture_output=True, text=True, cwd=root, timeout=240, env=dict(os.environ, PYTHONPATH=root))
    assert r.returncode == 0, r.stderr[-2000:]
    assert json.loads(r.stdout.strip().splitlines()[-1])["ids"] == [want]


def test_forty_requests_at_once_decode_together(folders):
    from gesso_amd import Session
    from noise import supported
    cfg, _ = CONFIGS["C"]
    model_dir = write_tiny(folders, "C", torch.bfloat16)
    pc, pw = P.read_config(model_dir), P.read_weights(model_dir)
    prompts = [random_ids(3 + (7 * i) % 40, cfg.vocab, 2000 + i) for i in range(40)]
    session = Session(model_dir, dtype="bfloat16", device=DEV, context_length=128, max_num_seqs=64)
    try:
        got = session.generate(prompts, max_new_tokens=10)
        alone = session.generate([prompts[0]], max_new_tokens=10)[0]
    finally:
        session.close()
    assert [len(g_) for g_ in got] == [len(p) + 10 for p in prompts]
    for p, ids in ((prompts[0], got[0]), (prompts[17], got[17]), (prompts[39], got[39]), (prompts[0], alone)):
        lg = P.forward(pc, pw, ids).numpy()
        assert all(supported(lg[j - 1], ids[j], 0.5) for j in range(len(p), len(ids)))


def random_bilolix(seed: int):
    """A configuration drawn from a seed: two to five layers of the three kinds in any order, with and without a loop, turns,
    windows, feed-forwards of either kind or none, sizes with and without whole tiles."""
    from gesso_amd.config import (BilolixConfig, BilolixLayer, ChannelDeltaConfig, FadingConfig, GeluFFConfig, LoopConfig,
                                  MapAttentionConfig, PairTurn, SoftmaxMoEConfig)
    rng = random.Random(seed)

    def mlp():
        r = rng.random()
        if r < 0.15:
            return None
        if r < 0.5:
            return GeluFFConfig(rng.choice([8, 24, 40, 64, 200]))
        E = rng.choice([1, 2, 3, 5, 8, 12])
        return SoftmaxMoEConfig(E, rng.randint(1, min(4, E)), rng.choice([8, 12, 24, 40, 64]))

    def heads():
        G = rng.choice([1, 2, 3])
        return G * rng.choice([1, 2, 3, 4]), G

    layers = []
    for _ in range(rng.randint(2, 5)):
        kind = rng.choice(["attention", "gla", "channel_delta"])
        n, m = rng.choice([4, 8, 16, 32, 64]), rng.choice([4, 8, 24, 64])
        H, G = heads()
        if kind == "attention":
            d, vd = rng.choice([(6, 8), (16, 32), (32, 64), (24, 48), (64, 128), (32, 32), (48, 20)])
            dims = rng.choice([x for x in (0, 2, 6, 8, 16, 32, 64) if x <= d])
            rot = PairTurn(rng.choice([1e2, 1e4, 2.5e5]), dims) if dims else None
            mixer = MapAttentionConfig(H, G, d, vd, rng.choice([0.1, 0.2, 0.35]), rng.choice([0.0, 0.2, 0.5, 0.8]), rot,
                                       rng.choice([None, 1, 5, 16, 33, 64, 100]))
        elif kind == "gla":
            mixer = FadingConfig(rng.choice([1, 2, 3, 6]), n, m, rng.choice([1.0, 4.0, 16.0]), rng.choice([1, 3, 8, 16]))
        else:
            mixer = ChannelDeltaConfig(H, G, n, m, rng.choice([1, 2, 3, 4, 5]), rng.choice([1, 3, 8, 40]), rng.choice([2, 5, 16, 33]))
        layers.append(BilolixLayer(kind, mixer, mlp()))
    loop = None
    if rng.random() < 0.7:
        a = rng.randrange(len(layers))
        loop = LoopConfig(a, rng.randint(a + 1, len(layers)), rng.choice([1, 2, 3]))
    return BilolixConfig(vocab=rng.choice([97, 200, 333, 512]), width=rng.choice([64, 72, 96, 128, 160]),
                         norm_eps=rng.choice([1e-5, 1e-6, 1e-4]), max_position=512, layers=tuple(layers), loop=loop)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("seed", [71, 72, 73, 74, 75, 76])
def test_replay_of_configurations_drawn_at_random(seed, dtype, tmp_path):
    cfg = random_bilolix(seed)
    rng = random.Random(seed)
    model_dir = write_folder(str(tmp_path / "m"), cfg, seed, torch.float32 if dtype == "float32" else torch.bfloat16)
    lens = [rng.randint(1, 4), rng.randint(20, 60), rng.randint(70, 120), rng.randint(130, 180)]
    seqs = {f"s{i}": random_ids(n, cfg.vocab, seed * 10 + i) for i, n in enumerate(lens)}
    plain = R.Plain(model_dir, seqs, dtype)
    ways, big = four_ways(seqs, seed, tail=40)
    got, rc = R.run_trace(model_dir, dtype, str(tmp_path / "out"), big, cfg.vocab, extra=["--poison"])
    assert rc == 0
    for way in ways:
        mine = {k.split(".", 1)[1]: v for k, v in got.items() if k.startswith(way + ".")}
        assert {k: len(v) for k, v in mine.items()} == {k: len(v) for k, v in seqs.items()}, way
        check_rows(plain, mine, dtype, f"Bilolix drawn from {seed}, {way}")
