"""Vakesun on the GPU against the plain implementation: each kernel alone, each mixer and the side input alone (mixers with
their own cache: whole, token by token, in portions, in unequal batches, with pages and slots used again), the residual
stream after every layer, whole models replayed in the four ways of cutting, long decoding, and greedy generation through the
session, its scheduler and the command line.

Where random weights would hide a fault, the inputs are made so that it shows: one cached row is made to point along a query
(far back, on a page's first and last row, just inside and just outside a window) with sinks from negligible to dominant; a
memory that hardly forgets is given one key and, hundreds of tokens later, the query that meets it; gates run from keeping
almost nothing to keeping almost all, so that the running maximum is set by either.
"""
import math
import random

import pytest
import torch

import plain_vakesun as P
import replay as R
from test_gpu_kuditar import DEV, DTYPES, Pages, attention_case, check_rows, four_ways, gen, i32, renamed, starts_of, tol
from tiny import random_ids
from tiny_vakesun import CONFIGS, write_folder, write_tiny

pytestmark = pytest.mark.gpu

EPS = 1e-6


@pytest.fixture(scope="module")
def ops():
    from gesso_amd.kernels import ops
    ops.lib()
    return ops


@pytest.fixture(scope="module")
def folders(tmp_path_factory):
    return str(tmp_path_factory.mktemp("vakesun"))


# ------------------------------------------------------------------ kernels alone

@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("H", [96, 100, 7, 1030, 2048, 5000])
def test_the_pass_between_two_sub_layers(ops, dtype, H):
    """Every kind of norm on the output, every kind on what is read next, and none of either."""
    res, y = torch.randn(6, H, generator=gen(0)) * 3, (torch.randn(6, H, generator=gen(1)) * 4).to(dtype)
    w, b, w2, b2 = (torch.randn(H, generator=gen(2 + i)) for i in range(4))
    W = {"p": w.double(), "p.b": b.double(), "p.alpha": torch.tensor(0.4), "q": w2.double(), "q.b": b2.double(), "q.alpha": torch.tensor(0.9)}
    dev = lambda t: t.to(DEV)
    posts = {None: (None, lambda v: v), "rms": (ops.SeamNorm("rms", dev(w), eps=EPS), lambda v: P.rms(v, EPS) * w.double()),
             "dyt": (ops.SeamNorm("dyn_tanh", dev(w), dev(b), dev(torch.tensor([0.4]))), lambda v: P.dyt(v, W, "p"))}
    pres = {None: (None, lambda v: v), "rms": (ops.SeamNorm("rms", dev(w2), eps=EPS), lambda v: P.rms(v, EPS) * w2.double()),
            "dyt": (ops.SeamNorm("dyn_tanh", dev(w2), dev(b2), dev(torch.tensor([0.9]))), lambda v: P.dyt(v, W, "q"))}
    for post, fp in posts.values():
        for pre, fq in pres.values():
            r = res.clone().to(DEV)
            got = ops.norm_seam(r, y.to(DEV), post, 0.7, pre, dtype).cpu().double()
            x = res.double() + 0.7 * fp(y.double())
            assert float((r.cpu().double() - x).abs().max()) <= 4e-6 * max(1.0, float(x.abs().max()))
            want = fq(x)
            assert float((got - want).abs().max()) <= tol(dtype, want)
            # nothing is read next: the stream alone moves on
            r2 = res.clone().to(DEV)
            assert ops.norm_seam(r2, y.to(DEV), post, 0.7, None) is None and torch.equal(r2, r)
            # nothing is added, and chosen rows only: the stream stays
            r3 = res.clone().to(DEV)
            some = ops.norm_seam(r3, None, None, 1.0, pre, dtype, rows=i32([4, 0, 4])).cpu().double()
            want = fq(res.double())[[4, 0, 4]]
            assert float((some - want).abs().max()) <= tol(dtype, want) and torch.equal(r3.cpu(), res)


def test_a_row_whose_squares_overflow_is_not_a_number_after_the_pass(ops):
    y = torch.randn(2, 96, generator=gen(8))
    y[1] *= 1e25
    r = torch.zeros(2, 96, device=DEV)
    ops.norm_seam(r, y.to(DEV), ops.SeamNorm("rms", torch.ones(96, device=DEV), eps=EPS), 1.0, None)
    assert torch.isfinite(r[0]).all() and torch.isnan(r[1]).all()


@pytest.mark.parametrize("dtype", DTYPES)
def test_the_elementwise_norm_as_a_part(dtype):
    from gesso_amd.config import DynTanhSpec
    from gesso_amd.parts import ResidualStream, Runtime, build
    rt = Runtime(DEV, dtype)
    norm, other = build("norm", DynTanhSpec(100), rt), build("norm", DynTanhSpec(100), rt)
    W = {"n": torch.randn(100, generator=gen(9)), "n.b": torch.randn(100, generator=gen(10)), "n.alpha": torch.tensor(0.6)}
    for part in (norm, other):
        part.bind({"weight": W["n"].to(DEV), "bias": W["n.b"].to(DEV), "alpha": W["n.alpha"].to(DEV)})
    x, a, b = (torch.randn(5, 100, generator=gen(11 + i)) for i in range(3))
    for pend in (None, a.to(dtype), (a.to(dtype), None), (a.to(dtype), b.to(dtype))):
        on = tuple(None if t is None else t.to(DEV) for t in pend) if isinstance(pend, tuple) else None if pend is None else pend.to(DEV)
        s = ResidualStream(x.clone().to(DEV), pending=on)
        y = norm.add_norm(s)
        full = x.double() + sum(t.double() for t in (pend if isinstance(pend, tuple) else (pend,)) if t is not None)
        want = P.dyt(full, {k: v.double() for k, v in W.items()}, "n")
        assert s.pending is None and float((s.res.cpu().double() - full).abs().max()) <= 1e-5
        assert float((y.cpu().double() - want).abs().max()) <= tol(dtype, want)
    # rows that the last writer left for this norm are taken as they are; another norm makes its own
    s.normed, s.xs_for = y, norm
    assert norm.add_norm(s) is y
    assert other.add_norm(s) is not y


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("dim,width,H", [(12, 96, 96), (5, 64, 64), (7, 100, 100), (80, 128, 128), (200, 256, 256), (64, 512, 512)])
def test_a_tokens_own_input_alone(ops, dtype, dim, width, H):
    from gesso_amd.config import TokenSideSpec
    from gesso_amd.parts import Runtime, build, part_class
    from gesso_amd.weights import random_tensors
    from gesso_amd.weights.loader import held_dtype
    spec = TokenSideSpec(hidden=width, vocab=50, dim=dim, columns=3 * dim, offset=dim, eps=EPS)
    table = part_class("side", spec).tensor_specs(spec)
    w = random_tensors(table, 5, dtype, std=0.3)
    rt = Runtime(DEV, dtype)
    part = build("side", spec, rt)
    part.bind({k: v.to(DEV, held_dtype(v.dtype, table[k].role, dtype)) for k, v in w.items()})
    W = {"side.gate": w["gate.weight"].double(), "side.proj": w["proj.weight"].double(), "side.norm": w["norm.weight"].double()}

    class Ctx:
        pass

    for T in (1, 9, 70, 300):
        ids = random_ids(T, 50, T)
        x = torch.randn(T, width, generator=gen(20 + T)).to(dtype)
        ctx = Ctx()
        ctx.token_ids = i32(ids)
        y = part.forward(x.to(DEV), ctx)
        res = torch.randn(T, width, generator=gen(21))
        r = res.clone().to(DEV)
        ops.norm_seam(r, y, part.out_seam(), 0.7, None)
        e = w["table"].double()[ids, dim:2 * dim]
        want = res.double() + 0.7 * P.side_input(x.double(), W, "", e, EPS)
        assert float((r.cpu().double() - want).abs().max()) <= tol(dtype, want, 2e-5, 2e-2), T
    # the two products' spare columns are zeros whatever stands in the table beside this layer's columns
    z = torch.zeros(3, part.width, device=DEV) + 1.0
    g = ops.side_gate(z, part.table, i32([1, 2, 3]), dim, dim, part.width, dtype)
    assert float(g[:, dim:].abs().max() if part.width > dim else 0.0) == 0.0


@pytest.mark.parametrize("M,N,K", [(65, 16, 256), (300, 7, 1024), (70, 64, 96), (129, 40, 40), (2048, 32, 512), (1, 48, 8), (17, 33, 1000)])
def test_products_of_many_rows_with_few_outputs(ops, M, N, K):
    x, w = torch.randn(M, K + 8, generator=gen(30)).bfloat16(), (torch.randn(N, K, generator=gen(31)) / math.sqrt(K)).bfloat16()
    xd = x.to(DEV)[:, 8:] if K % 8 == 0 else x.to(DEV)
    want = x[:, 8:].double() @ w.double().T
    for out in (torch.float32, torch.bfloat16):
        got = ops.gemm_narrow(xd, w.to(DEV), out).cpu().double()
        assert float((got - want).abs().max()) <= (2e-5 if out == torch.float32 else 1e-2) * max(1.0, float(want.abs().max()))
    one = ops.gemm_narrow(xd[M // 2:M // 2 + 1], w.to(DEV))
    assert torch.equal(one[0], ops.gemm_narrow(xd, w.to(DEV))[M // 2])               # a row depends on nothing but the row


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("H,G,d,rd", [(4, 2, 96, 48), (3, 3, 64, 32), (2, 1, 96, 96), (2, 2, 24, 16), (5, 1, 40, 16), (4, 4, 128, 64), (2, 1, 256, 128),
                                      (3, 1, 64, 0), (2, 1, 16, 16), (2, 1, 10, 6), (2, 2, 96, 40)])
@pytest.mark.parametrize("normed", [True, False])
def test_cache_write_of_heads_turned_in_part(ops, dtype, H, G, d, rd, normed):
    from gesso_amd.config import ScaledRopeSpec
    from gesso_amd.parts.rope import scaled_rope_tables
    ps, T, start = 4, 23, 150
    sc = {"factor": 4.0, "original": 64.0, "fast": 8.0, "slow": 1.0}
    cos = sin = None
    if rd:
        cos, sin = (t.to(DEV) for t in scaled_rope_tables(ScaledRopeSpec(head_dim=d, rotary_dim=rd, theta=1e4, max_position=256, **sc)))
    x = (torch.randn(T, (H + 2 * G) * d, generator=gen(32)) * 2).to(dtype)
    qw, kw = (1 + 0.3 * torch.randn(d, generator=gen(33 + i)) for i in (0, 1))
    pos = [start + i for i in range(T)]
    pg = Pages(dtype, G, d, d, ps, [start + T], seed=1)
    xd = x.clone().to(DEV)
    ops.qknorm_rope_kv(xd, qw.to(DEV) if normed else None, kw.to(DEV) if normed else None, EPS, cos, sin, rd, i32(pos), i32([0] * T), pg.table,
                       ps, pg.k, pg.v, H, G, d)
    f, amp = P.yarn(rd, 1e4, sc) if rd else ([], 1.0)
    r = x.double()
    q, k, v = r[:, :H * d].reshape(T, H, d), r[:, H * d:(H + G) * d].reshape(T, G, d), r[:, (H + G) * d:].reshape(T, G, d)
    if normed:
        q, k = P.rms(q, EPS) * qw.double(), P.rms(k, EPS) * kw.double()
    q, k = P.rotate_half(q, pos, f, amp), P.rotate_half(k, pos, f, amp)
    out = xd.cpu().double()
    assert float((out[:, :H * d].reshape(T, H, d) - q).abs().max()) <= tol(dtype, q)
    assert torch.equal(out[:, H * d:], r[:, H * d:])                       # only q is rewritten in place
    table = pg.table[0].cpu().tolist()
    for t, p in enumerate(pos):
        page, row = table[p // ps], p % ps
        assert float((pg.k[page, :, row].double().cpu() - k[t]).abs().max()) <= tol(dtype, k)
        assert torch.equal(pg.v[page, :, row].double().cpu(), v[t])
    assert torch.isnan(pg.k[table[(start - 1) // ps], :, (start - 1) % ps]).all()     # nothing before the step's rows was written


@pytest.mark.parametrize("rows", [16, 32])
def test_heads_of_96_on_the_matrix_cores(ops, rows):
    """Prompt portions, single tokens behind them (the kernel for single queries, its keys split or not), groups of one to
    eight heads; one key that stands out far back and at page borders."""
    assert ops.attention_prefill_supports(8, 1, 96) and ops.attention_decode_supports(8, 1, 96)
    for nh, nkv, ps, window in ((1, 1, 8, None), (2, 1, 16, None), (3, 1, 4, 33), (8, 2, 16, None), (5, 1, 8, 64), (6, 1, 16, None), (7, 1, 16, None),
                                (8, 1, 8, 100)):
        if rows == 32 and nh // nkv > 4:
            continue
        lens = [230, 1, 97, 40]
        cuts = [[100, 64, 1, 33, 30, 1, 1], [1], [97], [2, 17, 1, 1, 17, 1, 1]]
        got, want = attention_case(ops, torch.bfloat16, nh, nkv, 96, 96, lens, cuts, ps=ps, window=window, seed=nh, tiled=rows)
        for s in range(len(lens)):
            assert float((got[s] - want[s]).abs().max()) <= tol(torch.bfloat16, want[s], 2e-5, 2e-2), (s, nh, nkv)
    T, query, ps = 340, 339, 16
    for place in (0, ps - 1, ps, query - 300, (query // ps) * ps - 1, query - 1):
        for cuts in ([[T]], [[query, 1]], [[query - 60] + [1] * 61], [[query - 70, 71]]):
            got, want = attention_case(ops, torch.bfloat16, 2, 1, 96, 96, [T], cuts, ps=ps, scale=1.0, seed=3, tiled=rows,
                                       plant=(0, place, query, 12.0))
            assert float((got[0] - want[0]).abs().max()) <= tol(torch.bfloat16, want[0], 2e-5, 2e-2), (place, cuts[0][:2])


# ------------------------------------------------------------------ latent rows with sinks

def latent_rows_case(ops, dtype, H, c, T, rows, window, ps, scale, sinks, seed, plant=None, cores=False, nsplit=1):
    """Queries in absorbed form over cached latent rows: the kernel's sums over the rows, and the plain attention's with the
    rows as keys and as values.  ``plant``: ``(row, size)``: that row points along the last query's first head."""
    g = gen(seed)
    z, qa = torch.randn(T, c, generator=g), torch.randn(T, H, c, generator=g)
    if plant is not None:
        q = qa[rows[-1], 0]
        z[plant[0]] = q / q.norm() * plant[1]
    z, qa = z.to(dtype), qa.to(dtype)
    pg = Pages(dtype, 1, c, 1, ps, [T], seed)
    table = pg.table[0].cpu().tolist()
    for t in range(T):
        pg.k[table[t // ps], 0, t % ps] = z[t].to(DEV)
    q = qa[rows].reshape(len(rows), H * c).contiguous().to(DEV)
    pos, sk = i32(rows), sinks.to(DEV)
    if cores:
        most, tiles, at = ops.attention_latent_mfma_tokens(H), [], 0
        while at < len(rows):
            n = 1
            while at + n < len(rows) and n < most and rows[at + n] == rows[at + n - 1] + 1:
                n += 1
            tiles.append((0, at, n))
            at += n
        tiles = torch.tensor(tiles, dtype=torch.int32).T.contiguous().to(DEV)
        if len(rows) == 1:
            tiles = None                                        # a step of single tokens
        o = ops.attention_latent_mfma(q, pg.k, pos, tiles, pg.table, ps, window, scale, H, c, 0, len(rows), nsplit=nsplit, sinks=sk)
    else:
        o = ops.attention_latent(q, pg.k, pos, i32([0] * len(rows)), pg.table, ps, window, scale, H, c, 0, len(rows), sinks=sk)
    zd, qd = z.double(), qa.double()
    want = torch.stack([P.softmax_head(qd[:, h], zd, zd, scale, window, sinks[h].double()) for h in range(H)], 1)[rows]
    return o.cpu().double().reshape(len(rows), H, c), want


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("H,c,window,ps", [(3, 48, 24, 8), (5, 36, 17, 16), (2, 32, None, 4), (4, 64, 40, 16), (1, 200, 1, 8), (16, 256, 100, 16),
                                           (6, 512, 65, 16), (70, 16, 30, 16)])
def test_latent_attention_with_a_sink_a_head(ops, dtype, H, c, window, ps):
    T = 150
    sinks = torch.linspace(-3.0, 4.0, H) if H > 1 else torch.tensor([1.5])
    for cores in ([False, True] if dtype == torch.bfloat16 and ops.attention_latent_mfma_supports(H, c, 0) else [False]):
        scale = 0.5 / math.sqrt(c)
        for rows in (list(range(T)), [0, 1, 2, 40, 41, 97, T - 2, T - 1]):
            got, want = latent_rows_case(ops, dtype, H, c, T, rows, window, ps, scale, sinks, 40, cores=cores)
            assert float((got - want).abs().max()) <= tol(dtype, want, 1e-5, 2e-2), (cores, len(rows))
        for nsplit in (1, 2, 5):
            got, want = latent_rows_case(ops, dtype, H, c, T, [T - 1], window, ps, scale, sinks, 40, cores=cores, nsplit=nsplit)
            assert float((got - want).abs().max()) <= tol(dtype, want, 1e-5, 2e-2), (cores, nsplit)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("window,ps", [(24, 8), (21, 8), (33, 16), (None, 16)])
def test_a_latent_row_that_stands_out_beside_a_sink(ops, dtype, window, ps):
    """A row that points along the query takes the weight if and only if the window lets the query see it; against a sink
    of the same score it takes half, against one far larger nothing."""
    T, H, c = 340, 2, 32
    query = T - 1
    edge = query - window + 1 if window else 0
    places = [query, query - 1, (query // ps) * ps, (query // ps) * ps - 1]
    places += [edge, edge + 1, edge - 1, edge - 2] if window else [query - 300, 0, ps - 1, ps]
    for place in places:
        base, _ = latent_rows_case(ops, torch.float32, H, c, T, [query], None, ps, 1.0, torch.tensor([-60.0, -60.0]), place, plant=(place, 40.0))
        for cores in ([False, True] if dtype == torch.bfloat16 else [False]):
            for sink in (-60.0, 5.0, 400.0):
                got, want = latent_rows_case(ops, dtype, H, c, T, [query - 5, query - 1, query], window, ps, 1.0, torch.tensor([sink, 0.0]), place,
                                             plant=(place, 40.0), cores=cores)
                assert float((got - want).abs().max()) <= tol(dtype, want, 2e-5, 2e-2), (place, cores, sink)
                seen = P.visible(query, place, window)
                size = float(got[2, 0].norm())
                assert (size > 30.0) == (seen and sink < 100.0), (place, cores, sink, size)
                if sink > 100.0:
                    assert size < 1e-3
    # a sink of the row's own score takes half of the weight
    q = torch.randn(T, c, generator=gen(99))
    z = torch.zeros(1, c)
    z[0] = q[0] / q[0].norm() * 6.0
    score = float((q[0].double() @ z[0].double()))
    one = P.softmax_head(q[:1].double(), z.double(), z.double(), 1.0, None, torch.tensor(score, dtype=torch.float64))
    assert torch.allclose(one[0], 0.5 * z[0].double())


# ------------------------------------------------------------------ the matrix memory

def plain_gate_rows(zi, zf, cap):
    """``(T, 3 H)``: what a memory keeps, with what it writes, the least it divides by, from the plain gates."""
    i, f = P.gates(zi.double(), zf.double(), cap)
    T, H = i.shape
    out = torch.zeros(T, 3 * H, dtype=torch.float64)
    for h in range(H):
        p = torch.zeros((), dtype=torch.float64)
        for t in range(T):
            new = torch.maximum(f[t, h] + p, i[t, h])
            out[t, h], out[t, H + h], out[t, 2 * H + h] = torch.exp(f[t, h] + p - new), torch.exp(i[t, h] - new), torch.exp(-new)
            p = new
    return out


@pytest.mark.parametrize("H,cap,spread", [(3, 15.0, 6.0), (1, 1.5, 3.0), (8, 30.0, 25.0), (5, 4.0, 0.5)])
def test_gates_and_their_running_maximum_over_unequal_sequences_and_any_cut(ops, H, cap, spread):
    lens = [1, 700, 64, 65, 2, 1300]
    z = [torch.randn(n, 2 * H + 5, generator=gen(50 + n)) * spread for n in lens]
    z[1][:, 2 + H:2 + 2 * H] += 4.0                                     # almost nothing forgotten
    z[5][:, 2 + H:2 + 2 * H] -= 3.0                                     # almost everything
    bi, bf = torch.randn(H, generator=gen(51)), torch.randn(H, generator=gen(52))
    want = [plain_gate_rows(r[:, 2:2 + H] + bi, r[:, 2 + H:2 + 2 * H] + bf, cap) for r in z]
    slots = [4, 0, 6, 2, 1, 5]
    for cuts in ([[n] for n in lens], [[1], [130, 1, 1, 300, 64, 204], [63, 1], [2, 63], [1, 1], [64, 600, 1, 635]]):
        peak = torch.full((8, H), float("nan"), device=DEV)
        peak[slots] = 0.0
        done, got, logs = [0] * len(lens), [[] for _ in lens], [[] for _ in lens]
        for step in range(max(len(c) for c in cuts)):
            live = [s for s in range(len(lens)) if step < len(cuts[s])]
            sizes = [cuts[s][step] for s in live]
            x = torch.cat([z[s][done[s]:done[s] + n] for s, n in zip(live, sizes)]).to(DEV)
            args = (x, 2, 2 + H, bi.to(DEV), bf.to(DEV), cap)
            at = (i32(starts_of(sizes)), i32([slots[s] for s in live]), len(live), H)
            kept = peak.clone()
            lg = ops.exp_gates(*args, kept, *at, longest=max(sizes), logs=True).cpu().double()
            g = ops.exp_gates(*args, peak, *at, longest=max(sizes)).cpu().double()
            assert torch.equal(kept[slots], peak[slots])
            a = 0
            for s, n in zip(live, sizes):
                got[s].append(g[a:a + n])
                logs[s].append(lg[a:a + n])
                a += n
                done[s] += n
        for s in range(len(lens)):
            g, lg = torch.cat(got[s]), torch.cat(logs[s])
            assert float((g - want[s]).abs().max() / max(1.0, float(want[s].abs().max()))) <= 2e-5, (s, cuts[s][:2])
            assert float((torch.exp2(lg[:, :2 * H]) - want[s][:, :2 * H]).abs().max()) <= 2e-5
            assert torch.equal(lg[:, 2 * H:], g[:, 2 * H:])
        assert torch.isnan(peak[[3, 7]]).all()


def memory_case(ops, dtype, H, n, m, lens, cuts, route, seed=0, segment=0, meet=None, slow=False):
    """A memory over sequences of ``lens`` tokens fed in the pieces ``cuts[s]``: gates, recurrence, and the divided, normed
    and gated outputs, states in shuffled slots.  ``route``: "scan" token by token (with ``segment`` in segments side by
    side), "steps" the same with the kernel for single tokens where a step brings nothing else, "cores" 32 tokens at a time
    on the matrix cores.  ``meet``: ``(t, u)``: one key of token ``t`` is met by the query
    of token ``u`` alone.  Returns the divided outputs' rows (with the gate at one half, no weight's effect) and the plain
    memory's, per sequence."""
    g = gen(seed)
    cols = 2 * H * n + 2 * H * m
    junk = 8
    q_scale = n ** -0.5
    xs, zs = [], []
    for L in lens:
        x, z = torch.randn(L, junk + cols, generator=g), torch.randn(L, 2 * H, generator=g) * 3.0
        z[:, H:] += torch.linspace(-2.0, 5.0, H)
        if slow:
            z[:, H:] = 9.0
            z[:, :H] *= 0.2
        x[:, junk + 2 * H * n + H * m:] = 0.0                              # the output's gate: one half
        if meet is not None and L > meet[1]:
            q, k = x[:, junk:junk + H * n].view(L, H, n), x[:, junk + H * n:junk + 2 * H * n].view(L, H, n)
            q[..., 0] = 0.0
            k[..., 0] = 0.0
            k[meet[0], :, 0] = 30.0                                        # one key along channel 0 ...
            q[meet[1]] = 0.0
            q[meet[1], :, 0] = 30.0                                        # ... and, later, the query along the same channel
        xs.append(x.to(dtype))
        zs.append(z)
    slots = torch.randperm(len(lens) + 2, generator=g)[:len(lens)].tolist()
    state = torch.full((len(lens) + 3, H, n, m + 1), float("nan"), device=DEV)
    peak = torch.full((len(lens) + 3, H), float("nan"), device=DEV)
    state[slots], peak[slots] = 0.0, 0.0
    zero, weight = torch.zeros(H, device=DEV), torch.ones(H * m, device=DEV)
    done, got = [0] * len(lens), [[] for _ in lens]
    for step in range(max(len(c) for c in cuts)):
        live = [s for s in range(len(lens)) if step < len(cuts[s])]
        sizes = [cuts[s][step] for s in live]
        cat = lambda parts: torch.cat([parts[s][done[s]:done[s] + k] for s, k in zip(live, sizes)]).to(DEV)
        x, z = cat(xs), cat(zs)
        starts, at = i32(starts_of(sizes)), i32([slots[s] for s in live])
        cores = route == "cores"
        gates = ops.exp_gates(z, 0, H, zero, zero, 15.0, peak, starts, at, len(live), H, longest=max(sizes), logs=cores)
        offs = (junk, junk + H * n, junk + 2 * H * n)
        den = None
        if route == "steps" and all(k == 1 for k in sizes):
            o, den = ops.memory_step(x, *offs, H, n, m, gates, state, at, q_scale=q_scale)
        elif cores:
            o, den = ops.memory_scan_chunks(x, *offs, H, n, m, gates, state, starts, at, sizes, q_scale=q_scale, segment=segment)
        else:
            kw = dict(q_scale=q_scale, beta=gates, ob=H, delta=False, ones=True)
            args = (x, *offs, H, H, n, m + 1, gates, 0, False, state)
            o = ops.gated_state_scan_segments(*args, sizes, at, segment, **kw) if segment else \
                ops.gated_state_scan(*args, starts, at, len(live), **kw)
        y = ops.memory_outnorm(o, den, gates, x, junk + 2 * H * n + H * m, weight, EPS, H, m, torch.float32)
        a = 0
        for s, k in zip(live, sizes):
            got[s].append(y[a:a + k].double().cpu())
            a += k
            done[s] += k
    want = []
    for s, L in enumerate(lens):
        x, z = xs[s].double(), zs[s].double()
        q, k, v = (x[:, o:o + w].reshape(L, H, -1) for o, w in ((junk, H * n), (junk + H * n, H * n), (junk + 2 * H * n, H * m)))
        i, f = P.gates(z[:, :H], z[:, H:], 15.0)
        want.append(torch.stack([P.rms(P.matrix_memory(q[:, h] * q_scale, k[:, h], v[:, h], i[:, h], f[:, h]), EPS) for h in range(H)], 1)
                    .reshape(L, H * m) * 0.5)
    spare = [s for s in range(state.shape[0]) if s not in slots]
    assert torch.isnan(state[spare]).all() and torch.isnan(peak[spare]).all()
    return [torch.cat(g_) for g_ in got], want


def near(got, want, bound):
    """Rows that are root-mean-square one apiece (a head divided by its own): the largest difference over a row's heads."""
    return float((got - want).abs().max()) <= bound * max(1.0, float(want.abs().max()))


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("H,n,m", [(4, 16, 24), (3, 8, 12), (2, 64, 128), (1, 128, 40), (5, 6, 14), (2, 14, 70), (1, 200, 33), (3, 32, 15)])
def test_the_memory_token_by_token_over_unequal_sequences_and_any_cut(ops, dtype, H, n, m):
    lens = [1, 23, 2, 41]
    pieces = [[1], [5, 1, 1, 2, 7, 3, 1, 3], [1, 1], [12, 9, 1, 17, 2]]
    for cuts in ([[1], [23], [2], [41]], pieces):
        got, want = memory_case(ops, dtype, H, n, m, lens, cuts, "scan", seed=n + m)
        for s in range(len(lens)):
            assert near(got[s], want[s], 1e-4), (s, cuts[s][:2])


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("H,n,m", [(4, 16, 24), (3, 8, 12), (2, 64, 128), (1, 128, 40), (5, 6, 14), (2, 13, 70), (1, 200, 33), (3, 32, 129), (2, 300, 8), (1, 1, 1)])
def test_the_memory_one_token_a_sequence(ops, dtype, H, n, m):
    """From nothing, and behind portions that the other kernels have walked."""
    if n <= 256:
        lens, cuts = [40, 23, 61], [[9] + [1] * 31, [23], [30] + [1] * 31]
        got, want = memory_case(ops, dtype, H, n, m, lens, cuts, "steps", seed=n + m)
        for s in range(len(lens)):
            assert near(got[s], want[s], 1e-4), s
    got, want = memory_case(ops, dtype, H, n, m, [30, 11], [[1] * 30, [1] * 11], "steps", seed=n + m + 1)
    for s in range(2):
        assert near(got[s], want[s], 1e-4), s


@pytest.mark.parametrize("H,n,m,seg", [(2, 64, 128, 128), (4, 16, 24, 64), (1, 40, 10, 32)])
def test_the_memory_in_segments_side_by_side(ops, H, n, m, seg):
    lens = [300, 1, 130, 64]
    for cuts in ([[300], [1], [130], [64]], [[150, 150], [1], [1, 128, 1], [64]]):
        got, want = memory_case(ops, torch.float32, H, n, m, lens, cuts, "scan", seed=n, segment=seg)
        for s in range(len(lens)):
            assert near(got[s], want[s], 2e-4), s


CHUNKS = [(4, 16, 24), (2, 64, 128), (1, 128, 256), (3, 32, 136), (2, 96, 64), (1, 200, 40), (2, 256, 8), (5, 8, 8), (2, 64, 264), (1, 24, 200)]


@pytest.mark.parametrize("H,n,m", CHUNKS)
@pytest.mark.parametrize("seg", [0, 32, 64, 128])
def test_the_memory_on_the_matrix_cores(ops, H, n, m, seg):
    """Runs of 32 tokens that begin and end anywhere, states carried over cuts of every size, single tokens among them."""
    lens = [330, 1, 97, 33, 32]
    for cuts in ([[330], [1], [97], [33], [32]], [[150, 1, 2, 64, 113], [1], [31, 33, 33], [1, 32], [8, 8, 8, 8]]):
        got, want = memory_case(ops, torch.bfloat16, H, n, m, lens, cuts, "cores", seed=n + m + seg, segment=seg)
        for s in range(len(lens)):
            # sixteen bits of every operand held in 32: a thousandth where sums nearly cancel
            assert near(got[s], want[s], 3e-3), (s, cuts[s][:2])


@pytest.mark.parametrize("route,dtype,bound", [("scan", torch.float32, 2e-4), ("steps", torch.float32, 2e-4), ("cores", torch.bfloat16, 3e-3)])
@pytest.mark.parametrize("cuts,seg", [([[420]], 0), ([[420]], 128), ([[40] + [1] * 380], 0), ([[200, 220]], 64)])
def test_a_memory_keeps_what_it_was_given_hundreds_of_tokens_before(ops, route, dtype, bound, cuts, seg):
    """Nothing else has a share in the channel that the late query asks for: what it finds is the one value, 380 tokens old."""
    H, n, m = 2, 16, 24
    got, want = memory_case(ops, dtype, H, n, m, [420], cuts, route, seed=7, slow=True, meet=(20, 400), segment=seg)
    assert near(got[0], want[0], bound)
    quiet, _ = memory_case(ops, dtype, H, n, m, [420], cuts, route, seed=7, slow=True, segment=seg)
    assert float((got[0][400] - quiet[0][400]).abs().max()) > 0.3
    v = want[0][400].reshape(H, m)
    assert float(((v * v).mean(-1).sqrt() - 0.5).abs().max()) < 1e-2          # a whole value, not a remainder that eps swallows


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("H,m", [(3, 24), (4, 128), (5, 6), (1, 700)])
def test_divided_normed_and_gated_outputs(ops, dtype, H, m):
    T = 7
    o, gates = torch.randn(T, H * (m + 1), generator=gen(70)) * 3, torch.rand(T, 3 * H, generator=gen(71)) * 2
    rows, w = torch.randn(T, H * m + 10, generator=gen(72)).to(dtype), 1 + 0.2 * torch.randn(H * m, generator=gen(73))
    od = o.double().reshape(T, H, m + 1)
    u = od[..., :m] / (torch.maximum(od[..., m].abs(), gates[:, 2 * H:].double()) + 1e-6)[..., None]
    want = P.rms(u, EPS).reshape(T, H * m) * w.double() * torch.sigmoid(rows[:, 10:].double())
    got = ops.memory_outnorm(o.to(DEV), None, gates.to(DEV), rows.to(DEV), 10, w.to(DEV), EPS, H, m, dtype).cpu().double()
    assert float((got - want).abs().max()) <= tol(dtype, want)
    apart = o.reshape(T, H, m + 1)
    got = ops.memory_outnorm(apart[..., :m].reshape(T, H * m).contiguous().to(DEV), apart[..., m].contiguous().to(DEV), gates.to(DEV),
                             rows.to(DEV), 10, w.to(DEV), EPS, H, m, dtype).cpu().double()
    assert float((got - want).abs().max()) <= tol(dtype, want)


@pytest.mark.parametrize("dtype", DTYPES)
def test_the_square_of_relu(ops, dtype):
    for F in (96, 7):
        x = (torch.randn(5, F, generator=gen(74)) * 3).to(dtype)
        got = ops.activate(x.to(DEV), "relu_squared", dtype).cpu().double()
        want = torch.relu(x.double()) ** 2
        assert float((got - want).abs().max()) <= tol(dtype, want)


# ------------------------------------------------------------------ mixers alone

ATT = {"q_proj.weight": "q", "k_proj.weight": "k", "v_proj.weight": "v", "q_norm.weight": "q.norm", "k_norm.weight": "k.norm", "out_proj.weight": "o"}
MEMORY = {"q_proj.weight": "q", "k_proj.weight": "k", "v_proj.weight": "v", "gate_proj.weight": "g", "input_gate.weight": "i", "input_gate.bias": "i.b",
          "forget_gate.weight": "f", "forget_gate.bias": "f.b", "out_norm.weight": "norm", "out_proj.weight": "o"}
LATENT = {"q_down.weight": "dq", "q_norm.weight": "dq.norm", "q_up.weight": "uq", "kv_down.weight": "dkv", "kv_norm.weight": "dkv.norm",
          "k_up.weight": "uk", "v_up.weight": "uv", "sinks": "sink", "gate.weight": "g", "out.weight": "o"}


def mixer_harness(kind, dtype, W=96, page_size=8, num_pages=64, seed=11, **kw):
    """A mixer of the design with its cache, and the plain function of the same tensors."""
    from test_gpu_kuditar import _harness
    from gesso_amd.config import AttentionSpec, LatentAttentionSpec, MatrixMemorySpec, NoPositionSpec, RMSNormSpec, ScaledRopeSpec
    g = gen(seed)
    if kind == "attention":
        H, G, d, vd, rd = kw.get("H", 4), kw.get("G", 2), kw.get("d", 24), kw.get("vd", 16), kw.get("rd", 16)
        sc = kw.get("scaling", {"factor": 4.0, "original": 64.0, "fast": 8.0, "slow": 1.0})
        pos = ScaledRopeSpec(head_dim=d, rotary_dim=rd, theta=1e4, max_position=1024, **(sc or {})) if rd else NoPositionSpec()
        spec = AttentionSpec(hidden=W, n_heads=H, n_kv_heads=G, head_dim=d, value_dim=vd, position=pos, qk_norm=RMSNormSpec(d, EPS), scale=0.4)
        h = _harness(spec, dtype, seed, page_size, num_pages, {})
        w = renamed(h.tensors, ATT, "m.")
        m = {"heads": H, "kv_heads": G, "dim": d, "vdim": vd, "scale": 0.4, "rot": {"base": 1e4, "dims": rd, "scaling": sc} if rd else None}
        return h, lambda x: P.attention(x.double(), w, "m.", m, range(x.shape[0]), EPS)
    if kind == "memory":
        H, n, m_, cap = kw.get("H", 4), kw.get("n", 16), kw.get("m", 24), kw.get("cap", 15.0)
        spec = MatrixMemorySpec(hidden=W, n_heads=H, key_dim=n, value_dim=m_, gate_cap=cap, eps=EPS)
        sharp = {"forget_gate.bias": torch.linspace(-2.0, 6.0, H), "input_gate.bias": torch.rand(H, generator=g) * 6 - 3}
        h = _harness(spec, dtype, seed, page_size, num_pages, sharp)
        w = renamed(h.tensors, MEMORY, "m.")
        # a head's output is divided by its own root mean square: where its products with the query all but cancel (at the
        # first token, where key and query are nearly at right angles), their sign is the roundings'
        store = P.to_bfloat16 if dtype == torch.bfloat16 else P._keep
        return h, lambda x: P.mlstm(x.double(), w, "m.", {"heads": H, "dim": n, "vdim": m_, "gate_cap": cap}, EPS, store)
    H, n, dv, qr, c, window = kw.get("H", 4), kw.get("n", 16), kw.get("dv", 20), kw.get("qr", 24), kw.get("c", 32), kw.get("window", 21)
    spec = LatentAttentionSpec(hidden=W, n_heads=H, plain_dim=n, rot_dim=0, value_dim=dv, q_rank=qr, kv_rank=c, scale=0.5, eps=EPS,
                               position=NoPositionSpec(), window=window, sinks=True)
    h = _harness(spec, dtype, seed, page_size, num_pages, {"sinks": torch.linspace(-2.0, 3.0, H)})
    w = renamed(h.tensors, LATENT, "m.")
    m = {"heads": H, "dim": n, "vdim": dv, "scale": 0.5, "mask": {"size": window} if window else None}
    return h, lambda x: P.latent_attention(x.double(), w, "m.", m, EPS, P.latent(x.double(), w, "m.", EPS))


def agree(got, want, bound, kind, dtype):
    """Every row within the bound; for memories in bfloat16 all but a few (see :func:`mixer_harness`)."""
    off = (got - want).abs().amax(-1) > bound
    few = 0.06 if kind == "memory" and dtype == torch.bfloat16 else 0.0
    assert bool(torch.isfinite(got).all()) and float(off.double().mean()) <= few, (int(off.sum()), off.nonzero().flatten()[:8].tolist())


CASES = [("attention", dict()), ("attention", dict(W=64, H=3, G=3, d=10, vd=22, rd=6)), ("attention", dict(W=64, H=2, G=1, d=12, vd=12, rd=0)),
         ("attention", dict(W=128, H=4, G=1, d=96, vd=96, rd=48, page_size=16)), ("attention", dict(W=128, H=4, G=2, d=64, vd=64, rd=64, scaling=None)),
         ("attention", dict(W=128, H=6, G=1, d=32, vd=32, rd=16)),
         ("memory", dict()), ("memory", dict(W=64, H=2, n=24, m=8, cap=1.5)), ("memory", dict(W=128, H=2, n=64, m=128, cap=8.0)),
         ("memory", dict(W=100, H=5, n=10, m=6, cap=4.0)), ("memory", dict(W=128, H=1, n=128, m=72)),
         ("latent", dict()), ("latent", dict(W=64, H=3, n=12, dv=8, qr=16, c=36, window=None)), ("latent", dict(W=64, H=1, n=8, dv=4, qr=8, c=20, window=1)),
         ("latent", dict(W=128, H=4, n=32, dv=32, qr=64, c=64, window=32, page_size=16)), ("latent", dict(W=128, H=8, n=16, dv=64, qr=32, c=128, window=40))]


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("kind,kw", CASES)
def test_mixers_whole_token_by_token_in_portions_and_in_batches(dtype, kind, kw):
    h, plain = mixer_harness(kind, dtype, **kw)
    W, T = kw.get("W", 96), 90
    x = torch.randn(T, W, generator=gen(60)).to(dtype)
    want = plain(x)
    bound = tol(dtype, want, 5e-5, 3e-2)
    agree(h.mixer(x, [("whole", T)]), want, bound, kind, dtype)
    # most of it at once, the rest token by token across the window's edge; the first tokens one by one
    got = [h.mixer(x[:40], [("tail", 40)])] + [h.mixer(x[i:i + 1], [("tail", 1)]) for i in range(40, T)]
    agree(torch.cat(got), want, bound, kind, dtype)
    got = [h.mixer(x[i:i + 1], [("first", 1)]) for i in range(6)]
    agree(torch.cat(got), want[:6], bound, kind, dtype)
    at, got = 0, []
    for size in (2, 7, 2, 13, 3, 16, 5, 2, 31, 9):
        got.append(h.mixer(x[at:at + size], [("cut", size)]))
        at += size
    assert at == T
    agree(torch.cat(got), want, bound, kind, dtype)
    for rid in ("whole", "tail", "first", "cut"):
        h.manager.release(rid)
    # unequal requests side by side: a single token of one, a portion of another, a whole short one
    y, u = torch.randn(30, W, generator=gen(61)).to(dtype), torch.randn(5, W, generator=gen(62)).to(dtype)
    h.mixer(y[:29], [("b", 29)])
    h.mixer(x[:50], [("a", 50)])
    out = h.mixer(torch.cat([y[29:30], x[50:70], u]), [("b", 1), ("a", 20), ("c", 5)])
    agree(out[:1], plain(y)[29:30], bound, kind, dtype)
    agree(out[1:21], want[50:70], bound, kind, dtype)
    agree(out[21:], plain(u), bound, kind, dtype)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("kind,kw", [("memory", dict()), ("memory", dict(W=128, H=2, n=64, m=128)), ("latent", dict(W=128, H=4, n=32, dv=32, c=64, window=200)),
                                     ("attention", dict(W=128, H=4, G=1, d=96, vd=96, rd=48, page_size=16))])
def test_mixers_with_long_portions(dtype, kind, kw):
    """A prompt of several segments whole; the same in two long portions and single tokens; a long portion of one request
    beside a single token of another."""
    h, plain = mixer_harness(kind, dtype, num_pages=256, **kw)
    W, T = kw.get("W", 96), 640
    x = torch.randn(T, W, generator=gen(63)).to(dtype)
    want = plain(x)
    bound = tol(dtype, want, 5e-5, 3e-2)
    agree(h.mixer(x, [("whole", T)]), want, bound, kind, dtype)
    got = [h.mixer(x[:300], [("cut", 300)]), h.mixer(x[300:301], [("cut", 1)]), h.mixer(x[301:630], [("cut", 329)])]
    got += [h.mixer(x[i:i + 1], [("cut", 1)]) for i in range(630, T)]
    agree(torch.cat(got), want, bound, kind, dtype)
    h.manager.release("whole")
    h.manager.release("cut")
    y = torch.randn(30, W, generator=gen(64)).to(dtype)
    h.mixer(y[:29], [("b", 29)])
    h.mixer(x[:130], [("a", 130)])
    out = h.mixer(torch.cat([y[29:30], x[130:500]]), [("b", 1), ("a", 370)])
    agree(out[:1], plain(y)[29:30], bound, kind, dtype)
    agree(out[1:], want[130:500], bound, kind, dtype)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("kind,kw", [("attention", dict()), ("attention", dict(H=4, G=2, d=32, vd=32, rd=16)), ("memory", dict()), ("latent", dict()),
                                     ("latent", dict(window=None, c=64))])
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
        agree(torch.cat(got), want, tol(dtype, want, 5e-5, 3e-2), kind, dtype)
        h.manager.release(i)
        for pool in h.storage.keys + h.storage.values:
            pool[:, :-1].fill_(float("nan"))
        for pool, _ in h.storage.state_pools:
            pool[:, :-1].fill_(float("nan"))


def test_a_mixer_without_rows_of_its_own_refuses_a_cache_of_its_own():
    from gesso_amd.config import LatentAttentionSpec, NoPositionSpec
    from gesso_amd.errors import InvalidPlan
    from test_gpu_parts import Harness
    spec = LatentAttentionSpec(hidden=64, n_heads=2, plain_dim=8, rot_dim=0, value_dim=8, q_rank=16, kv_rank=16, scale=0.4, eps=EPS,
                               position=NoPositionSpec(), window=5, sinks=True, own_rows=False)
    h = Harness("mixer", spec, torch.float32, seed=1)
    with pytest.raises(InvalidPlan):
        h.mixer(torch.randn(3, 64), [("a", 3)])


# ------------------------------------------------------------------ whole models

LENGTHS = {"A": (1, 23, 70, 130), "B": (2, 40, 77), "C": (5, 64, 150, 300), "D": (3, 52, 110)}


def sequences(name):
    cfg, seed = CONFIGS[name]
    return {f"s{i}": random_ids(n, cfg.vocab, 100 * seed + i) for i, n in enumerate(LENGTHS[name])}


@pytest.mark.parametrize("name", ["A", "B", "D"])
def test_the_residual_stream_after_every_layer(name, folders):
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
            assert stream.pending is None
            got.append(stream.res.double().cpu())
        b.forward = wrapped
    eng.add_request("r")
    eng.step([StepEntry("r", ids[:29], [])])
    first = list(got)
    got.clear()
    eng.step([StepEntry("r", ids[29:], [])])
    assert len(first) == len(got) == len(want) == len(cfg.layers)
    for i, w in enumerate(want):
        mine = torch.cat([first[i], got[i]])
        assert float((mine - w).abs().max()) <= 3e-5 * max(1.0, float(w.abs().max())), f"layer {i}"


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
        check_rows(plain, mine, dtype, f"Vakesun {name} {way}")


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", ["A", "D"])
def test_long_decoding_token_by_token(name, dtype, folders, tmp_path):
    """A short prompt, then two hundred tokens one by one: memories carried, windows passed and pages begun and given back
    many times over, one layer's rows kept for another whose window is wider."""
    cfg, seed = CONFIGS[name]
    model_dir = write_tiny(folders, name, torch.float32 if dtype == "float32" else torch.bfloat16)
    seqs = {"long": random_ids(230, cfg.vocab, 7000 + seed), "other": random_ids(201, cfg.vocab, 7100 + seed)}
    plain = R.Plain(model_dir, seqs, dtype)
    got, rc = R.run_trace(model_dir, dtype, str(tmp_path / "out"), R.trace_tail(seqs, tail=200), cfg.vocab)
    assert rc == 0 and {k: len(v) for k, v in got.items()} == {"long": 230, "other": 201}
    check_rows(plain, got, dtype, f"Vakesun {name}, 200 tokens one by one")


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
        check_rows(plain, got, dtype, f"Vakesun {name}, pages of 8, poisoned, {way}")


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


def test_the_command_line_serves_a_vakesun_folder(folders):
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


@pytest.mark.parametrize("count", [40, 70])
def test_many_requests_at_once_decode_together(count, folders):
    """As many as the fused decode loop takes, and more than its products take rows."""
    from gesso_amd import Session
    from noise import supported
    cfg, _ = CONFIGS["C"]
    model_dir = write_tiny(folders, "C", torch.bfloat16)
    pc, pw = P.read_config(model_dir), P.read_weights(model_dir)
    prompts = [random_ids(3 + (7 * i) % 40, cfg.vocab, 2000 + i) for i in range(count)]
    session = Session(model_dir, dtype="bfloat16", device=DEV, context_length=128, max_num_seqs=count)
    try:
        got = session.generate(prompts, max_new_tokens=10)
        alone = session.generate([prompts[0]], max_new_tokens=10)[0]
    finally:
        session.close()
    assert [len(g_) for g_ in got] == [len(p) + 10 for p in prompts]
    for p, ids in ((prompts[0], got[0]), (prompts[17], got[17]), (prompts[count - 1], got[count - 1]), (prompts[0], alone)):
        lg = P.forward(pc, pw, ids).numpy()
        assert all(supported(lg[j - 1], ids[j], 0.5) for j in range(len(p), len(ids)))


def test_recorded_decode_steps_replay_what_was_launched(folders):
    """The recorded step several times over, with launched steps of the same engine in between: the same tokens as the
    same requests fed token by token through launched steps."""
    from gesso_amd.engine.batch import StepEntry
    from gesso_amd.engine.decode import DecodeLoop
    from gesso_amd.engine.engine import Engine
    cfg, seed = CONFIGS["A"]
    model_dir = write_tiny(folders, "A", torch.bfloat16)
    eng = Engine.from_folder(model_dir, dtype="bfloat16", device=DEV, page_size=16, max_tokens=2048, num_slots=8)
    prompts = [random_ids(n, cfg.vocab, 300 + n) for n in (30, 7, 51)]
    out = {}
    for kind in ("recorded", "launched"):
        rids, first = [], []
        for i, p in enumerate(prompts):
            rid = (kind, i)
            eng.add_request(rid)
            rids.append(rid)
            first.append(int(eng.step([StepEntry(rid, p, [len(p) - 1])])[0].argmax()))
        rows = [first]
        if kind == "recorded":
            loop = DecodeLoop(eng, rids, first)
            for n in (5, 1, 11, 3):
                rows += loop.run(n)
                eng.add_request("between")
                eng.step([StepEntry("between", prompts[0][:9], [8])])
                eng.step([StepEntry("between", [3], [0])])
                eng.finish_request("between")
        else:
            for _ in range(20):
                lg = eng.step([StepEntry(r, [t], [0]) for r, t in zip(rids, rows[-1])])
                rows.append(lg.argmax(1).tolist())
        for r in rids:
            eng.finish_request(r)
        out[kind] = rows
    assert eng.model.graph_safe
    # (the fused and the launched step may round differently where two logits nearly tie: the tokens up to there agree)
    from noise import supported
    pc, pw = P.read_config(model_dir), P.read_weights(model_dir)
    assert len(out["recorded"]) == len(out["launched"]) == 21
    for i, p in enumerate(prompts):
        ids = list(p) + [row[i] for row in out["recorded"]]
        lg = P.forward(pc, pw, ids).numpy()
        assert all(supported(lg[j - 1], ids[j], 0.5) for j in range(len(p), len(ids)))
    same = sum(a == b for a, b in zip(out["recorded"], out["launched"]))
    assert same >= 1


def random_vakesun(seed: int):
    """A configuration drawn from a seed: two to six layers of the three kinds in any order, latent layers that read an
    earlier one's rows, turns whole, in part or none, windows, feed-forwards or none, sizes with and without whole tiles."""
    from tiny_vakesun import attention, latent, memory
    from gesso_amd.config import VakesunConfig
    rng = random.Random(seed)
    layers, own = [], []
    for i in range(rng.randint(2, 6)):
        kind = rng.choice(["attention", "memory", "latent"])
        ff = rng.choice([None, 8, 24, 40, 64, 200])
        G = rng.choice([1, 2, 3])
        H = G * rng.choice([1, 2, 3, 4])
        if kind == "attention":
            d = rng.choice([6, 16, 24, 32, 64, 96])
            vd = rng.choice([d, d, d, 8, 20])
            dims = rng.choice([x for x in (0, 2, 6, 16, 32, 48, 64, 96) if x <= d])
            scaling = rng.choice([None, (2.0, 64.0, 16.0, 1.0), (8.0, 32.0, 32.0, 0.5)])
            layers.append(attention(H, G, d, vd, rng.choice([0.1, 0.2, 0.4]), ff, rng.choice([1e2, 1e4, 5e5]), dims, scaling))
        elif kind == "memory":
            layers.append(memory(rng.choice([1, 2, 3, 6]), rng.choice([4, 8, 16, 32, 64, 100]), rng.choice([4, 8, 24, 64, 130]),
                                 rng.choice([1.0, 4.0, 15.0, 40.0]), ff))
        else:
            src = rng.choice(own) if own and rng.random() < 0.6 else None
            c = layers[src].mixer.kv_rank if src is not None else rng.choice([16, 20, 32, 64, 96])
            if src is None:
                own.append(i)
            layers.append(latent(H, rng.choice([4, 8, 16, 32]), rng.choice([4, 12, 32, 64]), rng.choice([0.2, 0.5]), rng.choice([8, 20, 64]), c, ff,
                                 rng.choice([None, 1, 5, 16, 33, 64, 100]), src))
    return VakesunConfig(vocab=rng.choice([97, 200, 333, 512]), width=rng.choice([64, 72, 96, 128, 160]), layers=tuple(layers),
                         embedding_scale=rng.choice([1.0, 3.0, 12.0]), norm_eps=rng.choice([1e-5, 1e-6, 1e-4]),
                         residual_mult=rng.choice([0.3, 0.7, 1.0]), side_dim=rng.choice([3, 8, 33, 64, 70]), max_position=512)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("seed", [81, 82, 83, 84, 85, 86])
def test_replay_of_configurations_drawn_at_random(seed, dtype, tmp_path):
    cfg = random_vakesun(seed)
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
        check_rows(plain, mine, dtype, f"Vakesun drawn from {seed}, {way}")
