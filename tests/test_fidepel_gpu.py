"""Fidepel on the GPU: every kernel of its path, in bfloat16 and float32,
against the plain implementation of fidepel_oracle."""
import pytest
import torch

import fidepel_oracle as O
import fidepel_util as U
from llmlb_amd.backend.ragged import RaggedBatch
from llmlb_amd.backend.sampler import SamplingParams
from llmlb_amd.ops import hybrid as hy
from llmlb_amd.ops.reference import build_cos_sin_table
from test_fidepel_cpu import greedy_oracle, oracle

pytestmark = pytest.mark.gpu
DEV = "cuda:0"
F32, B16 = torch.float32, torch.bfloat16
DTYPES = pytest.mark.parametrize("dtype", [B16, F32], ids=["bf16", "f32"])
NAMES = pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
# rms logit error over the logits' spread
LOGIT_TOL = {"float32": 1e-4, "bfloat16": 0.1}


@pytest.fixture(scope="module", params=["ODD", "TILED", "PLAIN"])
def model(request, tmp_path_factory):
    cfg = getattr(U, request.param)
    w = U.weights(cfg, seed=len(request.param))
    return cfg, w, U.write_model(tmp_path_factory.mktemp(request.param),
                                 cfg, w)


@pytest.fixture(scope="module")
def plain(tmp_path_factory):
    cfg = U.PLAIN
    w = U.weights(cfg, seed=3)
    return cfg, w, U.write_model(tmp_path_factory.mktemp("plain"), cfg, w)


def close(got, want, dtype, rel=None):
    """Largest difference over the largest value."""
    rel = rel or (2e-2 if dtype == B16 else 2e-5)
    err = (got.double().cpu() - want).abs().max() / want.abs().max()
    assert err < rel, float(err)


# -- whole models ----------------------------------------------------------

@NAMES
def test_prompt_portions_and_decoding(model, dtype):
    cfg, w, folder = model
    toks = U.tokens(150, cfg["vocab"], 1)
    want = oracle(toks, w, cfg)
    eng = U.engine(folder, DEV, dtype)
    for cuts in ([], range(1, 150), range(2, 150, 2), range(9, 150, 9),
                 range(64, 150, 17), [140] + list(range(141, 150))):
        err = U.clear_error(U.run_cuts(eng, toks, cuts), *want, dtype)
        assert err < LOGIT_TOL[dtype], (cuts, err)
    assert eng._graphs and eng.use_graphs, "decode steps were not captured"


@NAMES
def test_unequal_batches_alone_and_together(model, dtype):
    """Every request's logits in mixed batches with reused pages and
    slots are those of the request alone."""
    cfg, w, folder = model
    eng = U.engine(folder, DEV, dtype, blocks=22, rows=4)
    reqs = [U.tokens(n, cfg["vocab"], 30 + n)
            for n in (1, 70, 2, 23, 80, 17, 66, 40)]
    want = [oracle(t, w, cfg) for t in reqs]
    free = eng.kv.free_blocks()
    got = U.serve_at_random(eng, reqs, 4, (1, 1, 2, 5, 16, 19, 33))
    assert eng.kv.free_blocks() == free
    for i, rows in got.items():
        if U.clear_rows(want[i][1], dtype).float().mean() > 0.3:
            assert U.clear_error(rows, *want[i], dtype) \
                < LOGIT_TOL[dtype], i


@NAMES
def test_long_decoding(plain, dtype):
    cfg, w, folder = plain
    toks = U.tokens(400, cfg["vocab"], 8)
    eng = U.engine(folder, DEV, dtype)
    got = U.run_cuts(eng, toks, range(3, 400))
    assert U.clear_error(got, *oracle(toks, w, cfg), dtype) \
        < LOGIT_TOL[dtype]


def test_captured_steps_match_eager_steps(model):
    """Replays with other work and synchronizations between them; batch
    sizes that pad their bucket."""
    cfg, _, folder = model
    engines = [U.engine(folder, DEV, "bfloat16", rows=6) for _ in range(2)]
    engines[1].use_graphs = False
    seqs = [[e.open_sequence() for _ in range(5)] for e in engines]
    for e, ss in zip(engines, seqs):
        for n, s in enumerate(ss):
            e.run_batch([(s, U.tokens(7 * n + 3, cfg["vocab"], n), [])])
    worst = []
    for step in range(8):
        live = range(step % 2, 5 - step % 3)
        res = []
        for e, ss in zip(engines, seqs):
            res.append(e.run_batch(
                [(ss[i], U.tokens(1, cfg["vocab"], 50 * step + i), [0])
                 for i in live]).clone())
            e.run_batch([(ss[4], [step, step + 1], [])])
            torch.cuda.synchronize()
        worst += ((res[0] - res[1]).abs().amax(-1) / res[1].std()).tolist()
    # matrix products of other heights may round a close choice of
    # experts to the other side
    assert sorted(worst)[int(0.9 * len(worst))] < 0.05, worst
    assert engines[0]._graphs and not engines[1]._graphs


@NAMES
def test_captured_steps_with_lists_of_experts(plain, dtype, monkeypatch):
    """Decode steps that build experts' lists, replayed several times."""
    monkeypatch.setattr(hy, "FEW_PAIRS", 0)
    cfg, w, folder = plain
    toks = U.tokens(40, cfg["vocab"], 18)
    eng = U.engine(folder, DEV, dtype, rows=3)
    other = eng.open_sequence()
    want = oracle(toks, w, cfg)
    seq, got = eng.open_sequence(), []
    for t in toks:
        got.append(eng.run_batch([(seq, [t], [0])]).cpu().double())
        eng.run_batch([(other, U.tokens(3, cfg["vocab"], t), [])])
        torch.cuda.synchronize()
    assert eng._graphs
    assert U.clear_error(torch.cat(got), *want, dtype) < LOGIT_TOL[dtype]


def test_greedy_generation(plain):
    cfg, w, folder = plain
    eng = U.engine(folder, DEV, "float32", blocks=40, rows=3,
                   prefill_step_budget=24)
    prompts = [U.tokens(n, cfg["vocab"], n) for n in (5, 60, 1, 31)]
    want = [greedy_oracle(w, cfg, p, 6) for p in prompts]
    queues = [eng.submit(p, SamplingParams(max_new_tokens=6))[1]
              for p in prompts]
    for _ in range(200):
        if not eng.step():
            break
    for q, expect in zip(queues, want):
        assert [q.get_nowait()[0] for _ in range(q.qsize())] == expect
    assert eng.kv.free_blocks() == eng.kv.num_blocks - 1


def test_preset_and_embeddings():
    from llmlb_amd.backend.launcher import build_engine
    eng = build_engine("fidepel-tiny", DEV, kv_blocks=64, max_batch=4)
    assert len(eng.generate_sync(list(range(40)), 5).token_ids) == 5
    h = eng.model.forward_dense(torch.tensor([[1, 2, 3]] * 2, device=DEV))
    assert torch.equal(h[0], h[1]) and h.isfinite().all()


# -- windowed attention alone ----------------------------------------------

# heads, kv_heads, dim, vdim, window, rotated: every tile shape with and
# without a remainder; more than 16 and more than 128 heads to a key/value
# head; whole, partial and no rotation; sizes only the general kernel takes
ATTENTION = [
    (2, 1, 32, 64, 70, 32), (3, 3, 24, 128, 64, 16), (2, 2, 16, 256, 33, 0),
    (8, 2, 64, 64, None, 64), (4, 1, 40, 96, 129, 32), (2, 1, 64, 200, 90, 48),
    (2, 2, 96, 40, 128, 96), (2, 1, 80, 128, 65, 16), (1, 1, 88, 256, 150, 88),
    (2, 1, 128, 64, 100, 128), (3, 1, 112, 128, 77, 64),
    (2, 2, 104, 136, 81, 64), (2, 1, 256, 64, 45, 128),
    (1, 1, 136, 128, 63, 16), (1, 1, 192, 256, 16, 192),
    (8, 8, 8, 8, 17, 8), (17, 1, 16, 24, 50, 16), (40, 2, 8, 40, None, 0),
    (130, 1, 8, 16, 40, 0), (6, 2, 7, 9, 31, 6), (2, 1, 264, 16, 80, 32),
    (2, 2, 24, 300, 96, 24), (1, 1, 20, 600, 48, 12), (4, 2, 12, 20, 1, 4),
    (10, 2, 16, 32, 2, 16),
]


@pytest.mark.parametrize("sizes", ATTENTION, ids=str)
@DTYPES
def test_attention_planted(sizes, dtype):
    """Scores that stand out at the window's edges, at page and tile
    borders, at the first tokens and just after the query; whole, in
    portions, and decoded."""
    H, G, D, V, window, rot = sizes
    m = U.attention(H, G, D, V, window, rot, base=3e3, factor=1.5,
                    scale=9.0 / D)
    T, width = 210, U.planted_width(m)
    w = U.attention_case(m, width, H + G + D + V)
    h = U.plant(m, w, U.inputs(T, width, 3), U.edge_pairs(window, T))
    want = O.attention(h, w, "", m, 1e-5)
    run = U.MixerRun(U.mixer(m, w, 1e-5, width, DEV, dtype), 2, T)
    for cuts in ([], [130, 132, 135] + list(range(136, T)),
                 list(range(9, T, 9)), [64, 128, 129, 192]):
        run.restart(1)
        close(run.cuts(1, h, cuts), want, dtype,
              rel=5e-2 if dtype == B16 else 5e-5)


def test_window_error_would_show():
    """The tolerance above is far below what a window one off costs."""
    H, G, D, V, window, rot = ATTENTION[4]
    m = U.attention(H, G, D, V, window, rot, base=3e3, factor=1.5,
                    scale=9.0 / D)
    T, width = 210, U.planted_width(m)
    w = U.attention_case(m, width, H + G + D + V)
    h = U.plant(m, w, U.inputs(T, width, 3), U.edge_pairs(window, T))
    want = O.attention(h, w, "", m, 1e-5)
    for off in (-1, 1):
        wrong = O.attention(h, w, "", dict(m, mask={"size": window + off}),
                            1e-5)
        assert (wrong - want).abs().max() / want.abs().max() > 0.1


@pytest.mark.parametrize("parts", [1, 2, 3, 8, 64])
@pytest.mark.parametrize("heads", [(7, 1, 117), (42, 2, None)], ids=str)
def test_decode_parts(parts, heads, monkeypatch):
    monkeypatch.setattr(hy, "window_parts", lambda *a: parts)
    m = U.attention(heads[0], heads[1], 16, 24, heads[2])
    width = 96
    lens = (1, 2, 16, 17, 64, 117, 118, 200)
    w = U.attention_case(m, width, heads[0])
    run = U.MixerRun(U.mixer(m, w, 1e-5, width, DEV, B16), len(lens), 208)
    hs = [U.inputs(n, width, n) for n in lens]
    run.step([(i, h[:-1]) for i, h in enumerate(hs) if len(h) > 1])
    got = run.step([(i, h[-1:]) for i, h in enumerate(hs)])
    for i, h in enumerate(hs):
        close(got[i][0], O.attention(h, w, "", m, 1e-5)[-1], B16, 3e-2)


def test_pages_of_others_do_not_matter():
    """What earlier sequences left in a page's unused places, even
    numbers that are none, changes nothing."""
    for dtype in (B16, F32):
        m = U.attention(4, 2, 16, 24, 40)
        w = U.attention_case(m, 64, 5)
        run = U.MixerRun(U.mixer(m, w, 1e-5, 64, DEV, dtype), 1, 112)
        for pages in run.cache.pages.values():
            pages.fill_(float("nan"))
        h = U.inputs(101, 64, 2)
        for cuts in ([], [70, 71, 72], range(1, 101)):
            run.restart(0)
            close(run.cuts(0, h, cuts), O.attention(h, w, "", m, 1e-5),
                  dtype, 3e-2 if dtype == B16 else 5e-5)


# -- experts alone ---------------------------------------------------------

# experts, choices a token, (groups, kept), width, tokens: up to 16, 32, 64
# and 256 experts in the matrix-core kernel, more in the general one
ROUTES = [(3, 1, (1, 1), 24, 5), (15, 4, (5, 3), 200, 70),
          (16, 16, (1, 1), 1000, 33), (20, 6, (5, 3), 264, 129),
          (32, 2, (8, 2), 64, 16), (64, 8, (8, 4), 520, 50),
          (63, 5, (9, 9), 128, 17), (70, 3, (7, 3), 96, 40),
          (256, 8, (64, 8), 72, 21), (240, 9, (80, 5), 72, 21),
          (300, 4, (10, 3), 40, 9), (1024, 40, (8, 8), 16, 4),
          (9, 3, (3, 3), 51, 30)]


@pytest.mark.parametrize("case", ROUTES, ids=str)
@DTYPES
def test_route(case, dtype):
    E, top, groups, W, T = case
    router = {"experts": E, "top": top, "scale": 1.7,
              "groups": dict(zip(("count", "keep"), groups))}
    g = torch.Generator().manual_seed(E + W)
    w = (3.0 * W ** -0.5 * torch.randn(E, W, generator=g)).bfloat16()
    h = torch.randn(T, W, generator=g).bfloat16()
    sure = O.margins(h.double(), w.double(), router) > 1e-4
    want = O.routing(h.double(), w.double(), router)
    assert sure.float().mean() > 0.7
    for lists in (False, True):
        index, weight, kept = hy.route(
            h.to(DEV, dtype), w.to(DEV, dtype), top, *groups, 1.7, lists)
        index, weight = index.cpu(), weight.cpu()
        for t in sure.nonzero().flatten().tolist():
            assert sorted(index[t].tolist()) == sorted(
                e for e, _ in want[t])
            for e, x in zip(index[t].tolist(), weight[t].tolist()):
                assert abs(x - dict(want[t])[e]) < 1e-5
        if lists:
            counts, pairs = (x.cpu() for x in kept)
            for e in range(E):
                mine = (index == e).flatten().nonzero().flatten().tolist()
                assert sorted(pairs[e, :counts[e]].tolist()) == mine
        else:
            assert kept is None


def test_route_survives_numbers_that_are_none():
    """Whatever the logits, a token's experts are different ones that
    exist."""
    for E, groups, W in ((12, 3, 64), (100, 10, 64), (5, 1, 7)):
        w = torch.randn(E, W).bfloat16()
        h = torch.randn(6, W).bfloat16()
        h[0], h[1, 2], h[2, 3] = float("nan"), float("inf"), 1e30
        w[1] = float("nan")
        index, _, kept = hy.route(h.to(DEV), w.to(DEV), 4, groups, groups,
                                  1.0, True)
        for row in index.tolist():
            assert len(set(row)) == 4 and 0 <= min(row) and max(row) < E
        assert int(kept[0].sum()) == 24


# experts, choices, width, ff, tokens: depths and heights with and without
# remainders, experts with no pair, one pair and many
EXPERTS = [(4, 2, 64, 32, 1), (14, 5, 264, 88, 60), (5, 1, 72, 40, 130),
           (3, 3, 200, 264, 90), (16, 4, 128, 136, 700), (8, 2, 320, 520, 64),
           (40, 3, 48, 8, 33), (2, 1, 1032, 24, 300)]


@pytest.mark.parametrize("case", EXPERTS, ids=str)
@pytest.mark.parametrize("form", ["few", 0, 1, 2, "general"])
def test_experts(case, form, monkeypatch):
    E, top, W, ff, T = case
    if form == "few" and T * top > 2048:
        pytest.skip("more pairs than a workgroup's list holds")
    dtype = F32 if form == "general" else B16
    mlp = U.moe(E, top, ff)
    w = U.experts_case(mlp, W, E)
    h = U.inputs(T, W, 5)
    # unequal loads: half of the tokens prefer the first experts
    w["router"][:top] += 0.5 * h[: T // 2 + 1].mean(0)
    h[: T // 2] = h[0]
    w["router"] = w["router"].bfloat16().double()
    monkeypatch.setattr(hy, "FEW_PAIRS", 2048 if form == "few" else 0)
    monkeypatch.setattr(hy, "expert_tile", lambda *a: form)
    got = U.run_experts(U.experts_module(mlp, w, W, DEV, dtype), h)
    want = O.mixture(h, w, "", mlp)
    sure = O.margins(h, w["router"], mlp["router"]) > 1e-4
    close(got[sure], want[sure], dtype)


@pytest.mark.parametrize("W,ff", [(50, 12), (64, 15), (31, 33)])
@DTYPES
def test_experts_of_odd_sizes(W, ff, dtype):
    mlp = U.moe(6, 2, ff, groups=(3, 2), scale=2.0)
    w = U.experts_case(mlp, W, 3)
    h = U.inputs(77, W, 5)
    got = U.run_experts(U.experts_module(mlp, w, W, DEV, dtype), h)
    sure = O.margins(h, w["router"], mlp["router"]) > 1e-4
    close(got[sure], O.mixture(h, w, "", mlp)[sure], dtype)


def test_expert_results_do_not_depend_on_the_batch():
    """A token's result is the same to the bit wherever it lies."""
    mlp = U.moe(6, 2, 64)
    w = U.experts_case(mlp, 128, 3)
    ff = U.experts_module(mlp, w, 128, DEV, B16)
    x = U.inputs(600, 128, 5).to(DEV, B16)
    index, weight, lists = hy.route(x, *ff.routing(x)[1:-1], True)
    z = ff.routed(x, index, lists)
    order = torch.randperm(600, device=DEV)[:411]
    y = x[order].contiguous()
    index2, weight2, lists = hy.route(y, *ff.routing(y)[1:-1], True)
    assert torch.equal(index2, index[order])
    assert torch.equal(ff.routed(y, index2, lists), z[order])


# -- between the projections and attention ---------------------------------

# heads, kv_heads, dim, vdim, rotated, experts, shared: every number of
# units a lane, both for queries and keys; the last ones run unfused
FRONT = [(4, 2, 64, 24, 64, 12, 40), (16, 4, 128, 128, 128, 16, 520),
         (16, 16, 128, 64, 32, 24, 8), (32, 8, 128, 128, 128, 16, 1280),
         (30, 30, 128, 16, 0, 64, 64), (64, 8, 128, 128, 128, 100, None),
         (60, 60, 128, 8, 96, 8, 16), (3, 1, 16, 8, 16, 5, 24),
         (8, 2, 24, 8, 16, 8, 16), (4, 2, 64, 24, 8, 12, 40),
         (4, 2, 64, 20, 64, 12, 40), (4, 4, 64, 24, 64, 300, 40),
         (4, 2, 64, 24, 64, 12, 44)]


@pytest.mark.parametrize("case", FRONT, ids=str)
@pytest.mark.parametrize("T", [1, 3, 70])
def test_front(case, T):
    H, G, D, V, rot, E, ff = case
    W, eps = 136, 1e-5
    g = torch.Generator().manual_seed(H + T)

    def rand(*shape):
        return torch.randn(shape, generator=g)

    up = lambda n: n + -n % 8
    k_off = up(H * D)
    v_off = k_off + up(G * D)
    u_off = v_off + up(G * V)
    proj = rand(T, u_off + up(ff or 0)).bfloat16()
    wq, wk = (1 + 0.3 * rand(n * D) for n in (H, G))
    table = build_cos_sin_table(300, rot, 500.0) if rot else None
    h, w = rand(T, W).bfloat16(), (0.3 * rand(E, W)).bfloat16()
    bt = (torch.randperm(21, generator=g) + 1).int().view(1, 21)
    b = RaggedBatch.build([(0, 200, [0] * T)], bt.to(DEV))
    cache = torch.full((22, 16, G * (D + V)), 5.0, dtype=B16, device=DEV)
    dev = proj.to(DEV)
    out = torch.full((T, up(ff or 0) + 8), 7.0, dtype=B16, device=DEV)
    index, weight, kept = hy.window_front(
        (dev, H, G, D, V, rot, k_off, v_off, wq.to(DEV), wk.to(DEV), eps,
         table if table is None else table.to(DEV), b, cache),
        (h.to(DEV), w.to(DEV), 2, 1, 1, 1.0, True),
        (out[:, :ff], dev[:, u_off:u_off + ff]) if ff else None)

    x = proj.double()
    turned = torch.zeros(200 + T, H + G, D).double()
    turned[200:, :H] = (O.rms(x[:, :H * D], eps) * wq).view(T, H, D)
    turned[200:, H:] = (O.rms(x[:, k_off:k_off + G * D], eps)
                        * wk).view(T, G, D)
    turned = O.rotate(turned, rot and {"base": 500.0, "dims": rot})[200:]
    close(dev[:, :H * D], turned[:, :H].reshape(T, -1), B16, 1e-2)
    rows = cache.view(22, G, 16, D + V).cpu()
    for t in range(T):
        p = 200 + t
        row = rows[int(bt[0, p // 16]), :, p % 16]
        close(row[:, :D], turned[t, H:], B16, 1e-2)
        assert torch.equal(row[:, D:].reshape(-1),
                           proj[t, v_off:v_off + G * V])
    assert int((rows != 5.0).any(-1).sum()) == T * G
    if ff:
        close(out[:, :ff], x[:, u_off:u_off + ff].clamp(min=0) ** 2, B16,
              1e-2)
        assert (out[:, ff:] == 7.0).all()
    alone = hy.route(h.to(DEV), w.to(DEV), 2, 1, 1, 1.0, True)
    assert torch.equal(index, alone[0]) and torch.equal(weight, alone[1])
    assert torch.equal(kept[0], alone[2][0])


# -- rows ------------------------------------------------------------------

@pytest.mark.parametrize("width", [52, 256, 2048, 8200, 16384])
@pytest.mark.parametrize("top", [0, 1, 3, 8])
@DTYPES
def test_add_norms_with_routed_rows(width, top, dtype):
    g = torch.Generator().manual_seed(width + top)
    x = 3 * torch.randn(21, width, generator=g)
    y = torch.randn(21, width, generator=g).to(dtype)
    z = torch.randn(21, max(top, 1), width, generator=g).to(dtype)
    zw = torch.rand(21, max(top, 1), generator=g)
    total = y.double()
    if top:
        total = total + torch.einsum("tkw,tk->tw", z.double(), zw.double())
    total = x.double() + 0.7 * total
    tol = 1e-2 if dtype == B16 else 2e-6
    routed = (z.to(DEV), zw.to(DEV)) if top else None
    row = 1 + 0.3 * torch.randn(width, generator=g)
    for wt in (torch.tensor(0.8), row, None):
        dev = x.to(DEV)
        h1, h2 = hy.add_norms(dev, y.to(DEV),
                              None if wt is None else wt.to(DEV), None,
                              1e-3, dtype, 0.7, routed)
        close(dev, total, F32, 2e-6)
        assert h2 is None
        if wt is None:
            assert h1 is None
        else:
            close(h1, O.rms(total, 1e-3) * wt, dtype, tol)
    index = torch.tensor([20, 3, 3], dtype=torch.int32, device=DEV)
    close(hy.norm_rows(total.float().to(DEV), index,
                       torch.tensor(0.8, device=DEV), 1e-3, dtype),
          (O.rms(total, 1e-3) * 0.8)[[20, 3, 3]], dtype, tol)


@pytest.mark.parametrize("ff", [8, 70, 416, 5000])
@DTYPES
def test_squared_relu(ff, dtype):
    g = torch.Generator().manual_seed(ff)
    u = torch.randn(21, ff + 16, generator=g).to(dtype)
    out = torch.full((21, ff + 5), 7.0, dtype=dtype, device=DEV)
    hy.squared_relu(out[:, 5:], u.to(DEV)[:, 16:])
    close(out[:, 5:], u[:, 16:].double().clamp(min=0) ** 2, dtype,
          1e-2 if dtype == B16 else 1e-6)
    assert (out[:, :5] == 7.0).all()


def test_sizes_out_of_bounds_are_refused():
    """The host checks sizes before a kernel is launched."""
    h, w = torch.zeros(2, 8, device=DEV), torch.zeros(6, 8, device=DEV)
    for args in ((7, 1, 1), (2, 4, 2), (2, 3, 4), (3, 3, 1), (0, 1, 1)):
        with pytest.raises(RuntimeError):
            hy.route(h, w, *args, 1.0)
    with pytest.raises(RuntimeError):
        hy.route(h, torch.zeros(1025, 8, device=DEV), 1, 1, 1, 1.0)
    m = U.attention(1, 1, 1032, 8)
    w = U.attention_case(m, 24, 1)
    run = U.MixerRun(U.mixer(m, w, 1e-5, 24, DEV, F32), 1, 32)
    with pytest.raises(RuntimeError):
        run.step([(0, U.inputs(3, 24, 1))])
