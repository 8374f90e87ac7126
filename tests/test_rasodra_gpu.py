"""Rasodra on the GPU: every kernel of its path, in bfloat16 and float32,
against the plain implementation of rasodra_oracle."""
import pytest
import torch

import rasodra_oracle as O
import rasodra_util as U
from llmlb_amd.backend.sampler import SamplingParams
from llmlb_amd.ops import hybrid as hy
from test_rasodra_cpu import greedy_oracle

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
    want = O.forward(toks, w, cfg)
    eng = U.engine(folder, DEV, dtype)
    for cuts in ([], range(1, 150), range(2, 150, 2), range(9, 150, 9),
                 range(64, 150, 17), [140] + list(range(141, 150))):
        err = U.error(U.run_cuts(eng, toks, cuts), want)
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
    want = [O.forward(t, w, cfg) for t in reqs]
    free = eng.kv.free_blocks()
    got = U.serve_at_random(eng, reqs, 4, (1, 1, 2, 5, 16, 19, 33))
    assert eng.kv.free_blocks() == free
    for i, rows in got.items():
        assert U.error(rows, want[i]) < LOGIT_TOL[dtype], i


@NAMES
def test_long_decoding(plain, dtype):
    cfg, w, folder = plain
    toks = U.tokens(400, cfg["vocab"], 8)
    want = O.forward(toks, w, cfg)
    eng = U.engine(folder, DEV, dtype)
    got = U.run_cuts(eng, toks, range(3, 400))
    assert U.error(got, want) < LOGIT_TOL[dtype]


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
    for step in range(8):
        live = range(step % 2, 5 - step % 3)
        res = []
        for e, ss in zip(engines, seqs):
            res.append(e.run_batch(
                [(ss[i], U.tokens(1, cfg["vocab"], 50 * step + i), [0])
                 for i in live]).clone())
            e.run_batch([(ss[4], [step, step + 1], [])])
            torch.cuda.synchronize()
        d = (res[0] - res[1]).abs().max() / res[1].std()
        assert d < 0.05, (step, float(d))
    assert engines[0]._graphs and not engines[1]._graphs


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
    eng = build_engine("rasodra-tiny", DEV, kv_blocks=64, max_batch=4)
    assert len(eng.generate_sync(list(range(40)), 5).token_ids) == 5
    h = eng.model.forward_dense(torch.tensor([[1, 2, 3]] * 2, device=DEV))
    assert torch.equal(h[0], h[1]) and h.isfinite().all()


# -- attention alone -------------------------------------------------------

# heads, kv_heads, dim, chunk, rotated: every tile with and without a
# remainder, more than 16 heads to a key/value head, chunks of one token,
# of pages, between pages, of a tile and more; sizes only the general
# kernels take
ATTENTION = [
    (2, 1, 32, 16, 32), (3, 3, 24, 40, 16), (2, 2, 96, 64, 48),
    (8, 2, 64, 100, 64), (4, 1, 128, 65, 96), (2, 1, 256, 37, 256),
    (17, 1, 16, 50, 16), (40, 2, 16, 33, 0), (6, 2, 80, 128, 80),
    (1, 1, 64, 1, 64), (2, 1, 112, None, 32), (6, 2, 7, 30, 6),
    (4, 2, 40, 63, 10), (2, 1, 280, 48, 16), (5, 5, 8, 17, 8),
]


def planted_attention(sizes, T=210):
    heads, kv, dim, chunk, rot = sizes
    ly = U.attention(heads, kv, dim, chunk, rot=rot, scale=16.0 / dim)
    width = U.planted_width("attention", ly["mixer"])
    oracle, m, w = U.case(ly, width, heads + dim)
    if chunk is None:
        pairs = U.far_pairs(T)
    else:
        pairs = U.chunk_pairs(T, chunk) if chunk > 3 else []
    taken = {i for i, _ in pairs}
    pairs = [(i, j) for i, j in pairs if j not in taken]
    h = U.plant("attention", m, w, U.inputs(T, width, 3), pairs, 1e-5)
    return m, w, h, oracle(h, w, "", m, 1e-5)


@pytest.mark.parametrize("sizes", ATTENTION, ids=str)
@DTYPES
def test_attention_planted(sizes, dtype):
    """Scores that stand out just inside and just outside every chunk's
    edge; whole, in portions, and decoded."""
    T = 210
    m, w, h, want = planted_attention(sizes, T)
    run = U.MixerRun(U.mixer("attention", m, w, 1e-5, h.shape[1], DEV,
                             dtype), 2, T)
    for cuts in ([], [130, 132, 135] + list(range(136, T)),
                 list(range(9, T, 9)), [64, 128, 129, 192],
                 list(range(2, T, 2))):
        run.restart(1)
        close(run.cuts(1, h, cuts), want, dtype,
              rel=5e-2 if dtype == B16 else 5e-5)


@pytest.mark.parametrize("parts", [1, 2, 3, 8, 64])
def test_attention_decode_parts(parts, monkeypatch):
    monkeypatch.setattr(hy, "window_parts", lambda *a: parts)
    T = 210
    m, w, h, want = planted_attention((18, 1, 16, 150, 16), T)
    run = U.MixerRun(U.mixer("attention", m, w, 1e-5, h.shape[1], DEV, B16),
                     2, T)
    close(run.cuts(0, h, [140, 145, 148] + list(range(149, T))), want, B16,
          5e-2)


# heads, dim, rotated, vdim, rank: as above
LATENT = [(2, 32, 16, 64, 64), (17, 48, 8, 40, 96), (6, 64, 32, 128, 136),
          (4, 104, 64, 24, 264), (20, 16, 24, 136, 512), (3, 72, 56, 96, 72),
          (1, 128, 64, 200, 40), (3, 12, 6, 20, 30), (2, 24, 8, 9, 24),
          (2, 200, 72, 16, 32), (3, 40, 2, 272, 600)]


@pytest.mark.parametrize("sizes", LATENT, ids=str)
@DTYPES
def test_latent_planted(sizes, dtype):
    """Scores that stand out at the first tokens, at page and tile
    borders, just before and just after the query, beside a sink."""
    T = 210
    ly = U.latent(*sizes)
    width = min(U.planted_width("latent_attention", ly["mixer"]), 2400)
    oracle, m, w = U.case(ly, width, sum(sizes))
    h = U.plant("latent_attention", m, w, U.inputs(T, width, 3),
                U.far_pairs(T), 1e-5)
    want = oracle(h, w, "", m, 1e-5)
    run = U.MixerRun(U.mixer("latent_attention", m, w, 1e-5, width, DEV,
                             dtype), 2, T)
    for cuts in ([], [130, 132, 135] + list(range(136, T)),
                 list(range(9, T, 9)), [64, 128, 129, 192]):
        run.restart(1)
        close(run.cuts(1, h, cuts), want, dtype,
              rel=5e-2 if dtype == B16 else 5e-5)


@pytest.mark.parametrize("parts", [1, 2, 3, 8, 16])
@pytest.mark.parametrize("heads", [5, 21])
def test_latent_decode_parts(parts, heads, monkeypatch):
    """The sink counts once, however a query's keys are split."""
    monkeypatch.setattr(hy, "decode_parts", lambda *a: parts)
    ly = U.latent(heads, 16, 8, 24, 40)
    width = 96
    lens = (1, 2, 16, 17, 64, 65, 128, 200)
    oracle, m, w = U.case(ly, width, heads)
    run = U.MixerRun(U.mixer("latent_attention", m, w, 1e-5, width, DEV,
                             B16), len(lens), 208)
    hs = [U.inputs(n, width, n) for n in lens]
    run.step([(i, h[:-1]) for i, h in enumerate(hs) if len(h) > 1])
    got = run.step([(i, h[-1:]) for i, h in enumerate(hs)])
    for i, h in enumerate(hs):
        close(got[i][0], oracle(h, w, "", m, 1e-5)[-1], B16, 3e-2)


@pytest.mark.parametrize("ly", [U.attention(4, 2, 16, 37),
                                U.latent(4, 16, 8, 24, 40),
                                U.memory(3, 24, 16)], ids=str)
@DTYPES
def test_what_others_left_does_not_matter(ly, dtype):
    """What earlier sequences left in pages and slots, even numbers that
    are none, changes nothing."""
    oracle, m, w = U.case(ly, 64, 5)
    run = U.MixerRun(U.mixer(ly["type"], m, w, 1e-5, 64, DEV, dtype), 1, 112)
    c = run.cache
    for n in (101, 1, 2, 30):
        h = U.inputs(n, 64, n)
        want = oracle(h, w, "", m, 1e-5)
        for cuts in ([], [70, 71, 72], range(1, n)):
            for t in (*c.pages.values(), *c.state.values(),
                      *c.extra.values()):
                t.fill_(float("nan"))
            run.restart(0)
            close(run.cuts(0, h, [c for c in cuts if c < n]), want, dtype,
                  3e-2 if dtype == B16 else 5e-5)


# -- matrix memory alone ---------------------------------------------------

# rows per lane 1..32 and every tile of the matrix cores, with and without
# a remainder; caps that bind and that do not
MEMORY = [U.memory(2, 16, 16), U.memory(3, 7, 9, cap=2.0),
          U.memory(3, 32, 48), U.memory(8, 64, 96, cap=15.0),
          U.memory(20, 24, 64), U.memory(2, 128, 128, cap=30.0),
          U.memory(3, 104, 40), U.memory(2, 256, 24, cap=4.0),
          U.memory(2, 200, 72), U.memory(1, 512, 16), U.memory(1, 300, 600),
          U.memory(2, 50, 36), U.memory(1, 64, 200, cap=6.0),
          U.memory(5, 8, 8), U.memory(2, 96, 7)]


# the operation on given projections: what is rounded is the output alone
MEMORY_TOL = {B16: 8e-3, F32: 5e-5}


@pytest.mark.parametrize("ly", MEMORY, ids=str)
@DTYPES
def test_memory(ly, dtype):
    T = 205
    op = U.memory_op(ly, 3, DEV, dtype)
    x = op.rows(T, 2)
    want = op.oracle(x)
    run = U.MixerRun(op, 2, T)
    for cuts in ([], range(1, T), range(2, T, 2),
                 [30, 33, 34, 35, 99, 163, 164]):
        run.restart(1)
        close(run.cuts(1, x, cuts), want, dtype, MEMORY_TOL[dtype])


@pytest.mark.parametrize("ly", MEMORY[:7], ids=str)
@DTYPES
def test_memory_with_projections(ly, dtype):
    """The whole mixer.  Where a query meets little of the state, the head
    norm enlarges the rounding of 16-bit projections: there the error is
    the root mean square over the output."""
    width, T = 48, 100
    oracle, m, w = U.case(ly, width, sum(map(ord, str(ly))) % 1000)
    h = U.inputs(T, width, 2)
    want = oracle(h, w, "", m, 1e-4)
    run = U.MixerRun(U.mixer(ly["type"], m, w, 1e-4, width, DEV, dtype),
                     2, T)
    for cuts in ([], range(1, T), [30, 33, 34, 64, 99]):
        run.restart(1)
        got = run.cuts(1, h, cuts)
        if dtype == F32:
            close(got, want, F32, 5e-5)
        else:
            d = (got - want).pow(2).mean().sqrt() / want.pow(2).mean().sqrt()
            assert d < 2e-2, float(d)


@pytest.mark.parametrize("forget", [-6.0, 0.0, 8.0, 14.0])
@pytest.mark.parametrize("put", [-9.0, 0.0, 9.0])
@DTYPES
def test_memory_gate_ranges(forget, put, dtype):
    """Gates at both ends of their ranges: everything forgotten at once
    or kept for good; the normaliser's lower bound decides, or never."""
    T = 150
    for eps in (1e-6, 1.0):
        op = U.memory_op(U.memory(4, 32, 40, cap=10.0), 3, DEV, dtype, eps)
        x = op.rows(T, 2, put, forget)
        want = op.oracle(x)
        run = U.MixerRun(op, 2, T)
        for cuts in ([], range(1, T), [64, 65, 100]):
            run.restart(1)
            # with the small eps also near-zero scores are normed
            close(run.cuts(1, x, cuts), want, dtype,
                  max(MEMORY_TOL[dtype], 3e-4))


@DTYPES
def test_memory_remembers_far_tokens(dtype):
    """One token with a large input gate, followed by many with small
    ones: its value stays, across chunks and portions."""
    T = 400
    op = U.memory_op(U.memory(2, 16, 24, cap=12.0), 3, DEV, dtype)
    x = op.rows(T, 2, -9.0, 14.0)
    at = op.offs[4]
    x[5, at:at + 2] = 8.0
    want = op.oracle(x)
    lost = x.clone()
    lost[5, at:at + 2] = -9.0
    d = (op.oracle(lost) - want)[300:].abs().amax(-1)
    assert (d > 0.3 * want.abs().max()).any()
    run = U.MixerRun(op, 2, T)
    for cuts in ([], range(3, T), range(50, T, 50)):
        run.restart(1)
        close(run.cuts(1, x, cuts), want, dtype, MEMORY_TOL[dtype])


@pytest.mark.parametrize("rows", [3, 9, 33])
@pytest.mark.parametrize("ly", [U.memory(8, 64, 128), U.memory(16, 128, 64),
                                U.memory(16, 96, 40), U.memory(8, 32, 72)],
                         ids=str)
@DTYPES
def test_memory_full_chip(ly, rows, dtype):
    """Enough sequences for the wide forms; unequal lengths, portions
    beside single tokens."""
    op = U.memory_op(ly, rows, DEV, dtype)
    xs = [op.rows(5 + 7 * (i % 12), i) for i in range(rows)]
    run = U.MixerRun(op, rows, 96)
    first = run.step([(i, x[:-3 - i % 2]) for i, x in enumerate(xs)])
    second = run.step([(i, x[-3 - i % 2:-1] if i % 3 else
                        x[-3 - i % 2:-2 - i % 2])
                       for i, x in enumerate(xs)])
    for i, x in enumerate(xs):
        got = torch.cat([first[i], second[i]])
        close(got, op.oracle(x)[:len(got)], dtype, MEMORY_TOL[dtype])


# -- rows ------------------------------------------------------------------

@pytest.mark.parametrize("width", [7, 52, 256, 2048, 4096, 8200, 16384,
                                   9001])
@DTYPES
def test_post_pre_norm(width, dtype):
    g = torch.Generator().manual_seed(width)
    x = 3 * torch.randn(33, width, generator=g) + 5
    y = (torch.randn(33, width, generator=g) - 2).to(dtype)
    w1, w2 = (1 + 0.3 * torch.randn(width, generator=g) for _ in range(2))
    tol = 1e-2 if dtype == B16 else 2e-6
    for centred in (True, False):
        for eps in (1e-5, 0.5):
            def norm(v, w):
                return O.layer_norm(v, w, eps) if centred \
                    else O.rms(v, eps) * w

            for add, pre in ((y, w2), (None, w2), (y, None)):
                dev = x.to(DEV)
                total = x.double() + (0 if add is None else
                                      norm(add.double(), w1.double()))
                h = hy.post_pre_norm(
                    dev, None if add is None else add.to(DEV), w1.to(DEV),
                    None if pre is None else pre.to(DEV), eps, dtype,
                    centred)
                close(dev, total, F32, 2e-6)
                if pre is None:
                    assert h is None
                else:
                    close(h, norm(total, w2.double()), dtype, tol)
            rows = torch.tensor([4, 30, 4], dtype=torch.int32, device=DEV)
            got = hy.norm_rows(x.to(DEV), rows, w1.to(DEV), eps, dtype, 0.0,
                               centred)
            close(got, norm(x.double(), w1.double())[[4, 30, 4]], dtype, tol)


@pytest.mark.parametrize("width", [8, 256, 520, 1024])
@DTYPES
def test_post_pre_norm_of_many_rows(width, dtype):
    g = torch.Generator().manual_seed(width)
    x = 3 * torch.randn(2051, width, generator=g) + 5
    y = (torch.randn(2051, width, generator=g) - 2).to(dtype)
    w1, w2 = (1 + 0.3 * torch.randn(width, generator=g) for _ in range(2))
    total = x.double() + O.layer_norm(y.double(), w1.double(), 1e-4)
    dev = x.to(DEV)
    h = hy.post_pre_norm(dev, y.to(DEV), w1.to(DEV), w2.to(DEV), 1e-4, dtype,
                         True)
    close(dev, total, F32, 2e-6)
    close(h, O.layer_norm(total, w2.double(), 1e-4), dtype,
          1e-2 if dtype == B16 else 4e-6)


@pytest.mark.parametrize("sizes", [(3, 9, 7), (16, 40, 64), (1, 3, 136)],
                         ids=str)
@DTYPES
def test_join_heads(sizes, dtype):
    H, N, V = sizes
    g = torch.Generator().manual_seed(V)
    o = torch.randn(H, N, V, generator=g).to(dtype)
    proj = (4 * torch.randn(N + 2, H * V + 24, generator=g)).to(dtype)
    for off in (8, 5):
        out = torch.empty(N, H * V, dtype=dtype, device=DEV)
        hy.join_heads(out, o.to(DEV), proj.to(DEV), off)
        gate = O.sigmoid(proj[:N, off:off + H * V].double())
        want = o.double().transpose(0, 1).reshape(N, -1) * gate
        close(out, want, dtype, 1e-2 if dtype == B16 else 1e-6)


@pytest.mark.parametrize("parts", [(5, 7), (3, 128), (4, 129), (2, 256),
                                   (2, 520)], ids=str)
@DTYPES
def test_norm_with_sigmoid_gate(parts, dtype):
    groups, size = parts
    W = groups * size
    g = torch.Generator().manual_seed(W)
    y = torch.randn(9, W, generator=g)
    gate = torch.randn(9, W + 16, generator=g).to(dtype)
    w = 1 + 0.3 * torch.randn(W, generator=g)
    want = O.rms(y.double().view(9, groups, size), 1e-2).reshape(9, W) \
        * w.double() * O.sigmoid(gate[:, 8:8 + W].double())
    out = torch.empty(9, W, dtype=dtype, device=DEV)
    hy._gated_norm(out, y.to(DEV), gate.to(DEV), 8, w.to(DEV), groups, False,
                   1e-2, True)
    close(out, want, dtype, 1e-2 if dtype == B16 else 1e-6)


def test_sizes_out_of_bounds_are_refused():
    """The host checks sizes before a kernel is launched."""
    ly = U.memory(1, 513, 8)
    _, m, w = U.case(ly, 24, 1)
    for dtype in (B16, F32):
        run = U.MixerRun(U.mixer("mlstm", m, w, 1e-5, 24, DEV, dtype), 1, 32)
        for n in (3, 1):
            with pytest.raises(RuntimeError):
                run.step([(0, U.inputs(n, 24, 1))])
