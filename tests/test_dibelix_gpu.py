"""Dibelix on the GPU: every kernel of the hybrid path, in bfloat16 and
float32, against the plain implementation of dibelix_oracle."""
import pytest
import torch

import dibelix_oracle as O
import dibelix_util as U
from llmlb_amd.backend.sampler import SamplingParams
from llmlb_amd.ops import hybrid as hy
from test_dibelix_cpu import edge_pairs, greedy_oracle

pytestmark = pytest.mark.gpu
DEV = "cuda:0"
F32, B16 = torch.float32, torch.bfloat16
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

@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
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


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
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


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
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
    eng = build_engine("dibelix-tiny", DEV, kv_blocks=64, max_batch=4)
    assert len(eng.generate_sync(list(range(40)), 5).token_ids) == 5
    h = eng.model.forward_dense(torch.tensor([[1, 2, 3]] * 2, device=DEV))
    assert torch.equal(h[0], h[1]) and h.isfinite().all()


# -- latent attention alone ------------------------------------------------

# heads, dim, rot, vdim, rank, window: one line per tile shape of the
# prompt kernel and per rank class and head tiling of the decode kernel,
# then sizes only the general kernel takes
LATENT = [
    (3, 32, 16, 48, 40, 70), (2, 64, 32, 64, 136, 64),
    (4, 96, 32, 64, 256, 33), (2, 128, 64, 40, 264, 129),
    (2, 192, 64, 64, 64, 90), (5, 40, 24, 100, 128, 128),
    (2, 96, 32, 128, 512, 65), (3, 128, 64, 128, 400, 150),
    (2, 192, 64, 128, 200, 100), (1, 120, 64, 250, 320, 77),
    (18, 16, 8, 24, 72, 80), (33, 8, 8, 16, 136, 63),
    (20, 16, 8, 16, 512, 50), (17, 16, 16, 16, 256, 81),
    (3, 10, 6, 9, 30, 60), (2, 24, 8, 20, 600, 45),
]


@pytest.mark.parametrize("sizes", LATENT, ids=str)
@pytest.mark.parametrize("dtype", [B16, F32], ids=["bf16", "f32"])
def test_latent_attention_planted(sizes, dtype):
    """Scores that stand out at the window's edges, at page and tile
    borders, at the first tokens; whole, in portions, and decoded."""
    spec = U.latent(*sizes, base=3e4)["mixer"]
    H, D, R = sizes[:3]
    T, width = 210, max(H * (D + R), 64) + 8
    pairs = edge_pairs(spec["mask"]["size"], T)
    w, h = U.planted_attention(spec, width, T, pairs, seed=sum(sizes))
    want = O.latent_attention(h, w, "", spec, 1e-5)[0]
    mix = U.latent_mixer(spec, w, 1e-5, width, DEV, dtype)
    run = U.MixerRun(mix, 2, T)
    for cuts in ([], [130, 132, 135] + list(range(136, T)),
                 list(range(9, T, 9)), [64, 128, 129, 192]):
        run.restart(1)
        close(run.cuts(1, h, cuts), want, dtype,
              rel=5e-2 if dtype == B16 else 2e-5)


def test_window_error_would_show():
    """The tolerance above is far below what a window one off costs."""
    sizes = LATENT[7]
    spec = U.latent(*sizes, base=3e4)["mixer"]
    T, width = 210, sizes[0] * (sizes[1] + sizes[2]) + 8
    w, h = U.planted_attention(spec, width, T,
                               edge_pairs(spec["mask"]["size"], T))
    want = O.latent_attention(h, w, "", spec, 1e-5)[0]
    for off in (-1, 1):
        other = dict(spec, mask={"size": spec["mask"]["size"] + off})
        wrong = O.latent_attention(h, w, "", other, 1e-5)[0]
        assert (wrong - want).abs().max() / want.abs().max() > 0.08


@pytest.mark.parametrize("parts", [1, 2, 3, 8, 16])
@pytest.mark.parametrize("heads", [7, 21])
def test_decode_parts(parts, heads, monkeypatch):
    monkeypatch.setattr(hy, "decode_parts", lambda *a: parts)
    spec = U.latent(heads, 16, 16, 24, 136, 117)["mixer"]
    width = heads * 32
    lens = (1, 2, 16, 17, 64, 117, 118, 200)
    w, _ = U.planted_attention(spec, width, 4, [], seed=heads)
    mix = U.latent_mixer(spec, w, 1e-5, width, DEV, B16)
    run = U.MixerRun(mix, len(lens), 208)
    g = torch.Generator().manual_seed(1)
    hs = [torch.randn(n, width, generator=g).bfloat16().double()
          for n in lens]
    run.step([(i, h[:-1]) for i, h in enumerate(hs) if len(h) > 1])
    got = run.step([(i, h[-1:]) for i, h in enumerate(hs)])
    for i, h in enumerate(hs):
        want = O.latent_attention(h, w, "", spec, 1e-5)[0]
        close(got[i][0], want[-1], B16)


# -- gated delta rule alone ------------------------------------------------

def delta_case(heads, kv_heads, dim, vdim, taps, width, seed):
    cfg = U.config([U.delta(heads, kv_heads, dim, vdim, taps)], 8, width, 8)
    w = {k[len("l0.mix."):]: t.double()
         for k, t in U.weights(cfg, seed).items() if k.startswith("l0.mix.")}
    return cfg["layers"][0]["mixer"], w


# heads, kv_heads, dim, vdim, taps: rows per lane 1..32 with and without
# a remainder, every convolution length, grouped heads
DELTA = [(2, 2, 16, 16, 4), (4, 2, 11, 7, 3), (3, 1, 32, 48, 2),
         (4, 4, 30, 64, 1), (8, 2, 64, 96, 4), (4, 2, 50, 40, 6),
         (2, 1, 128, 128, 4), (3, 3, 100, 36, 3), (2, 2, 256, 24, 4),
         (2, 1, 200, 50, 2), (1, 1, 512, 16, 4), (2, 1, 300, 300, 5)]


@pytest.mark.parametrize("sizes", DELTA, ids=str)
@pytest.mark.parametrize("dtype", [B16, F32], ids=["bf16", "f32"])
def test_delta_rule(sizes, dtype):
    width, T = 48, 75
    m, w = delta_case(*sizes, width, seed=sum(sizes))
    g = torch.Generator().manual_seed(2)
    h = torch.randn(T, width, generator=g).bfloat16().double()
    want = O.channel_delta(h, w, "", m, 1e-4)
    mix = U.delta_mixer(m, w, 1e-4, width, DEV, dtype)
    run = U.MixerRun(mix, 2, T)
    for cuts in ([], range(1, T), range(2, T, 2),
                 [30, 33, 34, 35, 36, 60, 62]):
        run.restart(1)
        close(run.cuts(1, h, cuts), want, dtype,
              rel=3e-2 if dtype == B16 else 5e-5)


@pytest.mark.parametrize("rows", [3, 9, 33])
def test_delta_rule_full_chip(rows):
    """Enough sequences for the scan's wide lanes; unequal lengths,
    portions beside single tokens."""
    width = 40
    m, w = delta_case(8, 8, 64, 128, 4, width, seed=rows)
    g = torch.Generator().manual_seed(3)
    hs = [torch.randn(5 + 2 * i, width, generator=g).bfloat16().double()
          for i in range(rows)]
    mix = U.delta_mixer(m, w, 1e-5, width, DEV, F32)
    run = U.MixerRun(mix, rows, 80)
    first = run.step([(i, h[:-3 - i % 2]) for i, h in enumerate(hs)])
    second = run.step([(i, h[-3 - i % 2:-1] if i % 3 else
                        h[-3 - i % 2:-2 - i % 2])
                       for i, h in enumerate(hs)])
    for i, h in enumerate(hs):
        got = torch.cat([first[i], second[i]])
        want = O.channel_delta(h, w, "", m, 1e-5)
        close(got, want[:len(got)], F32)


def test_slots_start_empty():
    """A slot's next sequence sees nothing of the last one, also when it
    is shorter than the convolution."""
    width = 40
    m, w = delta_case(4, 2, 32, 32, 4, width, seed=1)
    g = torch.Generator().manual_seed(4)
    run = U.MixerRun(U.delta_mixer(m, w, 1e-5, width, DEV, F32), 1, 64)
    for n in (30, 2, 1, 3, 17):
        h = torch.randn(n, width, generator=g).bfloat16().double()
        for cuts in ([], range(1, n)):
            run.restart(0)
            close(run.cuts(0, h, cuts), O.channel_delta(h, w, "", m, 1e-5),
                  F32)


# -- rows ------------------------------------------------------------------

@pytest.mark.parametrize("width", [52, 256, 2048, 8200, 16384])
@pytest.mark.parametrize("dtype", [B16, F32], ids=["bf16", "f32"])
def test_rows(width, dtype):
    g = torch.Generator().manual_seed(width)
    table = torch.randn(40, width, generator=g).to(dtype)
    ids = torch.randint(0, 40, (33,), generator=g).to(torch.int32)
    y = torch.randn(33, width, generator=g).to(dtype)
    wn = 0.3 * torch.randn(width, generator=g)
    x, xb = hy.embed_rows(table.to(DEV), ids.to(DEV))
    assert torch.equal(x.cpu(), table[ids.long()].float())
    assert torch.equal(xb.cpu(), table[ids.long()])
    for eps in (1e-5, 0.3):
        want = x.double().cpu() + O.post_norm(y.double(), wn.double(), eps)
        hy.post_norm_add(x, xb, y.to(DEV), wn.to(DEV), eps, 1.0)
        close(x, want, F32, 1e-6)
        assert torch.equal(xb, x.to(dtype))
    index = torch.tensor([5, 0, 32], dtype=torch.int32, device=DEV)
    got = hy.norm_rows(x, index, wn.to(DEV), 0.1, dtype, 1.0)
    close(got, O.post_norm(x.double().cpu()[[5, 0, 32]], wn.double(), 0.1),
          dtype, 1e-2 if dtype == B16 else 1e-6)
    z = (4 * torch.randn(33, width, generator=g)).to(dtype)
    close(hy.soft_cap(z.to(DEV), 3.0), 3 * torch.tanh(z.double() / 3), F32,
          1e-6)
    assert torch.equal(hy.soft_cap(z.to(DEV), None).cpu(), z.float())
    close(hy.gelu_tanh_(z.to(DEV)), O.gelu_tanh(z.double()), dtype,
          1e-2 if dtype == B16 else 1e-6)
