"""Dibelix on the CPU: scheduler, cache, state and the reference ops,
in 32-bit, against the plain implementation of dibelix_oracle."""
import json

import pytest
import torch

import dibelix_oracle as O
import dibelix_util as U
from llmlb_amd.backend.sampler import SamplingParams

TOL = 2e-5


@pytest.fixture(scope="module", params=["ODD", "TILED", "PLAIN"])
def model(request, tmp_path_factory):
    cfg = getattr(U, request.param)
    w = U.weights(cfg, seed=len(request.param))
    folder = U.write_model(tmp_path_factory.mktemp(request.param), cfg, w)
    return cfg, w, folder


@pytest.fixture(scope="module")
def plain(tmp_path_factory):
    cfg = U.PLAIN
    w = U.weights(cfg, seed=3)
    return cfg, w, U.write_model(tmp_path_factory.mktemp("plain"), cfg, w)


def test_whole_prompt_and_token_by_token(model):
    cfg, w, folder = model
    toks = U.tokens(45, cfg["vocab"], 1)
    want = O.forward(toks, w, cfg)
    eng = U.engine(folder)
    assert U.error(U.run_cuts(eng, toks, []), want) < TOL
    assert U.error(U.run_cuts(eng, toks, range(1, 45)), want) < TOL


@pytest.mark.parametrize("size", [2, 3, 7, 16, 17])
def test_portions(model, size):
    cfg, w, folder = model
    toks = U.tokens(51, cfg["vocab"], 2)
    want = O.forward(toks, w, cfg)
    got = U.run_cuts(U.engine(folder), toks, range(size, 51, size))
    assert U.error(got, want) < TOL


def test_layers_one_by_one(model):
    cfg, w, folder = model
    toks = U.tokens(21, cfg["vocab"], 5)
    want, got = [], []
    O.forward(toks, w, cfg, want)
    eng = U.engine(folder)
    from llmlb_amd.backend.ragged import RaggedBatch
    bt = torch.arange(1, 3, dtype=torch.int32).view(1, 2)
    eng.model(RaggedBatch.build([(0, 0, toks)], bt), eng.kv,
              on_layer=lambda i, x: got.append(x.clone()))
    assert len(got) == len(want) == len(cfg["layers"])
    for a, b in zip(got, want):
        assert (a.double() - b).abs().max() < 1e-3


def test_unequal_batch_and_reuse(model):
    """Sequences of all lengths side by side, some left out of steps;
    pages and slots of finished ones serve new ones."""
    cfg, w, folder = model
    eng = U.engine(folder, blocks=12, rows=3)
    reqs = [U.tokens(n, cfg["vocab"], 30 + n)
            for n in (1, 40, 2, 23, 50, 17, 33)]
    want = [O.forward(t, w, cfg) for t in reqs]
    free = eng.kv.free_blocks()
    got = U.serve_at_random(eng, reqs, 3, (1, 2, 5, 16, 19))
    assert eng.kv.free_blocks() == free
    for i, rows in got.items():
        assert U.error(rows, want[i]) < TOL, i


def greedy_oracle(w, cfg, prompt, n):
    toks = list(prompt)
    for _ in range(n):
        toks.append(int(O.forward(toks, w, cfg)[-1].argmax()))
    return toks[len(prompt):]


def test_generate_through_the_scheduler(plain):
    cfg, w, folder = plain
    eng = U.engine(folder, blocks=40, rows=3, max_prefill_tokens=24,
                   prefill_step_budget=24)
    prompts = [U.tokens(n, cfg["vocab"], n) for n in (5, 60, 1, 31)]
    want = [greedy_oracle(w, cfg, p, 6) for p in prompts]
    queues = [eng.submit(p, SamplingParams(max_new_tokens=6))[1]
              for p in prompts]
    for _ in range(200):
        if not eng.step():
            break
    for q, expect in zip(queues, want):
        out = [q.get_nowait() for _ in range(q.qsize())]
        assert [t for t, _, _ in out] == expect
        assert out[-1][1] == "length"
    assert not eng.running and len(eng._free_rows) == 3
    assert eng.kv.free_blocks() == eng.kv.num_blocks - 1
    # and one at a time, through the blocking entry point
    assert eng.generate_sync(prompts[1], 6).token_ids == want[1]


def test_requests_that_cannot_run(plain):
    cfg, _, folder = plain
    eng = U.engine(folder, blocks=20, rows=2, max_pos=64)
    for prompt in ([], [cfg["vocab"]], [-1], [1] * 64):
        _, q = eng.submit(prompt, SamplingParams(max_new_tokens=2))
        for _ in range(5):
            eng.step()
        assert q.get_nowait()[1] == "error"
    assert len(eng.generate_sync([1, 2, 3], 2).token_ids) == 2
    seq = eng.open_sequence()
    for bad in ([cfg["vocab"]], [], [1] * 65):
        with pytest.raises(ValueError):
            eng.run_batch([(seq, bad, [])])
    with pytest.raises(ValueError):
        eng.run_batch([(seq, [1], []), (seq, [2], [])])
    eng.open_sequence()
    with pytest.raises(RuntimeError):
        eng.open_sequence()


def test_pool_exhaustion_changes_nothing(plain):
    cfg, w, folder = plain
    eng = U.engine(folder, blocks=4, rows=2)       # three pages
    toks = U.tokens(40, cfg["vocab"], 9)
    seq, other = eng.open_sequence(), eng.open_sequence()
    eng.run_batch([(seq, toks[:30], [])])
    with pytest.raises(MemoryError):
        eng.run_batch([(seq, toks[30:32], []), (other, [1] * 30, [])])
    got = eng.run_batch([(seq, toks[30:], [9])]).double()
    assert U.error(got, O.forward(toks, w, cfg)[-1:]) < TOL


def test_abort_and_sampling(plain):
    cfg, _, folder = plain
    eng = U.engine(folder, blocks=40, rows=2)
    rid, _ = eng.submit([1, 2, 3], SamplingParams(max_new_tokens=50))
    for _ in range(3):
        eng.step()
    eng.abort(rid)
    eng.step()
    assert not eng.running
    p = SamplingParams(temperature=0.8, top_p=0.9, seed=5, logprobs=2)
    _, q = eng.submit([4, 5], p)
    p.max_new_tokens = 3
    for _ in range(4):
        eng.step()
    tok, _, extra = q.get_nowait()
    assert 0 <= tok < cfg["vocab"] and len(extra["top"]) == 2


def test_embeddings_and_presets():
    from llmlb_amd.backend.launcher import build_engine
    eng = build_engine("dibelix-tiny", "cpu", kv_blocks=32, max_batch=2)
    h = eng.model.forward_dense(torch.tensor([[1, 2, 3], [4, 5, 6]]))
    assert h.shape == (2, 3, eng.cfg.model.width)
    alone = eng.model.forward_dense(torch.tensor([[4, 5, 6]]))
    assert torch.allclose(h[1], alone[0], atol=1e-5)
    assert len(eng.generate_sync([1, 2, 3], 4).token_ids) == 4


def test_served_over_http_payloads(plain):
    from llmlb_amd.backend.server import BackendServer
    _, _, folder = plain
    srv = BackendServer(U.engine(folder), "dibelix")
    assert srv.health_payload()["status"] == "ok"
    assert srv.models_payload()["data"][0]["id"] == "dibelix"
    _, _, ids = srv.submit_completion({"prompt": "a b c", "max_tokens": 2})
    assert ids and max(ids) < U.PLAIN["vocab"]


def test_weights_are_checked(tmp_path):
    w = U.weights(U.PLAIN)
    bad = dict(w)
    del bad["l0.mix.uk"]
    with pytest.raises(KeyError):
        U.engine(U.write_model(tmp_path / "a", U.PLAIN, bad))
    bad = dict(w, **{"l1.mix.b": w["l1.mix.b"][:1].clone()})
    with pytest.raises(ValueError):
        U.engine(U.write_model(tmp_path / "b", U.PLAIN, bad))


def test_configurations_that_are_refused(tmp_path):
    def broken(change):
        cfg = json.loads(json.dumps(U.ODD))
        change(cfg["layers"])
        return cfg

    for i, change in enumerate((
            lambda ls: ls[2]["mixer"].update(kv_from=1),
            lambda ls: ls[2]["mixer"].update(kv_from=3),
            lambda ls: ls[0].update(type="other"),
            lambda ls: ls[0]["mlp"].update(kind="other"))):
        w = U.weights(U.ODD)
        with pytest.raises((ValueError, KeyError)):
            U.engine(U.write_model(tmp_path / str(i), broken(change), w))


def test_registry(tmp_path):
    from llmlb_amd.models.registry import resolve
    assert resolve("llama-tiny")[1] is None
    with pytest.raises(SystemExit):
        resolve("no-such-model")
    (tmp_path / "config.json").write_text('{"architecture": "Nope"}')
    with pytest.raises(SystemExit):
        resolve(str(tmp_path))


def test_trace_replay(plain, tmp_path):
    import numpy as np

    from llmlb_amd.backend import trace_replay as R
    cfg, w, folder = plain
    args = R.parse_args(["--model", str(folder), "--dtype", "float32",
                         "--out", str(tmp_path), "--max-tokens", "80",
                         "--max-live", "2", "--device", "cpu"])
    eng = R.open_engine(args)
    assert eng.kv.free_blocks() == 5
    a, b = U.tokens(20, cfg["vocab"], 1), U.tokens(33, cfg["vocab"], 2)
    steps = [
        {"step": 0, "entries": [
            {"id": "a", "tokens": a[:19], "want": [0, 18]},
            {"id": "b", "tokens": b[:2], "want": [1]}], "end": []},
        {"step": 1, "entries": [
            {"id": "b", "tokens": b[2:32], "want": []}], "end": []},
        {"step": 2, "entries": [
            {"id": "b", "tokens": b[32:], "want": [0]},
            {"id": "a", "tokens": a[19:], "want": [0]}],
         "end": ["a", "b"]}]
    said = []
    R.replay(eng, map(json.dumps, steps), str(tmp_path), said.append)
    assert said == ["done 0", "done 1", "done 2"]
    assert not (tmp_path / "1.f32").exists()
    la, lb = O.forward(a, w, cfg), O.forward(b, w, cfg)

    def read(n):
        return torch.from_numpy(np.fromfile(
            tmp_path / f"{n}.f32", dtype="<f4")).view(-1, cfg["vocab"])

    assert U.error(read(0), torch.stack([la[0], la[18], lb[1]])) < TOL
    assert U.error(read(2), torch.stack([lb[32], la[19]])) < TOL
    assert eng.kv.free_blocks() == 5


# -- planted scores: the mechanism alone -----------------------------------

def edge_pairs(window, T):
    """(query, key) at the edges of the window, at page borders, at the
    first tokens and far back."""
    out = []
    for i, back in ((T - 1, window - 1), (T - 3, window), (T - 5, window + 1),
                    (window - 1, window - 1), (T - 8, 1), (T - 20, 5)):
        if 0 <= i - back:
            out.append((i, i - back))
    for j in (0, 1, 15, 16, 31, 32):
        i = j + window - 2
        if i < T and all(i != a and i != b and j != a for a, b in out):
            out.append((i, j))
    return out


@pytest.mark.parametrize("window", [19, 48])
def test_planted_scores(window):
    spec = U.latent(3, 16, 8, 12, 40, window)["mixer"]
    T = 90
    pairs = edge_pairs(window, T)
    w, h = U.planted_attention(spec, 80, T, pairs)
    want = O.latent_attention(h, w, "", spec, 1e-5)[0]
    mix = U.latent_mixer(spec, w, 1e-5, 80)
    run = U.MixerRun(mix, 2, T)
    for cuts in ([], range(1, T), [40, 42, 75], range(2, T, 2)):
        run.restart(1)
        got = run.cuts(1, h, cuts)
        assert (got - want).abs().max() < 1e-4
    # a window one off, either way, shows at its edge
    for off in (-1, 1):
        other = dict(spec, mask={"size": window + off})
        wrong = O.latent_attention(h, w, "", other, 1e-5)[0]
        assert (wrong - want).abs().amax(-1)[[T - 1, T - 3]].max() > 0.05
