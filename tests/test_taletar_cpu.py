"""Taletar on the CPU: scheduler, cache, state and the reference ops, in
32-bit, against the plain implementation of taletar_oracle."""
import json
import math

import pytest
import torch

import taletar_oracle as O
import taletar_util as U
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
              on_layer=lambda i, x: got.append((i, x.clone())))
    assert [i for i, _ in got] == list(range(len(cfg["layers"])))
    for (_, a), b in zip(got, want):
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


def test_embeddings_and_presets():
    from llmlb_amd.backend.launcher import build_engine
    eng = build_engine("taletar-tiny", "cpu", kv_blocks=32, max_batch=2)
    h = eng.model.forward_dense(torch.tensor([[1, 2, 3], [4, 5, 6]]))
    assert h.shape == (2, 3, eng.cfg.model.width)
    alone = eng.model.forward_dense(torch.tensor([[4, 5, 6]]))
    assert torch.allclose(h[1], alone[0], atol=1e-5)
    assert len(eng.generate_sync([1, 2, 3], 4).token_ids) == 4


def test_served_over_http_payloads(plain):
    from llmlb_amd.backend.server import BackendServer
    _, _, folder = plain
    srv = BackendServer(U.engine(folder), "taletar")
    assert srv.models_payload()["data"][0]["id"] == "taletar"
    _, _, ids = srv.submit_completion({"prompt": "a b c", "max_tokens": 2})
    assert ids and max(ids) < U.PLAIN["vocab"]


def test_weights_and_configurations_are_checked(tmp_path):
    w = U.weights(U.PLAIN)
    bad = dict(w)
    del bad["l0.mix.a2.b"]
    with pytest.raises(KeyError):
        U.engine(U.write_model(tmp_path / "a", U.PLAIN, bad))
    bad = dict(w, **{"l1.mlp.up": w["l1.mlp.up"][:-1].clone()})
    with pytest.raises(ValueError):
        U.engine(U.write_model(tmp_path / "b", U.PLAIN, bad))
    for n, (i, part, change) in enumerate((
            (1, "mixer", {"heads": 4, "kv_heads": 3}),
            (2, "mixer", {"groups": 3}), (2, "mixer", {"norm_groups": 7}),
            (0, "mlp", {"kind": "other"}))):
        cfg = json.loads(json.dumps(U.PLAIN))
        cfg["layers"][i][part].update(change)
        with pytest.raises(ValueError):
            U.engine(U.write_model(tmp_path / str(n), cfg, w))
    cfg = json.loads(json.dumps(U.PLAIN))
    cfg["layers"][1]["type"] = "other"
    with pytest.raises(ValueError):
        U.engine(U.write_model(tmp_path / "c", cfg, w))


def test_trace_replay(plain, tmp_path):
    import numpy as np

    from llmlb_amd.backend import trace_replay as R
    cfg, w, folder = plain
    args = R.parse_args(["--model", str(folder), "--dtype", "float32",
                         "--out", str(tmp_path), "--max-tokens", "80",
                         "--max-live", "2", "--device", "cpu"])
    eng = R.open_engine(args)
    a, b = U.tokens(20, cfg["vocab"], 1), U.tokens(33, cfg["vocab"], 2)
    steps = [
        {"step": 0, "entries": [
            {"id": "a", "tokens": a[:19], "want": [0, 18]},
            {"id": "b", "tokens": b[:2], "want": [1]}], "end": []},
        {"step": 1, "entries": [
            {"id": "b", "tokens": b[2:], "want": [30]},
            {"id": "a", "tokens": a[19:], "want": [0]}],
         "end": ["a", "b"]}]
    R.replay(eng, map(json.dumps, steps), str(tmp_path), lambda s: None)
    la, lb = O.forward(a, w, cfg), O.forward(b, w, cfg)

    def read(n):
        return torch.from_numpy(np.fromfile(
            tmp_path / f"{n}.f32", dtype="<f4")).view(-1, cfg["vocab"])

    assert U.error(read(0), torch.stack([la[0], la[18], lb[1]])) < TOL
    assert U.error(read(1), torch.stack([lb[32], la[19]])) < TOL
    assert eng.kv.free_blocks() == 5


# -- mechanisms alone ------------------------------------------------------

@pytest.mark.parametrize("q_temp", [(0.4, 17), (0.1, 1), (0.7, 2.5), None])
def test_query_scale_table(q_temp):
    from llmlb_amd.models.taletar import query_scale_table
    temp = q_temp and {"coef": q_temp[0], "every": q_temp[1]}
    got = query_scale_table(200, 0.3, temp)
    want = [0.3 * O.temperature(p, temp) for p in range(200)]
    assert (got.double() - torch.tensor(want).double()).abs().max() < 1e-6
    if q_temp == (0.4, 17):       # steps at the 17th token, not the 18th
        assert got[15] == got[0]
        assert math.isclose(got[16], 0.3 * (1 + 0.4 * math.log(2)),
                            rel_tol=1e-6)


MIXERS = [U.attention(4, 2, 12, 20), U.attention(3, 3, 8, 7, softcap=None,
                                                 q_temp=None),
          U.gla(3, 12, 20), U.gla(2, 7, 5, tau=1.0),
          U.mamba2(4, 6, 10, groups=2, taps=3, norm_groups=3),
          U.mamba2(3, 8, 5, taps=1)]


@pytest.mark.parametrize("ly", MIXERS, ids=str)
def test_mixer_alone(ly):
    oracle, m, w = U.case(ly, 40, 2)
    h = U.inputs(41, 40, 1)
    want = oracle(h, w, "", m, 1e-4)
    run = U.MixerRun(U.mixer(ly["type"], m, w, 1e-4, 40), 2, 41)
    for cuts in ([], range(1, 41), range(2, 41, 2), [17, 19, 20, 33]):
        run.restart(1)
        got = run.cuts(1, h, cuts)
        assert (got - want).abs().max() / want.abs().max() < 1e-5


def test_planted_scores():
    """A key that stands out changes the output by far more than the
    tolerance when it is lost, added or taken by the other map."""
    ly = U.attention(3, 1, 12, 16, q_temp=(0.3, 50))
    T, width = 170, U.planted_width(ly["mixer"])
    _, m, w = U.case(ly, width, 4)
    triples = U.far_triples(T)
    h = U.plant(m, w, U.inputs(T, width, 3), triples)
    want = O.attention(h, w, "", m, 1e-5)
    run = U.MixerRun(U.mixer("attention", m, w, 1e-5, width), 2, T)
    for cuts in ([], [130, 132, 135] + list(range(136, T)),
                 range(2, T, 2), [64, 128]):
        run.restart(1)
        got = run.cuts(1, h, cuts)
        assert (got - want).abs().max() < 1e-4
    size = want.abs().max()
    rows = [i for i, _, _ in triples]

    def change(**kw):
        wrong = O.attention(h, w, "", dict(m, **kw), 1e-5)
        return (wrong - want).abs().amax(-1)[rows] / size

    orig = O.causal_attention
    try:
        # the first token is lost
        O.causal_attention = lambda q, k, v, s, c: orig(
            q, torch.cat([k[:1] * 0, k[1:]]), v, s, c)
        assert change()[0] > 0.08
        # every query sees one key more
        O.causal_attention = lambda q, k, v, s, c: torch.cat(
            [orig(torch.cat([q[i:i + 1]] * (i + 2)), k[:i + 2], v[:i + 2],
                  s, c)[-1:] for i in range(T - 1)]
            + [orig(q, k, v, s, c)[-1:]])
        assert change()[rows.index(T - 15)] > 0.08
    finally:
        O.causal_attention = orig
    assert change(softcap=None).max() > 0.02
    assert change(q_temp=None).max() > 0.02
    assert change(diff=m["diff"] + 0.1).max() > 0.02
