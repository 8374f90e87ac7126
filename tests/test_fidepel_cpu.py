"""Fidepel on the CPU: scheduler, cache, loops and the reference ops, in
32-bit, against the plain implementation of fidepel_oracle."""
import json

import pytest
import torch

import fidepel_oracle as O
import fidepel_util as U
from llmlb_amd.backend.sampler import SamplingParams

TOL = 2e-5
MODELS = ["ODD", "TILED", "PLAIN"]


@pytest.fixture(scope="module", params=MODELS)
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


def check(got, want, margin):
    assert U.clear_error(got, want, margin, "float32") < TOL


def oracle(toks, w, cfg):
    margin = []
    return O.forward(toks, w, cfg, clear=margin), margin


def test_whole_prompt_and_token_by_token(model):
    cfg, w, folder = model
    toks = U.tokens(60, cfg["vocab"], 1)
    want = oracle(toks, w, cfg)
    eng = U.engine(folder)
    check(U.run_cuts(eng, toks, []), *want)
    check(U.run_cuts(eng, toks, range(1, 60)), *want)


@pytest.mark.parametrize("size", [2, 3, 7, 16, 17])
def test_portions(model, size):
    cfg, w, folder = model
    toks = U.tokens(61, cfg["vocab"], 2)
    check(U.run_cuts(U.engine(folder), toks, range(size, 61, size)),
          *oracle(toks, w, cfg))


def test_layer_runs_one_by_one(model):
    """The residual stream after every layer run; a looped layer counts
    each time, and every run has pages of its own."""
    cfg, w, folder = model
    toks = U.tokens(21, cfg["vocab"], 5)
    want, got = [], []
    O.forward(toks, w, cfg, want)
    eng = U.engine(folder)
    from llmlb_amd.backend.ragged import RaggedBatch
    bt = torch.arange(1, 3, dtype=torch.int32).view(1, 2)
    eng.model(RaggedBatch.build([(0, 0, toks)], bt), eng.kv,
              on_layer=lambda i, x: got.append((i, x.clone())))
    runs = O.layer_runs(cfg)
    assert [i for i, _ in got] == list(range(len(runs)))
    assert sorted(eng.kv.pages) == list(range(len(runs)))
    for (_, a), b in zip(got, want):
        assert (a.double() - b).abs().max() < 1e-4 * b.abs().max()


def test_unequal_batch_and_reuse(model):
    """Sequences of all lengths side by side, some left out of steps;
    pages and slots of finished ones serve new ones."""
    cfg, w, folder = model
    eng = U.engine(folder, blocks=12, rows=3)
    reqs = [U.tokens(n, cfg["vocab"], 30 + n)
            for n in (1, 40, 2, 23, 50, 17, 33)]
    want = [oracle(t, w, cfg) for t in reqs]
    free = eng.kv.free_blocks()
    got = U.serve_at_random(eng, reqs, 3, (1, 2, 5, 16, 19))
    assert eng.kv.free_blocks() == free
    for i, rows in got.items():
        check(rows, *want[i])


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
    eng = build_engine("fidepel-tiny", "cpu", kv_blocks=32, max_batch=2)
    h = eng.model.forward_dense(torch.tensor([[1, 2, 3], [4, 5, 6]]))
    assert h.shape == (2, 3, eng.cfg.model.width)
    alone = eng.model.forward_dense(torch.tensor([[4, 5, 6]]))
    assert torch.allclose(h[1], alone[0], atol=1e-5)
    assert len(eng.generate_sync([1, 2, 3], 4).token_ids) == 4


def test_served_over_http_payloads(plain):
    from llmlb_amd.backend.server import BackendServer
    _, _, folder = plain
    srv = BackendServer(U.engine(folder), "fidepel")
    assert srv.models_payload()["data"][0]["id"] == "fidepel"
    _, _, ids = srv.submit_completion({"prompt": "a b c", "max_tokens": 2})
    assert ids and max(ids) < U.PLAIN["vocab"]


def test_weights_and_configurations_are_checked(tmp_path):
    w = U.weights(U.PLAIN)
    bad = dict(w)
    del bad["l0.mlp.e3.up"]
    with pytest.raises(KeyError):
        U.engine(U.write_model(tmp_path / "a", U.PLAIN, bad))
    bad = dict(w, **{"l0.norm1": w["l0.mix.temp"].clone()})
    with pytest.raises(ValueError):
        U.engine(U.write_model(tmp_path / "b", U.PLAIN, bad))

    def changed(n, change):
        cfg = json.loads(json.dumps(U.PLAIN))
        change(cfg)
        with pytest.raises(ValueError):
            U.engine(U.write_model(tmp_path / str(n), cfg, w))

    for n, change in enumerate((
            lambda c: c["layers"][0]["mixer"].update(heads=4, kv_heads=3),
            lambda c: c["layers"][0]["mixer"]["rot"].update(dims=18),
            lambda c: c["layers"][0]["mixer"]["rot"].update(dims=3),
            lambda c: c["layers"][0]["mixer"]["mask"].update(size=-1),
            lambda c: c["layers"][0]["mlp"]["router"].update(top=5),
            lambda c: c["layers"][0]["mlp"]["router"]["groups"].update(
                count=4),
            lambda c: c["layers"][0]["mlp"]["router"]["groups"].update(
                keep=4),
            lambda c: c["layers"][0]["mlp"].update(kind="dense"),
            lambda c: c["layers"][1].update(type="other"),
            lambda c: c.update(loop={"start": 1, "stop": 3, "times": 2}),
            lambda c: c.update(loop={"start": 0, "stop": 1, "times": 0}))):
        changed(n, change)


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

def test_loops():
    from llmlb_amd.models.fidepel import FidepelConfig
    for loop, want in (((1, 3, 2), [0, 1, 2, 1, 2, 3]),
                       ((0, 4, 1), [0, 1, 2, 3]), ((2, 2, 3), [0, 1, 2, 3]),
                       ((0, 1, 3), [0, 0, 0, 1, 2, 3]),
                       ((3, 4, 2), [0, 1, 2, 3, 3]), (None, [0, 1, 2, 3])):
        cfg = U.config(
            [(U.attention(1, 1, 2, 2), None)] * 4,
                       8, 4, 1.0, loop)
        assert FidepelConfig.from_json(cfg).runs() == want
        assert O.layer_runs(cfg) == want


def test_linear_scaling_of_frequencies():
    from llmlb_amd.ops.reference import build_cos_sin_table
    a, b = build_cos_sin_table(40, 6, 100.0), build_cos_sin_table(
        160, 6, 100.0, factor=4.0)
    assert torch.allclose(a[1:40], b[4:160:4], atol=1e-6)


ATTENTION = [U.attention(4, 2, 12, 20, window=19),
             U.attention(3, 3, 8, 7, dims=0),
             U.attention(6, 1, 10, 6, window=1, dims=4),
             U.attention(2, 1, 16, 24, window=40, factor=2.5, base=77.0)]


@pytest.mark.parametrize("m", ATTENTION, ids=str)
def test_attention_alone(m):
    w = U.attention_case(m, 40, 2)
    h = U.inputs(61, 40, 1)
    want = O.attention(h, w, "", m, 1e-4)
    run = U.MixerRun(U.mixer(m, w, 1e-4, 40), 2, 61)
    for cuts in ([], range(1, 61), range(2, 61, 2), [17, 19, 20, 33]):
        run.restart(1)
        got = run.cuts(1, h, cuts)
        assert (got - want).abs().max() / want.abs().max() < 1e-5


def test_planted_scores():
    """A key that stands out changes the output by far more than the
    tolerance when the window is one off, the key is lost or the turn is
    another."""
    m = U.attention(3, 1, 16, 16, window=33, scale=0.6)
    T, width = 120, U.planted_width(m)
    w = U.attention_case(m, width, 4)
    pairs = U.edge_pairs(33, T)
    h = U.plant(m, w, U.inputs(T, width, 3), pairs)
    want = O.attention(h, w, "", m, 1e-5)
    run = U.MixerRun(U.mixer(m, w, 1e-5, width), 2, T)
    for cuts in ([], [70, 72, 75] + list(range(76, T)), range(2, T, 2),
                 [64, 96]):
        run.restart(1)
        assert (run.cuts(1, h, cuts) - want).abs().max() < 1e-4
    size = want.abs().max()
    inside = [i for i, j in pairs if i - j == 32]
    outside = [i for i, j in pairs if i - j == 33]
    assert len(inside) > 2 and len(outside) > 2

    def change(rows, **kw):
        wrong = O.attention(h, w, "", dict(m, **kw), 1e-5)
        return ((wrong - want).abs().amax(-1)[rows] / size).min()

    assert change(inside, mask={"size": 32}) > 0.05
    assert change(outside, mask={"size": 34}) > 0.05
    rows = [i for i, j in pairs if 2 < i - j < 33]
    assert change(rows, rot={"base": 1e4, "dims": 8}) > 0.01
    assert change(rows, rot={"base": 1e4, "dims": 16,
                             "scaling": {"factor": 2.0}}) > 0.01


EXPERTS = [U.moe(6, 2, 12), U.moe(8, 3, 20, groups=(4, 2), scale=2.0),
           U.moe(9, 9, 4), U.moe(6, 1, 5, groups=(6, 1)),
           U.moe(12, 4, 7, groups=(2, 1), scale=0.3)]


@pytest.mark.parametrize("mlp", EXPERTS, ids=str)
def test_experts_alone(mlp):
    w = U.experts_case(mlp, 24, 3)
    h = U.inputs(40, 24, 5)
    want = O.mixture(h, w, "", mlp)
    got = U.run_experts(U.experts_module(mlp, w, 24), h)
    assert (got - want).abs().max() / want.abs().max() < 1e-5


def test_routing_details():
    """Groups by their best score; a good expert of a group that is not
    kept is left out; weights are those of all experts' softmax."""
    from llmlb_amd.ops import hybrid as hy
    z = torch.tensor([[3.0, 0.0, 2.5, 2.4, 2.6, -9.0]])
    eye = torch.eye(6)
    index, weight, _ = hy.route(z, eye, 2, 3, 2, 1.5)
    assert index.tolist() == [[0, 4]]
    p = torch.softmax(z[0], -1)
    assert torch.allclose(weight[0], 1.5 * p[[0, 4]] / (p[0] + p[4]))
    index, _, _ = hy.route(z, eye, 3, 3, 2, 1.0)
    assert index.tolist() == [[0, 4, 1]]        # not 2 and 3
    index, _, _ = hy.route(z, eye, 3, 1, 1, 1.0)
    assert index.tolist() == [[0, 4, 2]]
