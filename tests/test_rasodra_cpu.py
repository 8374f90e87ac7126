"""Rasodra on the CPU: scheduler, cache, state and the reference ops, in
32-bit, against the plain implementation of rasodra_oracle."""
import json

import pytest
import torch

import rasodra_oracle as O
import rasodra_util as U
from llmlb_amd.backend.sampler import SamplingParams

TOL = 3e-5


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
    toks = U.tokens(55, cfg["vocab"], 1)
    want = O.forward(toks, w, cfg)
    eng = U.engine(folder)
    assert U.error(U.run_cuts(eng, toks, []), want) < TOL
    assert U.error(U.run_cuts(eng, toks, range(1, 55)), want) < TOL


def test_portions(model):
    cfg, w, folder = model
    toks = U.tokens(51, cfg["vocab"], 2)
    want = O.forward(toks, w, cfg)
    eng = U.engine(folder)
    for size in (2, 3, 7, 13, 16, 17):
        got = U.run_cuts(eng, toks, range(size, 51, size))
        assert U.error(got, want) < TOL, size


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
    reqs = [U.tokens(n, cfg["vocab"], 30 + n) for n in (1, 40, 2, 23, 53, 17)]
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
    eng = build_engine("rasodra-tiny", "cpu", kv_blocks=32, max_batch=2)
    h = eng.model.forward_dense(torch.tensor([[1, 2, 3], [4, 5, 6]]))
    assert h.shape == (2, 3, eng.cfg.model.width)
    alone = eng.model.forward_dense(torch.tensor([[4, 5, 6]]))
    assert torch.allclose(h[1], alone[0], atol=1e-5)
    assert len(eng.generate_sync([1, 2, 3], 4).token_ids) == 4


def test_served_over_http_payloads(plain):
    from llmlb_amd.backend.server import BackendServer
    _, _, folder = plain
    srv = BackendServer(U.engine(folder), "rasodra")
    assert srv.models_payload()["data"][0]["id"] == "rasodra"
    _, _, ids = srv.submit_completion({"prompt": "a b c", "max_tokens": 2})
    assert ids and max(ids) < U.PLAIN["vocab"]


def test_layers_share_weights_not_state(plain):
    """A layer that uses another's weights has pages or a state of its
    own, and adds no parameters."""
    cfg, _, folder = plain
    model = U.engine(folder).model
    assert model.layers_[3] is model.layers_[0]
    assert model.owners == [0, 1, 2] and len(model.specs) == 4
    assert not any(k.startswith("l3.") for k in model.weight_shapes())
    kv = model.make_cache(4, 2)
    assert set(kv.state) == set(kv.extra) == {0, 3}
    assert set(kv.pages) == {1, 2}
    assert kv.state_bytes(model.specs, 2, torch.float32) == sum(
        t.numel() * 4 for d in (kv.state, kv.extra) for t in d.values())


def test_weights_and_configurations_are_checked(tmp_path):
    w = U.weights(U.PLAIN)
    for name in ("l0.mix.f.b", "l0.norm1b", "l1.mix.k.b", "l2.mix.sink"):
        bad = dict(w)
        del bad[name]
        with pytest.raises(KeyError):
            U.engine(U.write_model(tmp_path / name, U.PLAIN, bad))
    bad = dict(w, **{"l1.mlp.up": w["l1.mlp.up"][:-1].clone()})
    with pytest.raises(ValueError):
        U.engine(U.write_model(tmp_path / "b", U.PLAIN, bad))

    def changed(n, i, **change):
        cfg = json.loads(json.dumps(U.PLAIN))
        for part, value in change.items():
            if isinstance(value, dict):
                cfg["layers"][i][part].update(value)
            else:
                cfg["layers"][i][part] = value
        return U.write_model(tmp_path / f"c{n}", cfg, w)

    for n, (i, change) in enumerate((
            (1, {"mixer": {"kv_heads": 2}}), (1, {"mixer": {"vdim": 8}}),
            (1, {"mixer": {"rot": {"base": 9.0, "dims": 18}}}),
            (2, {"mixer": {"rot": {"base": 9.0, "dims": 4}}}),
            (0, {"mlp": {"kind": "other"}}), (1, {"type": "other"}),
            (3, {"weights_of": 4}), (3, {"weights_of": 3}),
            (3, {"mixer": {"gate_cap": 1.0}}), (3, {"mlp": None}))):
        with pytest.raises(ValueError):
            U.engine(changed(n, i, **change))


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

MIXERS = [U.attention(4, 2, 12, 9, rot=8), U.attention(3, 3, 8, None),
          U.attention(2, 1, 10, 16, rot=0), U.attention(2, 2, 6, 1),
          U.latent(4, 12, 8, 20, 24), U.latent(3, 7, 2, 5, 9),
          U.memory(3, 12, 20), U.memory(2, 7, 5, cap=2.0),
          U.memory(1, 16, 8, cap=40.0)]


@pytest.mark.parametrize("ly", MIXERS, ids=str)
def test_mixer_alone(ly):
    oracle, m, w = U.case(ly, 40, 2)
    h = U.inputs(41, 40, 1)
    want = oracle(h, w, "", m, 1e-4)
    run = U.MixerRun(U.mixer(ly["type"], m, w, 1e-4, 40), 2, 41)
    for cuts in ([], range(1, 41), range(2, 41, 2), [17, 19, 20, 33]):
        run.restart(1)
        got = run.cuts(1, h, cuts)
        assert (got - want).abs().max() / want.abs().max() < 2e-5


def change(oracle, h, w, m, want, rows, **kw):
    wrong = oracle(h, {k: kw.get(k, t) for k, t in w.items()}, "",
                   {k: kw.get(k, v) for k, v in m.items()}, 1e-5)
    return (wrong - want).abs().amax(-1)[rows] / want.abs().max()


@pytest.mark.parametrize("size", [16, 25])
def test_planted_chunk_edges(size):
    """Keys that stand out just inside and just outside a chunk's edge: a
    chunk one longer or shorter, or counted from another place, changes
    the output by far more than the tolerance."""
    ly = U.attention(3, 1, 12, size, rot=8, scale=2.0)
    T = 4 * size + 5
    width = U.planted_width("attention", ly["mixer"])
    oracle, m, w = U.case(ly, width, 4)
    pairs = U.chunk_pairs(T, size)
    h = U.plant("attention", m, w, U.inputs(T, width, 3), pairs, 1e-5)
    want = oracle(h, w, "", m, 1e-5)
    run = U.MixerRun(U.mixer("attention", m, w, 1e-5, width), 2, T)
    for cuts in ([], [size, size + 2], range(1, T), range(2, T, 2)):
        run.restart(1)
        assert (run.cuts(1, h, cuts) - want).abs().max() < 1e-4
    rows = [i for i, _ in pairs]
    orig = O.sees
    wrongs = [lambda i, j, s: j <= i and i - j < s,          # a window
              lambda i, j, s: orig(i, j, s) or j == i // s * s - 1,
              lambda i, j, s: orig(i, j, s) and (j % s or j == i)]
    try:
        for O.sees in wrongs:
            assert change(oracle, h, w, m, want, rows).max() > 0.1
    finally:
        O.sees = orig


def test_planted_latents():
    """Far keys, keys at borders and the sink."""
    ly = U.latent(3, 10, 6, 12, 20)
    T, width = 170, U.planted_width("latent_attention", ly["mixer"])
    oracle, m, w = U.case(ly, width, 4)
    pairs = U.far_pairs(T)
    h = U.plant("latent_attention", m, w, U.inputs(T, width, 3), pairs, 1e-5)
    want = oracle(h, w, "", m, 1e-5)
    run = U.MixerRun(U.mixer("latent_attention", m, w, 1e-5, width), 2, T)
    for cuts in ([], [130, 132, 135] + list(range(136, T)),
                 range(2, T, 2), [64, 128]):
        run.restart(1)
        assert (run.cuts(1, h, cuts) - want).abs().max() < 1e-4
    first = list(range(6))
    assert change(oracle, h, w, m, want, first,
                  sink=w["sink"] - 90.0).min() > 0.02
    lost = h.clone()
    lost[0] = 0.0                   # the first token is another one
    wrong = oracle(lost, w, "", m, 1e-5)
    assert (wrong - want)[T - 1].abs().max() / want.abs().max() > 0.1


def test_memory_gates_matter():
    """What the running maximum's start, the caps and the normaliser's
    lower bound change is far above the tolerance."""
    ly = U.memory(2, 12, 16, cap=4.0)
    oracle, m, w = U.case(ly, 40, 5)
    h = U.inputs(30, 40, 6)
    want = oracle(h, w, "", m, 1e-5)
    rows = list(range(30))
    assert change(oracle, h, w, m, want, rows, gate_cap=5.0).max() > 0.02
    orig = O.memory

    def no_bound(q, k, v, li, lf):
        # as if the lower bound were never reached
        return orig(q, k, v, li + 30.0, lf)

    try:
        O.memory = no_bound
        h2 = h * 1e-2               # small queries: the bound decides
        small = w | {"q": w["q"] * 1e-3}
        a = O.mlstm(h2, small, "", m, 1e-1)
        O.memory = orig
        b = O.mlstm(h2, small, "", m, 1e-1)
        assert (a - b).abs().max() / b.abs().max() > 0.1
    finally:
        O.memory = orig
