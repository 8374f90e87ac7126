"""Small random Taletar models and mixers for tests.

Configurations are plain dictionaries in the layout of config.json, so
that the oracle and the served model read the same thing.
"""
from __future__ import annotations

import torch
import torch.nn as nn

import taletar_oracle as O
from llmlb_amd.models.mixers import (DifferentialAttention,
                                     GatedLinearAttention,
                                     StateSpaceDuality)
from llmlb_amd.models.taletar import query_scale_table
from packed_util import (MixerRun, engine, error, run_cuts,  # noqa: F401
                         serve_at_random, tokens, write_model)


def attention(heads, kv_heads, dim, vdim, softcap=30.0, diff=0.5,
              q_temp=(0.4, 17), scale=None):
    return {"type": "attention", "mixer": {
        "heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim,
        "diff": diff, "softcap": softcap,
        "q_temp": q_temp and {"coef": q_temp[0], "every": q_temp[1]},
        "scale": scale or 1.3 * dim ** -0.5}}


def gla(heads, dim, vdim, tau=8.0, low=12):
    return {"type": "gla", "low": low, "mixer": {
        "heads": heads, "dim": dim, "vdim": vdim, "tau": tau}}


def mamba2(heads, vdim, state, groups=1, taps=4, norm_groups=1):
    return {"type": "mamba2", "mixer": {
        "heads": heads, "vdim": vdim, "state": state, "groups": groups,
        "conv": taps, "norm_groups": norm_groups}}


def config(layers, vocab, width, ff, limit, eps=1e-5):
    """ff, limit: one value for all layers, or a list (None: no
    feed-forward)."""
    n = len(layers)
    ffs = ff if isinstance(ff, list) else [ff] * n
    limits = limit if isinstance(limit, list) else [limit] * n
    return {"architecture": "Taletar", "vocab": vocab, "width": width,
            "norm": {"eps": eps},
            "layers": [{**ly, "mlp": None if f is None else
                        {"kind": "dense", "ff": f, "limit": lim}}
                       for ly, f, lim in zip(layers, ffs, limits)]}


# sizes that fit no vector or tile, a layer without a feed-forward, no
# cap, no temperature, one tap
ODD = config([mamba2(6, 5, 11, groups=3, taps=2, norm_groups=5),
              attention(6, 3, 7, 9, softcap=None, q_temp=None, diff=0.35),
              gla(3, 10, 13, tau=1.0, low=5),
              attention(5, 1, 10, 11, softcap=5.0, diff=0.7),
              mamba2(2, 9, 17, groups=1, taps=1, norm_groups=2)],
             vocab=131, width=52, ff=[70, 33, None, 44, 58],
             limit=[0.7, 1.1, 0, 5.0, 0.4], eps=1e-4)
# sizes of the tiled kernels; more than 16 heads to a key/value head,
# grouped heads, a cap above what the fixed reference takes
TILED = config([attention(20, 1, 40, 72, softcap=25.0, q_temp=(0.2, 16)),
                mamba2(8, 48, 64, groups=4, taps=3, norm_groups=2),
                attention(8, 4, 24, 136, softcap=90.0, diff=0.45,
                          q_temp=(0.5, 33)),
                gla(4, 64, 96, tau=4.0, low=24),
                gla(2, 128, 40, tau=16.0, low=8),
                attention(6, 6, 72, 64, softcap=None, diff=0.2)],
               vocab=320, width=256, ff=208, limit=0.8, eps=1e-6)
# one layer of each kind, for long runs
PLAIN = config([gla(2, 32, 24, low=9), attention(3, 1, 16, 40),
                mamba2(4, 16, 24, groups=2)],
               vocab=97, width=64, ff=96, limit=1.5)


def mixer_weights(rand, out, p, ly, W):
    """Weights of one mixer; ``rand(name, *shape, std=)`` fills ``out``."""
    m = ly["mixer"]
    H, V = m["heads"], m["vdim"]
    if ly["type"] == "attention":
        D, G = m["dim"], m["kv_heads"]
        rand(p + "q", H * 2 * D, W)
        rand(p + "k", G * 2 * D, W)
        rand(p + "v", G * V, W)
        rand(p + "g", H * V, W)
        for n in ("lq1", "lk1", "lq2", "lk2"):
            rand(p + n, D, std=0.8 * D ** -0.25)
    elif ly["type"] == "gla":
        D, low = m["dim"], ly["low"]
        for name, rows in (("q", H * D), ("k", H * D), ("v", H * V),
                           ("g", H * V), ("a1", low)):
            rand(p + name, rows, W)
        rand(p + "a2", H * D, low)
        rand(p + "a2.b", H * D, std=1.5)
        rand(p + "norm", V, std=0.3)
        out[p + "norm"] += 1
    else:
        N, G, inner = m["state"], m["groups"], H * V
        C = inner + 2 * G * N
        rand(p + "in", inner + C + H, W)
        rand(p + "conv", C, m["conv"], std=0.6)
        rand(p + "conv.b", C, std=0.4)
        rand(p + "dt_bias", H, std=1.0)
        out[p + "dt_bias"] -= 2
        rand(p + "A_log", H, std=0.9)
        rand(p + "D", H, std=1.0)
        rand(p + "norm", inner, std=0.3)
        out[p + "norm"] += 1
    rand(p + "o", W, H * V)


def weights(cfg, seed=0, dtype=torch.bfloat16):
    g = torch.Generator().manual_seed(seed)
    W, V = cfg["width"], cfg["vocab"]
    out = {}

    def rand(name, *shape, std=None):
        out[name] = (torch.randn(*shape, generator=g)
                     * (shape[-1] ** -0.5 if std is None else std)).to(dtype)

    rand("embed", V, W, std=1.0)
    rand("head", V, W)
    norms = ["final.norm"]
    for i, ly in enumerate(cfg["layers"]):
        mixer_weights(rand, out, f"l{i}.mix.", ly, W)
        norms.append(f"l{i}.norm1")
        if ly["mlp"] is not None:
            norms.append(f"l{i}.norm2")
            for name in ("gate", "up"):
                rand(f"l{i}.mlp.{name}", ly["mlp"]["ff"], W)
            rand(f"l{i}.mlp.down", W, ly["mlp"]["ff"])
    for name in norms:
        rand(name, W, std=0.2)
        out[name] += 1
    return out


# -- one mixer alone -------------------------------------------------------

class Projected(nn.Module):
    """A mixer for parallel layers with its output projection, in double
    precision; the mixer writes into columns of wider rows, and must
    leave the others alone."""

    def __init__(self, mix, w_o):
        super().__init__()
        self.mix, self.w_o = mix, w_o.double()
        self.device, self.dtype = mix.device, mix.dtype
        self.cache_spec = mix.cache_spec

    def forward(self, x, b, cache, index):
        n = self.mix.out_width
        rows = torch.full((b.n_tok, n + 8), 3.0, dtype=x.dtype,
                          device=x.device)
        self.mix.inner(x, b, cache, index, rows[:, :n])
        assert (rows[:, n:] == 3.0).all()
        return rows[:, :n].cpu().double() @ self.w_o.T


def mixer(kind, m, w, eps, width, device="cpu", dtype=torch.float32,
          max_pos=1024):
    common = dict(width=width, eps=eps, dtype=dtype,
                  device=torch.device(device))
    if kind == "attention":
        mix = DifferentialAttention(
            heads=m["heads"], kv_heads=m["kv_heads"], dim=m["dim"],
            vdim=m["vdim"], softcap=m["softcap"], diff=m["diff"], **common)
        mix.q_scale = query_scale_table(max_pos, m["scale"],
                                        m["q_temp"]).to(device)
    elif kind == "gla":
        mix = GatedLinearAttention(
            heads=m["heads"], dim=m["dim"], vdim=m["vdim"], tau=m["tau"],
            decay_rank=w["a1"].shape[0], **common)
    else:
        mix = StateSpaceDuality(
            heads=m["heads"], vdim=m["vdim"], state=m["state"],
            groups=m["groups"], taps=m["conv"],
            norm_groups=m["norm_groups"], **common)
    mix.load({k: w[k] for k in mix.weight_shapes()})
    return Projected(mix, w["o"])


def case(ly, width, seed):
    """(oracle function, mixer sizes, weights in double)."""
    cfg = config([ly], 8, width, None, 0)
    w = {k[len("l0.mix."):]: t.double()
         for k, t in weights(cfg, seed).items() if k.startswith("l0.mix.")}
    return O.MIXERS[ly["type"]], ly["mixer"], w


def inputs(T, width, seed):
    g = torch.Generator().manual_seed(seed)
    return torch.randn(T, width, generator=g).bfloat16().double()


def plant(m, w, h, triples, strength=9.0):
    """Change the inputs of the queries so that for every (i, j1, j2) in
    ``triples`` query i's score with key j1 stands out in map 1 of every
    head, and with key j2 in map 2: W_q h_i is ``strength`` times the
    key over its squared length and the score's factor, and W_k h_i is
    zero, so that it is no outstanding key itself."""
    H, G, D = m["heads"], m["kv_heads"], m["dim"]
    assert w["q"].shape[1] > planted_width(m) - 8
    queries = {i for i, _, _ in triples}
    assert not any(j in queries for _, *js in triples for j in js)
    k = (h @ w["k"].T).view(-1, G, 2, D)[:, torch.arange(H) // (H // G)]
    h = h.clone()
    both = torch.cat([w["q"], w["k"]])
    for i, j1, j2 in triples:
        key = torch.stack([k[j1, :, 0], k[j2, :, 1]], 1)      # [H, 2, D]
        factor = m["scale"] * O.temperature(i, m["q_temp"])
        t = key / key.pow(2).sum(-1, keepdim=True) * strength / factor
        t = torch.cat([t.reshape(-1), torch.zeros(G * 2 * D).double()])
        h[i] = torch.linalg.lstsq(both, t[:, None],
                                  driver="gelsd").solution[:, 0]
    return h.bfloat16().double()


def planted_width(m):
    """A width at which ``plant`` has solutions of ordinary size."""
    return 3 * (m["heads"] + m["kv_heads"]) * m["dim"] + 8


def far_triples(T):
    """(query, key of map 1, key of map 2) for the first tokens, page
    and tile borders, keys just before the query, keys far back, and
    keys after the query, which must not count."""
    return [(T - 1, 0, 31), (T - 2, 15, 1), (T - 4, 16, 64), (T - 6, 63, 2),
            (T - 9, 32, 127), (T - 11, T - 12, 0), (T - 15, T - 14, 5),
            (T - 30, 128, T - 29), (100, 3, 101), (66, 65, 17), (35, 1, 33)]
