"""Small random Fidepel models and mixers for tests.

Configurations are plain dictionaries in the layout of config.json, so
that the oracle and the served model read the same thing.
"""
from __future__ import annotations

import torch
import torch.nn as nn

import fidepel_oracle as O
from llmlb_amd.models.mixers import (RoutedExperts, WindowedAttention,
                                     _stack_rows)
from llmlb_amd.ops.reference import build_cos_sin_table
from packed_util import (MixerRun, engine, error, run_cuts,  # noqa: F401
                         serve_at_random, tokens, write_model)


def attention(heads, kv_heads, dim, vdim, window=None, dims=None, base=1e4,
              factor=1.0, scale=None):
    """window None: all keys; dims None: the whole head turns, 0: none."""
    m = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim,
         "scale": scale or 4.0 / dim}
    if window is not None:
        m["mask"] = {"size": window}
    if dims != 0:
        m["rot"] = {"base": base, "dims": dim if dims is None else dims}
        if factor != 1.0:
            m["rot"]["scaling"] = {"factor": factor}
    return m


def moe(experts, top, ff, groups=None, shared=None, scale=1.0):
    """groups: (count, keep)."""
    out = {"kind": "moe", "expert": {"ff": ff},
           "router": {"experts": experts, "top": top, "scale": scale}}
    if groups:
        out["router"]["groups"] = dict(zip(("count", "keep"), groups))
    if shared:
        out["shared"] = {"ff": shared}
    return out


def config(layers, vocab, width, mult, loop=None, eps=1e-5):
    """layers: (mixer, mlp) pairs; loop: (start, stop, times)."""
    cfg = {"architecture": "Fidepel", "vocab": vocab, "width": width,
           "norm": {"eps": eps}, "residual_mult": mult,
           "layers": [{"type": "attention", "mixer": m, "mlp": f}
                      for m, f in layers]}
    if loop:
        cfg["loop"] = dict(zip(("start", "stop", "times"), loop))
    return cfg


# sizes that fit no vector or tile; no window, no rotation, no groups, no
# shared expert, no feed-forward, a window of one token; the last layer
# loops
ODD = config([(attention(6, 3, 7, 9, window=13, dims=4), moe(5, 2, 11)),
              (attention(5, 1, 10, 11, dims=0), None),
              (attention(3, 3, 9, 5, window=1, dims=8, factor=3.0),
               moe(6, 1, 13, groups=(3, 1), shared=7, scale=1.7)),
              (attention(4, 2, 6, 15, window=30),
               moe(7, 7, 5, shared=10, scale=0.6))],
             vocab=131, width=52, mult=0.6, loop=(2, 4, 3), eps=1e-4)
# sizes of the tiled kernels; more than 16 heads to a key/value head
TILED = config([(attention(20, 1, 48, 72, window=50, dims=32, factor=2.0),
                 moe(12, 3, 88, groups=(4, 2), shared=40, scale=1.3)),
                (attention(6, 2, 32, 24, window=37, base=500.0),
                 moe(24, 5, 40, groups=(6, 3), shared=136)),
                (attention(2, 2, 80, 136, window=96, dims=48),
                 moe(9, 2, 64)),
                (attention(4, 4, 16, 64, dims=0),
                 moe(70, 4, 24, groups=(10, 4), shared=8, scale=2.5))],
               vocab=320, width=200, mult=0.5, loop=(1, 3, 2), eps=1e-6)
# two layers, for long runs
PLAIN = config([(attention(3, 1, 16, 40, window=45),
                 moe(6, 2, 32, groups=(3, 2), shared=48)),
                (attention(4, 2, 24, 16, window=70, factor=4.0),
                 moe(4, 1, 40))],
               vocab=97, width=64, mult=0.8)


def weights(cfg, seed=0, dtype=torch.bfloat16):
    g = torch.Generator().manual_seed(seed)
    W, vocab = cfg["width"], cfg["vocab"]
    out = {}

    def rand(name, *shape, std=None, mean=0.0):
        out[name] = (torch.randn(shape, generator=g) * (
            shape[-1] ** -0.5 if std is None else std) + mean).to(dtype)

    rand("embed", vocab, W, std=1.0)
    rand("head", vocab, W)
    rand("final.norm", std=0.2, mean=1.0)
    for i, ly in enumerate(cfg["layers"]):
        rand(f"l{i}.norm1", std=0.2, mean=1.0)
        mixer_weights(rand, f"l{i}.mix.", ly["mixer"], W)
        if ly["mlp"] is not None:
            expert_weights(rand, f"l{i}.mlp.", ly["mlp"], W)
    return out


def mixer_weights(rand, p, m, W):
    H, G, D, V = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    rand(p + "q", H * D, W)
    rand(p + "k", G * D, W)
    rand(p + "v", G * V, W)
    rand(p + "g", H, W)
    rand(p + "o", W, H * V)
    rand(p + "q.norm", H * D, std=0.3, mean=1.0)
    rand(p + "k.norm", G * D, std=0.3, mean=1.0)
    rand(p + "temp", H, std=0.3, mean=1.2)


def expert_weights(rand, p, mlp, W):
    rand(p + "router", mlp["router"]["experts"], W, std=3.0 * W ** -0.5)
    parts = [(f"e{e}", mlp["expert"]["ff"])
             for e in range(mlp["router"]["experts"])]
    if mlp.get("shared"):
        parts.append(("shared", mlp["shared"]["ff"]))
    for name, ff in parts:
        rand(f"{p}{name}.up", ff, W)
        rand(f"{p}{name}.down", W, ff)


def clear_rows(margin, dtype):
    """Positions whose choice of experts the rounding of ``dtype`` does
    not decide."""
    return torch.tensor(margin) > (0.05 if dtype == "bfloat16" else 1e-4)


def clear_error(got, want, margin, dtype):
    """``error`` over the positions with clear choices; in bfloat16 the
    worst in fifty of them may still have gone the other way."""
    keep = clear_rows(margin, dtype)
    assert keep.float().mean() > 0.3
    d = (got.cpu().double() - want)[keep].pow(2).mean(-1).sqrt().sort().values
    spare = -(-len(d) // 50) if dtype == "bfloat16" and len(d) > 10 else 0
    return (d[len(d) - 1 - spare] / want.std()).item()


# -- one mixer alone -------------------------------------------------------

class Projected(nn.Module):
    """Windowed attention with its input and output projections; the
    mixer writes into columns of wider rows, and must leave the others
    alone."""

    def __init__(self, mix, w):
        super().__init__()
        self.mix, self.w_o = mix, w["o"].double()
        stacked, offs = _stack_rows([w[k] for k in mix.inputs])
        mix.place(offs)
        self.w_in = stacked.to(mix.dtype).to(mix.device)
        self.device, self.dtype = mix.device, mix.dtype
        self.cache_spec = mix.cache_spec

    def forward(self, x, b, cache, index):
        n = self.mix.out_width
        rows = torch.full((b.n_tok, n + -n % 8 + 8), 3.0, dtype=x.dtype,
                          device=x.device)
        self.mix.inner(x @ self.w_in.T, b, cache, index, rows[:, :n])
        assert (rows[:, n:] == 3.0).all()
        return rows[:, :n].cpu().double() @ self.w_o.T


def mixer(m, w, eps, width, device="cpu", dtype=torch.float32, max_pos=1024):
    rot = m.get("rot") or {}
    mix = WindowedAttention(
        width=width, heads=m["heads"], kv_heads=m["kv_heads"], dim=m["dim"],
        vdim=m["vdim"], rot=rot.get("dims", 0), scale=m["scale"],
        window=(m.get("mask") or {}).get("size"), eps=eps, dtype=dtype,
        device=torch.device(device))
    mix.load({k: w[k] for k in mix.weight_shapes()})
    if rot:
        mix.cos_sin = build_cos_sin_table(
            max_pos, rot["dims"], rot["base"], factor=(
                rot.get("scaling") or {}).get("factor", 1.0)).to(device)
    return Projected(mix, w)


def attention_case(m, width, seed):
    """Weights of one attention mixer, in double precision."""
    g = torch.Generator().manual_seed(seed)
    out = {}

    def rand(name, *shape, std=None, mean=0.0):
        out[name] = (torch.randn(shape, generator=g) * (
            shape[-1] ** -0.5 if std is None else std)
            + mean).bfloat16().double()

    mixer_weights(rand, "", m, width)
    return out


def inputs(T, width, seed):
    g = torch.Generator().manual_seed(seed)
    return torch.randn(T, width, generator=g).bfloat16().double()


def planted_width(m):
    """A width at which ``plant`` has solutions."""
    return m["heads"] * m["dim"] + 16


def plant(m, w, h, pairs, eps=1e-5):
    """Change the inputs of the queries so that for every (i, j) in
    ``pairs`` query i's score with key j stands out in every head: before
    its norm, the query is the key at j turned back from j's place to
    i's, the norm's weights divided out."""
    H, G, D = m["heads"], m["kv_heads"], m["dim"]
    assert not {j for _, j in pairs} & {i for i, _ in pairs}
    k = O.rms(h @ w["k"].T, eps) * w["k.norm"]
    k = O.rotate(k.view(-1, G, D), m.get("rot"))
    h = h.clone()
    for i, j in pairs:
        key = k[j, torch.arange(H) // (H // G)]             # [H, D]
        rows = torch.zeros(i + 1, H, D, dtype=h.dtype)
        rows[i] = key
        # turning by -p: flip the sign of the second half before and after
        t = rows[i]
        if m.get("rot"):
            n = m["rot"]["dims"]
            sign = torch.ones(D, dtype=h.dtype)
            sign[n // 2:n] = -1
            t = O.rotate(rows * sign, m["rot"])[i] * sign
        t = t.reshape(-1) / w["q.norm"]
        h[i] = torch.linalg.lstsq(w["q"], t[:, None],
                                  driver="gelsd").solution[:, 0]
    return h.bfloat16().double()


def edge_pairs(window, T):
    """(query, key) at the window's edges, just inside and just outside,
    at page and tile borders, the first tokens, and the next token."""
    W = window or T
    out = []
    spare = iter(range(T - 1, 0, -3))      # queries, none of them a key
    keys = [0, 1, 15, 16, 17, 31, 32, 63, 64, 65]
    queries = []
    for j in keys:
        for i in (j + W - 1, j + W):       # last to see j, first not to
            if j < i < T and i not in keys and i not in queries:
                queries.append(i)
                out.append((i, j))
    used = set(keys)
    for back in (1, 2, W - 1, W, W + 1):
        for i in spare:
            j = i - back
            if j < 0:
                break
            if i in queries or i in used or j in queries or j == i:
                continue
            queries.append(i)
            used.add(j)
            out.append((i, j))
            break
    for i in spare:                        # a key after the query
        if i + 1 < T and i not in used and i not in queries \
                and i + 1 not in queries:
            out.append((i, i + 1))
            break
    assert not {j for _, j in out} & {i for i, _ in out}
    return out


def experts_module(mlp, w, width, device="cpu", dtype=torch.float32):
    groups = mlp["router"].get("groups") or {"count": 1, "keep": 1}
    ff = RoutedExperts(
        width=width, ff=mlp["expert"]["ff"],
        experts=mlp["router"]["experts"], top=mlp["router"]["top"],
        groups=groups["count"], keep=groups["keep"],
        scale=mlp["router"]["scale"],
        shared=(mlp.get("shared") or {}).get("ff"), dtype=dtype,
        device=torch.device(device))
    ff.load({k: w[k] for k in ff.weight_shapes()})
    return ff


def experts_case(mlp, width, seed):
    g = torch.Generator().manual_seed(seed)
    out = {}

    def rand(name, *shape, std=None, mean=0.0):
        out[name] = (torch.randn(shape, generator=g) * (
            shape[-1] ** -0.5 if std is None else std)
            + mean).bfloat16().double()

    expert_weights(rand, "", mlp, width)
    return out


def run_experts(ff, h):
    """The routed experts' sum alone, in double precision."""
    from llmlb_amd.ops import hybrid as hy
    x = h.to(ff.dtype).to(ff.device).contiguous()
    index, weight, lists = hy.route(*ff.routing(x))
    z = ff.routed(x, index, lists)
    return torch.einsum("tkw,tk->tw", z.cpu().double(),
                        weight.cpu().double())
