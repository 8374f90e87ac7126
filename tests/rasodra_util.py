"""Small random Rasodra models and mixers for tests.

Configurations are plain dictionaries in the layout of config.json, so
that the oracle and the served model read the same thing.
"""
from __future__ import annotations

import math

import torch

import rasodra_oracle as O
from llmlb_amd.backend.kv_cache import StateSpec
from llmlb_amd.models.mixers import (GroupedAttention, LatentAttention,
                                     MatrixMemory)
from llmlb_amd.ops import hybrid as hy
from llmlb_amd.ops.reference import build_cos_sin_table
from packed_util import (MixerRun, engine, error, run_cuts,  # noqa: F401
                         serve_at_random, tokens, write_model)


def attention(heads, kv_heads, dim, chunk, rot=None, base=3000.0,
              scale=None):
    rot = dim // 2 * 2 if rot is None else rot
    return {"type": "attention", "mixer": {
        "heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": dim,
        "mask": chunk and {"size": chunk},
        "rot": rot and {"base": base, "dims": rot},
        "scale": scale or 1.7 * dim ** -0.5}}


def latent(heads, dim, rot, vdim, rank, base=900.0, scale=None):
    return {"type": "latent_attention", "mixer": {
        "heads": heads, "dim": dim, "rot_dim": rot, "vdim": vdim,
        "kv_rank": rank, "rot": {"base": base, "dims": rot},
        "scale": scale or 1.4 * (dim + rot) ** -0.5}}


def memory(heads, dim, vdim, cap=9.0):
    return {"type": "mlstm", "mixer": {"heads": heads, "dim": dim,
                                       "vdim": vdim, "gate_cap": cap}}


def config(layers, vocab, width, ff, eps=1e-5):
    """``layers``: mixers, or the number of the layer whose weights serve
    once more; ff: one width for all, or a list (None: no feed-forward)."""
    out = []
    ffs = ff if isinstance(ff, list) else [ff] * len(layers)
    for ly, f in zip(layers, ffs):
        if isinstance(ly, int):
            out.append({**out[ly], "weights_of": ly})
        else:
            out.append({**ly, "mlp": None if f is None else
                        {"kind": "dense", "ff": f}})
    return {"architecture": "Rasodra", "vocab": vocab, "width": width,
            "norm": {"eps": eps}, "layers": out}


# sizes that fit no vector or tile; weights used again across other
# layers, and through a layer that uses another's itself
ODD = config([memory(3, 7, 9, cap=3.0), latent(5, 7, 6, 9, 11),
              attention(6, 3, 10, 13, rot=6), 1, memory(2, 11, 5), 2, 0, 5],
             vocab=131, width=52, ff=[None, 70, 33, 0, 44, 0, 0, 0],
             eps=1e-4)
# sizes of the tiled kernels; more than 16 heads to a key/value head and
# to a latent
TILED = config([attention(20, 1, 48, 50, rot=32), latent(20, 40, 24, 72, 96),
                memory(8, 48, 64), attention(6, 6, 80, 33, rot=80, scale=0.3),
                latent(6, 64, 32, 128, 136), memory(3, 128, 40, cap=20.0), 1,
                2, 3],
               vocab=320, width=256, ff=[208, None, 104, 160, 96, None, 0, 0,
                                         0], eps=1e-6)
# one layer of each kind, for long runs
PLAIN = config([memory(2, 32, 24), attention(3, 1, 16, 37),
                latent(4, 24, 8, 16, 40), 0], vocab=97, width=64, ff=96)


def mixer_weights(rand, out, p, ly, W):
    """Weights of one mixer; ``rand(name, *shape, std=)`` fills ``out``."""
    m = ly["mixer"]
    H, D, V = m["heads"], m["dim"], m["vdim"]

    def around_one(name, n):
        rand(p + name, n, std=0.3)
        out[p + name] += 1

    if ly["type"] == "attention":
        G = m["kv_heads"]
        for name, n in (("q", H), ("k", G)):
            rand(p + name, n * D, W)
            rand(p + name + ".b", n * D, std=0.6)
            around_one(name + ".norm", D)
    elif ly["type"] == "latent_attention":
        R, rank = m["rot_dim"], m["kv_rank"]
        rand(p + "q", H * (D + R), W)
        rand(p + "dkv", rank + R, W)
        around_one("dkv.norm", rank)
        rand(p + "uk", H * D, rank)
        rand(p + "uv", H * V, rank)
        rand(p + "sink", H, std=1.2)
        out[p + "sink"] += 1
        rand(p + "g", H * V, W)
    else:
        rand(p + "q", H * D, W)
        rand(p + "k", H * D, W)
        rand(p + "v", H * V, W)
        rand(p + "g", H * V, W)
        around_one("norm", H * V)
        for name, mean in (("i", -1.0), ("f", 2.5)):
            rand(p + name, H, W, std=1.5 * W ** -0.5)
            rand(p + name + ".b", H, std=1.0)
            out[p + name + ".b"] += mean
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
        if "weights_of" in ly:
            continue
        mixer_weights(rand, out, f"l{i}.mix.", ly, W)
        norms += [f"l{i}.norm1", f"l{i}.norm1b"]
        if ly["mlp"] is not None:
            norms += [f"l{i}.norm2", f"l{i}.norm2b"]
            rand(f"l{i}.mlp.up", ly["mlp"]["ff"], W)
            rand(f"l{i}.mlp.down", W, ly["mlp"]["ff"])
    for name in norms:
        rand(name, W, std=0.2)
        out[name] += 1
    return out


# -- one mixer alone -------------------------------------------------------

def mixer(kind, m, w, eps, width, device="cpu", dtype=torch.float32,
          max_pos=1024):
    common = dict(width=width, eps=eps, dtype=dtype,
                  device=torch.device(device))
    rot = m.get("rot")
    if kind == "attention":
        mix = GroupedAttention(
            heads=m["heads"], kv_heads=m["kv_heads"], dim=m["dim"],
            vdim=m["vdim"], rot=rot["dims"] if rot else 0, scale=m["scale"],
            window=(m["mask"] or {}).get("size"), chunk=True, bias=True,
            tied=True, interleaved=True, **common)
    elif kind == "latent_attention":
        mix = LatentAttention(
            heads=m["heads"], dim=m["dim"], rot_dim=m["rot_dim"],
            vdim=m["vdim"], kv_rank=m["kv_rank"], scale=m["scale"],
            window=None, kv_from=None, interleaved=True, sink=True,
            gate=True, **common)
    else:
        mix = MatrixMemory(heads=m["heads"], dim=m["dim"], vdim=m["vdim"],
                           gate_cap=m["gate_cap"], **common)
    if rot:
        mix.cos_sin = build_cos_sin_table(max_pos, rot["dims"],
                                          rot["base"]).to(device)
    mix.load({k: w[k] for k in mix.weight_shapes()})
    return mix


def case(ly, width, seed):
    """(oracle function, mixer sizes, weights in double)."""
    cfg = config([ly], 8, width, None)
    w = {k[len("l0.mix."):]: t.double()
         for k, t in weights(cfg, seed).items() if k.startswith("l0.mix.")}
    return O.MIXERS[ly["type"]], ly["mixer"], w


def inputs(T, width, seed):
    g = torch.Generator().manual_seed(seed)
    return torch.randn(T, width, generator=g).bfloat16().double()


class MemoryOp:
    """Matrix memory without its projections, as MixerRun takes it: the
    inputs are rows q | k | v | gate | i | f."""

    def __init__(self, ly, bias, norm, eps, device, dtype):
        self.m, self.eps = ly["mixer"], eps
        self.device, self.dtype = torch.device(device), dtype
        self.bias = bias.float().to(device)
        self.norm = norm.float().to(device)
        H, D, V = (self.m[k] for k in ("heads", "dim", "vdim"))
        at, self.offs = 0, []
        for n in (H * D, H * D, H * V, H * V, 2 * H):
            self.offs.append(at)
            at += n + -n % 8
        self.width = at

    def cache_spec(self):
        H, D, V = (self.m[k] for k in ("heads", "dim", "vdim"))
        return StateSpec(H, V, D, 0, 0, hy.memory_extra(D))

    def __call__(self, x, b, cache, index):
        H, D, V = (self.m[k] for k in ("heads", "dim", "vdim"))
        out = torch.full((b.n_tok, H * V + 8), 3.0, dtype=x.dtype,
                         device=x.device)
        hy.matrix_memory(out[:, :H * V], x, *self.offs[1:], self.bias,
                         self.m["gate_cap"], cache.state[index],
                         cache.extra[index], b, self.norm, H, D, V, self.eps)
        assert (out[:, H * V:] == 3.0).all()
        return out[:, :H * V]

    def rows(self, T, seed, put=-1.0, forget=2.5):
        """Random inputs, bf16 numbers; gates around ``put`` and
        ``forget``."""
        x = inputs(T, self.width, seed)
        at, H = self.offs[4], self.m["heads"]
        x[:, at:at + H] = 1.5 * x[:, at:at + H] + put
        x[:, at + H:at + 2 * H] = 1.5 * x[:, at + H:at + 2 * H] + forget
        return x.bfloat16().double()

    def oracle(self, x):
        T = x.shape[0]
        H, D, V = (self.m[k] for k in ("heads", "dim", "vdim"))
        q, k, v, g, z = (x[:, a:a + n] for a, n in zip(
            self.offs, (H * D, H * D, H * V, H * V, 2 * H)))
        bias = self.bias.double().cpu()
        li, lf = O.gates(z[:, :H] + bias[0], z[:, H:] + bias[1],
                         self.m["gate_cap"])
        o = O.memory(q.reshape(T, H, D) * D ** -0.5, k.reshape(T, H, D),
                     v.reshape(T, H, V), li, lf)
        o = O.rms(o, self.eps).reshape(T, H * V) * self.norm.double().cpu()
        return o * O.sigmoid(g)


def memory_op(ly, seed, device="cpu", dtype=torch.float32, eps=1e-4):
    m = ly["mixer"]
    g = torch.Generator().manual_seed(seed)
    return MemoryOp(ly, 0.5 * torch.randn(2, m["heads"], generator=g),
                    1 + 0.3 * torch.randn(m["heads"] * m["vdim"],
                                          generator=g), eps, device, dtype)


def turn_back(x, p, rot):
    """x [heads, D] rotated from position p to position 0."""
    out = x.clone()
    for i in range(rot["dims"] // 2 if rot else 0):
        a = -p * rot["base"] ** (-2.0 * i / rot["dims"])
        u, v = x[:, 2 * i], x[:, 2 * i + 1]
        out[:, 2 * i] = u * math.cos(a) - v * math.sin(a)
        out[:, 2 * i + 1] = v * math.cos(a) + u * math.sin(a)
    return out


def planted_width(kind, m):
    """A width at which ``plant`` has solutions of ordinary size."""
    H, D = m["heads"], m["dim"]
    if kind == "attention":
        return 3 * (H + m["kv_heads"]) * D + 8
    return 3 * (H * (D + m["rot_dim"]) + m["kv_rank"] + m["rot_dim"]) + 8


def plant(kind, m, w, h, pairs, eps, strength=9.0):
    """Change the inputs of the queries so that for every (i, j) in
    ``pairs`` query i's scores point at key j in every head, and query i's
    own key is nothing special."""
    H, D, T = m["heads"], m["dim"], h.shape[0]
    queries = {i for i, _ in pairs}
    assert not any(j in queries for _, j in pairs)
    h = h.clone()
    if kind == "attention":
        # normed queries all have one length: only their direction counts
        G = m["kv_heads"]
        k = (h @ w["k"].T + w["k.b"]).view(T, G, D)
        k = O.rms(k, eps) * w["k.norm"]
        rot = m["rot"]
        if rot:
            k = O.rotate(k, rot["base"], rot["dims"])
        both = torch.cat([w["q"], w["k"]])
        group = torch.arange(H) // (H // G)
        for i, j in pairs:
            q = turn_back(k[j, group], i, rot) / w["q.norm"]
            q = q / q.pow(2).mean(-1, keepdim=True).sqrt()
            t = torch.cat([q.reshape(-1) - w["q.b"],
                           torch.zeros(G * D).double()])
            h[i] = torch.linalg.lstsq(both, t[:, None],
                                      driver="gelsd").solution[:, 0]
    else:
        R, rot = m["rot_dim"], m["rot"]
        c, kr = torch.split(h @ w["dkv"].T, [m["kv_rank"], R], -1)
        c = O.rms(c, eps) * w["dkv.norm"]
        k = (c @ w["uk"].T).view(T, H, D)
        kr = O.rotate(kr[:, None], rot["base"], R)[:, 0]
        both = torch.cat([w["q"], w["dkv"]])
        for i, j in pairs:
            full = torch.cat([k[j], turn_back(
                kr[j].expand(H, R), i, rot)], -1)
            q = full / full.pow(2).sum(-1, keepdim=True) * (
                strength / m["scale"])
            t = torch.cat([q.reshape(-1), torch.zeros(
                w["dkv"].shape[0]).double()])
            h[i] = torch.linalg.lstsq(both, t[:, None],
                                      driver="gelsd").solution[:, 0]
    return h.bfloat16().double()


def far_pairs(T):
    """(query, key) for the first tokens, page and tile borders, keys
    just before the query, keys far back, and keys after the query, which
    must not count."""
    return [(T - 1, 0), (T - 2, 15), (T - 4, 16), (T - 6, 63), (T - 9, 32),
            (T - 11, 64), (T - 13, T - 14), (T - 15, T - 16),
            (T - 17, T - 18), (T - 30, T - 29), (100, 3), (66, 65), (35, 1),
            (130, 127), (131, 128), (40, 41)]


def chunk_pairs(T, size):
    """(query, key): the first key of the query's chunk and the one just
    before it, for queries at a chunk's start, in it, and at its end."""
    out = []
    for c in range(1, T // size):
        first = c * size
        out += [(first + 1, first if c % 2 else first - 1),
                (first + size // 2, first - 1 if c % 2 else first),
                (first + size - 2, first if c % 3 else first - 1)]
    return [(i, j) for i, j in out if 0 <= j and i < T and i != j]
