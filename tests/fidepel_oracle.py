"""Plain, slow Fidepel in double precision: one function per mechanism.

Tests compare the served model with this.  It imports nothing from
llmlb_amd, keeps no cache, and always runs a sequence from its start.
``w`` maps tensor names to tensors, ``cfg`` is the parsed config.json.
"""
from __future__ import annotations

import torch

F64 = torch.float64


def rms(x, eps):
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def sigmoid(x):
    return 1.0 / (1.0 + torch.exp(-x))


# -- attention -------------------------------------------------------------

def rotate(x, rot):
    """x [T, heads, D]: the first rot.dims numbers of every head turned
    by position times frequency, pairs half of them apart."""
    if not rot:
        return x
    n = rot["dims"]
    half = n // 2
    out = x.clone()
    factor = (rot.get("scaling") or {}).get("factor", 1.0)
    for p in range(x.shape[0]):
        for i in range(half):
            a = torch.tensor(p * rot["base"] ** (-2.0 * i / n) / factor,
                             dtype=x.dtype)
            u, v = x[p, :, i], x[p, :, i + half]
            out[p, :, i] = u * a.cos() - v * a.sin()
            out[p, :, i + half] = v * a.cos() + u * a.sin()
    return out


def sees(i, j, window):
    """Whether the query at i sees the key at j."""
    return 0 <= i - j and (window is None or i - j < window)


def windowed_attention(q, k, v, scale, temp, window):
    """q [T, H, D], k [T, G, D], v [T, G, V] -> [T, H, V]."""
    T, H, _ = q.shape
    group = torch.arange(H) // (H // k.shape[1])
    out = torch.zeros(T, H, v.shape[-1], dtype=q.dtype)
    for i in range(T):
        js = [j for j in range(i + 1) if sees(i, j, window)]
        s = torch.einsum("hd,jhd->hj", q[i], k[js][:, group]) * scale
        a = torch.softmax(s * temp[:, None], -1)
        out[i] = torch.einsum("hj,jhv->hv", a, v[js][:, group])
    return out


def attention(h, w, p, m, eps):
    T = h.shape[0]
    H, G, D, V = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q = rms(h @ w[p + "q"].T, eps) * w[p + "q.norm"]
    k = rms(h @ w[p + "k"].T, eps) * w[p + "k.norm"]
    v = (h @ w[p + "v"].T).view(T, G, V)
    q = rotate(q.view(T, H, D), m.get("rot"))
    k = rotate(k.view(T, G, D), m.get("rot"))
    o = windowed_attention(q, k, v, m["scale"], w[p + "temp"],
                           (m.get("mask") or {}).get("size"))
    o = o * sigmoid(h @ w[p + "g"].T)[:, :, None]
    return o.reshape(T, H * V) @ w[p + "o"].T


# -- mixture of experts ----------------------------------------------------

def expert(h, w, p):
    up = torch.clamp(h @ w[p + "up"].T, min=0.0)
    return (up * up) @ w[p + "down"].T


def choose(scores, top, groups):
    """Indices of the chosen experts of one token, by its scores."""
    E = scores.numel()
    count, keep = (groups or {}).get("count", 1), (groups or {}).get(
        "keep", 1)
    size = E // count
    best = sorted(range(count),
                  key=lambda g: -scores[g * size:(g + 1) * size].max())
    allowed = [e for e in range(E) if e // size in best[:keep]]
    return sorted(allowed, key=lambda e: -scores[e])[:top]


def routing(h, w_router, router):
    """[(expert, weight)] of every token."""
    scores = torch.softmax(h @ w_router.T, -1)
    out = []
    for s in scores:
        chosen = choose(s, router["top"], router.get("groups"))
        total = sum(s[e] for e in chosen) + 1e-20
        out.append([(e, s[e] / total * router["scale"]) for e in chosen])
    return out


def margins(h, w_router, router):
    """By how much each token's choice of experts is clear, as the ratio
    of scores (logarithm): between the last expert taken and the first
    one left, and between the last group kept and the next."""
    out = []
    count = (router.get("groups") or {}).get("count", 1)
    keep = (router.get("groups") or {}).get("keep", 1)
    for z in h @ w_router.T:
        chosen = choose(torch.softmax(z, -1), router["top"],
                        router.get("groups"))
        best = z.view(count, -1).amax(-1).sort(descending=True).values
        gaps = [best[keep - 1] - best[keep]] if keep < count else []
        size = z.numel() // count
        open_ = z.view(count, -1).amax(-1) >= best[keep - 1]
        rest = [z[e] for e in range(z.numel())
                if open_[e // size] and e not in chosen]
        if rest:
            gaps.append(z[chosen[-1]] - max(rest))
        out.append(float(min(gaps)) if gaps else float("inf"))
    return torch.tensor(out)


def mixture(h, w, p, mlp):
    y = torch.zeros_like(h)
    picks = routing(h, w[p + "router"], mlp["router"])
    for e in range(mlp["router"]["experts"]):
        rows = [t for t, pick in enumerate(picks) if e in dict(pick)]
        if rows:
            g = torch.stack([dict(picks[t])[e] for t in rows])
            y[rows] += g[:, None] * expert(h[rows], w, f"{p}e{e}.")
    if mlp.get("shared"):
        y = y + expert(h, w, p + "shared.")
    return y


# -- the model -------------------------------------------------------------

def layer_runs(cfg):
    """Layer index of every layer run, in order."""
    n, loop = len(cfg["layers"]), cfg.get("loop")
    if not loop:
        return list(range(n))
    return (list(range(loop["start"]))
            + list(range(loop["start"], loop["stop"])) * loop["times"]
            + list(range(loop["stop"], n)))


def forward(tokens, w, cfg, layers_out=None, clear=None):
    """Logits [T, vocab] in double precision.  ``clear`` (a list) gets
    every position's smallest margin over all layer runs."""
    w = {k: t.to(F64) for k, t in w.items()}
    eps, mult = cfg["norm"]["eps"], cfg["residual_mult"]
    x = w["embed"][torch.tensor(tokens, dtype=torch.long)]
    least = torch.full((len(tokens),), float("inf"))
    for i in layer_runs(cfg):
        layer = cfg["layers"][i]
        h = rms(x, eps) * w[f"l{i}.norm1"]
        y = attention(h, w, f"l{i}.mix.", layer["mixer"], eps)
        if layer.get("mlp") is not None:
            y = y + mixture(h, w, f"l{i}.mlp.", layer["mlp"])
            if clear is not None:
                least = torch.minimum(least, margins(
                    h, w[f"l{i}.mlp.router"], layer["mlp"]["router"]))
        x = x + mult * y
        if layers_out is not None:
            layers_out.append(x)
    if clear is not None:
        clear.extend(least.tolist())
    return (rms(x, eps) * w["final.norm"]) @ w["head"].T
