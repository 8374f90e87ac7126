"""Plain, slow Rasodra in double precision: one function per mechanism,
one token after another where the mechanism is a recurrence.

Tests compare the served model with this.  It imports nothing from
llmlb_amd, keeps no cache, and always runs a sequence from its start.
``w`` maps tensor names to tensors, ``cfg`` is the parsed config.json.
"""
from __future__ import annotations

import torch

F64 = torch.float64


def rms(x, eps):
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def layer_norm(x, w, eps):
    d = x - x.mean(-1, keepdim=True)
    return d / torch.sqrt((d * d).mean(-1, keepdim=True) + eps) * w


def sigmoid(x):
    return 1.0 / (1.0 + torch.exp(-x))


def log_sigmoid(x):
    return -torch.logaddexp(-x, torch.zeros_like(x))


def rotate(x, base, n):
    """x [T, heads, D]: neighbours (2i, 2i + 1) among the first n numbers
    of every head turn by position times base^(-2i/n)."""
    out = x.clone()
    p = torch.arange(x.shape[0], dtype=F64)[:, None]
    for i in range(n // 2):
        a = p * base ** (-2.0 * i / n)
        u, v = x[:, :, 2 * i], x[:, :, 2 * i + 1]
        out[:, :, 2 * i] = u * a.cos() - v * a.sin()
        out[:, :, 2 * i + 1] = v * a.cos() + u * a.sin()
    return out


# -- matrix memory ---------------------------------------------------------

def gates(zi, zf, cap):
    """Log input and forget gates."""
    return cap * torch.tanh(zi / cap), log_sigmoid(cap * torch.tanh(zf / cap))


def memory(q, k, v, li, lf):
    """q, k [T, H, D] (q scaled), v [T, H, V], log gates [T, H]
    -> [T, H, V]."""
    T, H, D = q.shape
    S = torch.zeros(H, D, v.shape[-1], dtype=q.dtype)
    n = torch.zeros(H, D, dtype=q.dtype)
    m = torch.zeros(H, dtype=q.dtype)
    out = torch.zeros(T, H, v.shape[-1], dtype=q.dtype)
    for t in range(T):
        new = torch.maximum(lf[t] + m, li[t])
        keep = torch.exp(lf[t] + m - new)[:, None]
        put = torch.exp(li[t] - new)[:, None] * k[t]
        S = keep[:, :, None] * S + put[:, :, None] * v[t][:, None, :]
        n = keep * n + put
        m = new
        den = torch.maximum((n * q[t]).sum(-1).abs(), torch.exp(-m)) + 1e-6
        out[t] = torch.einsum("hdv,hd->hv", S, q[t]) / den[:, None]
    return out


def mlstm(h, w, p, m, eps):
    T = h.shape[0]
    H, D, V = m["heads"], m["dim"], m["vdim"]
    q = (h @ w[p + "q"].T).view(T, H, D) * D ** -0.5
    k = (h @ w[p + "k"].T).view(T, H, D)
    v = (h @ w[p + "v"].T).view(T, H, V)
    li, lf = gates(h @ w[p + "i"].T + w[p + "i.b"],
                   h @ w[p + "f"].T + w[p + "f.b"], m["gate_cap"])
    o = rms(memory(q, k, v, li, lf), eps).reshape(T, H * V) * w[p + "norm"]
    return (o * sigmoid(h @ w[p + "g"].T)) @ w[p + "o"].T


# -- attention -------------------------------------------------------------

def sink_softmax(s, sink):
    """s [H, keys]; exp(sink) [H] takes part in the sum only."""
    top = torch.maximum(s.amax(-1), sink)[:, None]
    e = torch.exp(s - top)
    return e / (e.sum(-1, keepdim=True) + torch.exp(sink[:, None] - top))


def latent_attention(h, w, p, m, eps):
    T = h.shape[0]
    H, D, R, V = m["heads"], m["dim"], m["rot_dim"], m["vdim"]
    base = m["rot"]["base"]
    q = (h @ w[p + "q"].T).view(T, H, D + R)
    c, kr = torch.split(h @ w[p + "dkv"].T, [m["kv_rank"], R], -1)
    c = rms(c, eps) * w[p + "dkv.norm"]
    k = (c @ w[p + "uk"].T).view(T, H, D)
    v = (c @ w[p + "uv"].T).view(T, H, V)
    qr = rotate(q[:, :, D:], base, R)
    kr = rotate(kr[:, None], base, R)[:, 0]
    out = torch.zeros(T, H, V, dtype=h.dtype)
    for i in range(T):
        s = torch.einsum("hd,jhd->hj", q[i, :, :D], k[:i + 1]) \
            + qr[i] @ kr[:i + 1].T
        a = sink_softmax(s * m["scale"], w[p + "sink"])
        out[i] = torch.einsum("hj,jhv->hv", a, v[:i + 1])
    return (out.reshape(T, H * V) * sigmoid(h @ w[p + "g"].T)) @ w[p + "o"].T


def sees(i, j, size):
    """Whether the query at i sees the key at j: both in one chunk."""
    return j <= i and (size is None or i // size == j // size)


def attention(h, w, p, m, eps):
    T = h.shape[0]
    H, G, D = m["heads"], m["kv_heads"], m["dim"]
    rot = m.get("rot") or {"base": 1.0, "dims": 0}
    q = (h @ w[p + "q"].T + w[p + "q.b"]).view(T, H, D)
    v = (h @ w[p + "k"].T + w[p + "k.b"]).view(T, G, D)
    q = rotate(rms(q, eps) * w[p + "q.norm"], rot["base"], rot["dims"])
    k = rotate(rms(v, eps) * w[p + "k.norm"], rot["base"], rot["dims"])
    group = torch.arange(H) // (H // G)
    size = (m.get("mask") or {}).get("size")
    out = torch.zeros(T, H, D, dtype=h.dtype)
    for i in range(T):
        js = [j for j in range(i + 1) if sees(i, j, size)]
        s = torch.einsum("hd,jhd->hj", q[i], k[js][:, group]) * m["scale"]
        out[i] = torch.einsum("hj,jhv->hv", torch.softmax(s, -1),
                              v[js][:, group])
    return out.reshape(T, H * D) @ w[p + "o"].T


# -- the model -------------------------------------------------------------

def feed_forward(h, w, p):
    up = torch.clamp(h @ w[p + "up"].T, min=0.0)
    return (up * up) @ w[p + "down"].T


MIXERS = {"mlstm": mlstm, "latent_attention": latent_attention,
          "attention": attention}


def owner(layers, i):
    """The layer whose tensors layer i uses."""
    while layers[i].get("weights_of") is not None:
        i = layers[i]["weights_of"]
    return i


def forward(tokens, w, cfg, layers_out=None):
    """Logits [T, vocab] in double precision."""
    w = {k: t.to(F64) for k, t in w.items()}
    eps = cfg["norm"]["eps"]
    x = w["embed"][torch.tensor(tokens, dtype=torch.long)]
    for i, layer in enumerate(cfg["layers"]):
        p = f"l{owner(cfg['layers'], i)}."
        h = layer_norm(x, w[p + "norm1"], eps)
        y = MIXERS[layer["type"]](h, w, p + "mix.", layer["mixer"], eps)
        x = x + layer_norm(y, w[p + "norm1b"], eps)
        if layer.get("mlp") is not None:
            y = feed_forward(layer_norm(x, w[p + "norm2"], eps), w,
                             p + "mlp.")
            x = x + layer_norm(y, w[p + "norm2b"], eps)
        if layers_out is not None:
            layers_out.append(x)
    return layer_norm(x, w["final.norm"], eps) @ w["head"].T
