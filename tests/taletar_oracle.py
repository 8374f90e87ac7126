"""Plain, slow Taletar in double precision: one function per mechanism,
one token after another where the mechanism is a recurrence.

Tests compare the served model with this.  It imports nothing from
llmlb_amd, keeps no cache, and always runs a sequence from its start.
``w`` maps tensor names to tensors, ``cfg`` is the parsed config.json.
"""
from __future__ import annotations

import math

import torch

F64 = torch.float64


def rms(x, eps):
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def sigmoid(x):
    return 1.0 / (1.0 + torch.exp(-x))


def silu(x):
    return x * sigmoid(x)


def softplus(x):
    return torch.logaddexp(x, torch.zeros_like(x))


# -- differential attention ------------------------------------------------

def temperature(p, temp):
    """Factor of the query at position p."""
    if temp is None:
        return 1.0
    return 1.0 + temp["coef"] * math.log(
        math.floor((p + 1) / temp["every"]) + 1)


def cap_scores(s, cap):
    return cap * torch.tanh(s / cap) if cap else s


def causal_attention(q, k, v, scale, cap):
    """q [T, H, D], k [T, G, D], v [T, G, V] -> [T, H, V]."""
    T, H, _ = q.shape
    group = torch.arange(H) // (H // k.shape[1])
    out = torch.zeros(T, H, v.shape[-1], dtype=q.dtype)
    for i in range(T):
        s = torch.einsum("hd,jhd->hj", q[i], k[:i + 1, group]) * scale
        a = torch.softmax(cap_scores(s, cap), -1)
        out[i] = torch.einsum("hj,jhv->hv", a, v[:i + 1, group])
    return out


def mix_factor(w, p, diff):
    a = torch.exp((w[p + "lq1"] * w[p + "lk1"]).sum())
    b = torch.exp((w[p + "lq2"] * w[p + "lk2"]).sum())
    return a - b + diff


def attention(h, w, p, m, eps):
    T = h.shape[0]
    H, G, D, V = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q = (h @ w[p + "q"].T).view(T, H, 2, D)
    k = (h @ w[p + "k"].T).view(T, G, 2, D)
    v = (h @ w[p + "v"].T).view(T, G, V)
    t = torch.tensor([temperature(i, m.get("q_temp")) for i in range(T)],
                     dtype=h.dtype)
    q = q * t[:, None, None, None]
    a1, a2 = (causal_attention(q[:, :, n], k[:, :, n], v, m["scale"],
                               m.get("softcap")) for n in (0, 1))
    o = a1 - mix_factor(w, p, m["diff"]) * a2
    o = rms(o, eps) * (1.0 - m["diff"])
    o = o.reshape(T, H * V) * sigmoid(h @ w[p + "g"].T)
    return o @ w[p + "o"].T


# -- linear recurrences ----------------------------------------------------

def scan(q, k, v, g, S=None):
    """S <- diag(g) S + k v^T, o = S^T q.  q, k, g [T, H, D],
    v [T, H, V] -> o [T, H, V] and the last state [H, D, V]."""
    T, H, D = q.shape
    S = torch.zeros(H, D, v.shape[-1], dtype=q.dtype) if S is None else S
    out = torch.zeros(T, H, v.shape[-1], dtype=q.dtype)
    for t in range(T):
        S = g[t][:, :, None] * S + k[t][:, :, None] * v[t][:, None, :]
        out[t] = torch.einsum("hdv,hd->hv", S, q[t])
    return out, S


def gla(h, w, p, m, eps):
    T = h.shape[0]
    H, D, V = m["heads"], m["dim"], m["vdim"]
    q = (h @ w[p + "q"].T).view(T, H, D) * D ** -0.5
    k = (h @ w[p + "k"].T).view(T, H, D)
    v = (h @ w[p + "v"].T).view(T, H, V)
    z = (h @ w[p + "a1"].T) @ w[p + "a2"].T + w[p + "a2.b"]
    alpha = sigmoid(z) ** (1.0 / m["tau"])
    o, _ = scan(q, k, v, alpha.view(T, H, D))
    o = (rms(o, eps) * w[p + "norm"]).reshape(T, H * V)
    return (o * silu(h @ w[p + "g"].T)) @ w[p + "o"].T


def short_conv(x, taps, bias):
    """Causal convolution per channel then silu; taps [C, K], the last
    column is the current token's."""
    T, C = x.shape
    K = taps.shape[1]
    pad = torch.cat([torch.zeros(K - 1, C, dtype=x.dtype), x])
    y = bias.expand(T, C).clone()
    for i in range(K):
        y += pad[i:i + T] * taps[:, i]
    return silu(y)


def mamba2(h, w, p, m, eps):
    T = h.shape[0]
    H, V, N, G = m["heads"], m["vdim"], m["state"], m["groups"]
    inner = H * V
    z, x, B, C, dt = torch.split(
        h @ w[p + "in"].T, [inner, inner, G * N, G * N, H], -1)
    x, B, C = torch.split(
        short_conv(torch.cat([x, B, C], -1), w[p + "conv"],
                   w[p + "conv.b"]), [inner, G * N, G * N], -1)
    x = x.view(T, H, V)
    head = torch.arange(H) // (H // G)
    B, C = (t.view(T, G, N)[:, head] for t in (B, C))
    dt = softplus(dt + w[p + "dt_bias"])
    g = torch.exp(-torch.exp(w[p + "A_log"]) * dt)
    y, _ = scan(C, B, dt[:, :, None] * x, g[:, :, None].expand(T, H, N))
    y = (y + w[p + "D"][:, None] * x).reshape(T, inner) * silu(z)
    y = rms(y.view(T, m["norm_groups"], -1), eps).reshape(T, inner)
    return (y * w[p + "norm"]) @ w[p + "o"].T


# -- the model -------------------------------------------------------------

def feed_forward(h, w, p, limit):
    g = torch.clamp(h @ w[p + "gate"].T, max=limit)
    u = torch.clamp(h @ w[p + "up"].T, -limit, limit)
    return (g * sigmoid(1.702 * g) * (u + 1.0)) @ w[p + "down"].T


MIXERS = {"attention": attention, "gla": gla, "mamba2": mamba2}


def forward(tokens, w, cfg, layers_out=None):
    """Logits [T, vocab] in double precision."""
    w = {k: t.to(F64) for k, t in w.items()}
    eps = cfg["norm"]["eps"]
    x = w["embed"][torch.tensor(tokens, dtype=torch.long)]
    for i, layer in enumerate(cfg["layers"]):
        n = rms(x, eps)
        y = MIXERS[layer["type"]](n * w[f"l{i}.norm1"], w, f"l{i}.mix.",
                                  layer["mixer"], eps)
        if layer["mlp"] is not None:
            y = y + feed_forward(n * w[f"l{i}.norm2"], w, f"l{i}.mlp.",
                                 layer["mlp"]["limit"])
        x = x + y
        if layers_out is not None:
            layers_out.append(x)
    return (rms(x, eps) * w["final.norm"]) @ w["head"].T
