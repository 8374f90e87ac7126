"""Plain, slow Dibelix in double precision: one function per mechanism,
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


def post_norm(y, weight, eps):
    """RMS norm whose stored weight is the distance from one."""
    return rms(y, eps) * (1.0 + weight)


def silu(x):
    return x / (1.0 + torch.exp(-x))


def gelu_tanh(z):
    inner = math.sqrt(2.0 / math.pi) * (z + 0.044715 * z ** 3)
    return 0.5 * z * (1.0 + torch.tanh(inner))


def rotate(x, pos, base):
    """x [T, ..., R] rotated at positions pos [T]; channel i turns with
    channel i + R/2."""
    R = x.shape[-1]
    half = R // 2
    out = x.clone()
    for i in range(half):
        ang = pos.to(F64) * base ** (-2.0 * i / R)
        ang = ang.reshape([-1] + [1] * (x.dim() - 2))
        u, v = x[..., i], x[..., i + half]
        out[..., i] = u * torch.cos(ang) - v * torch.sin(ang)
        out[..., i + half] = v * torch.cos(ang) + u * torch.sin(ang)
    return out


def latent_kv(h, w, p, m, eps):
    """(latent [T, rank], rotated key part [T, rot]) of one layer."""
    T = h.shape[0]
    r = m["kv_rank"]
    d = h @ w[p + "dkv"].T
    c = rms(d[:, :r], eps) * w[p + "dkv.norm"]
    return c, rotate(d[:, r:], torch.arange(T), m["rot"]["base"])


def window_attention(q, k, v, scale, size):
    """q, k [T, H, D], v [T, H, V]; key j is seen by i when
    0 <= i - j < size."""
    T, H, _ = q.shape
    out = torch.zeros(T, H, v.shape[-1], dtype=q.dtype)
    for i in range(T):
        lo = max(0, i - size + 1)
        s = torch.einsum("hd,jhd->hj", q[i], k[lo:i + 1]) * scale
        a = torch.softmax(s, -1)
        out[i] = torch.einsum("hj,jhv->hv", a, v[lo:i + 1])
    return out


def latent_attention(h, w, p, m, eps, shared=None):
    """Returns (output, latent, rotated key).  ``shared`` is another
    layer's (latent, rotated key)."""
    T = h.shape[0]
    H, D, R, V = m["heads"], m["dim"], m["rot_dim"], m["vdim"]
    c, kr = shared if shared is not None else latent_kv(h, w, p, m, eps)
    q = (h @ w[p + "q"].T).view(T, H, D + R)
    qr = rotate(q[..., D:], torch.arange(T), m["rot"]["base"])
    k = (c @ w[p + "uk"].T).view(T, H, D)
    v = (c @ w[p + "uv"].T).view(T, H, V)
    o = window_attention(
        torch.cat([q[..., :D], qr], -1),
        torch.cat([k, kr[:, None].expand(T, H, R)], -1), v,
        m["scale"], m["mask"]["size"])
    return o.reshape(T, H * V) @ w[p + "o"].T, c, kr


def short_conv(x, taps):
    """Causal convolution per channel then silu; taps [C, K], the last
    column is the current token's."""
    T, C = x.shape
    K = taps.shape[1]
    pad = torch.cat([torch.zeros(K - 1, C, dtype=x.dtype), x])
    y = torch.zeros_like(x)
    for i in range(K):
        y += pad[i:i + T] * taps[:, i]
    return silu(y)


def unit(x):
    return x / torch.sqrt((x * x).sum(-1, keepdim=True) + 1e-6)


def delta_rule(q, k, v, g, beta):
    """q, k, g [T, H, D], v [T, H, V], beta [T, H] -> o [T, H, V] and
    the final state [H, D, V]."""
    T, H, D = q.shape
    V = v.shape[-1]
    S = torch.zeros(H, D, V, dtype=q.dtype)
    out = torch.zeros(T, H, V, dtype=q.dtype)
    for t in range(T):
        for n in range(H):
            S[n] = g[t, n][:, None] * S[n]
            u = beta[t, n] * (v[t, n] - S[n].T @ k[t, n])
            S[n] = S[n] + torch.outer(k[t, n], u)
            out[t, n] = S[n].T @ q[t, n]
    return out, S


def decay(h, w, p, H, D):
    z = (h @ w[p + "a1"].T) @ w[p + "a2"].T + w[p + "dt_bias"]
    z = z.view(h.shape[0], H, D)
    return torch.exp(-torch.exp(w[p + "A_log"])[:, None]
                     * torch.nn.functional.softplus(z, threshold=50.0))


def channel_delta(h, w, p, m, eps):
    T = h.shape[0]
    H, KH, D, V = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q = short_conv(h @ w[p + "q"].T, w[p + "q.conv"]).view(T, KH, D)
    k = short_conv(h @ w[p + "k"].T, w[p + "k.conv"]).view(T, KH, D)
    v = short_conv(h @ w[p + "v"].T, w[p + "v.conv"]).view(T, H, V)
    q, k = unit(q) * D ** -0.5, unit(k)
    head = torch.arange(H) // (H // KH)
    beta = torch.sigmoid(h @ w[p + "b"].T)
    o, _ = delta_rule(q[:, head], k[:, head], v, decay(h, w, p, H, D), beta)
    gate = torch.sigmoid((h @ w[p + "g1"].T) @ w[p + "g2"].T).view(T, H, V)
    o = rms(o, eps) * w[p + "norm"] * gate
    return o.reshape(T, H * V) @ w[p + "o"].T


def forward(tokens, w, cfg, layers_out=None):
    """Logits [T, vocab] in double precision."""
    w = {k: t.to(F64) for k, t in w.items()}
    eps = cfg["norm"]["eps"]
    x = w["embed"][torch.tensor(tokens, dtype=torch.long)]
    kept = {}
    for i, layer in enumerate(cfg["layers"]):
        p, m = f"l{i}.mix.", layer["mixer"]
        if layer["type"] == "latent_attention":
            shared = kept[m["kv_from"]] if "kv_from" in m else None
            y, c, kr = latent_attention(x, w, p, m, eps, shared)
            if shared is None:
                kept[i] = (c, kr)
        else:
            y = channel_delta(x, w, p, m, eps)
        x = x + post_norm(y, w[f"l{i}.norm1"], eps)
        if layer["mlp"] is not None:
            y = gelu_tanh(x @ w[f"l{i}.mlp.up"].T) @ w[f"l{i}.mlp.down"].T
            x = x + post_norm(y, w[f"l{i}.norm2"], eps)
        if layers_out is not None:
            layers_out.append(x)
    z = post_norm(x, w["final.norm"], eps) @ w["head"].T
    cap = cfg["logit_softcap"]
    return cap * torch.tanh(z / cap)
