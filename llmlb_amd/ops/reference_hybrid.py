"""Pure-PyTorch versions of the hybrid-model ops for CPU tensors, with
the kernels' arguments, layouts and in-place effects."""
from __future__ import annotations

import torch
import torch.nn.functional as F

PAGE = 16


def _rms(x, eps):
    return x * torch.rsqrt(x.pow(2).mean(-1, keepdim=True) + eps)


def embed_rows(table, ids):
    x = table[ids.long()].float()
    return x, x if table.dtype == torch.float32 else x.to(table.dtype)


def post_norm_add(x, xb, y, w, eps, w_offset):
    x += _rms(y.float(), eps) * (w_offset + w)
    if xb is not x:
        xb.copy_(x)


def norm_rows(x, index, w, eps, dtype, w_offset):
    rows = x if index is None else x[index.long()]
    return (_rms(rows, eps) * (w_offset + w)).to(dtype)


def gelu_tanh_(y):
    return y.copy_(F.gelu(y.float(), approximate="tanh"))


def soft_cap(logits, cap):
    z = logits.float()
    return cap * torch.tanh(z / cap) if cap else z


def _turn(x, cs):
    """x [T, ..., R] by table rows cs [T, R]."""
    half = x.shape[-1] // 2
    cs = cs.reshape([cs.shape[0]] + [1] * (x.dim() - 2) + [-1])
    u, v = x[..., :half].float(), x[..., half:].float()
    c, s = cs[..., :half], cs[..., half:]
    return torch.cat([u * c - v * s, v * c + u * s], -1).to(x.dtype)


def latent_prep(proj, heads, dim, rot, rank, c_off, w_norm, eps, cos_sin, b,
                cache, writes_kv):
    T = b.n_tok
    cs = cos_sin[b.pos.long()]
    q = proj[:, :heads * (dim + rot)].view(T, heads, dim + rot)
    q[..., dim:] = _turn(q[..., dim:], cs)
    if not writes_kv:
        return
    page = b.block_tables[b.row.long(), b.pos.long() // PAGE].long()
    off = b.pos.long() % PAGE
    c = proj[:, c_off:c_off + rank].float()
    cache[page, off, :rank] = (_rms(c, eps) * w_norm).to(cache.dtype)
    cache[page, off, rank:] = _turn(
        proj[:, c_off + rank:c_off + rank + rot], cs)


def latent_rows(qa, proj, dim, rot, cache, b, window, scale):
    H, N, rank = qa.shape
    out = torch.empty_like(qa)
    q = proj[:N, :H * (dim + rot)].reshape(N, H, dim + rot)
    for n in range(N):
        p = int(b.pos[n])
        js = torch.arange(max(0, p - window + 1), p + 1)
        page = b.block_tables[int(b.row[n]), js // PAGE].long()
        key = cache[page, js % PAGE].float()
        full = torch.cat([qa[:, n], q[n, :, dim:]], -1).float()
        a = torch.softmax(full @ key.T * scale, -1)
        out[:, n] = (a @ key[:, :rank]).to(out.dtype)
    return out


def gated_delta(proj, b_off, dec, gate, state, ring, b, wconv, a_log,
                dt_bias, w_norm, kv_heads, heads, dim, vdim, taps, eps):
    KH, H, D, V = kv_heads, heads, dim, vdim
    C = 2 * KH * D + H * V
    group = torch.arange(H) // (H // KH)
    outs = []
    for start, n, pos, row in b.entries:
        x = proj[start:start + n, :C]
        past = torch.zeros(taps - 1, C, dtype=x.dtype)
        for back in range(1, taps):
            if pos - back >= 0:
                past[taps - 1 - back] = ring[row, (pos - back) % taps]
        full = torch.cat([past, x]).float()
        y = F.silu(sum(full[i:i + n] * wconv[i] for i in range(taps)))
        q = y[:, :KH * D].view(n, KH, D)
        k = y[:, KH * D:2 * KH * D].view(n, KH, D)
        v = y[:, 2 * KH * D:].view(n, H, V)
        q = q * torch.rsqrt(q.pow(2).sum(-1, keepdim=True) + 1e-6) \
            * D ** -0.5
        k = k * torch.rsqrt(k.pow(2).sum(-1, keepdim=True) + 1e-6)
        z = (dec[start:start + n].float() + dt_bias).view(n, H, D)
        g = torch.exp(-a_log.exp()[:, None] * F.softplus(z, threshold=60.0))
        beta = torch.sigmoid(proj[start:start + n, b_off:b_off + H].float())
        S = state[row].clone() if pos else torch.zeros(H, V, D)
        o = torch.empty(n, H, V)
        for t in range(n):
            kt, qt = k[t, group], q[t, group]
            S *= g[t][:, None]
            u = beta[t][:, None] * (v[t] - torch.einsum("hvd,hd->hv", S, kt))
            S += u[..., None] * kt[:, None]
            o[t] = torch.einsum("hvd,hd->hv", S, qt)
        state[row] = S
        for t in range(max(0, n - taps), n):
            ring[row, (pos + t) % taps] = x[t]
        o = _rms(o, eps) * w_norm * torch.sigmoid(
            gate[start:start + n].float().view(n, H, V))
        outs.append(o.reshape(n, H * V))
    return torch.cat(outs).to(proj.dtype)
