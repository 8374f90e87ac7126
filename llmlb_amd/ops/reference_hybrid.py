"""Pure-PyTorch versions of the hybrid-model ops for CPU tensors, with
the kernels' arguments, layouts and in-place effects."""
from __future__ import annotations

import torch
import torch.nn.functional as F

PAGE = 16
LN2 = 0.6931471805599453


def _rms(x, eps):
    return x * torch.rsqrt(x.pow(2).mean(-1, keepdim=True) + eps)


def embed_rows(table, ids, copy):
    x = table[ids.long()].float()
    if not copy:
        return x, None
    return x, x if table.dtype == torch.float32 else x.to(table.dtype)


def post_norm_add(x, xb, y, w, eps, w_offset):
    x += _rms(y.float(), eps) * (w_offset + w)
    if xb is not x:
        xb.copy_(x)


def add_norms(x, y, w1, w2, eps, dtype, mult=1.0, routed=None):
    if y is not None:
        x += mult * y.float()
    if routed is not None:
        z, g = routed
        x += mult * torch.einsum("tkw,tk->tw", z.float(), g)
    if w1 is None:
        return None, None
    n = _rms(x, eps)
    return (n * w1).to(dtype), None if w2 is None else (n * w2).to(dtype)


def _norm(x, eps, centred):
    return _rms(x - x.mean(-1, keepdim=True) if centred else x, eps)


def post_pre_norm(x, y, w_post, w_pre, eps, dtype, centred):
    if y is not None:
        x += _norm(y.float(), eps, centred) * w_post
    return None if w_pre is None else (_norm(x, eps, centred)
                                       * w_pre).to(dtype)


def norm_rows(x, index, w, eps, dtype, w_offset, centred):
    rows = x if index is None else x[index.long()]
    return (_norm(rows, eps, centred) * (w_offset + w)).to(dtype)


def gelu_tanh_(y):
    return y.copy_(F.gelu(y.float(), approximate="tanh"))


def clamped_swiglu(out, gu, u_off, limit, sharpness):
    n = out.shape[1]
    g = gu[:, :n].float().clamp(max=limit)
    u = gu[:, u_off:u_off + n].float().clamp(-limit, limit)
    out.copy_(g * torch.sigmoid(sharpness * g) * (u + 1.0))


def squared_relu(out, u):
    out.copy_(u.float().clamp(min=0).square())


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


def latent_rows(qa, proj, dim, rot, cache, b, window, scale, sink):
    H, N, rank = qa.shape
    out = torch.empty_like(qa)
    q = proj[:N, :H * (dim + rot)].reshape(N, H, dim + rot)
    for n in range(N):
        p = int(b.pos[n])
        js = torch.arange(max(0, p - window + 1), p + 1)
        page = b.block_tables[int(b.row[n]), js // PAGE].long()
        key = cache[page, js % PAGE].float()
        full = torch.cat([qa[:, n], q[n, :, dim:]], -1).float()
        s = full @ key.T * scale
        if sink is not None:
            s = torch.cat([s, sink[:, None]], -1)
        a = torch.softmax(s, -1)[:, :len(js)]
        out[:, n] = (a @ key[:, :rank]).to(out.dtype)
    return out


def join_heads(out, o, proj, g_off):
    H, N, V = o.shape
    gate = torch.sigmoid(proj[:N, g_off:g_off + H * V].float())
    out.copy_(o.transpose(0, 1).reshape(N, H * V) * gate)


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


def pair_append(proj, k_off, v_off, kv_heads, dim, vdim, b, cache):
    T, G = b.n_tok, kv_heads
    page = b.block_tables[b.row.long(), b.pos.long() // PAGE].long()
    rows = cache.view(cache.shape[0], G, PAGE, 2 * dim + vdim)
    k = proj[:, k_off:k_off + G * 2 * dim].reshape(T, G, 2 * dim)
    v = proj[:, v_off:v_off + G * vdim].reshape(T, G, vdim)
    rows[page, :, b.pos.long() % PAGE] = torch.cat([k, v], -1)


def pair_attention(out, proj, g_off, heads, kv_heads, dim, vdim, cache, b,
                   q_scale, softcap, lam, gain, eps):
    H, G, D, V = heads, kv_heads, dim, vdim
    rows = cache.view(cache.shape[0], G, PAGE, 2 * D + V)
    head = torch.arange(H) // (H // G)
    for t in range(b.n_tok):
        p = int(b.pos[t])
        js = torch.arange(p + 1)
        page = b.block_tables[int(b.row[t]), js // PAGE].long()
        kv = rows[page, :, js % PAGE].float()[:, head]         # [j, H, ..]
        q = proj[t, :H * 2 * D].view(H, 2, D).float()
        s = torch.einsum("hmd,jhmd->mhj", q,
                         kv[..., :2 * D].unflatten(-1, (2, D))) * q_scale[p]
        if softcap > 0:
            s = softcap * torch.tanh(s / softcap)
        a = torch.einsum("mhj,jhv->mhv", torch.softmax(s, -1),
                         kv[..., 2 * D:])
        o = _rms(a[0] - lam * a[1], eps) * gain
        gate = torch.sigmoid(proj[t, g_off:g_off + H * V].float())
        out[t] = (o.reshape(-1) * gate).to(out.dtype)


def _scan(q, k, v, g, S, o):
    """S [H, V, D] in place; q, k, g [n, H, D] (g may be [n, H, 1]),
    v [n, H, V]; o [n, H, V] is filled."""
    for t in range(q.shape[0]):
        S *= g[t][:, None]
        S += v[t][..., None] * k[t][:, None]
        o[t] = torch.einsum("hvd,hd->hv", S, q[t])


def gated_linear(out, proj, k_off, v_off, g_off, dec, dec_bias, state, b,
                 w_norm, heads, dim, vdim, tau, eps):
    H, D, V = heads, dim, vdim
    for start, n, pos, row in b.entries:
        x = proj[start:start + n].float()
        z = dec[start:start + n].float() + dec_bias
        g = torch.exp(F.logsigmoid(z) / tau).view(n, H, D)
        S = state[row] if pos else state[row].zero_()
        o = torch.empty(n, H, V)
        _scan(x[:, :H * D].view(n, H, D) * D ** -0.5,
              x[:, k_off:k_off + H * D].view(n, H, D),
              x[:, v_off:v_off + H * V].view(n, H, V), g, S, o)
        o = (_rms(o, eps) * w_norm).reshape(n, H * V)
        out[start:start + n] = (
            o * F.silu(x[:, g_off:g_off + H * V])).to(out.dtype)


def state_space(out, proj, z_off, dt_off, state, ring, b, wconv, bconv,
                per_head, w_norm, groups, heads, dim, vdim, taps,
                norm_groups, eps):
    G, H, N, V = groups, heads, dim, vdim
    C = H * V + 2 * G * N
    group = torch.arange(H) // (H // G)
    for start, n, pos, row in b.entries:
        x = proj[start:start + n, :C]
        past = torch.zeros(taps - 1, C, dtype=x.dtype)
        for back in range(1, taps):
            if pos - back >= 0:
                past[taps - 1 - back] = ring[row, (pos - back) % taps]
        full = torch.cat([past, x]).float()
        y = F.silu(bconv + sum(full[i:i + n] * wconv[i]
                               for i in range(taps)))
        xs = y[:, :H * V].view(n, H, V)
        B = y[:, H * V:H * V + G * N].view(n, G, N)[:, group]
        Cq = y[:, H * V + G * N:].view(n, G, N)[:, group]
        dt = F.softplus(proj[start:start + n, dt_off:dt_off + H].float()
                        + per_head[0], threshold=60.0)
        g = torch.exp(-per_head[1] * dt)
        S = state[row] if pos else state[row].zero_()
        o = torch.empty(n, H, V)
        _scan(Cq, B, dt[..., None] * xs, g[..., None], S, o)
        for t in range(max(0, n - taps), n):
            ring[row, (pos + t) % taps] = x[t]
        o = (o + per_head[2][:, None] * xs).reshape(n, H * V)
        o = o * F.silu(proj[start:start + n, z_off:z_off + H * V].float())
        o = _rms(o.view(n, norm_groups, -1), eps).reshape(n, H * V) * w_norm
        out[start:start + n] = o.to(out.dtype)


def matrix_memory(out, proj, k_off, v_off, g_off, i_off, gate_bias, cap,
                  state, extra, b, w_norm, heads, dim, vdim, eps):
    H, D, V = heads, dim, vdim
    for start, n, pos, row in b.entries:
        x = proj[start:start + n].float()
        q = x[:, :H * D].view(n, H, D) * D ** -0.5
        k = x[:, k_off:k_off + H * D].view(n, H, D)
        v = x[:, v_off:v_off + H * V].view(n, H, V)
        z = x[:, i_off:i_off + 2 * H].view(n, 2, H) + gate_bias.view(2, H)
        z = cap * torch.tanh(z / cap)
        li, lf = z[:, 0], F.logsigmoid(z[:, 1])
        S, N, m = state[row], extra[row, :, :D], extra[row, :, -4]
        if not pos:
            for t in (S, N, m):
                t.zero_()
        o = torch.empty(n, H, V)
        for t in range(n):
            now = torch.maximum(lf[t] + m, li[t])
            keep = torch.exp(lf[t] + m - now)[:, None]
            put = torch.exp(li[t] - now)[:, None] * k[t]
            S *= keep[..., None]
            S += v[t][..., None] * put[:, None]
            N.mul_(keep).add_(put)
            m.copy_(now)
            den = torch.maximum((N * q[t]).sum(-1).abs(), torch.exp(-m))
            o[t] = torch.einsum("hvd,hd->hv", S, q[t]) \
                / (den + 1e-6)[:, None]
        o = _rms(o, eps).reshape(n, H * V) * w_norm
        gate = torch.sigmoid(x[:, g_off:g_off + H * V])
        out[start:start + n] = (o * gate).to(out.dtype)


# -- windowed attention ----------------------------------------------------

def head_prep(proj, heads, kv_heads, dim, vdim, rot, k_off, v_off, bq, bk,
              wq, wk, eps, cos_sin, b, cache):
    T, H, G, D, V = b.n_tok, heads, kv_heads, dim, vdim
    pos = b.pos.long()

    def section(at, n, bias):
        x = proj[:, at:at + n * D].float()
        return (x if bias is None else x + bias).view(T, n, D)

    def normed(x, w):
        y = _rms(x, eps) * w
        if rot:
            y = torch.cat([_turn(y[..., :rot], cos_sin[pos]), y[..., rot:]],
                          -1)
        return y.to(proj.dtype)

    q, k = section(0, H, bq), section(k_off, G, bk)
    v = k if v_off is None else proj[:, v_off:v_off + G * V].reshape(T, G, V)
    proj[:, :H * D] = normed(q, wq).reshape(T, -1)
    page = b.block_tables[b.row.long(), pos // PAGE].long()
    rows = cache.view(cache.shape[0], G, PAGE, D + V)
    rows[page, :, pos % PAGE] = torch.cat(
        [normed(k, wk), v.to(proj.dtype)], -1)


def window_prep(proj, heads, kv_heads, dim, vdim, rot, k_off, v_off, wq, wk,
                eps, cos_sin, b, cache):
    T, H, G, D, V = b.n_tok, heads, kv_heads, dim, vdim
    pos = b.pos.long()

    def normed(at, n, w):
        x = proj[:, at:at + n * D]
        y = (_rms(x.float(), eps) * w).view(T, n, D)
        if rot:
            y = torch.cat([_turn(y[..., :rot], cos_sin[pos]), y[..., rot:]],
                          -1)
        return y.to(proj.dtype)

    proj[:, :H * D] = normed(0, H, wq).reshape(T, -1)
    page = b.block_tables[b.row.long(), pos // PAGE].long()
    rows = cache.view(cache.shape[0], G, PAGE, D + V)
    v = proj[:, v_off:v_off + G * V].reshape(T, G, V)
    rows[page, :, pos % PAGE] = torch.cat([normed(k_off, G, wk), v], -1)


def window_attention(out, proj, g_off, heads, kv_heads, dim, vdim, cache, b,
                     window, chunk):
    H, G, D, V = heads, kv_heads, dim, vdim
    rows = cache.view(cache.shape[0], G, PAGE, D + V)
    head = torch.arange(H) // (H // G)
    for t in range(b.n_tok):
        p = int(b.pos[t])
        first = p - p % window if chunk else max(0, p - window + 1)
        js = torch.arange(first, p + 1)
        page = b.block_tables[int(b.row[t]), js // PAGE].long()
        kv = rows[page, :, js % PAGE].float()[:, head]         # [j, H, ..]
        s = torch.einsum("hd,jhd->hj", proj[t, :H * D].view(H, D).float(),
                         kv[..., :D])
        a = torch.softmax(s * LN2, -1)
        o = torch.einsum("hj,jhv->hv", a, kv[..., D:])
        if g_off is not None:
            o = o * torch.sigmoid(proj[t, g_off:g_off + H].float())[:, None]
        out[t] = o.reshape(-1).to(out.dtype)


# -- mixture of experts ----------------------------------------------------

def route(h, w, top, groups, keep, scale):
    s = torch.softmax(h.float() @ w.float().T, -1)
    T, E = s.shape
    best = s.view(T, groups, -1).amax(-1).topk(keep, -1).indices
    allowed = torch.zeros(T, groups, dtype=torch.bool).scatter_(
        1, best, True).repeat_interleave(E // groups, 1)
    g, index = s.masked_fill(~allowed, -1.0).topk(top, -1)
    return index.int(), g / (g.sum(-1, keepdim=True) + 1e-20) * scale


def experts(h, index, w_up, w_down):
    T, top = index.shape
    z = torch.empty(T, top, h.shape[1], dtype=h.dtype)
    for e in index.unique().tolist():
        t, k = (index == e).nonzero(as_tuple=True)
        u = (h[t].float() @ w_up[e].float().T).to(h.dtype)
        u = u.float().clamp(min=0).square().to(h.dtype)
        z[t, k] = (u.float() @ w_down[e].float().T).to(h.dtype)
    return z
