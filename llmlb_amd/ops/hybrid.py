"""Ops of the hybrid models: a 32-bit residual stream with norms before
or after the sublayers or both, latent, differential, windowed and chunked
attention over pages, gated delta rule, linear recurrences and mixtures of
experts.

The native library (csrc/hybrid) is loaded at first use.  GPU tensors
always run the HIP kernels, in bfloat16 and in float32; CPU tensors run
``reference_hybrid`` (tests, machines without a GPU).  ``b`` is a
backend.ragged.RaggedBatch.
"""
from __future__ import annotations

import ctypes

import torch

from . import NativeKernelsMissing, _check, _ptr, _stream
from . import reference_hybrid as ref
from .build import library_path

_lib: ctypes.CDLL | None = None


def native() -> ctypes.CDLL:
    global _lib
    if _lib is None:
        path = library_path("hybrid")
        if not path.exists():
            raise NativeKernelsMissing(
                f"{path} is not built (python -m llmlb_amd.ops.build "
                "hybrid); there is no eager fallback on GPU")
        lib = ctypes.CDLL(str(path))
        lib.hy_delta_ws_floats.restype = ctypes.c_longlong
        _lib = lib
    return _lib


def _i(v) -> ctypes.c_int:
    return ctypes.c_int(int(v))


def _f(v) -> ctypes.c_float:
    return ctypes.c_float(float(v))


def _p(t):
    return None if t is None else _ptr(t)


def _dt(dtype: torch.dtype) -> ctypes.c_int:
    if dtype == torch.bfloat16:
        return _i(0)
    if dtype == torch.float32:
        return _i(1)
    raise TypeError(f"hybrid kernels take bfloat16 or float32, not {dtype}")


# -- rows ------------------------------------------------------------------

def embed_rows(table, ids, copy: bool = True):
    """(x float32 [T, W], the same in the storage type; None without
    ``copy``)."""
    if not table.is_cuda:
        return ref.embed_rows(table, ids, copy)
    T, W = ids.shape[0], table.shape[1]
    x = torch.empty(T, W, dtype=torch.float32, device=table.device)
    xb = None
    if copy:
        xb = x if table.dtype == torch.float32 else torch.empty(
            T, W, dtype=table.dtype, device=table.device)
    _check(native().hy_embed_rows(
        _ptr(x), None if xb is x else _p(xb), _ptr(table), _ptr(ids),
        _i(T), _i(W), _i(table.shape[0]), _dt(table.dtype), _stream()),
        "hy_embed_rows")
    return x, xb


def post_norm_add(x, xb, y, w, eps, w_offset=0.0) -> None:
    """In place: x += rmsnorm(y) * (w_offset + w); xb = x in the storage
    type (xb may be x itself)."""
    if not x.is_cuda:
        ref.post_norm_add(x, xb, y, w, eps, w_offset)
        return
    assert y.is_contiguous() and y.shape == x.shape
    _check(native().hy_post_norm_add(
        _ptr(x), None if xb is x else _ptr(xb), _ptr(y), _ptr(w),
        _f(w_offset), _i(x.shape[0]), _i(x.shape[1]), _f(eps), _dt(y.dtype),
        _stream()), "hy_post_norm_add")


def add_norms(x, y, w1, w2, eps, dtype, mult=1.0, routed=None):
    """In place: x += mult * y (None: nothing to add).  Returns
    rmsnorm(x) * w1 and rmsnorm(x) * w2 in ``dtype``, None for a weight
    that is None (w2 alone may not be given); weights are rows or single
    numbers.  ``routed``: (z [T, n, W], g [T, n]) whose weighted sum
    over n is added to y first."""
    if not x.is_cuda:
        return ref.add_norms(x, y, w1, w2, eps, dtype, mult, routed)
    assert y is None or (y.is_contiguous() and y.shape == x.shape
                         and y.dtype == dtype)
    z, g = routed or (None, None)
    n = 0
    if z is not None:
        n = z.shape[1]
        assert z.is_contiguous() and g.is_contiguous() and z.dtype == dtype \
            and z.shape == (x.shape[0], n, x.shape[1]) \
            and g.shape == (x.shape[0], n)
    one = w1 is not None and w1.numel() == 1 and x.shape[1] > 1
    for w in (w1, w2):
        assert w is None or w.numel() == (1 if one else x.shape[1])
    h1, h2 = (None if w is None else
              torch.empty(x.shape, dtype=dtype, device=x.device)
              for w in (w1, w2))
    _check(native().hy_add_norms(
        _ptr(x), _p(y), _p(z), _p(g), _i(n), _f(mult), _p(w1), _p(w2),
        _i(one), _p(h1), _p(h2), _i(x.shape[0]), _i(x.shape[1]), _f(eps),
        _dt(dtype), _stream()), "hy_add_norms")
    return h1, h2


def post_pre_norm(x, y, w_post, w_pre, eps, dtype, centred: bool):
    """In place: x += norm(y) * w_post (y None: nothing to add).  Returns
    norm(x) * w_pre in ``dtype`` (w_pre None: nothing).  ``centred``:
    layer norms, else RMS norms."""
    if not x.is_cuda:
        return ref.post_pre_norm(x, y, w_post, w_pre, eps, dtype, centred)
    assert x.is_contiguous()
    assert y is None or (y.is_contiguous() and y.shape == x.shape
                         and y.dtype == dtype
                         and w_post.numel() == x.shape[1])
    assert w_pre is None or w_pre.numel() == x.shape[1]
    h = None if w_pre is None else torch.empty(x.shape, dtype=dtype,
                                               device=x.device)
    _check(native().hy_post_pre_norm(
        _ptr(x), _p(y), None if y is None else _ptr(w_post), _p(w_pre),
        _p(h), _i(centred), _i(x.shape[0]), _i(x.shape[1]), _f(eps),
        _dt(dtype), _stream()), "hy_post_pre_norm")
    return h


def norm_rows(x, index, w, eps, dtype, w_offset=0.0, centred=False):
    """norm(x[index]) * (w_offset + w) in ``dtype``; index may be None
    (every row), w a row or a single number.  ``centred``: a layer norm,
    else an RMS norm."""
    if not x.is_cuda:
        return ref.norm_rows(x, index, w, eps, dtype, w_offset, centred)
    n = x.shape[0] if index is None else index.shape[0]
    one = w.numel() == 1 and x.shape[1] > 1
    assert w.numel() == (1 if one else x.shape[1])
    out = torch.empty(n, x.shape[1], dtype=dtype, device=x.device)
    _check(native().hy_norm_rows(
        _ptr(out), _ptr(x), _p(index), _ptr(w), _i(one), _f(w_offset),
        _i(centred), _i(n), _i(x.shape[1]), _f(eps), _dt(dtype), _stream()),
        "hy_norm_rows")
    return out


def gelu_tanh_(y):
    """In place, the tanh form of gelu."""
    if not y.is_cuda:
        return ref.gelu_tanh_(y)
    assert y.is_contiguous()
    _check(native().hy_gelu_tanh(
        _ptr(y), ctypes.c_longlong(y.numel()), _dt(y.dtype), _stream()),
        "hy_gelu_tanh")
    return y


def clamped_swiglu(out, gu, u_off, limit, sharpness) -> None:
    """out = g sigmoid(sharpness g) (u + 1), with g = min(gate, limit)
    from the first columns of ``gu`` and u = clamp(up, -limit, limit)
    from those at ``u_off``.  ``out`` may be columns of wider rows."""
    if not gu.is_cuda:
        ref.clamped_swiglu(out, gu, u_off, limit, sharpness)
        return
    assert gu.stride(1) == 1 and out.stride(1) == 1
    _check(native().hy_clamped_swiglu(
        _ptr(out), _i(out.stride(0)), _ptr(gu), _i(gu.stride(0)), _i(u_off),
        _i(out.shape[0]), _i(out.shape[1]), _f(limit), _f(sharpness),
        _dt(gu.dtype), _stream()), "hy_clamped_swiglu")


def squared_relu(out, u) -> None:
    """out = max(u, 0)^2; both may be columns of wider rows."""
    if not u.is_cuda:
        ref.squared_relu(out, u)
        return
    assert u.stride(1) == 1 and out.stride(1) == 1 and u.shape == out.shape
    _check(native().hy_squared_relu(
        _ptr(out), _i(out.stride(0)), _ptr(u), _i(u.stride(0)),
        _i(out.shape[0]), _i(out.shape[1]), _dt(u.dtype), _stream()),
        "hy_squared_relu")


def soft_cap(logits, cap):
    """cap * tanh(logits / cap) in float32; no cap: a widening."""
    if not logits.is_cuda:
        return ref.soft_cap(logits, cap)
    assert logits.is_contiguous()
    out = torch.empty(logits.shape, dtype=torch.float32,
                      device=logits.device)
    _check(native().hy_soft_cap(
        _ptr(out), _ptr(logits), _f(cap or 0.0),
        ctypes.c_longlong(logits.numel()), _dt(logits.dtype), _stream()),
        "hy_soft_cap")
    return out


# -- latent attention ------------------------------------------------------

def latent_prep(proj, heads, dim, rot, rank, c_off, w_norm, eps, cos_sin, b,
                cache, writes_kv: bool) -> None:
    """Rotate the query parts of ``proj`` in place; with ``writes_kv``
    also norm the latent, rotate the shared key part and append both to
    the paged cache."""
    if not proj.is_cuda:
        ref.latent_prep(proj, heads, dim, rot, rank, c_off, w_norm, eps,
                        cos_sin, b, cache, writes_kv)
        return
    assert proj.stride(1) == 1
    _check(native().hy_latent_prep(
        _ptr(proj), _i(proj.stride(0)), _i(heads), _i(dim), _i(rot),
        _i(c_off), _i(rank), _p(w_norm), _f(eps), _ptr(cos_sin),
        _ptr(b.pos), _ptr(b.row), _ptr(b.block_tables),
        _i(b.block_tables.shape[1]), _ptr(cache), _i(writes_kv),
        _i(b.n_tok), _dt(proj.dtype), _stream()), "hy_latent_prep")


def latent_rows(qa, proj, dim, rot, cache, b, window, scale, sink=None):
    """Absorbed attention: qa [H, N, rank] (the batch's first N tokens)
    -> weighted latents [H, N, rank].  ``sink`` [H] float32 (None: none):
    a score of every head that has no key and no value."""
    if not qa.is_cuda:
        return ref.latent_rows(qa, proj, dim, rot, cache, b, window, scale,
                               sink)
    H, N, rank = qa.shape
    assert qa.is_contiguous()
    out = torch.empty_like(qa)
    _check(native().hy_latent_rows(
        _ptr(out), _ptr(qa), _ptr(proj), _i(proj.stride(0)), _i(H), _i(dim),
        _i(rot), _i(rank), _ptr(cache), _ptr(b.pos), _ptr(b.row),
        _ptr(b.block_tables), _i(b.block_tables.shape[1]), _i(window),
        _f(scale), _p(sink), _i(N), _dt(qa.dtype), _stream()),
        "hy_latent_rows")
    return out


def can_decode_tiled(dtype, dim, rot, rank) -> bool:
    """Sizes that ``latent_decode`` takes."""
    return (dtype == torch.bfloat16 and rank % 8 == 0 and rot % 8 == 0
            and dim % 8 == 0 and rot <= 64 and rank <= 512)


def decode_parts(n: int, heads: int, window: int, max_keys: int) -> int:
    """How many workgroups share one query's keys: enough to fill the
    chip, with at least two tiles of keys each."""
    groups = n * ((heads + 31) // 32 if heads > 16 else 1)
    keys = min(window, max_keys)
    return max(1, min(256 // groups, keys // 64, 16))


def latent_decode(qa, proj, dim, rot, cache, b, window, scale, sink=None):
    """``latent_rows`` on the matrix cores (bf16, GPU)."""
    H, N, rank = qa.shape
    assert qa.is_contiguous()
    bt = b.block_tables
    parts = decode_parts(N, H, window, b.max_keys)
    out = torch.empty_like(qa)
    acc = ml = None
    if parts > 1:
        acc = torch.empty(N, H, parts, rank, dtype=torch.float32,
                          device=qa.device)
        ml = torch.empty(N, H, parts, 2, dtype=torch.float32,
                         device=qa.device)
    _check(native().hy_latent_decode(
        _ptr(out), _p(acc), _p(ml), _ptr(qa), _ptr(proj),
        _i(proj.stride(0)), _i(H), _i(dim), _i(rot), _i(rank), _ptr(cache),
        _ptr(b.pos), _ptr(b.row), _ptr(bt), _i(bt.shape[1]), _i(window),
        _f(scale), _p(sink), _i(N), _i(parts), _stream()),
        "hy_latent_decode")
    return out


def join_heads(out, o, proj, g_off) -> None:
    """out [N, H * V] = the heads of o [H, N, V] side by side, times the
    sigmoid of the columns of ``proj`` from ``g_off`` on."""
    if not o.is_cuda:
        ref.join_heads(out, o, proj, g_off)
        return
    H, N, V = o.shape
    gate = proj[:N, g_off:g_off + H * V]
    assert o.is_contiguous() and out.is_contiguous() \
        and out.shape == gate.shape == (N, H * V) and gate.stride(1) == 1
    _check(native().hy_join_heads(
        _ptr(out), _ptr(o), _ptr(gate), _i(proj.stride(0)), _i(N), _i(H),
        _i(V), _dt(o.dtype), _stream()), "hy_join_heads")


def can_flash(dtype, dim, rot, rank, vdim) -> bool:
    """Sizes that ``latent_flash`` takes."""
    return (dtype == torch.bfloat16 and dim % 8 == 0 and rot % 8 == 0
            and rank % 8 == 0 and dim + rot <= 256 and vdim <= 256)


def latent_flash(out, proj, heads, dim, rot, w_uk, w_uv, cache, b, window,
                 scale, sink=None, g_off=None) -> None:
    """Attention of the batch's long entries into ``out`` [T, H * vdim]:
    their visible latents are copied out of the pages and expanded to
    keys and (transposed) values.  w_uk [H, dim, rank], w_uv
    [H, vdim, rank].  With ``g_off`` times the sigmoid of the columns of
    ``proj`` from there on."""
    H, V, rank = w_uv.shape
    blocks, items, n_blocks, n_items = b.long_plan(window)
    n = 64 * n_blocks
    lib, bt, st = native(), b.block_tables, _stream()
    c = torch.empty(n, rank, dtype=proj.dtype, device=proj.device)
    kr = torch.empty(n, rot, dtype=proj.dtype, device=proj.device)
    _check(lib.hy_latent_gather(
        _ptr(c), _ptr(kr), _ptr(cache), _ptr(blocks), _i(n_blocks), _ptr(bt),
        _i(bt.shape[1]), _i(rank), _i(rot), st), "hy_latent_gather")
    kx = torch.nn.functional.linear(c, w_uk.view(H * dim, rank))
    vt = torch.nn.functional.linear(w_uv.view(H * V, rank), c)
    _check(lib.hy_latent_flash(
        _ptr(out), _ptr(proj), _i(proj.stride(0)), _ptr(kx), _ptr(kr),
        _ptr(vt), _i(n), _ptr(items), _i(n_items), _i(H), _i(dim), _i(rot),
        _i(V), _i(window), _f(scale), _p(sink),
        _i(-1 if g_off is None else g_off), st), "hy_latent_flash")


# -- gated delta rule ------------------------------------------------------

def gated_delta(proj, b_off, dec, gate, state, ring, b, wconv, a_log,
                dt_bias, w_norm, kv_heads, heads, dim, vdim, taps, eps):
    """Convolutions, unit norms, decays, the recurrence, head norm and
    output gate of a packed batch -> [T, heads * vdim].

    proj columns start with the convolved q | k | v; beta's projection
    is at ``b_off``.  dec [T, heads * dim] and gate [T, heads * vdim]
    are the low-rank projections.  Updates ``state`` and ``ring``."""
    if not proj.is_cuda:
        return ref.gated_delta(proj, b_off, dec, gate, state, ring, b, wconv,
                               a_log, dt_bias, w_norm, kv_heads, heads, dim,
                               vdim, taps, eps)
    lib = native()
    T, H, KH, D, V = b.n_tok, heads, kv_heads, dim, vdim
    assert proj.stride(1) == 1 and dec.is_contiguous() \
        and gate.is_contiguous()
    dt, ld, st = _dt(proj.dtype), _i(proj.stride(0)), _stream()
    sizes = (_i(KH), _i(H), _i(D), _i(V))
    q_scale = _f(D ** -0.5)
    out = torch.empty(T, H * V, dtype=proj.dtype, device=proj.device)
    if b.decode:
        _check(lib.hy_delta_step(
            _ptr(out), _ptr(state), _ptr(ring), _ptr(proj), ld, _i(b_off),
            _ptr(dec), _ptr(gate), _ptr(wconv), _ptr(a_log), _ptr(dt_bias),
            _ptr(w_norm), _ptr(b.pos), _ptr(b.row), _i(T), *sizes, _i(taps),
            q_scale, _f(eps), dt, st), "hy_delta_step")
        return out
    ws = torch.empty(T, int(lib.hy_delta_ws_floats(*sizes)),
                     dtype=torch.float32, device=proj.device)
    o = torch.empty(T, H * V, dtype=torch.float32, device=proj.device)
    _check(lib.hy_delta_prep(
        _ptr(ws), _ptr(proj), ld, _i(b_off), _ptr(dec), _ptr(ring),
        _ptr(wconv), _ptr(a_log), _ptr(dt_bias), _ptr(b.pos), _ptr(b.row),
        _ptr(b.tstart), _i(T), *sizes, _i(taps), q_scale, dt, st),
        "hy_delta_prep")
    _check(lib.hy_delta_scan(
        _ptr(o), _ptr(state), _ptr(ws), _ptr(b.e_start), _ptr(b.e_len),
        _ptr(b.e_pos), _ptr(b.e_row), _i(len(b.entries)), *sizes, st),
        "hy_delta_scan")
    _check(lib.hy_delta_out(
        _ptr(out), _ptr(o), _ptr(gate), _ptr(w_norm), _f(eps), _ptr(proj),
        ld, _ptr(ring), _ptr(b.pos), _ptr(b.row), _ptr(b.tend), _i(T),
        *sizes, _i(taps), dt, st), "hy_delta_out")
    return out


# -- differential attention ------------------------------------------------

def pair_append(proj, k_off, v_off, kv_heads, dim, vdim, b, cache) -> None:
    """Put every token's keys (both maps) and values into its page."""
    if not proj.is_cuda:
        ref.pair_append(proj, k_off, v_off, kv_heads, dim, vdim, b, cache)
        return
    assert proj.stride(1) == 1
    _check(native().hy_pair_append(
        _ptr(cache), _ptr(proj), _i(proj.stride(0)), _i(k_off), _i(v_off),
        _i(kv_heads), _i(dim), _i(vdim), _ptr(b.pos), _ptr(b.row),
        _ptr(b.block_tables), _i(b.block_tables.shape[1]), _i(b.n_tok),
        _dt(proj.dtype), _stream()), "hy_pair_append")


def can_pair_mfma(dtype, dim, vdim) -> bool:
    """Sizes that the matrix-core kernels take."""
    return (dtype == torch.bfloat16 and dim % 8 == 0 and vdim % 8 == 0
            and dim <= 128 and vdim <= 256)


def pair_parts(n: int, kv_heads: int, group: int, max_keys: int) -> int:
    """How many workgroups share one query's keys: enough to fill the
    chip, with at least two tiles of keys each."""
    groups = n * kv_heads * ((group + 15) // 16)
    return max(1, min(1024 // groups, max_keys // 128, 32))


def pair_attention(out, proj, g_off, heads, kv_heads, dim, vdim, cache, b,
                   q_scale, softcap, lam, gain, eps) -> None:
    """Both maps' attention, their difference a1 - lam * a2, its norm per
    head times ``gain`` and the sigmoid gate, into ``out`` [T, H * vdim]
    (columns of wider rows).  ``proj`` starts with the queries."""
    if not proj.is_cuda:
        ref.pair_attention(out, proj, g_off, heads, kv_heads, dim, vdim,
                           cache, b, q_scale, softcap, lam, gain, eps)
        return
    assert proj.stride(1) == 1 and out.stride(1) == 1
    lib, bt, st = native(), b.block_tables, _stream()
    H, G, D, V = heads, kv_heads, dim, vdim
    assert cache.shape[0] * G * 16 < 2 ** 31    # rows are 32-bit numbers
    dst = (_ptr(out), _i(out.stride(0)))
    src = (_ptr(proj), _i(proj.stride(0)), _i(g_off), _ptr(cache))
    sizes = (_i(H), _i(G), _i(D), _i(V))
    consts = (_ptr(q_scale), _f(softcap), _f(lam), _f(gain), _f(eps))
    where = (_ptr(bt), _i(bt.shape[1]))
    # vector accesses need whole vectors in every row
    if not (can_pair_mfma(proj.dtype, D, V) and proj.stride(0) % 8 == 0
            and g_off % 8 == 0 and out.stride(0) % 8 == 0):
        _check(lib.hy_pair_rows(
            *dst, *src, _ptr(b.pos), _ptr(b.row), *where, *sizes, *consts,
            _i(b.n_tok), _dt(proj.dtype), st), "hy_pair_rows")
        return
    n = b.n_short
    if n:
        parts = pair_parts(n, G, H // G, b.max_keys)
        acc = torch.empty(n, H, 2, parts, V, dtype=torch.float32,
                          device=proj.device)
        ml = torch.empty(n, H, 2, parts, 2, dtype=torch.float32,
                         device=proj.device)
        _check(lib.hy_pair_decode(
            *dst, _ptr(acc), _ptr(ml), *src, _ptr(b.pos), _ptr(b.row),
            *where, *sizes, *consts, _i(n), _i(parts), st),
            "hy_pair_decode")
    if n < b.n_tok:
        items, n_items = b.query_tiles(64)
        _check(lib.hy_pair_flash(
            *dst, *src, _ptr(items), _i(n_items), *where, *sizes, *consts,
            st), "hy_pair_flash")


# -- linear recurrences ----------------------------------------------------

def _gated_norm(out, y, gate, g_off, w, groups, gate_first: bool, eps,
                sigm: bool = False) -> None:
    """Rows of ``groups`` equal parts, each normed by its own rms and
    times ``w`` (repeated along the row); silu(gate) before or after, or
    sigmoid(gate) after (``sigm``)."""
    T, W = y.shape
    _check(native().hy_gated_norm(
        _ptr(out), _i(out.stride(0)), _ptr(y), _ptr(gate),
        _i(gate.stride(0)), _i(g_off), _ptr(w), _i(w.shape[0]), _i(T),
        _i(groups), _i(W // groups), _i(gate_first), _i(sigm), _f(eps),
        _dt(out.dtype), _stream()), "hy_gated_norm")


def gated_linear(out, proj, k_off, v_off, g_off, dec, dec_bias, state, b,
                 w_norm, heads, dim, vdim, tau, eps) -> None:
    """Gated linear attention of a packed batch into ``out``
    [T, H * vdim] (columns of wider rows).  ``proj`` starts with the
    queries; ``dec`` [T, H * dim] is the decays' projection.  Updates
    ``state``."""
    if not proj.is_cuda:
        ref.gated_linear(out, proj, k_off, v_off, g_off, dec, dec_bias,
                         state, b, w_norm, heads, dim, vdim, tau, eps)
        return
    assert proj.stride(1) == 1 and out.stride(1) == 1 \
        and dec.is_contiguous()
    lib, dt, st = native(), _dt(proj.dtype), _stream()
    T, H, D, V = b.n_tok, heads, dim, vdim
    ld, q_scale, rate = _i(proj.stride(0)), _f(D ** -0.5), _f(1.0 / tau)
    if b.decode:
        _check(lib.hy_gla_step(
            _ptr(out), _i(out.stride(0)), _ptr(state), _ptr(proj), ld,
            _i(k_off), _i(v_off), _i(g_off), _ptr(dec), _ptr(dec_bias),
            _ptr(w_norm), _ptr(b.pos), _ptr(b.row), _i(T), _i(H), _i(D),
            _i(V), q_scale, rate, _f(eps), dt, st), "hy_gla_step")
        return
    g = torch.empty(T, H * D, dtype=torch.float32, device=proj.device)
    o = torch.empty(T, H * V, dtype=torch.float32, device=proj.device)
    _check(lib.hy_gla_decay(
        _ptr(g), _ptr(dec), _ptr(dec_bias), _i(T), _i(H * D), rate, dt, st),
        "hy_gla_decay")
    _check(lib.hy_linear_scan(
        _ptr(o), _ptr(state), _ptr(proj), ld, _i(0), _i(k_off), _i(v_off),
        _ptr(g), None, None, _ptr(b.e_start), _ptr(b.e_len), _ptr(b.e_pos),
        _ptr(b.e_row), _i(len(b.entries)), _i(H), _i(H), _i(D), _i(V),
        q_scale, None, None, dt, st), "hy_linear_scan")
    _gated_norm(out, o, proj, g_off, w_norm, H, False, eps)


def state_space(out, proj, z_off, dt_off, state, ring, b, wconv, bconv,
                per_head, w_norm, groups, heads, dim, vdim, taps,
                norm_groups, eps) -> None:
    """Mamba-2 of a packed batch into ``out`` [T, H * vdim] (columns of
    wider rows).  ``proj`` starts with the convolved x | B | C;
    ``per_head`` rows are dt's bias, the decay rate and the skip factor.
    Updates ``state`` and ``ring``."""
    if not proj.is_cuda:
        ref.state_space(out, proj, z_off, dt_off, state, ring, b, wconv,
                        bconv, per_head, w_norm, groups, heads, dim, vdim,
                        taps, norm_groups, eps)
        return
    assert proj.stride(1) == 1 and out.stride(1) == 1
    lib, dt, st = native(), _dt(proj.dtype), _stream()
    T, G, H, N, V = b.n_tok, groups, heads, dim, vdim
    C = H * V + 2 * G * N
    ld = _i(proj.stride(0))
    o = torch.empty(T, H * V, dtype=torch.float32, device=proj.device)
    conv = (_ptr(ring), _ptr(wconv), _ptr(bconv), _ptr(per_head))
    if b.decode:
        _check(lib.hy_ssm_step(
            _ptr(o), _ptr(state), _ptr(proj), ld, _i(dt_off), *conv,
            _ptr(b.pos), _ptr(b.row), _i(T), _i(G), _i(H), _i(N), _i(V),
            _i(taps), dt, st), "hy_ssm_step")
    else:
        xbc = torch.empty(T, C, dtype=proj.dtype, device=proj.device)
        steps = torch.empty(2, T, H, dtype=torch.float32,
                            device=proj.device)
        _check(lib.hy_ssm_prep(
            _ptr(xbc), _ptr(steps), _ptr(proj), ld, _i(dt_off), *conv,
            _ptr(b.pos), _ptr(b.row), _ptr(b.tstart), _i(T), _i(C), _i(H),
            _i(taps), dt, st), "hy_ssm_prep")
        _check(lib.hy_ring_store(
            _ptr(ring), _ptr(proj), ld, _ptr(b.e_start), _ptr(b.e_len),
            _ptr(b.e_pos), _ptr(b.e_row), _i(len(b.entries)), _i(C),
            _i(taps), dt, st), "hy_ring_store")
        _check(lib.hy_linear_scan(
            _ptr(o), _ptr(state), _ptr(xbc), _i(C), _i(H * V + G * N),
            _i(H * V), _i(0), _ptr(steps[0]), _ptr(steps[1]),
            _ptr(per_head[2]), _ptr(b.e_start), _ptr(b.e_len),
            _ptr(b.e_pos), _ptr(b.e_row), _i(len(b.entries)), _i(G), _i(H),
            _i(N), _i(V), _f(1.0), None, None, dt, st), "hy_linear_scan")
    _gated_norm(out, o, proj, z_off, w_norm, norm_groups, True, eps)


def memory_extra(dim: int) -> int:
    """Floats per head that matrix memory keeps beside its matrix: the
    normaliser, padded to whole vectors, and a vector whose first number
    is the running maximum."""
    return -(-dim // 4) * 4 + 4


def can_memory_mfma(dtype, dim, vdim) -> bool:
    """Sizes that the matrix-core kernel takes."""
    return (dtype == torch.bfloat16 and dim % 8 == 0 and vdim % 8 == 0
            and dim <= 256)


def matrix_memory(out, proj, k_off, v_off, g_off, i_off, gate_bias, cap,
                  state, extra, b, w_norm, heads, dim, vdim, eps) -> None:
    """mLSTM of a packed batch into ``out`` [T, H * vdim] (columns of
    wider rows): recurrence, head norms and output gate.  ``proj`` starts
    with the queries; the input gates are H columns from ``i_off`` on,
    the forget gates the next H; ``gate_bias`` [2, H].  ``w_norm``
    [H * vdim].  Updates ``state`` [slots, H, vdim, dim] and ``extra``
    [slots, H, memory_extra(dim)]."""
    if not proj.is_cuda:
        ref.matrix_memory(out, proj, k_off, v_off, g_off, i_off, gate_bias,
                          cap, state, extra, b, w_norm, heads, dim, vdim,
                          eps)
        return
    T, H, D, V = b.n_tok, heads, dim, vdim
    assert proj.stride(1) == 1 and out.stride(1) == 1 \
        and extra.shape[1:] == (H, memory_extra(D)) \
        and w_norm.numel() == H * V and gate_bias.numel() == 2 * H
    lib, dt, st = native(), _dt(proj.dtype), _stream()
    ld, q_scale = _i(proj.stride(0)), _f(D ** -0.5)
    if b.decode:
        _check(lib.hy_memory_step(
            _ptr(out), _i(out.stride(0)), _ptr(state), _ptr(extra),
            _ptr(proj), ld, _i(k_off), _i(v_off), _i(g_off), _i(i_off),
            _ptr(gate_bias), _ptr(w_norm), _ptr(b.pos), _ptr(b.row), _i(T),
            _i(H), _i(D), _i(V), q_scale, _f(cap), _f(eps), dt, st),
            "hy_memory_step")
        return
    E = len(b.entries)
    f32 = dict(dtype=torch.float32, device=proj.device)
    steps = torch.empty(3, T, H, **f32)
    o = torch.empty(T, H * V, **f32)
    runs = (_ptr(b.e_start), _ptr(b.e_len), _ptr(b.e_pos), _ptr(b.e_row),
            _i(E))
    if can_memory_mfma(proj.dtype, D, V) and proj.stride(0) % 8 == 0 \
            and k_off % 8 == 0 and v_off % 8 == 0:
        carry = torch.empty(E, H, memory_extra(D), **f32)
        _check(lib.hy_memory_chunk(
            _ptr(o), _ptr(steps), _ptr(carry), _ptr(state), _ptr(extra),
            _ptr(proj), ld, _i(k_off), _i(v_off), _i(i_off),
            _ptr(gate_bias), *runs, _i(max(n for _, n, _, _ in b.entries)),
            _i(T), _i(H), _i(D), _i(V), q_scale, _f(cap), st),
            "hy_memory_chunk")
        _gated_norm(out, o, proj, g_off, w_norm, H, False, eps, True)
        return
    n0 = torch.empty(E, H, D, **f32)
    _check(lib.hy_memory_gates(
        _ptr(steps), _ptr(n0), _ptr(extra), _ptr(proj), ld, _i(i_off),
        _ptr(gate_bias), *runs, _i(T), _i(H), _i(D), _f(cap), dt, st),
        "hy_memory_gates")
    _check(lib.hy_linear_scan(
        _ptr(o), _ptr(state), _ptr(proj), ld, _i(0), _i(k_off), _i(v_off),
        _ptr(steps[0]), _ptr(steps[1]), _ptr(steps[2]), *runs, _i(H), _i(H),
        _i(D), _i(V), q_scale, _ptr(n0), _ptr(extra), dt, st),
        "hy_linear_scan")
    _gated_norm(out, o, proj, g_off, w_norm, H, False, eps, True)


# -- windowed attention ----------------------------------------------------

def head_prep(proj, heads, kv_heads, dim, vdim, rot, k_off, v_off, bq, bk,
              wq, wk, eps, cos_sin, b, cache) -> None:
    """Add biases (``bq``, ``bk`` float32, None: none) to queries (the
    first columns of ``proj``) and keys, norm each head by itself with
    the weights ``wq`` and ``wk`` [dim], rotate its first ``rot`` numbers
    (pairs half of them apart), the queries in place; put keys and values
    into the pages.  ``v_off`` None: the values are the keys with their
    biases, before norm and rotation.  ``wq`` carries the scores' scale
    and log2(e)."""
    if not proj.is_cuda:
        ref.head_prep(proj, heads, kv_heads, dim, vdim, rot, k_off, v_off,
                      bq, bk, wq, wk, eps, cos_sin, b, cache)
        return
    assert proj.stride(1) == 1 and wq.numel() == dim == wk.numel() \
        and (bq is None or bq.numel() == heads * dim) \
        and (bk is None or bk.numel() == kv_heads * dim)
    bt = b.block_tables
    _check(native().hy_head_prep(
        _ptr(proj), _i(proj.stride(0)), _ptr(cache), _i(k_off),
        _i(-1 if v_off is None else v_off), _i(heads), _i(kv_heads), _i(dim),
        _i(vdim), _i(rot), _p(bq), _p(bk), _ptr(wq), _ptr(wk), _p(cos_sin),
        _f(eps), _ptr(b.pos), _ptr(b.row), _ptr(bt), _i(bt.shape[1]),
        _i(b.n_tok), _dt(proj.dtype), _stream()), "hy_head_prep")


def window_prep(proj, heads, kv_heads, dim, vdim, rot, k_off, v_off, wq, wk,
                eps, cos_sin, b, cache) -> None:
    """Norm queries (the first columns of ``proj``) and keys over all
    heads, rotate the first ``rot`` numbers of each head, the queries in
    place; put keys and values into the pages.  ``wq`` carries the
    scores' scale and log2(e)."""
    if not proj.is_cuda:
        ref.window_prep(proj, heads, kv_heads, dim, vdim, rot, k_off, v_off,
                        wq, wk, eps, cos_sin, b, cache)
        return
    assert proj.stride(1) == 1 and wq.numel() == heads * dim \
        and wk.numel() == kv_heads * dim
    bt = b.block_tables
    _check(native().hy_window_prep(
        _ptr(proj), _i(proj.stride(0)), _ptr(cache), _i(k_off), _i(v_off),
        _i(heads), _i(kv_heads), _i(dim), _i(vdim), _i(rot), _ptr(wq),
        _ptr(wk), _p(cos_sin), _f(eps), _ptr(b.pos), _ptr(b.row), _ptr(bt),
        _i(bt.shape[1]), _i(b.n_tok), _dt(proj.dtype), _stream()),
        "hy_window_prep")


def window_front(prep, routing, act=None):
    """``window_prep(*prep)``, ``route(*routing)`` and, with ``act``,
    ``squared_relu(*act)`` of columns of the same ``proj``: what a
    parallel layer does between its input projections and its attention,
    in one launch.  Returns what ``route`` does."""
    proj = prep[0]
    if proj.is_cuda:
        (proj, heads, kv_heads, dim, vdim, rot, k_off, v_off, wq, wk, eps,
         cos_sin, b, cache) = prep
        h, w, top, groups, keep, scale, lists = routing
        out, u = act or (None, None)
        u_off = ff = ld_act = 0
        if act:
            assert out.stride(1) == 1 and out.shape == u.shape \
                and u.stride() == proj.stride() and u.dtype == proj.dtype
            u_off = (u.data_ptr() - proj.data_ptr()) // proj.element_size()
            ff, ld_act = u.shape[1], out.stride(0)
        assert proj.stride(1) == 1 and wq.numel() == heads * dim \
            and wk.numel() == kv_heads * dim and h.shape[0] == b.n_tok
        index, weight, counts, pairs = _routing_buffers(h, w, top, lists)
        bt = b.block_tables
        done = native().hy_window_front(
            _ptr(index), _ptr(weight), _p(counts), _p(pairs), _ptr(h),
            _ptr(w), _i(h.shape[1]), _i(w.shape[0]), _i(top), _i(groups),
            _i(keep), _f(scale), _ptr(proj), _i(proj.stride(0)), _ptr(cache),
            _i(k_off), _i(v_off), _i(heads), _i(kv_heads), _i(dim), _i(vdim),
            _i(rot), _ptr(wq), _ptr(wk), _p(cos_sin), _f(eps), _ptr(b.pos),
            _ptr(b.row), _ptr(bt), _i(bt.shape[1]), _p(out), _i(ld_act),
            _i(u_off), _i(ff), _i(b.n_tok), _dt(proj.dtype), _stream())
        if done == 1:
            return index, weight, (counts, pairs) if lists else None
        _check(done, "hy_window_front")
    window_prep(*prep)
    if act:
        squared_relu(*act)
    return route(*routing)


def can_window_mfma(dtype, group, dim, vdim) -> bool:
    """Sizes that the matrix-core kernels take."""
    return (dtype == torch.bfloat16 and dim % 8 == 0 and vdim % 8 == 0
            and dim <= 256 and vdim <= 256 and group <= 128)


def window_parts(n: int, kv_heads: int, group: int, keys: int) -> int:
    """How many workgroups share one query's keys: enough to fill the
    chip, with at least two tiles of keys each."""
    groups = n * kv_heads * ((group + 15) // 16)
    return max(1, min(256 // groups, keys // 128, 64))


def window_attention(out, proj, g_off, heads, kv_heads, dim, vdim, cache, b,
                     window, chunk: bool = False) -> None:
    """Attention of the prepared queries over the last ``window`` tokens,
    or (``chunk``) over those of the query's own run of ``window``
    positions, times the sigmoid of the heads' numbers at column
    ``g_off`` (None: no gate), into ``out`` [T, H * vdim] (columns of
    wider rows)."""
    if not proj.is_cuda:
        ref.window_attention(out, proj, g_off, heads, kv_heads, dim, vdim,
                             cache, b, window, chunk)
        return
    g_off = -1 if g_off is None else g_off
    assert proj.stride(1) == 1 and out.stride(1) == 1
    lib, bt, st = native(), b.block_tables, _stream()
    H, G, D, V = heads, kv_heads, dim, vdim
    assert cache.shape[0] * G * 16 < 2 ** 31    # rows are 32-bit numbers
    dst = (_ptr(out), _i(out.stride(0)))
    src = (_ptr(proj), _i(proj.stride(0)), _i(g_off), _ptr(cache))
    where = (_ptr(bt), _i(bt.shape[1]))
    sizes = (_i(H), _i(G), _i(D), _i(V), _i(window), _i(chunk))
    # vector accesses need whole vectors in every row
    if not (can_window_mfma(proj.dtype, H // G, D, V)
            and proj.stride(0) % 8 == 0 and out.stride(0) % 8 == 0):
        _check(lib.hy_window_rows(
            *dst, *src, _ptr(b.pos), _ptr(b.row), *where, *sizes,
            _i(b.n_tok), _dt(proj.dtype), st), "hy_window_rows")
        return
    n = b.n_short
    if n:
        parts = window_parts(n, G, H // G, min(window, b.max_keys))
        acc = ml = None
        if parts > 1:
            acc = torch.empty(n, H, parts, V, dtype=torch.float32,
                              device=proj.device)
            ml = torch.empty(n, H, parts, 2, dtype=torch.float32,
                             device=proj.device)
        _check(lib.hy_window_decode(
            *dst, _p(acc), _p(ml), *src, _ptr(b.pos), _ptr(b.row), *where,
            *sizes, _i(n), _i(parts), st), "hy_window_decode")
    if n < b.n_tok:
        items, n_items = b.query_tiles(128 // (H // G))
        _check(lib.hy_window_flash(
            *dst, *src, _ptr(items), _i(n_items), *where, *sizes, st),
            "hy_window_flash")


# -- mixture of experts ----------------------------------------------------

FEW_PAIRS = 512      # (token, choice) pairs that need no lists of experts


def can_expert_mfma(dtype, width, ff) -> bool:
    """Sizes that the matrix-core kernels take."""
    return dtype == torch.bfloat16 and width % 8 == 0 and ff % 8 == 0


def _routing_buffers(h, w, top, lists: bool):
    T, E = h.shape[0], w.shape[0]
    assert h.is_contiguous() and w.is_contiguous() \
        and w.shape[1] == h.shape[1] and w.dtype == h.dtype
    index = torch.empty(T, top, dtype=torch.int32, device=h.device)
    weight = torch.empty(T, top, dtype=torch.float32, device=h.device)
    if not lists:
        return index, weight, None, None
    return (index, weight,
            torch.zeros(E, dtype=torch.int32, device=h.device),
            torch.empty(E, T, dtype=torch.int32, device=h.device))


def route(h, w, top, groups, keep, scale, lists: bool = True):
    """The experts of every token: (index [T, top] int32, weight [T, top]
    float32, lists).  Logits w h in 32-bit, softmax over all experts, the
    ``top`` best among the ``keep`` groups of neighbours with the largest
    best score, weights over their sum times ``scale``.  ``lists``: also
    every expert's (token, choice) pairs, as (counts, pairs)."""
    if not h.is_cuda:
        return *ref.route(h, w, top, groups, keep, scale), None
    T, W = h.shape
    E = w.shape[0]
    index, weight, counts, pairs = _routing_buffers(h, w, top, lists)
    _check(native().hy_route(
        _ptr(index), _ptr(weight), _p(counts), _p(pairs), _ptr(h), _ptr(w),
        _i(W), _i(E), _i(top), _i(groups), _i(keep), _f(scale), _i(T),
        _dt(h.dtype), _stream()), "hy_route")
    return index, weight, (counts, pairs) if lists else None


def expert_tile(pairs: int, experts: int, n: int, k: int) -> int:
    """Tile of ``hy_expert_tiles`` for products of depth k with n
    outputs: 128 x 128 where experts have few pairs or outputs, 256 x 256
    for deep products, 128 x 256 (two a compute unit, so that one stores
    while the other multiplies) for shallow ones."""
    if pairs < 192 * experts or n <= 256:
        return 0
    return 1 if k > 1024 else 2


def experts(h, index, lists, w_up, w_down):
    """down(relu(up h)^2) of every token's experts -> [T, top, W].
    w_up [E, ff, W], w_down [E, W, ff]; ``lists``: of ``route``, may be
    None for few pairs on the matrix cores."""
    if not h.is_cuda:
        return ref.experts(h, index, w_up, w_down)
    T, top = index.shape
    E, F, W = w_up.shape
    assert h.is_contiguous() and w_up.is_contiguous() \
        and w_down.is_contiguous() and w_down.shape == (E, W, F) \
        and h.shape == (T, W)
    lib, st = native(), _stream()
    u = torch.empty(T * top, F, dtype=h.dtype, device=h.device)
    z = torch.empty(T, top, W, dtype=h.dtype, device=h.device)
    up = (_ptr(u), _ptr(h), _ptr(w_up))
    down = (_ptr(z), _ptr(u), _ptr(w_down))
    up_size = (_i(E), _i(F), _i(W), _i(top), _i(1))
    down_size = (_i(E), _i(W), _i(F), _i(1), _i(0))
    if lists is None:
        for data, size in ((up, up_size), (down, down_size)):
            _check(lib.hy_expert_few(*data, _ptr(index), *size, _i(T * top),
                                     st), "hy_expert_few")
        return z
    where = (_ptr(lists[0]), _ptr(lists[1]))
    tiles = can_expert_mfma(h.dtype, W, F)
    for data, size, n, k in ((up, up_size, F, W), (down, down_size, W, F)):
        args = (*data, *where, *size, _i(T), _i(T * top))
        if tiles:
            _check(lib.hy_expert_tiles(
                *args, _i(expert_tile(T * top, E, n, k)), st),
                "hy_expert_tiles")
        else:
            _check(lib.hy_expert_rows(*args, _dt(h.dtype), st),
                   "hy_expert_rows")
    return z
