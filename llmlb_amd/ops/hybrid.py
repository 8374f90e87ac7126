"""Ops of the hybrid models: 32-bit residual stream with a norm on the
sublayer's output, latent attention over pages, gated delta rule.

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

def embed_rows(table, ids):
    """(x float32 [T, W], the same in the storage type)."""
    if not table.is_cuda:
        return ref.embed_rows(table, ids)
    T, W = ids.shape[0], table.shape[1]
    x = torch.empty(T, W, dtype=torch.float32, device=table.device)
    xb = x if table.dtype == torch.float32 else torch.empty(
        T, W, dtype=table.dtype, device=table.device)
    _check(native().hy_embed_rows(
        _ptr(x), None if xb is x else _ptr(xb), _ptr(table), _ptr(ids),
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


def norm_rows(x, index, w, eps, dtype, w_offset=0.0):
    """rmsnorm(x[index]) * (w_offset + w) in ``dtype``; index may be
    None (every row)."""
    if not x.is_cuda:
        return ref.norm_rows(x, index, w, eps, dtype, w_offset)
    n = x.shape[0] if index is None else index.shape[0]
    out = torch.empty(n, x.shape[1], dtype=dtype, device=x.device)
    _check(native().hy_norm_rows(
        _ptr(out), _ptr(x), _p(index), _ptr(w), _f(w_offset), _i(n),
        _i(x.shape[1]), _f(eps), _dt(dtype), _stream()), "hy_norm_rows")
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


def latent_rows(qa, proj, dim, rot, cache, b, window, scale):
    """Absorbed attention: qa [H, N, rank] (the batch's first N tokens)
    -> weighted latents [H, N, rank]."""
    if not qa.is_cuda:
        return ref.latent_rows(qa, proj, dim, rot, cache, b, window, scale)
    H, N, rank = qa.shape
    assert qa.is_contiguous()
    out = torch.empty_like(qa)
    _check(native().hy_latent_rows(
        _ptr(out), _ptr(qa), _ptr(proj), _i(proj.stride(0)), _i(H), _i(dim),
        _i(rot), _i(rank), _ptr(cache), _ptr(b.pos), _ptr(b.row),
        _ptr(b.block_tables), _i(b.block_tables.shape[1]), _i(window),
        _f(scale), _i(N), _dt(qa.dtype), _stream()), "hy_latent_rows")
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


def latent_decode(qa, proj, dim, rot, cache, b, window, scale):
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
        _f(scale), _i(N), _i(parts), _stream()), "hy_latent_decode")
    return out


def can_flash(dtype, dim, rot, rank, vdim) -> bool:
    """Sizes that ``latent_flash`` takes."""
    return (dtype == torch.bfloat16 and dim % 8 == 0 and rot % 8 == 0
            and rank % 8 == 0 and dim + rot <= 256 and vdim <= 256)


def latent_flash(out, proj, heads, dim, rot, w_uk, w_uv, cache, b, window,
                 scale) -> None:
    """Attention of the batch's long entries into ``out`` [T, H * vdim]:
    their visible latents are copied out of the pages and expanded to
    keys and (transposed) values.  w_uk [H, dim, rank], w_uv
    [H, vdim, rank]."""
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
        _i(V), _i(window), _f(scale), st), "hy_latent_flash")


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
