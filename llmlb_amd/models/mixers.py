"""Token mixers and feed-forwards of the hybrid models.

Each takes its sizes and constants as arguments and reads the layer's
input [T, width] in the storage type.  Projections of the same input are
one matrix product.

``forward`` returns the sublayer's output before any norm.  Modules for
parallel layers have ``inner`` instead: it writes what the output
projection reads (``out_width`` columns of a wider row), so that the
layer applies the projections of mixer and feed-forward as one product.
Where both also read the same norm, ``inputs`` names the weights of a
module's input projections, and the layer stacks them into one product,
whose sections start at the columns given to ``place``.
"""
from __future__ import annotations

import math

import torch
import torch.nn as nn
import torch.nn.functional as F

from ..backend.kv_cache import StateSpec, PageSpec
from ..ops import hybrid as hy
from ..ops import linear_decode

FULL_CONTEXT = 2 ** 30     # the window of an unmasked causal layer


def _linear(x, w):
    return linear_decode(x, w) if x.shape[0] <= 128 else F.linear(x, w)


def _param(t):
    return nn.Parameter(t, requires_grad=False)


def _stack_rows(parts, align: int = 8):
    """Concatenate weights along their output rows, each part padded to
    a multiple of ``align`` so that every section of the product starts
    on a whole vector.  Returns (weight, offsets)."""
    rows, offs, at = [], [], 0
    for w in parts:
        offs.append(at)
        rows.append(w)
        at += w.shape[0]
        gap = -at % align
        if gap:
            rows.append(w.new_zeros(gap, w.shape[1]))
            at += gap
    return torch.cat(rows).contiguous(), offs


def _halves(dim: int, rot: int) -> torch.Tensor:
    """Order of a head's ``dim`` numbers that takes neighbours (2i, 2i+1)
    of the first ``rot`` to places i and i + rot/2, where the kernels
    rotate pairs.  Scores do not change when queries and keys share an
    order."""
    order = torch.arange(dim)
    turned = order[:rot]
    return torch.cat([turned[0::2], turned[1::2], order[rot:]])


class LatentAttention(nn.Module):
    """Multi-head attention whose keys and values are linear maps of one
    cached latent per token, plus a rotated key part shared by the
    heads.  ``kv_from`` names the layer whose latents this one reads
    (None: its own).  ``interleaved``: neighbouring numbers turn
    together.  ``sink``: the softmax has a learned score per head without
    a key.  ``gate``: the heads' outputs are multiplied with the sigmoid
    of a projection of the layer's input."""

    def __init__(self, *, width, heads, dim, rot_dim, vdim, kv_rank, scale,
                 window, kv_from, eps, dtype, device, interleaved=False,
                 sink=False, gate=False):
        super().__init__()
        self.interleaved, self.sink, self.gate = interleaved, sink, gate
        self.heads, self.dim, self.rot, self.vdim = heads, dim, rot_dim, vdim
        self.rank, self.scale, self.kv_from = kv_rank, scale, kv_from
        self.window = min(window or FULL_CONTEXT, FULL_CONTEXT)
        self.eps, self.width = eps, width
        self.dtype, self.device = dtype, device
        self.tiled = hy.can_decode_tiled(dtype, dim, rot_dim, kv_rank)
        self.flash = hy.can_flash(dtype, dim, rot_dim, kv_rank, vdim)
        self.cos_sin = None            # set by the model, [max_pos, rot]

    def weight_shapes(self) -> dict[str, tuple]:
        H, R = self.heads, self.rank
        out = {"q": (H * (self.dim + self.rot), self.width),
               "uk": (H * self.dim, R), "uv": (H * self.vdim, R),
               "o": (self.width, H * self.vdim)}
        if self.kv_from is None:
            out["dkv"] = (R + self.rot, self.width)
            out["dkv.norm"] = (R,)
        if self.sink:
            out["sink"] = (H,)
        if self.gate:
            out["g"] = (H * self.vdim, self.width)
        return out

    def load(self, w: dict[str, torch.Tensor]) -> None:
        to = dict(dtype=self.dtype, device=self.device)
        own = self.kv_from is None
        parts = {"q": w["q"]}
        if own:
            parts["dkv"] = w["dkv"]
        if self.interleaved:
            turn = self.dim + _halves(self.rot, self.rot)
            order = torch.cat([torch.arange(self.dim), turn])
            parts["q"] = w["q"].view(self.heads, -1, self.width)[
                :, order].reshape(w["q"].shape)
            if own:
                parts["dkv"] = w["dkv"][torch.cat(
                    [torch.arange(self.rank), turn - self.dim + self.rank])]
        if self.gate:
            parts["g"] = w["g"]
        stacked, offs = _stack_rows(list(parts.values()))
        offs = dict(zip(parts, offs))
        self.w_in = _param(stacked.to(**to))
        self.c_off = offs.get("dkv", 0)
        self.g_off = offs.get("g")
        self.w_sink = _param(w["sink"].float().to(self.device).contiguous()) \
            if self.sink else None
        self.w_uk = _param(w["uk"].reshape(
            self.heads, self.dim, self.rank).to(**to).contiguous())
        uv = w["uv"].reshape(self.heads, self.vdim, self.rank).to(**to)
        self.w_uv = _param(uv.contiguous())
        self.w_uv_t = _param(uv.transpose(1, 2).contiguous())
        self.w_o = _param(w["o"].to(**to))
        self.w_norm = _param(w["dkv.norm"].float().to(self.device)) \
            if own else None

    def cache_spec(self):
        return PageSpec(self.rank + self.rot) \
            if self.kv_from is None else None

    def forward(self, x, b, cache, index: int):
        own = self.kv_from is None
        pages = cache.pages[index if own else self.kv_from]
        proj = _linear(x, self.w_in)
        hy.latent_prep(proj, self.heads, self.dim, self.rot, self.rank,
                       self.c_off, self.w_norm, self.eps, self.cos_sin, b,
                       pages, own)
        T = b.n_tok
        n = b.n_short if self.flash and x.is_cuda else T
        if n == T:
            o = self._absorbed(proj, b, pages, n)
        else:
            o = torch.empty(T, self.heads * self.vdim, dtype=x.dtype,
                            device=x.device)
            if n:
                self._absorbed(proj, b, pages, n, o[:n])
            hy.latent_flash(o, proj, self.heads, self.dim, self.rot,
                            self.w_uk, self.w_uv, pages, b, self.window,
                            self.scale, self.w_sink, self.g_off)
        return _linear(o, self.w_o)

    def _absorbed(self, proj, b, pages, n, out=None):
        """The first n tokens of the batch -> [n, heads * vdim]."""
        H, D = self.heads, self.dim
        q = proj[:n, :H * (D + self.rot)].unflatten(
            1, (H, D + self.rot))[..., :D].transpose(0, 1)
        qa = torch.bmm(q, self.w_uk)
        attend = hy.latent_decode if self.tiled and proj.is_cuda \
            else hy.latent_rows
        lat = attend(qa, proj, D, self.rot, pages, b, self.window,
                     self.scale, self.w_sink)
        o = torch.bmm(lat, self.w_uv_t)                 # [H, n, vdim]
        if self.gate:
            if out is None:
                out = torch.empty(n, H * self.vdim, dtype=o.dtype,
                                  device=o.device)
            hy.join_heads(out, o, proj, self.g_off)
            return out
        o = o.transpose(0, 1).reshape(n, H * self.vdim)
        return o if out is None else out.copy_(o)


class ChannelDelta(nn.Module):
    """Gated delta rule with a decay per head and key channel, short
    convolutions on q, k and v, and a gated norm on each head's
    output."""

    def __init__(self, *, width, heads, kv_heads, dim, vdim, taps,
                 decay_rank, gate_rank, eps, dtype, device):
        super().__init__()
        if heads % kv_heads:
            raise ValueError("heads must be a multiple of kv_heads")
        self.heads, self.kv_heads, self.dim, self.vdim = \
            heads, kv_heads, dim, vdim
        self.taps, self.eps, self.width = taps, eps, width
        self.decay_rank, self.gate_rank = decay_rank, gate_rank
        self.dtype, self.device = dtype, device

    def weight_shapes(self) -> dict[str, tuple]:
        W, qk, v = self.width, self.kv_heads * self.dim, \
            self.heads * self.vdim
        n = self.heads * self.dim
        return {"q": (qk, W), "k": (qk, W), "v": (v, W),
                "q.conv": (qk, self.taps), "k.conv": (qk, self.taps),
                "v.conv": (v, self.taps), "b": (self.heads, W),
                "A_log": (self.heads,), "norm": (self.vdim,),
                "a1": (self.decay_rank, W), "a2": (n, self.decay_rank),
                "dt_bias": (n,), "g1": (self.gate_rank, W),
                "g2": (v, self.gate_rank), "o": (W, v)}

    def load(self, w: dict[str, torch.Tensor]) -> None:
        to = dict(dtype=self.dtype, device=self.device)
        qkv = torch.cat([w["q"], w["k"], w["v"]])
        stacked, (_, self.a_off, self.g_off, self.b_off) = _stack_rows(
            [qkv, w["a1"], w["g1"], w["b"]])
        self.w_in = _param(stacked.to(**to))
        self.w_a2 = _param(w["a2"].to(**to))
        self.w_g2 = _param(w["g2"].to(**to))
        self.w_o = _param(w["o"].to(**to))

        def wide(t):
            return _param(t.float().to(self.device).contiguous())

        self.w_conv = wide(torch.cat(
            [w["q.conv"], w["k.conv"], w["v.conv"]]).t())   # [taps, C]
        self.a_log, self.dt_bias = wide(w["A_log"]), wide(w["dt_bias"])
        self.w_norm = wide(w["norm"])

    def cache_spec(self):
        C = 2 * self.kv_heads * self.dim + self.heads * self.vdim
        return StateSpec(self.heads, self.vdim, self.dim, C, self.taps)

    def forward(self, x, b, cache, index: int):
        proj = _linear(x, self.w_in)
        dec = _linear(proj[:, self.a_off:self.a_off + self.decay_rank],
                      self.w_a2)
        gate = _linear(proj[:, self.g_off:self.g_off + self.gate_rank],
                       self.w_g2)
        o = hy.gated_delta(
            proj, self.b_off, dec, gate, cache.state[index],
            cache.ring[index], b, self.w_conv, self.a_log, self.dt_bias,
            self.w_norm, self.kv_heads, self.heads, self.dim, self.vdim,
            self.taps, self.eps)
        return _linear(o, self.w_o)


class DenseFF(nn.Module):
    """down(act(up x)); ``act``: "gelu" (its tanh form) or "relu2", the
    square of relu."""

    def __init__(self, *, width, ff, dtype, device, act="gelu"):
        super().__init__()
        if act not in ("gelu", "relu2"):
            raise ValueError(f"unknown activation '{act}'")
        self.width, self.ff, self.dtype, self.device = \
            width, ff, dtype, device
        self.act = act

    def weight_shapes(self) -> dict[str, tuple]:
        return {"up": (self.ff, self.width), "down": (self.width, self.ff)}

    def load(self, w: dict[str, torch.Tensor]) -> None:
        to = dict(dtype=self.dtype, device=self.device)
        # an uneven depth would keep the staged decode GEMM from the
        # product down; what is added is zero in both matrices
        gap = -self.ff % 256 if self.ff >= 4096 else 0
        self.w_up = _param(F.pad(w["up"], (0, 0, 0, gap)).to(**to))
        self.w_down = _param(F.pad(w["down"], (0, gap)).to(**to))

    def forward(self, x):
        u = _linear(x, self.w_up)
        if self.act == "gelu":
            hy.gelu_tanh_(u)
        else:
            hy.squared_relu(u, u)
        return _linear(u, self.w_down)


class DifferentialAttention(nn.Module):
    """Causal attention with two score maps over the same values,
    combined as a1 - lam * a2, normed per head and gated by a projection
    of the layer's input.

    ``q_scale`` ([max_pos], set by the model) is the score factor of a
    query at each position; ``softcap`` (None: off) bounds scores to
    softcap * tanh(score / softcap)."""

    def __init__(self, *, width, heads, kv_heads, dim, vdim, softcap, diff,
                 eps, dtype, device):
        super().__init__()
        if heads % kv_heads:
            raise ValueError("heads must be a multiple of kv_heads")
        self.heads, self.kv_heads, self.dim, self.vdim = \
            heads, kv_heads, dim, vdim
        self.softcap, self.diff = softcap or 0.0, diff
        self.eps, self.width = eps, width
        self.dtype, self.device = dtype, device
        self.out_width = heads * vdim
        self.q_scale = None

    def weight_shapes(self) -> dict[str, tuple]:
        W, H, G, D, V = (self.width, self.heads, self.kv_heads, self.dim,
                         self.vdim)
        return {"q": (H * 2 * D, W), "k": (G * 2 * D, W), "v": (G * V, W),
                "lq1": (D,), "lk1": (D,), "lq2": (D,), "lk2": (D,),
                "g": (H * V, W), "o": (W, H * V)}

    def load(self, w: dict[str, torch.Tensor]) -> None:
        stacked, offs = _stack_rows([w["q"], w["k"], w["v"], w["g"]])
        self.w_in = _param(stacked.to(dtype=self.dtype, device=self.device))
        _, self.k_off, self.v_off, self.g_off = offs
        d1, d2 = ((w[f"lq{n}"].float() * w[f"lk{n}"].float()).sum().exp()
                  for n in (1, 2))
        self.lam = float(d1 - d2 + self.diff)

    def cache_spec(self):
        return PageSpec(self.kv_heads * (2 * self.dim + self.vdim))

    def inner(self, x, b, cache, index: int, out) -> None:
        proj = _linear(x, self.w_in)
        pages = cache.pages[index]
        hy.pair_append(proj, self.k_off, self.v_off, self.kv_heads,
                       self.dim, self.vdim, b, pages)
        hy.pair_attention(out, proj, self.g_off, self.heads, self.kv_heads,
                          self.dim, self.vdim, pages, b, self.q_scale,
                          self.softcap, self.lam, 1.0 - self.diff, self.eps)


class GatedLinearAttention(nn.Module):
    """S <- diag(alpha) S + k v^T, o = S^T q, with a decay per head and
    key channel from a low-rank projection: alpha = sigmoid(z)^(1/tau).
    Each head's output is normed and gated."""

    def __init__(self, *, width, heads, dim, vdim, tau, decay_rank, eps,
                 dtype, device):
        super().__init__()
        self.heads, self.dim, self.vdim, self.tau = heads, dim, vdim, tau
        self.decay_rank, self.eps, self.width = decay_rank, eps, width
        self.dtype, self.device = dtype, device
        self.out_width = heads * vdim

    def weight_shapes(self) -> dict[str, tuple]:
        W, n, v = self.width, self.heads * self.dim, self.heads * self.vdim
        return {"q": (n, W), "k": (n, W), "v": (v, W), "g": (v, W),
                "o": (W, v), "norm": (self.vdim,),
                "a1": (self.decay_rank, W), "a2": (n, self.decay_rank),
                "a2.b": (n,)}

    def load(self, w: dict[str, torch.Tensor]) -> None:
        to = dict(dtype=self.dtype, device=self.device)
        stacked, offs = _stack_rows(
            [w["q"], w["k"], w["v"], w["g"], w["a1"]])
        self.w_in = _param(stacked.to(**to))
        _, self.k_off, self.v_off, self.g_off, self.a_off = offs
        self.w_a2 = _param(w["a2"].to(**to).contiguous())
        self.b_a2, self.w_norm = (
            _param(w[n].float().to(self.device).contiguous())
            for n in ("a2.b", "norm"))

    def cache_spec(self):
        return StateSpec(self.heads, self.vdim, self.dim, 0, 0)

    def inner(self, x, b, cache, index: int, out) -> None:
        proj = _linear(x, self.w_in)
        dec = _linear(proj[:, self.a_off:self.a_off + self.decay_rank],
                      self.w_a2)
        hy.gated_linear(out, proj, self.k_off, self.v_off, self.g_off, dec,
                        self.b_a2, cache.state[index], b, self.w_norm,
                        self.heads, self.dim, self.vdim, self.tau, self.eps)


class StateSpaceDuality(nn.Module):
    """Mamba-2: S <- exp(-exp(A) dt) S + dt B x^T, y = S^T C + D x, with
    x, B and C from a short convolution and B, C shared by the heads of a
    group; y is gated first and then normed in ``norm_groups`` parts."""

    def __init__(self, *, width, heads, vdim, state, groups, taps,
                 norm_groups, eps, dtype, device):
        super().__init__()
        if heads % groups or heads * vdim % norm_groups:
            raise ValueError("groups must divide heads, and norm_groups "
                             "heads * vdim")
        self.heads, self.vdim, self.state, self.groups = \
            heads, vdim, state, groups
        self.taps, self.norm_groups = taps, norm_groups
        self.eps, self.width = eps, width
        self.dtype, self.device = dtype, device
        self.out_width = heads * vdim
        self.channels = heads * vdim + 2 * groups * state

    def weight_shapes(self) -> dict[str, tuple]:
        W, inner, C, H = self.width, self.out_width, self.channels, self.heads
        return {"in": (inner + C + H, W), "conv": (C, self.taps),
                "conv.b": (C,), "dt_bias": (H,), "A_log": (H,), "D": (H,),
                "norm": (inner,), "o": (W, inner)}

    def load(self, w: dict[str, torch.Tensor]) -> None:
        inner, C = self.out_width, self.channels
        z, xbc, dt = torch.split(w["in"], [inner, C, self.heads])
        # convolved channels first, as the kernels index them
        stacked, (_, self.z_off, self.dt_off) = _stack_rows([xbc, z, dt])
        self.w_in = _param(stacked.to(dtype=self.dtype, device=self.device))

        def wide(t):
            return _param(t.float().to(self.device).contiguous())

        self.w_conv = wide(w["conv"].t())                  # [taps, C]
        self.b_conv, self.w_norm = wide(w["conv.b"]), wide(w["norm"])
        # per head: dt's bias, the rate exp(A_log), D
        self.per_head = wide(torch.stack(
            [w["dt_bias"].float(), w["A_log"].float().exp(),
             w["D"].float()]))

    def cache_spec(self):
        return StateSpec(self.heads, self.vdim, self.state, self.channels,
                         self.taps)

    def inner(self, x, b, cache, index: int, out) -> None:
        proj = _linear(x, self.w_in)
        hy.state_space(out, proj, self.z_off, self.dt_off,
                       cache.state[index], cache.ring[index], b, self.w_conv,
                       self.b_conv, self.per_head, self.w_norm, self.groups,
                       self.heads, self.state, self.vdim, self.taps,
                       self.norm_groups, self.eps)


class ClampedSwiGLU(nn.Module):
    """g sigmoid(sharpness g) (u + 1) with g = min(gate x, limit) and
    u = clamp(up x, -limit, limit)."""

    def __init__(self, *, width, ff, limit, dtype, device, sharpness=1.702):
        super().__init__()
        self.width, self.ff, self.limit = width, ff, limit
        self.sharpness = sharpness
        self.dtype, self.device = dtype, device
        self.out_width = ff

    def weight_shapes(self) -> dict[str, tuple]:
        return {"gate": (self.ff, self.width), "up": (self.ff, self.width),
                "down": (self.width, self.ff)}

    def load(self, w: dict[str, torch.Tensor]) -> None:
        stacked, (_, self.u_off) = _stack_rows([w["gate"], w["up"]])
        self.w_in = _param(stacked.to(dtype=self.dtype, device=self.device))

    def inner(self, x, out) -> None:
        hy.clamped_swiglu(out, _linear(x, self.w_in), self.u_off, self.limit,
                          self.sharpness)


class WindowedAttention(nn.Module):
    """Causal attention over the last ``window`` tokens (None: all).
    Queries and keys are normed over the whole projection and rotated on
    the first ``rot`` numbers of each head; every head has a score
    temperature and an output gate from a projection of the layer's
    input.  ``cos_sin`` ([max_pos, rot]) is set by the model."""

    inputs = ("q", "k", "v", "g")

    def __init__(self, *, width, heads, kv_heads, dim, vdim, rot, scale,
                 window, eps, dtype, device):
        super().__init__()
        if heads % kv_heads:
            raise ValueError("heads must be a multiple of kv_heads")
        if rot % 2 or not 0 <= rot <= dim:
            raise ValueError("rotated dimensions must be even and at most "
                             "the head size")
        if window is not None and window < 1:
            raise ValueError("a window holds at least one token")
        self.heads, self.kv_heads, self.dim, self.vdim = \
            heads, kv_heads, dim, vdim
        self.rot, self.scale = rot, scale
        self.window = min(window or FULL_CONTEXT, FULL_CONTEXT)
        self.eps, self.width = eps, width
        self.dtype, self.device = dtype, device
        self.out_width = heads * vdim
        self.cos_sin = None

    def weight_shapes(self) -> dict[str, tuple]:
        W, H, G, D, V = (self.width, self.heads, self.kv_heads, self.dim,
                         self.vdim)
        return {"q": (H * D, W), "k": (G * D, W), "v": (G * V, W),
                "q.norm": (H * D,), "k.norm": (G * D,), "temp": (H,),
                "g": (H, W), "o": (W, H * V)}

    def load(self, w: dict[str, torch.Tensor]) -> None:
        def wide(t):
            return _param(t.to(self.device).contiguous())

        # the kernels' softmax is of powers of two
        factor = w["temp"].float() * (self.scale * math.log2(math.e))
        self.w_q = wide(w["q.norm"].float()
                        * factor.repeat_interleave(self.dim))
        self.w_k = wide(w["k.norm"].float())

    def place(self, offsets) -> None:
        q, self.k_off, self.v_off, self.g_off = offsets
        assert q == 0, "queries are the first section"

    def cache_spec(self):
        return PageSpec(self.kv_heads * (self.dim + self.vdim))

    def prep(self, proj, b, cache, index: int) -> tuple:
        """Arguments of ``hybrid.window_prep``."""
        return (proj, self.heads, self.kv_heads, self.dim, self.vdim,
                self.rot, self.k_off, self.v_off, self.w_q, self.w_k,
                self.eps, self.cos_sin, b, cache.pages[index])

    def attend(self, proj, b, cache, index: int, out) -> None:
        hy.window_attention(out, proj, self.g_off, self.heads, self.kv_heads,
                            self.dim, self.vdim, cache.pages[index], b,
                            self.window)

    def inner(self, proj, b, cache, index: int, out) -> None:
        hy.window_prep(*self.prep(proj, b, cache, index))
        self.attend(proj, b, cache, index, out)


class GroupedAttention(nn.Module):
    """Causal attention with grouped key/value heads, over the last
    ``window`` tokens or (``chunk``) those of the query's own run of
    ``window`` positions (None: all).  Queries and keys are normed per
    head and rotated on the first ``rot`` numbers of each; with
    ``interleaved`` neighbouring numbers turn together.  ``bias``: their
    projections have biases.  ``tied``: the values are the keys as
    projected, before norm and rotation.  ``cos_sin`` ([max_pos, rot]) is
    set by the model."""

    def __init__(self, *, width, heads, kv_heads, dim, vdim, rot, scale,
                 window, chunk, bias, tied, interleaved, eps, dtype, device):
        super().__init__()
        if heads % kv_heads:
            raise ValueError("heads must be a multiple of kv_heads")
        if rot % 2 or not 0 <= rot <= dim:
            raise ValueError("rotated dimensions must be even and at most "
                             "the head size")
        if window is not None and window < 1:
            raise ValueError("a window or chunk holds at least one token")
        if tied and vdim != dim:
            raise ValueError("values that are the keys have their size")
        self.heads, self.kv_heads, self.dim, self.vdim = \
            heads, kv_heads, dim, vdim
        self.rot, self.scale = rot, scale
        self.window = min(window or FULL_CONTEXT, FULL_CONTEXT)
        self.chunk = chunk and window is not None
        self.bias, self.tied, self.interleaved = bias, tied, interleaved
        self.eps, self.width = eps, width
        self.dtype, self.device = dtype, device
        self.cos_sin = None

    def weight_shapes(self) -> dict[str, tuple]:
        W, H, G, D, V = (self.width, self.heads, self.kv_heads, self.dim,
                         self.vdim)
        out = {"q": (H * D, W), "k": (G * D, W), "q.norm": (D,),
               "k.norm": (D,), "o": (W, H * V)}
        if self.bias:
            out.update({"q.b": (H * D,), "k.b": (G * D,)})
        if not self.tied:
            out["v"] = (G * V, W)
        return out

    def load(self, w: dict[str, torch.Tensor]) -> None:
        D = self.dim
        order = _halves(D, self.rot) if self.interleaved \
            else torch.arange(D)

        def heads_in(t):
            """Rows of every head in the kernels' order."""
            return t.reshape(-1, D, *t.shape[1:])[:, order].reshape(t.shape)

        def wide(t):
            return _param(t.float().to(self.device).contiguous())

        to = dict(dtype=self.dtype, device=self.device)
        parts = [heads_in(w["q"]), heads_in(w["k"])]
        if not self.tied:
            parts.append(w["v"])
        stacked, offs = _stack_rows(parts)
        self.w_in = _param(stacked.to(**to))
        self.k_off = offs[1]
        self.v_off = None if self.tied else offs[2]
        self.b_q = wide(heads_in(w["q.b"])) if self.bias else None
        self.b_k = wide(heads_in(w["k.b"])) if self.bias else None
        # the kernels' softmax is of powers of two
        self.w_q = wide(w["q.norm"].float()[order]
                        * (self.scale * math.log2(math.e)))
        self.w_k = wide(w["k.norm"][order])
        w_o = w["o"]
        if self.tied:      # the heads' outputs are in the keys' order
            w_o = w_o.view(self.width, -1, D)[:, :, order].reshape(w_o.shape)
        self.w_o = _param(w_o.to(**to).contiguous())

    def cache_spec(self):
        return PageSpec(self.kv_heads * (self.dim + self.vdim))

    def forward(self, x, b, cache, index: int):
        H, G, D, V = self.heads, self.kv_heads, self.dim, self.vdim
        proj, pages = _linear(x, self.w_in), cache.pages[index]
        hy.head_prep(proj, H, G, D, V, self.rot, self.k_off, self.v_off,
                     self.b_q, self.b_k, self.w_q, self.w_k, self.eps,
                     self.cos_sin, b, pages)
        o = torch.empty(x.shape[0], H * V, dtype=x.dtype, device=x.device)
        hy.window_attention(o, proj, None, H, G, D, V, pages, b, self.window,
                            self.chunk)
        return _linear(o, self.w_o)


class MatrixMemory(nn.Module):
    """mLSTM: S <- exp(f) S + exp(i) k v^T with a normaliser n of the same
    gates, o = S^T q / max(|n . q|, 1), kept in range by a running
    maximum of the gates' logarithms; i = cap tanh(. / cap) and
    f = log sigmoid(cap tanh(. / cap)).  Each head's output is normed,
    weighted and gated."""

    def __init__(self, *, width, heads, dim, vdim, gate_cap, eps, dtype,
                 device):
        super().__init__()
        self.heads, self.dim, self.vdim, self.cap = \
            heads, dim, vdim, gate_cap
        self.eps, self.width = eps, width
        self.dtype, self.device = dtype, device

    def weight_shapes(self) -> dict[str, tuple]:
        W, H = self.width, self.heads
        n, v = H * self.dim, H * self.vdim
        return {"q": (n, W), "k": (n, W), "v": (v, W), "g": (v, W),
                "i": (H, W), "f": (H, W), "i.b": (H,), "f.b": (H,),
                "norm": (v,), "o": (W, v)}

    def load(self, w: dict[str, torch.Tensor]) -> None:
        to = dict(dtype=self.dtype, device=self.device)
        stacked, offs = _stack_rows(
            [w["q"], w["k"], w["v"], w["g"], torch.cat([w["i"], w["f"]])])
        self.w_in = _param(stacked.to(**to))
        _, self.k_off, self.v_off, self.g_off, self.i_off = offs

        def wide(t):
            return _param(t.float().to(self.device).contiguous())

        self.b_gate = wide(torch.stack([w["i.b"], w["f.b"]]))
        self.w_norm = wide(w["norm"])
        self.w_o = _param(w["o"].to(**to))

    def cache_spec(self):
        return StateSpec(self.heads, self.vdim, self.dim, 0, 0,
                         hy.memory_extra(self.dim))

    def forward(self, x, b, cache, index: int):
        proj = _linear(x, self.w_in)
        o = torch.empty(x.shape[0], self.heads * self.vdim, dtype=x.dtype,
                        device=x.device)
        hy.matrix_memory(o, proj, self.k_off, self.v_off, self.g_off,
                         self.i_off, self.b_gate, self.cap,
                         cache.state[index], cache.extra[index], b,
                         self.w_norm, self.heads, self.dim, self.vdim,
                         self.eps)
        return _linear(o, self.w_o)


class RoutedExperts(nn.Module):
    """Feed-forward experts down(relu(up x)^2), of which every token uses
    the ``top`` that a router scores highest, besides one that all tokens
    use (``shared``: its width, None: there is none).  Experts form
    ``groups`` runs of neighbours; only those of the ``keep`` groups with
    the largest best score can be chosen."""

    def __init__(self, *, width, ff, experts, top, groups, keep, scale,
                 shared, dtype, device):
        super().__init__()
        if groups < 1 or experts % groups or not 1 <= keep <= groups:
            raise ValueError("expert groups must be equal, and some kept")
        if not 1 <= top <= keep * (experts // groups):
            raise ValueError("more experts a token than can be chosen")
        self.width, self.ff, self.experts, self.top = width, ff, experts, top
        self.groups, self.keep, self.scale = groups, keep, scale
        self.dtype, self.device = dtype, device
        self.out_width = shared or 0
        self.inputs = ("shared.up",) if shared else ()

    def weight_shapes(self) -> dict[str, tuple]:
        W = self.width
        out = {"router": (self.experts, W)}
        for e in range(self.experts):
            out[f"e{e}.up"] = (self.ff, W)
            out[f"e{e}.down"] = (W, self.ff)
        if self.out_width:
            out["shared.up"] = (self.out_width, W)
            out["shared.down"] = (W, self.out_width)
        return out

    def load(self, w: dict[str, torch.Tensor]) -> None:
        to = dict(dtype=self.dtype, device=self.device)
        self.w_router = _param(w["router"].to(**to).contiguous())
        self.w_up, self.w_down = (
            _param(torch.stack([w[f"e{e}.{n}"] for e in range(self.experts)])
                   .to(**to)) for n in ("up", "down"))

    def place(self, offsets) -> None:
        self.u_off = offsets[0] if offsets else None

    def routing(self, x) -> tuple:
        """Arguments of ``hybrid.route``."""
        few = x.shape[0] * self.top <= hy.FEW_PAIRS \
            and hy.can_expert_mfma(x.dtype, self.width, self.ff)
        return (x, self.w_router, self.top, self.groups, self.keep,
                self.scale, not few)

    def act(self, proj, out) -> tuple | None:
        """Arguments of ``hybrid.squared_relu``: the shared expert's
        activation (None: there is none)."""
        n = self.out_width
        return (out, proj[:, self.u_off:self.u_off + n]) if n else None

    def routed(self, x, index, lists):
        """The chosen experts' outputs [T, top, width]."""
        return hy.experts(x, index, lists, self.w_up, self.w_down)
