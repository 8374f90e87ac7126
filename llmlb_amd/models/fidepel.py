"""Fidepel: a small decoder-only model of windowed attention and mixtures
of experts, some of whose layers run several times.

A layer is parallel with one norm: x += m (mixer(norm(x)) +
feed_forward(norm(x))), on a 32-bit residual stream; a norm has a single
number as its weight.  All input projections of a layer are one matrix
product, and so are the output projections of attention and the shared
expert; the residual sum takes in the routed experts' outputs and is
fused with the next layer's norm.

A run of layers may be repeated with the same weights; every pass has
pages of its own.
"""
from __future__ import annotations

import math
from dataclasses import dataclass
from pathlib import Path

import torch
import torch.nn as nn

from ..backend.kv_cache import HybridCache
from ..backend.ragged import RaggedBatch
from ..ops import hybrid as hy
from ..ops.reference import build_cos_sin_table
from ..parallel.tp import TPContext
from .mixers import (RoutedExperts, WindowedAttention, _linear, _param,
                     _stack_rows)
from .packed import PackedCausalLM, read_folder


@dataclass
class FidepelConfig:
    vocab: int
    width: int
    layers: list                      # as config.json lists them
    eps: float
    residual_mult: float
    loop: dict | None = None          # start, stop, times
    max_pos: int = 32768              # longest sequence served
    name: str = "fidepel"

    architecture = "Fidepel"
    logit_softcap = None

    @classmethod
    def from_json(cls, c: dict, **kw) -> "FidepelConfig":
        """``c``: parsed config.json."""
        return cls(vocab=c["vocab"], width=c["width"], layers=c["layers"],
                   eps=c["norm"]["eps"], residual_mult=c["residual_mult"],
                   loop=c.get("loop"), **kw)

    @classmethod
    def from_dir(cls, path) -> "FidepelConfig":
        c, _ = read_folder(path)
        return cls.from_json(c, name=Path(path).resolve().name)

    @classmethod
    def build(cls, n_layers: int, *, vocab, width, heads, kv_heads, dim,
              vdim, window, ff, experts, top, groups, keep, shared_ff,
              router_scale=1.0, rot_dims=None, base=10000.0, factor=1.0,
              residual_mult=1.0, loop=None, eps=1e-5, name="fidepel",
              max_pos=32768):
        """``n_layers`` layers of the same sizes; ``loop``: (start, stop,
        times)."""
        layer = {
            "type": "attention",
            "mixer": {"heads": heads, "kv_heads": kv_heads, "dim": dim,
                      "vdim": vdim, "scale": dim ** -0.5,
                      "mask": {"size": window},
                      "rot": {"base": base,
                              "dims": dim if rot_dims is None else rot_dims,
                              "scaling": {"factor": factor}}},
            "mlp": {"kind": "moe", "expert": {"ff": ff},
                    "router": {"experts": experts, "top": top,
                               "groups": {"count": groups, "keep": keep},
                               "scale": router_scale},
                    "shared": {"ff": shared_ff} if shared_ff else None}}
        return cls(vocab, width, [layer] * n_layers, eps, residual_mult,
                   loop and dict(zip(("start", "stop", "times"), loop)),
                   max_pos, name)

    @classmethod
    def tiny(cls) -> "FidepelConfig":
        """3 layers, one of them run twice, for smoke runs and tests."""
        return cls.build(3, vocab=512, width=192, heads=6, kv_heads=2,
                         dim=32, vdim=40, window=48, ff=72, experts=10, top=3,
                         groups=5, keep=3, shared_ff=104, router_scale=1.5,
                         rot_dims=16, factor=2.0, residual_mult=0.6,
                         loop=(1, 2, 2), max_pos=2048, name="fidepel-tiny")

    @classmethod
    def small(cls) -> "FidepelConfig":
        """~0.4B parameters, the layers of a real small model."""
        return cls.build(12, vocab=32000, width=1024, heads=16, kv_heads=4,
                         dim=64, vdim=64, window=1024, ff=512, experts=32,
                         top=4, groups=4, keep=2, shared_ff=512,
                         residual_mult=0.3, loop=(2, 10, 2),
                         name="fidepel-small")

    @classmethod
    def base_8b(cls) -> "FidepelConfig":
        """32 layers at the width of an 8B model."""
        return cls.build(32, vocab=128256, width=4096, heads=32, kv_heads=8,
                         dim=128, vdim=128, window=4096, ff=640, experts=32,
                         top=4, groups=8, keep=4, shared_ff=1280,
                         residual_mult=0.2, name="fidepel-8b")

    def runs(self) -> list[int]:
        """Layer index of every layer run of a forward pass."""
        n = len(self.layers)
        if not self.loop:
            return list(range(n))
        start, stop, times = (self.loop[k]
                              for k in ("start", "stop", "times"))
        if not (0 <= start <= stop <= n and times >= 1):
            raise ValueError(f"loop {self.loop} does not fit {n} layers")
        return (list(range(start)) + list(range(start, stop)) * times
                + list(range(stop, n)))


def _mixer(cfg: FidepelConfig, i: int, dtype, device):
    kind, m = cfg.layers[i]["type"], cfg.layers[i]["mixer"]
    if kind != "attention":
        raise ValueError(f"layer {i}: unknown mixer '{kind}'")
    return WindowedAttention(
        width=cfg.width, heads=m["heads"], kv_heads=m["kv_heads"],
        dim=m["dim"], vdim=m["vdim"], scale=m["scale"],
        rot=(m.get("rot") or {}).get("dims", 0),
        window=(m.get("mask") or {}).get("size"), eps=cfg.eps, dtype=dtype,
        device=device)


def _feed_forward(cfg: FidepelConfig, i: int, dtype, device):
    mlp = cfg.layers[i].get("mlp")
    if mlp is None:
        return None
    if mlp["kind"] != "moe":
        raise ValueError(f"layer {i}: unknown mlp '{mlp['kind']}'")
    router = mlp["router"]
    groups = router.get("groups") or {"count": 1, "keep": 1}
    return RoutedExperts(
        width=cfg.width, ff=mlp["expert"]["ff"], experts=router["experts"],
        top=router["top"], groups=groups["count"], keep=groups["keep"],
        scale=router["scale"], shared=(mlp.get("shared") or {}).get("ff"),
        dtype=dtype, device=device)


class FidepelLayer(nn.Module):
    def __init__(self, cfg: FidepelConfig, i: int, dtype, device):
        super().__init__()
        self.mix = _mixer(cfg, i, dtype, device)
        self.ff = _feed_forward(cfg, i, dtype, device)

    def forward(self, h, b, cache, run: int):
        """(what the joined output projections give, what the routed
        experts add or None)."""
        n = self.mix.out_width
        proj = _linear(h, self.w_in)
        mid = torch.empty(h.shape[0], self.w_out.shape[1], dtype=h.dtype,
                          device=h.device)
        if self.ff is None:
            self.mix.inner(proj, b, cache, run, mid[:, :n])
            return _linear(mid, self.w_out), None
        index, weight, lists = hy.window_front(
            self.mix.prep(proj, b, cache, run), self.ff.routing(h),
            self.ff.act(proj, mid[:, n:]))
        self.mix.attend(proj, b, cache, run, mid[:, :n])
        z = self.ff.routed(h, index, lists)
        return _linear(mid, self.w_out), (z, weight)


class FidepelForCausalLM(PackedCausalLM):
    shared_norm = True
    norm_shape = ()            # one number for all coordinates

    def __init__(self, cfg: FidepelConfig, tp: TPContext | None = None,
                 dtype: torch.dtype = torch.bfloat16, device="cpu",
                 seed: int = 1234, init_weights: bool = True):
        super().__init__(cfg, tp, dtype, device)
        self._runs = cfg.runs()
        self.layers_ = nn.ModuleList(
            [FidepelLayer(cfg, i, dtype, self.device)
             for i in range(len(cfg.layers))])
        tables: dict = {}
        for i, ly in enumerate(self.layers_):
            if ly.mix.rot:
                rot = cfg.layers[i]["mixer"]["rot"]
                key = (float(rot["base"]), ly.mix.rot, float(
                    (rot.get("scaling") or {}).get("factor", 1.0)))
                if key not in tables:
                    tables[key] = build_cos_sin_table(
                        cfg.max_pos, key[1], key[0],
                        factor=key[2]).to(self.device)
                ly.mix.cos_sin = tables[key]
        if init_weights:
            self._init_weights(seed)

    @property
    def runs(self) -> list[int]:
        return self._runs

    # -- weights ----------------------------------------------------------

    def load_layer(self, i: int, take, vec) -> None:
        ly = self.layers_[i]
        ly.norm1 = vec("norm1")
        mods = [(ly.mix, "mix")] + ([(ly.ff, "mlp")] if ly.ff else [])
        ins, outs = [], [take("mix.o")]
        for mod, p in mods:
            mod.load({k: take(f"{p}.{k}") for k in mod.weight_shapes()})
            ins += [take(f"{p}.{k}") for k in mod.inputs]
        if ly.ff is not None and ly.ff.out_width:
            outs.append(take("mlp.shared.down"))
        to = dict(dtype=self.dtype, device=self.device)
        stacked, offs = _stack_rows([w.to(**to) for w in ins])
        ly.w_in = _param(stacked)
        for mod, _ in mods:
            n = len(mod.inputs)
            mod.place(offs[:n])
            offs = offs[n:]
        ly.w_out = _param(torch.cat([w.to(**to) for w in outs],
                                    1).contiguous())

    def random_tensor(self, name: str, noise: torch.Tensor) -> torch.Tensor:
        if "norm" in name.rsplit(".", 1)[-1] or name.endswith(".temp"):
            return torch.ones_like(noise)
        if name in ("embed", "head"):
            return noise.mul_(0.02)
        depth = len(self._runs) if name.endswith((".o", ".down")) else 1
        return noise.mul_(noise.shape[-1] ** -0.5 / math.sqrt(depth))

    # -- forward ----------------------------------------------------------

    def forward(self, b: RaggedBatch, cache: HybridCache,
                on_layer=None) -> torch.Tensor:
        """Residual stream [T, width] in 32-bit after the last layer.
        ``on_layer(run, x)`` sees it after each layer run."""
        eps, mult = self.cfg.eps, self.cfg.residual_mult
        x, _ = hy.embed_rows(self.embed, b.ids, copy=False)
        y = routed = None
        for run, i in enumerate(self._runs):
            ly = self.layers_[i]
            h, _ = hy.add_norms(x, y, ly.norm1, None, eps, self.dtype, mult,
                                routed)
            if run and on_layer is not None:
                on_layer(run - 1, x)
            y, routed = ly(h, b, cache, run)
        if y is not None:
            hy.add_norms(x, y, None, None, eps, self.dtype, mult, routed)
            if on_layer is not None:
                on_layer(len(self._runs) - 1, x)
        return x
