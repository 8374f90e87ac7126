"""Taletar: a small decoder-only model that mixes differential attention,
gated linear attention and Mamba-2 layers.

A layer is parallel: x += mixer(norm1(x)) + feed_forward(norm2(x)), both
norms of the same 32-bit residual stream.  Its two output projections
are one matrix product, and the residual sum is fused with the next
layer's norms.  The list of layers names each layer's mixer and
feed-forward; sizes and constants come from the configuration, low-rank
sizes from the weights' shapes.
"""
from __future__ import annotations

import math
from dataclasses import dataclass, field
from pathlib import Path

import torch
import torch.nn as nn

from ..backend.kv_cache import HybridCache
from ..backend.ragged import RaggedBatch
from ..ops import hybrid as hy
from ..parallel.tp import TPContext
from .mixers import (ClampedSwiGLU, DifferentialAttention,
                     GatedLinearAttention, StateSpaceDuality, _linear,
                     _param)
from .packed import PackedCausalLM, read_folder


@dataclass
class TaletarConfig:
    vocab: int
    width: int
    layers: list                      # as config.json lists them
    eps: float
    # decay rank of each gated linear attention layer, by layer index
    low_rank: dict = field(default_factory=dict)
    max_pos: int = 32768              # longest sequence served
    name: str = "taletar"

    architecture = "Taletar"
    logit_softcap = None

    @classmethod
    def from_json(cls, c: dict, shapes: dict | None = None,
                  **kw) -> "TaletarConfig":
        """``c``: parsed config.json; ``shapes``: tensor name -> shape
        of its weights."""
        low = {i: shapes[f"l{i}.mix.a1"][0]
               for i, layer in enumerate(c["layers"])
               if layer["type"] == "gla"} if shapes is not None else {}
        return cls(vocab=c["vocab"], width=c["width"], layers=c["layers"],
                   eps=c["norm"]["eps"], low_rank=low, **kw)

    @classmethod
    def from_dir(cls, path) -> "TaletarConfig":
        c, shapes = read_folder(path)
        return cls.from_json(c, shapes, name=Path(path).resolve().name)

    @classmethod
    def build(cls, pattern: str, *, vocab, width, ff, heads, kv_heads, dim,
              vdim, gla_heads, gla_dim, gla_vdim, low_rank, ssm_heads,
              ssm_vdim, state, groups, norm_groups=1, taps=4, softcap=50.0,
              q_temp=(0.1, 8192), diff=0.8, tau=16.0, limit=7.0, eps=1e-5,
              name="taletar", max_pos=32768):
        """``pattern``: one letter a layer: A differential attention, G
        gated linear attention, M Mamba-2."""
        mixers = {
            "A": ("attention", {
                "heads": heads, "kv_heads": kv_heads, "dim": dim,
                "vdim": vdim, "scale": dim ** -0.5, "softcap": softcap,
                "q_temp": {"coef": q_temp[0], "every": q_temp[1]},
                "diff": diff}),
            "G": ("gla", {"heads": gla_heads, "dim": gla_dim,
                          "vdim": gla_vdim, "tau": tau}),
            "M": ("mamba2", {"heads": ssm_heads, "vdim": ssm_vdim,
                             "state": state, "groups": groups, "conv": taps,
                             "norm_groups": norm_groups}),
        }
        layers = [{"type": mixers[ch][0], "mixer": dict(mixers[ch][1]),
                   "mlp": {"kind": "dense", "ff": ff, "limit": limit}}
                  for ch in pattern]
        return cls(vocab, width, layers, eps,
                   {i: low_rank for i, ch in enumerate(pattern) if ch == "G"},
                   max_pos, name)

    @classmethod
    def tiny(cls) -> "TaletarConfig":
        """4 layers of every kind for smoke runs and tests."""
        return cls.build("AGMA", vocab=512, width=192, ff=320, heads=6,
                         kv_heads=2, dim=24, vdim=40, gla_heads=3,
                         gla_dim=40, gla_vdim=56, low_rank=12, ssm_heads=6,
                         ssm_vdim=24, state=32, groups=2, norm_groups=2,
                         max_pos=2048, name="taletar-tiny")

    @classmethod
    def small(cls) -> "TaletarConfig":
        """~0.2B parameters, the layers of a real small model."""
        return cls.build("AGMAGM", vocab=32000, width=1024, ff=2816,
                         heads=16, kv_heads=4, dim=32, vdim=64, gla_heads=16,
                         gla_dim=64, gla_vdim=64, low_rank=16, ssm_heads=32,
                         ssm_vdim=64, state=128, groups=1,
                         name="taletar-small")

    @classmethod
    def base_8b(cls) -> "TaletarConfig":
        """32 layers at the width of an 8B model."""
        return cls.build("AGMG" * 8, vocab=128256, width=4096, ff=14336,
                         heads=32, kv_heads=8, dim=64, vdim=128,
                         gla_heads=32, gla_dim=128, gla_vdim=128,
                         low_rank=128, ssm_heads=64, ssm_vdim=64, state=128,
                         groups=8, norm_groups=8, name="taletar-8b")


def query_scale_table(max_pos: int, scale: float, q_temp: dict | None
                      ) -> torch.Tensor:
    """Score factor of a query at each position, float32 [max_pos]:
    scale * (1 + coef ln(floor((p + 1) / every) + 1))."""
    if not q_temp:
        return torch.full((max_pos,), scale, dtype=torch.float32)
    p = torch.arange(1, max_pos + 1, dtype=torch.float64)
    steps = torch.floor(p / q_temp["every"])
    return (scale * (1.0 + q_temp["coef"] * torch.log(steps + 1.0))).float()


def _mixer(cfg: TaletarConfig, i: int, dtype, device):
    kind, m = cfg.layers[i]["type"], cfg.layers[i]["mixer"]
    common = dict(width=cfg.width, eps=cfg.eps, dtype=dtype, device=device)
    if kind == "attention":
        return DifferentialAttention(
            heads=m["heads"], kv_heads=m["kv_heads"], dim=m["dim"],
            vdim=m["vdim"], softcap=m.get("softcap"), diff=m["diff"],
            **common)
    if kind == "gla":
        return GatedLinearAttention(
            heads=m["heads"], dim=m["dim"], vdim=m["vdim"], tau=m["tau"],
            decay_rank=cfg.low_rank[i], **common)
    if kind == "mamba2":
        return StateSpaceDuality(
            heads=m["heads"], vdim=m["vdim"], state=m["state"],
            groups=m["groups"], taps=m["conv"],
            norm_groups=m["norm_groups"], **common)
    raise ValueError(f"layer {i}: unknown mixer '{kind}'")


class TaletarLayer(nn.Module):
    def __init__(self, cfg: TaletarConfig, i: int, dtype, device):
        super().__init__()
        self.mix = _mixer(cfg, i, dtype, device)
        mlp = cfg.layers[i].get("mlp")
        if mlp is not None and mlp["kind"] != "dense":
            raise ValueError(f"layer {i}: unknown mlp '{mlp['kind']}'")
        self.ff = None if mlp is None else ClampedSwiGLU(
            width=cfg.width, ff=mlp["ff"], limit=mlp["limit"], dtype=dtype,
            device=device)
        self.norm2 = None

    def forward(self, h1, h2, b, cache, index: int):
        """mixer(h1) + feed_forward(h2)."""
        n = self.mix.out_width
        mid = torch.empty(h1.shape[0], self.w_out.shape[1], dtype=h1.dtype,
                          device=h1.device)
        self.mix.inner(h1, b, cache, index, mid[:, :n])
        if self.ff is not None:
            self.ff.inner(h2, mid[:, n:])
        return _linear(mid, self.w_out)


class TaletarForCausalLM(PackedCausalLM):
    def __init__(self, cfg: TaletarConfig, tp: TPContext | None = None,
                 dtype: torch.dtype = torch.bfloat16, device="cpu",
                 seed: int = 1234, init_weights: bool = True):
        super().__init__(cfg, tp, dtype, device)
        self.layers_ = nn.ModuleList(
            [TaletarLayer(cfg, i, dtype, self.device)
             for i in range(len(cfg.layers))])
        tables: dict = {}
        for i, ly in enumerate(self.layers_):
            if isinstance(ly.mix, DifferentialAttention):
                m = cfg.layers[i]["mixer"]
                temp = m.get("q_temp")
                key = (m["scale"], *((temp or {}).get(k)
                                     for k in ("coef", "every")))
                if key not in tables:
                    tables[key] = query_scale_table(
                        cfg.max_pos, m["scale"], temp).to(self.device)
                ly.mix.q_scale = tables[key]
        if init_weights:
            self._init_weights(seed)

    # -- weights ----------------------------------------------------------

    def load_layer(self, i: int, take, vec) -> None:
        ly = self.layers_[i]
        ly.norm1 = vec("norm1")
        ly.mix.load({k: take(f"mix.{k}") for k in ly.mix.weight_shapes()})
        outs = [take("mix.o")]
        if ly.ff is not None:
            ly.norm2 = vec("norm2")
            ly.ff.load({k: take(f"mlp.{k}") for k in ly.ff.weight_shapes()})
            outs.append(take("mlp.down"))
        ly.w_out = _param(torch.cat(outs, 1).to(
            dtype=self.dtype, device=self.device).contiguous())

    def random_tensor(self, name: str, noise: torch.Tensor) -> torch.Tensor:
        if "norm" in name.rsplit(".", 1)[-1] or name.endswith("mix.D"):
            return torch.ones_like(noise)
        if name.endswith("A_log"):
            return noise.abs().mul_(0.5)
        if name.endswith("dt_bias"):
            return noise.mul_(0.5).sub_(4.0)
        if name.endswith("a2.b"):
            return noise.add_(2.0)
        if name.endswith("conv.b") or ".mix.l" in name:
            return noise.mul_(0.1)
        if name.endswith(".conv"):
            return noise.mul_(0.5)
        if name in ("embed", "head"):
            return noise.mul_(0.02)
        depth = len(self.layers_) if name.endswith((".o", ".down")) else 1
        return noise.mul_(noise.shape[-1] ** -0.5 / math.sqrt(depth))

    # -- forward ----------------------------------------------------------

    def forward(self, b: RaggedBatch, cache: HybridCache,
                on_layer=None) -> torch.Tensor:
        """Residual stream [T, width] in 32-bit after the last layer.
        ``on_layer(i, x)`` sees it after each layer."""
        eps = self.cfg.eps
        x, _ = hy.embed_rows(self.embed, b.ids, copy=False)
        y = None
        for i, ly in enumerate(self.layers_):
            h1, h2 = hy.add_norms(x, y, ly.norm1, ly.norm2, eps, self.dtype)
            if i and on_layer is not None:
                on_layer(i - 1, x)
            y = ly(h1, h2, b, cache, i)
        if y is not None:
            hy.add_norms(x, y, None, None, eps, self.dtype)
            if on_layer is not None:
                on_layer(len(self.layers_) - 1, x)
        return x
