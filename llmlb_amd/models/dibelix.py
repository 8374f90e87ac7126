"""Dibelix: a small decoder-only model that mixes windowed latent
attention with a gated delta rule.

Each sublayer reads the 32-bit residual stream itself and only its
output is normed on the way back: x += norm(sublayer(x)), with norm
weights stored as the distance from one.  The list of layers names each
layer's mixer and feed-forward; sizes and constants come from the
configuration, low-rank sizes from the weights' shapes.
"""
from __future__ import annotations

from dataclasses import dataclass, field
from pathlib import Path

import torch
import torch.nn as nn

from ..backend.kv_cache import HybridCache
from ..backend.ragged import RaggedBatch
from ..ops import hybrid as hy
from ..ops.reference import build_cos_sin_table
from ..parallel.tp import TPContext
from .mixers import ChannelDelta, DenseFF, LatentAttention
from .packed import PackedCausalLM, read_folder


@dataclass
class DibelixConfig:
    vocab: int
    width: int
    layers: list                      # as config.json lists them
    eps: float
    logit_softcap: float | None = None
    # (decay rank, gate rank) of each recurrent layer, by layer index
    low_rank: dict = field(default_factory=dict)
    max_pos: int = 32768              # longest sequence served
    name: str = "dibelix"

    architecture = "Dibelix"

    @classmethod
    def from_json(cls, c: dict, shapes: dict | None = None,
                  **kw) -> "DibelixConfig":
        """``c``: parsed config.json; ``shapes``: tensor name -> shape
        of its weights."""
        low = {}
        for i, layer in enumerate(c["layers"]):
            if layer["type"] == "channel_delta" and shapes is not None:
                low[i] = (shapes[f"l{i}.mix.a1"][0],
                          shapes[f"l{i}.mix.g1"][0])
        return cls(vocab=c["vocab"], width=c["width"], layers=c["layers"],
                   eps=c["norm"]["eps"], logit_softcap=c.get("logit_softcap"),
                   low_rank=low, **kw)

    @classmethod
    def from_dir(cls, path) -> "DibelixConfig":
        c, shapes = read_folder(path)
        return cls.from_json(c, shapes, name=Path(path).resolve().name)

    @classmethod
    def build(cls, pattern: str, *, vocab, width, ff, heads, dim, rot_dim,
              vdim, kv_rank, window, delta_heads, delta_kv_heads, delta_dim,
              delta_vdim, low_rank, taps=4, base=500000.0, eps=1e-5,
              softcap=30.0, name="dibelix", max_pos=32768):
        """``pattern``: one letter a layer: L latent attention, S latent
        attention on the latents of the last L, D gated delta rule."""
        layers, owner = [], None
        for i, ch in enumerate(pattern):
            if ch == "D":
                kind, m = "channel_delta", {
                    "heads": delta_heads, "kv_heads": delta_kv_heads,
                    "dim": delta_dim, "vdim": delta_vdim, "conv": taps}
            else:
                kind, m = "latent_attention", {
                    "heads": heads, "dim": dim, "rot_dim": rot_dim,
                    "vdim": vdim, "kv_rank": kv_rank,
                    "scale": (dim + rot_dim) ** -0.5,
                    "mask": {"size": window},
                    "rot": {"base": base, "dims": rot_dim}}
                if ch == "S":
                    m["kv_from"] = owner
                else:
                    owner = i
            layers.append({"type": kind, "mixer": m,
                           "mlp": {"kind": "dense", "ff": ff}})
        return cls(vocab, width, layers, eps, softcap,
                   {i: (low_rank, low_rank)
                    for i, ch in enumerate(pattern) if ch == "D"},
                   max_pos, name)

    @classmethod
    def tiny(cls) -> "DibelixConfig":
        """4 layers of every kind for smoke runs and tests."""
        return cls.build("LDSD", vocab=512, width=192, ff=320, heads=6,
                         dim=24, rot_dim=8, vdim=40, kv_rank=72, window=40,
                         delta_heads=4, delta_kv_heads=2, delta_dim=48,
                         delta_vdim=32, low_rank=20, max_pos=2048,
                         name="dibelix-tiny")

    @classmethod
    def small(cls) -> "DibelixConfig":
        """~0.4B parameters, the layers of a real small model."""
        return cls.build("LDDSLDDS", vocab=32000, width=1024, ff=4224,
                         heads=16, dim=64, rot_dim=32, vdim=64, kv_rank=256,
                         window=1024, delta_heads=16, delta_kv_heads=16,
                         delta_dim=64, delta_vdim=64, low_rank=64,
                         name="dibelix-small")

    @classmethod
    def base_8b(cls) -> "DibelixConfig":
        """32 layers at the width of an 8B model."""
        return cls.build("LDDS" * 8, vocab=128256, width=4096, ff=21504,
                         heads=32, dim=128, rot_dim=64, vdim=128,
                         kv_rank=512, window=2048, delta_heads=32,
                         delta_kv_heads=32, delta_dim=128, delta_vdim=128,
                         low_rank=128, name="dibelix-8b")


def _mixer(cfg: DibelixConfig, i: int, dtype, device):
    layer = cfg.layers[i]
    kind, m = layer["type"], layer["mixer"]
    common = dict(width=cfg.width, eps=cfg.eps, dtype=dtype, device=device)
    if kind == "latent_attention":
        src = m.get("kv_from")
        if src is not None and not (
                0 <= src < i
                and cfg.layers[src]["type"] == "latent_attention"
                and cfg.layers[src]["mixer"].get("kv_from") is None):
            raise ValueError(f"layer {i}: kv_from {src} is no earlier layer "
                             "with latents of its own")
        if m["rot"]["dims"] != m["rot_dim"]:
            raise ValueError(f"layer {i}: rot.dims must equal rot_dim")
        return LatentAttention(
            heads=m["heads"], dim=m["dim"], rot_dim=m["rot_dim"],
            vdim=m["vdim"], kv_rank=m["kv_rank"], scale=m["scale"],
            window=(m.get("mask") or {}).get("size"), kv_from=src, **common)
    if kind == "channel_delta":
        decay, gate = cfg.low_rank[i]
        return ChannelDelta(
            heads=m["heads"], kv_heads=m["kv_heads"], dim=m["dim"],
            vdim=m["vdim"], taps=m["conv"], decay_rank=decay,
            gate_rank=gate, **common)
    raise ValueError(f"layer {i}: unknown mixer '{kind}'")


class DibelixLayer(nn.Module):
    def __init__(self, cfg: DibelixConfig, i: int, dtype, device):
        super().__init__()
        self.mix = _mixer(cfg, i, dtype, device)
        mlp = cfg.layers[i].get("mlp")
        if mlp is not None and mlp["kind"] != "dense":
            raise ValueError(f"layer {i}: unknown mlp '{mlp['kind']}'")
        self.ff = None if mlp is None else DenseFF(
            width=cfg.width, ff=mlp["ff"], dtype=dtype, device=device)


class DibelixForCausalLM(PackedCausalLM):
    norm_offset = 1.0          # norm weights are stored around zero

    def __init__(self, cfg: DibelixConfig, tp: TPContext | None = None,
                 dtype: torch.dtype = torch.bfloat16, device="cpu",
                 seed: int = 1234, init_weights: bool = True):
        super().__init__(cfg, tp, dtype, device)
        self.layers_ = nn.ModuleList(
            [DibelixLayer(cfg, i, dtype, self.device)
             for i in range(len(cfg.layers))])
        tables: dict = {}
        for i, ly in enumerate(self.layers_):
            if isinstance(ly.mix, LatentAttention):
                key = (float(cfg.layers[i]["mixer"]["rot"]["base"]),
                       ly.mix.rot)
                if key not in tables:
                    tables[key] = build_cos_sin_table(
                        cfg.max_pos, key[1], key[0]).to(self.device)
                ly.mix.cos_sin = tables[key]
        if init_weights:
            self._init_weights(seed)

    # -- weights ----------------------------------------------------------

    def load_layer(self, i: int, take, vec) -> None:
        ly = self.layers_[i]
        ly.norm1 = vec("norm1")
        ly.mix.load({k: take(f"mix.{k}") for k in ly.mix.weight_shapes()})
        if ly.ff is not None:
            ly.norm2 = vec("norm2")
            ly.ff.load({k: take(f"mlp.{k}") for k in ly.ff.weight_shapes()})

    def random_tensor(self, name: str, noise: torch.Tensor) -> torch.Tensor:
        if name.endswith("mix.norm") or name.endswith("dkv.norm"):
            return torch.ones_like(noise)
        if ".norm" in name:
            return torch.zeros_like(noise)
        if name.endswith("A_log"):
            return noise.abs().mul_(0.5)
        if name.endswith("dt_bias"):
            return noise.mul_(0.5).sub_(4.0)
        if name.endswith(".conv"):
            return noise.mul_(0.5)
        return noise.mul_(0.02 if name in ("embed", "head")
                          else noise.shape[-1] ** -0.5)

    # -- forward ----------------------------------------------------------

    def forward(self, b: RaggedBatch, cache: HybridCache,
                on_layer=None) -> torch.Tensor:
        """Residual stream [T, width] in 32-bit after the last layer.
        ``on_layer(i, x)`` sees it after each layer."""
        eps = self.cfg.eps
        x, xb = hy.embed_rows(self.embed, b.ids)
        for i, ly in enumerate(self.layers_):
            hy.post_norm_add(x, xb, ly.mix(xb, b, cache, i), ly.norm1, eps,
                             self.norm_offset)
            if ly.ff is not None:
                hy.post_norm_add(x, xb, ly.ff(xb), ly.norm2, eps,
                                 self.norm_offset)
            if on_layer is not None:
                on_layer(i, x)
        return x
