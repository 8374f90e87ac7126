"""Rasodra: a small decoder-only model that mixes chunked attention,
mLSTM and latent attention.

Every sublayer has a layer norm before and one after it:
x += norm(mixer(norm(x))), then x += norm(feed_forward(norm(x))), on a
32-bit residual stream; what lies between two sublayers (a norm, the sum,
the next norm) is one kernel.  The list of layers names each layer's mixer
and feed-forward (which may be missing); a layer may use an earlier one's
weights, with a cache or state of its own.
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
from .mixers import (DenseFF, GroupedAttention, LatentAttention,
                     MatrixMemory)
from .packed import PackedCausalLM, read_folder


@dataclass
class RasodraConfig:
    vocab: int
    width: int
    layers: list                      # as config.json lists them
    eps: float
    max_pos: int = 32768              # longest sequence served
    name: str = "rasodra"

    architecture = "Rasodra"
    logit_softcap = None

    @classmethod
    def from_json(cls, c: dict, **kw) -> "RasodraConfig":
        """``c``: parsed config.json."""
        return cls(vocab=c["vocab"], width=c["width"], layers=c["layers"],
                   eps=c["norm"]["eps"], **kw)

    @classmethod
    def from_dir(cls, path) -> "RasodraConfig":
        c, _ = read_folder(path)
        return cls.from_json(c, name=Path(path).resolve().name)

    @classmethod
    def build(cls, pattern: str, *, vocab, width, ff, heads, kv_heads, dim,
              chunk, latent_heads, latent_dim, rot_dim, latent_vdim, kv_rank,
              memory_heads, memory_dim, memory_vdim, gate_cap=15.0,
              rot_dims=None, base=500000.0, repeats=1, eps=1e-5,
              name="rasodra", max_pos=32768):
        """``pattern``: one letter a layer: A chunked attention, L latent
        attention, M mLSTM, in lower case without a feed-forward; all of
        it ``repeats`` times, with the same weights."""
        mixers = {
            "A": ("attention", {
                "heads": heads, "kv_heads": kv_heads, "dim": dim,
                "vdim": dim, "scale": dim ** -0.5, "mask": {"size": chunk},
                "rot": {"base": base,
                        "dims": dim if rot_dims is None else rot_dims}}),
            "L": ("latent_attention", {
                "heads": latent_heads, "dim": latent_dim,
                "rot_dim": rot_dim, "vdim": latent_vdim, "kv_rank": kv_rank,
                "scale": (latent_dim + rot_dim) ** -0.5,
                "rot": {"base": base, "dims": rot_dim}}),
            "M": ("mlstm", {"heads": memory_heads, "dim": memory_dim,
                            "vdim": memory_vdim, "gate_cap": gate_cap}),
        }
        layers = []
        for r in range(repeats):
            for i, ch in enumerate(pattern):
                kind, m = mixers[ch.upper()]
                layers.append({
                    "type": kind, "mixer": dict(m),
                    "mlp": {"kind": "dense", "ff": ff} if ch.isupper()
                    else None})
                if r:
                    layers[-1]["weights_of"] = i
        return cls(vocab, width, layers, eps, max_pos, name)

    @classmethod
    def tiny(cls) -> "RasodraConfig":
        """3 layers of every kind, run twice, for smoke runs and tests."""
        return cls.build("AmL", vocab=512, width=192, ff=320, heads=6,
                         kv_heads=2, dim=32, chunk=48, latent_heads=5,
                         latent_dim=24, rot_dim=8, latent_vdim=40,
                         kv_rank=72, memory_heads=3, memory_dim=40,
                         memory_vdim=56, rot_dims=16, repeats=2,
                         max_pos=2048, name="rasodra-tiny")

    @classmethod
    def small(cls) -> "RasodraConfig":
        """~0.2B parameters, the layers of a real small model."""
        return cls.build("AMLM", vocab=32000, width=1024, ff=4224, heads=16,
                         kv_heads=4, dim=64, chunk=1024, latent_heads=16,
                         latent_dim=64, rot_dim=32, latent_vdim=64,
                         kv_rank=256, memory_heads=8, memory_dim=64,
                         memory_vdim=128, repeats=2, name="rasodra-small")

    @classmethod
    def base_8b(cls) -> "RasodraConfig":
        """32 layers at the width of an 8B model."""
        return cls.build("AMLM" * 8, vocab=128256, width=4096, ff=21504,
                         heads=32, kv_heads=8, dim=128, chunk=4096,
                         latent_heads=32, latent_dim=128, rot_dim=64,
                         latent_vdim=128, kv_rank=512, memory_heads=16,
                         memory_dim=128, memory_vdim=256, name="rasodra-8b")

    def owner(self, i: int) -> int:
        """The layer whose weights layer i uses."""
        seen = []
        while self.layers[i].get("weights_of") is not None:
            seen.append(i)
            i = self.layers[i]["weights_of"]
            if not 0 <= i < len(self.layers) or i in seen:
                raise ValueError(f"layer {seen[0]}: weights_of leads to no "
                                 "layer with weights")
        return i


def _mixer(cfg: RasodraConfig, i: int, dtype, device):
    kind, m = cfg.layers[i]["type"], cfg.layers[i]["mixer"]
    common = dict(width=cfg.width, eps=cfg.eps, dtype=dtype, device=device)
    if kind == "attention":
        return GroupedAttention(
            heads=m["heads"], kv_heads=m["kv_heads"], dim=m["dim"],
            vdim=m["vdim"], rot=(m.get("rot") or {}).get("dims", 0),
            scale=m["scale"], window=(m.get("mask") or {}).get("size"),
            chunk=True, bias=True, tied=True, interleaved=True, **common)
    if kind == "latent_attention":
        if m["rot"]["dims"] != m["rot_dim"]:
            raise ValueError(f"layer {i}: rot.dims must equal rot_dim")
        return LatentAttention(
            heads=m["heads"], dim=m["dim"], rot_dim=m["rot_dim"],
            vdim=m["vdim"], kv_rank=m["kv_rank"], scale=m["scale"],
            window=None, kv_from=None, interleaved=True, sink=True,
            gate=True, **common)
    if kind == "mlstm":
        return MatrixMemory(heads=m["heads"], dim=m["dim"], vdim=m["vdim"],
                            gate_cap=m["gate_cap"], **common)
    raise ValueError(f"layer {i}: unknown mixer '{kind}'")


class RasodraLayer(nn.Module):
    def __init__(self, cfg: RasodraConfig, i: int, dtype, device):
        super().__init__()
        self.mix = _mixer(cfg, i, dtype, device)
        mlp = cfg.layers[i].get("mlp")
        if mlp is not None and mlp["kind"] != "dense":
            raise ValueError(f"layer {i}: unknown mlp '{mlp['kind']}'")
        self.ff = None if mlp is None else DenseFF(
            width=cfg.width, ff=mlp["ff"], act="relu2", dtype=dtype,
            device=device)


class RasodraForCausalLM(PackedCausalLM):
    output_norms = True
    centred_norms = True

    def __init__(self, cfg: RasodraConfig, tp: TPContext | None = None,
                 dtype: torch.dtype = torch.bfloat16, device="cpu",
                 seed: int = 1234, init_weights: bool = True):
        super().__init__(cfg, tp, dtype, device)
        owner = [cfg.owner(i) for i in range(len(cfg.layers))]
        own = {j: RasodraLayer(cfg, j, dtype, self.device)
               for j in sorted(set(owner))}
        for i, j in enumerate(owner):
            if any(cfg.layers[i].get(k) != cfg.layers[j].get(k)
                   for k in ("type", "mixer", "mlp")):
                raise ValueError(f"layer {i} differs from layer {j}, whose "
                                 "weights it uses")
        self._owners = list(own)
        self.layers_ = nn.ModuleList([own[j] for j in owner])
        tables: dict = {}
        for i, ly in own.items():
            rot = cfg.layers[i]["mixer"].get("rot")
            if rot and rot["dims"]:
                key = (float(rot["base"]), rot["dims"])
                if key not in tables:
                    tables[key] = build_cos_sin_table(
                        cfg.max_pos, key[1], key[0]).to(self.device)
                ly.mix.cos_sin = tables[key]
        if init_weights:
            self._init_weights(seed)

    @property
    def owners(self) -> list[int]:
        return self._owners

    # -- weights ----------------------------------------------------------

    def load_layer(self, i: int, take, vec) -> None:
        ly = self.layers_[i]
        ly.norm1, ly.norm1b = vec("norm1"), vec("norm1b")
        ly.mix.load({k: take(f"mix.{k}") for k in ly.mix.weight_shapes()})
        if ly.ff is not None:
            ly.norm2, ly.norm2b = vec("norm2"), vec("norm2b")
            ly.ff.load({k: take(f"mlp.{k}") for k in ly.ff.weight_shapes()})

    def random_tensor(self, name: str, noise: torch.Tensor) -> torch.Tensor:
        last = name.rsplit(".", 1)[-1]
        if last in ("norm1b", "norm2b"):     # what each sublayer adds
            return torch.full_like(noise, len(self.layers_) ** -0.5)
        if "norm" in last:
            return torch.ones_like(noise)
        if name.endswith("f.b"):
            return noise.add_(4.0)
        if last in ("b", "sink"):
            return noise.mul_(0.1)
        if name in ("embed", "head"):
            return noise.mul_(0.02 if name == "head" else 1.0)
        return noise.mul_(noise.shape[-1] ** -0.5)

    # -- forward ----------------------------------------------------------

    def forward(self, b: RaggedBatch, cache: HybridCache,
                on_layer=None) -> torch.Tensor:
        """Residual stream [T, width] in 32-bit after the last layer.
        ``on_layer(i, x)`` sees it after each layer."""
        x, _ = hy.embed_rows(self.embed, b.ids, copy=False)
        y = w_post = None

        def between(w_pre):
            return hy.post_pre_norm(x, y, w_post, w_pre, self.cfg.eps,
                                    self.dtype, True)

        for i, ly in enumerate(self.layers_):
            h = between(ly.norm1)
            if i and on_layer is not None:
                on_layer(i - 1, x)
            y, w_post = ly.mix(h, b, cache, i), ly.norm1b
            if ly.ff is not None:
                y, w_post = ly.ff(between(ly.norm2)), ly.norm2b
        if y is not None:
            between(None)
            if on_layer is not None:
                on_layer(len(self.layers_) - 1, x)
        return x
