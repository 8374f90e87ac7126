"""Dibelix: a small decoder-only model that mixes windowed latent
attention with a gated delta rule.

Each sublayer reads the 32-bit residual stream itself and only its
output is normed on the way back: x += norm(sublayer(x)), with norm
weights stored as the distance from one.  The list of layers names each
layer's mixer and feed-forward; sizes and constants come from the
configuration, low-rank sizes from the weights' shapes.
"""
from __future__ import annotations

import json
from dataclasses import dataclass, field
from pathlib import Path

import torch
import torch.nn as nn

from ..backend.kv_cache import BLOCK_SIZE, HybridCache
from ..backend.ragged import RaggedBatch
from ..ops import hybrid as hy
from ..ops.reference import build_cos_sin_table
from ..parallel.tp import TPContext, get_tp_context
from .mixers import ChannelDelta, DenseFF, LatentAttention, _linear, _param

NORM_OFFSET = 1.0          # norm weights are stored around zero


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
        from safetensors import safe_open
        path = Path(path)
        shapes = {}
        for f in sorted(path.glob("*.safetensors")):
            with safe_open(str(f), framework="pt") as sf:
                for name in sf.keys():
                    shapes[name] = sf.get_slice(name).get_shape()
        return cls.from_json(json.loads((path / "config.json").read_text()),
                             shapes, name=path.resolve().name)

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


class DibelixForCausalLM(nn.Module):
    """Runs packed batches (backend.ragged.RaggedBatch) against a
    HybridCache; the engine owns both."""

    ragged = True

    def __init__(self, cfg: DibelixConfig, tp: TPContext | None = None,
                 dtype: torch.dtype = torch.bfloat16, device="cpu",
                 seed: int = 1234, init_weights: bool = True):
        super().__init__()
        self.tp = tp or get_tp_context()
        if self.tp.world_size != 1:
            raise ValueError("Dibelix runs on one GPU per replica "
                             "(tensor parallel size 1)")
        self.cfg, self.dtype = cfg, dtype
        self.device = torch.device(device)
        self.layers_ = nn.ModuleList(
            [DibelixLayer(cfg, i, dtype, self.device)
             for i in range(len(cfg.layers))])
        self.specs = [ly.mix.cache_spec() for ly in self.layers_]
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

    def weight_shapes(self) -> dict[str, tuple]:
        W = self.cfg.width
        out = {"embed": (self.cfg.vocab, W), "final.norm": (W,),
               "head": (self.cfg.vocab, W)}
        for i, ly in enumerate(self.layers_):
            out[f"l{i}.norm1"] = (W,)
            for k, s in ly.mix.weight_shapes().items():
                out[f"l{i}.mix.{k}"] = s
            if ly.ff is not None:
                out[f"l{i}.norm2"] = (W,)
                for k, s in ly.ff.weight_shapes().items():
                    out[f"l{i}.mlp.{k}"] = s
        return out

    def _assign(self, take) -> None:
        """``take(name)`` -> tensor.  Matrices keep the storage type;
        norms, convolutions and decay parameters are kept in 32-bit."""
        def mat(name):
            return _param(take(name).to(dtype=self.dtype,
                                        device=self.device).contiguous())

        def vec(name):
            return _param(take(name).float().to(self.device).contiguous())

        self.embed, self.head = mat("embed"), mat("head")
        self.final_norm = vec("final.norm")
        for i, ly in enumerate(self.layers_):
            ly.norm1 = vec(f"l{i}.norm1")
            ly.mix.load({k: take(f"l{i}.mix.{k}")
                         for k in ly.mix.weight_shapes()})
            if ly.ff is not None:
                ly.norm2 = vec(f"l{i}.norm2")
                ly.ff.load({k: take(f"l{i}.mlp.{k}")
                            for k in ly.ff.weight_shapes()})

    def load_safetensors(self, path) -> int:
        """Load a *.safetensors file or a folder of shards.  Returns the
        number of tensors consumed."""
        from safetensors import safe_open
        p = Path(path)
        files = sorted(p.glob("*.safetensors")) if p.is_dir() else [p]
        if not files:
            raise FileNotFoundError(f"no .safetensors under {path}")
        tensors = {}
        for f in files:
            with safe_open(str(f), framework="pt") as sf:
                for name in sf.keys():
                    tensors[name] = sf.get_tensor(name)
        want = self.weight_shapes()
        for name, shape in want.items():
            if name not in tensors:
                raise KeyError(f"{name} is missing from {path}")
            if tuple(tensors[name].shape) != tuple(shape):
                raise ValueError(
                    f"{name}: {tuple(tensors[name].shape)} in the file, "
                    f"{tuple(shape)} by the configuration")
        self._assign(lambda name: tensors[name])
        return len(want)

    def _init_weights(self, seed: int) -> None:
        shapes = self.weight_shapes()
        g = torch.Generator(device=self.device).manual_seed(seed)

        def take(name):
            s = shapes[name]
            n = torch.randn(s, generator=g, device=self.device)
            if name.endswith("mix.norm") or name.endswith("dkv.norm"):
                return torch.ones_like(n)
            if ".norm" in name:
                return torch.zeros_like(n)
            if name.endswith("A_log"):
                return n.abs().mul_(0.5)
            if name.endswith("dt_bias"):
                return n.mul_(0.5).sub_(4.0)
            if name.endswith(".conv"):
                return n.mul_(0.5)
            return n.mul_(0.02 if name in ("embed", "head")
                          else s[-1] ** -0.5)

        self._assign(take)

    # -- forward ----------------------------------------------------------

    def make_cache(self, num_blocks: int, slots: int) -> HybridCache:
        return HybridCache(self.specs, num_blocks, slots, self.device,
                           self.dtype)

    def forward(self, b: RaggedBatch, cache: HybridCache,
                on_layer=None) -> torch.Tensor:
        """Residual stream [T, width] in 32-bit after the last layer.
        ``on_layer(i, x)`` sees it after each layer."""
        eps = self.cfg.eps
        x, xb = hy.embed_rows(self.embed, b.ids)
        for i, ly in enumerate(self.layers_):
            hy.post_norm_add(x, xb, ly.mix(xb, b, cache, i), ly.norm1, eps,
                             NORM_OFFSET)
            if ly.ff is not None:
                hy.post_norm_add(x, xb, ly.ff(xb), ly.norm2, eps,
                                 NORM_OFFSET)
            if on_layer is not None:
                on_layer(i, x)
        return x

    def logits(self, x: torch.Tensor, index=None) -> torch.Tensor:
        """float32 logits of the rows ``index`` (int32; None: all)."""
        h = hy.norm_rows(x, index, self.final_norm, self.cfg.eps, self.dtype,
                         NORM_OFFSET)
        return hy.soft_cap(_linear(h, self.head), self.cfg.logit_softcap)

    @torch.inference_mode()
    def forward_dense(self, input_ids: torch.Tensor) -> torch.Tensor:
        """Final-norm hidden states [B, L, width] of whole sequences,
        through a cache of their own (embeddings)."""
        B, L = input_ids.shape
        nb = (L + BLOCK_SIZE - 1) // BLOCK_SIZE
        cache = self.make_cache(1 + B * nb, B)
        bt = torch.arange(1, 1 + B * nb, dtype=torch.int32,
                          device=self.device).view(B, nb)
        batch = RaggedBatch.build(
            [(i, 0, toks) for i, toks in enumerate(input_ids.tolist())], bt)
        x = self.forward(batch, cache)
        return hy.norm_rows(x, None, self.final_norm, self.cfg.eps,
                            self.dtype, NORM_OFFSET).view(B, L, -1)
