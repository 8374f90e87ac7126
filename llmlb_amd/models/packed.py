"""What the models that run packed batches have in common: reading a
model folder, loading and checking weights, the cache, embeddings.

A model's subclass builds ``layers_`` (modules with a mixer ``mix`` and a
feed-forward ``ff``, which may be None), loads their weights and
implements ``forward``.  Tensor names: ``embed``, ``head``,
``final.norm``, and per layer ``l<i>.norm1``, ``l<i>.mix.*``,
``l<i>.norm2`` (where mixer and feed-forward have norms of their own),
``l<i>.norm1b`` and ``l<i>.norm2b`` (where their outputs are normed too),
``l<i>.mlp.*``.  ``runs`` lists the layer index of every layer run of a
forward pass; each run has its own part of the cache.  ``owners`` lists
the layers that have tensors.
"""
from __future__ import annotations

import json
from pathlib import Path

import torch
import torch.nn as nn

from ..backend.kv_cache import BLOCK_SIZE, HybridCache
from ..backend.ragged import RaggedBatch
from ..ops import hybrid as hy
from ..parallel.tp import TPContext, get_tp_context
from .mixers import _linear, _param


def read_folder(path):
    """(parsed config.json, tensor name -> shape) of a model folder."""
    from safetensors import safe_open
    path = Path(path)
    shapes = {}
    for f in sorted(path.glob("*.safetensors")):
        with safe_open(str(f), framework="pt") as sf:
            for name in sf.keys():
                shapes[name] = tuple(sf.get_slice(name).get_shape())
    return json.loads((path / "config.json").read_text()), shapes


class PackedCausalLM(nn.Module):
    """Runs packed batches (backend.ragged.RaggedBatch) against a
    HybridCache; the engine owns both."""

    ragged = True
    norm_offset = 0.0          # what a stored norm weight is added to
    shared_norm = False        # one norm for mixer and feed-forward
    output_norms = False       # sublayers' outputs are normed as well
    centred_norms = False      # layer norms instead of RMS norms

    def __init__(self, cfg, tp: TPContext | None, dtype: torch.dtype,
                 device):
        super().__init__()
        self.tp = tp or get_tp_context()
        if self.tp.world_size != 1:
            raise ValueError(f"{cfg.architecture} runs on one GPU per "
                             "replica (tensor parallel size 1)")
        self.cfg, self.dtype = cfg, dtype
        self.device = torch.device(device)

    # -- weights ----------------------------------------------------------

    @property
    def norm_shape(self) -> tuple:
        """Shape of a norm's weight on the residual stream."""
        return (self.cfg.width,)

    def layer_shapes(self, i: int) -> dict[str, tuple]:
        """Names (without ``l<i>.``) and shapes of layer i's tensors."""
        ly = self.layers_[i]
        out = {"norm1": self.norm_shape}
        if self.output_norms:
            out["norm1b"] = self.norm_shape
        out.update({f"mix.{k}": s for k, s in ly.mix.weight_shapes().items()})
        if ly.ff is not None:
            if not self.shared_norm:
                out["norm2"] = self.norm_shape
            if self.output_norms:
                out["norm2b"] = self.norm_shape
            out.update({f"mlp.{k}": s
                        for k, s in ly.ff.weight_shapes().items()})
        return out

    def load_layer(self, i: int, take, vec) -> None:
        """``take(name)``: layer i's tensor as stored; ``vec(name)``: a
        32-bit parameter of it."""
        raise NotImplementedError

    def random_tensor(self, name: str, noise: torch.Tensor) -> torch.Tensor:
        """An initial value from unit normal ``noise``."""
        raise NotImplementedError

    def weight_shapes(self) -> dict[str, tuple]:
        W = self.cfg.width
        out = {"embed": (self.cfg.vocab, W), "final.norm": self.norm_shape,
               "head": (self.cfg.vocab, W)}
        for i in self.owners:
            for k, s in self.layer_shapes(i).items():
                out[f"l{i}.{k}"] = s
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
        for i in self.owners:
            self.load_layer(i, lambda k: take(f"l{i}.{k}"),
                            lambda k: vec(f"l{i}.{k}"))

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
        self._assign(lambda name: self.random_tensor(name, torch.randn(
            shapes[name], generator=g, device=self.device)))

    # -- forward ----------------------------------------------------------

    @property
    def owners(self) -> list[int]:
        return list(range(len(self.layers_)))

    @property
    def runs(self) -> list[int]:
        return list(range(len(self.layers_)))

    @property
    def specs(self):
        return [self.layers_[i].mix.cache_spec() for i in self.runs]

    def make_cache(self, num_blocks: int, slots: int) -> HybridCache:
        return HybridCache(self.specs, num_blocks, slots, self.device,
                           self.dtype)

    def final_rows(self, x: torch.Tensor, index=None) -> torch.Tensor:
        """Final-norm hidden states of the rows ``index`` (int32; None:
        all) of the residual stream."""
        return hy.norm_rows(x, index, self.final_norm, self.cfg.eps,
                            self.dtype, self.norm_offset,
                            self.centred_norms)

    def logits(self, x: torch.Tensor, index=None) -> torch.Tensor:
        """float32 logits of the rows ``index`` (int32; None: all)."""
        return hy.soft_cap(_linear(self.final_rows(x, index), self.head),
                           self.cfg.logit_softcap)

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
        return self.final_rows(self.forward(batch, cache)).view(B, L, -1)
