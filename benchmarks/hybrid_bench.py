#!/usr/bin/env python3
"""Prefill and decode throughput of the hybrid models (Dibelix, Taletar,
Fidepel, Rasodra) beside the Llama family at equal width, depth and
parameter count (random weights, one GPU).

  python bench.py --hybrid [--steps K --warmup W]      all sizes, one JSON
  python benchmarks/hybrid_bench.py --size m --only dibelix --phase decode

A prefill step is one wave of ``--prompts`` fresh prompts of
``--prompt-len`` tokens through ``Engine.step``; a decode step is one
token of every one of ``--batch`` sequences at contexts from
``--context`` on.  All engines run through the same entry points.
"""
from __future__ import annotations

import argparse
import json
import os
import sys
import time
from pathlib import Path

sys.path.insert(0, str(Path(__file__).resolve().parents[1]))
os.environ.setdefault("TORCH_BLAS_PREFER_HIPBLASLT", "1")

import torch  # noqa: E402

#        width layers heads head_dim kv_heads inter
SIZES = {
    "s": (1024, 8, 16, 64, 4, 2816),
    "m": (2048, 8, 16, 128, 4, 5632),
    "l": (4096, 8, 32, 128, 8, 14336),
}
VOCAB, WINDOW, CHUNK = 32000, 1024, 2048


def llama_config(size: str):
    from llmlb_amd.models.llama import LlamaConfig
    w, n, h, d, kv, inter = SIZES[size]
    return LlamaConfig(hidden=w, layers=n, q_heads=h, kv_heads=kv,
                       head_dim=d, inter=inter, vocab=VOCAB, max_pos=8192,
                       name=f"llama-{size}")


def dibelix_config(size: str):
    """The same width, depth and head sizes; the feed-forward takes up
    what remains of the Llama model's parameters."""
    from llmlb_amd.models.dibelix import DibelixConfig, DibelixForCausalLM
    w, n, h, d, kv, inter = SIZES[size]

    def build(ff):
        return DibelixConfig.build(
            "LDDS" * (n // 4), vocab=VOCAB, width=w, ff=ff, heads=h, dim=d,
            rot_dim=d // 2, vdim=d, kv_rank=4 * d, window=WINDOW,
            delta_heads=h, delta_kv_heads=h, delta_dim=d, delta_vdim=d,
            low_rank=d, max_pos=8192, name=f"dibelix-{size}")

    return build(fit_ff(DibelixForCausalLM, build, size, 2))


def fit_ff(cls, build, size: str, matrices: int) -> int:
    """The feed-forward width, of ``matrices`` matrices, at which
    ``build(ff)`` has the Llama model's parameters."""
    w, n, h, d, kv, inter = SIZES[size]
    probe = cls(build(64), device="meta", init_weights=False)
    rest = sum(torch.Size(s).numel() for k, s in probe.weight_shapes().items()
               if ".mlp." not in k and not k.startswith(("embed", "head")))
    target = n * (w * (h + 2 * kv) * d + h * d * w + 3 * w * inter)
    return max(64, round((target - rest) / (matrices * w * n) / 128) * 128)


def taletar_config(size: str):
    """The same width and depth; attention has the Llama model's heads
    with two score maps of half the size, recurrent layers its heads."""
    from llmlb_amd.models.taletar import TaletarConfig, TaletarForCausalLM
    w, n, h, d, kv, inter = SIZES[size]

    def build(ff):
        return TaletarConfig.build(
            "AGMG" * (n // 4), vocab=VOCAB, width=w, ff=ff, heads=h,
            kv_heads=kv, dim=d // 2, vdim=d, gla_heads=h, gla_dim=d,
            gla_vdim=d, low_rank=d, ssm_heads=h, ssm_vdim=d, state=d,
            groups=kv, norm_groups=kv, max_pos=8192, name=f"taletar-{size}")

    return build(fit_ff(TaletarForCausalLM, build, size, 3))


def fidepel_config(size: str):
    """The same width, depth and heads, with a window; 16 experts and a
    shared one take up the Llama model's feed-forward, 4 of 16 (and the
    shared one) compute a token."""
    from llmlb_amd.models.fidepel import FidepelConfig, FidepelForCausalLM
    w, n, h, d, kv, inter = SIZES[size]

    def build(ff):
        return FidepelConfig.build(
            n, vocab=VOCAB, width=w, heads=h, kv_heads=kv, dim=d, vdim=d,
            window=WINDOW, ff=ff, experts=16, top=4, groups=4, keep=2,
            shared_ff=ff, residual_mult=0.4, max_pos=8192,
            name=f"fidepel-{size}")

    return build(fit_ff(FidepelForCausalLM, build, size, 2 * 17))


def rasodra_config(size: str):
    """The same width, depth and heads in every mixer; chunks hold a whole
    prompt, so that attention sees what the Llama model's does."""
    from llmlb_amd.models.rasodra import RasodraConfig, RasodraForCausalLM
    w, n, h, d, kv, inter = SIZES[size]

    def build(ff):
        return RasodraConfig.build(
            "AMLM" * (n // 4), vocab=VOCAB, width=w, ff=ff, heads=h,
            kv_heads=kv, dim=d, chunk=CHUNK, latent_heads=h, latent_dim=d,
            rot_dim=d // 2, latent_vdim=d, kv_rank=4 * d, memory_heads=h,
            memory_dim=d, memory_vdim=d, max_pos=8192,
            name=f"rasodra-{size}")

    return build(fit_ff(RasodraForCausalLM, build, size, 2))


CONFIGS = {"llama": llama_config, "dibelix": dibelix_config,
           "taletar": taletar_config, "fidepel": fidepel_config,
           "rasodra": rasodra_config}


def make_engine(cfg, args):
    from llmlb_amd.backend.engine import Engine, EngineConfig
    tokens = max(args.prompts * args.prompt_len,
                 args.batch * (args.context + args.warmup + args.steps + 80))
    return Engine(EngineConfig(
        model=cfg, device="cuda:0", dtype="bfloat16",
        kv_cache_blocks=tokens // 16 + 16 * args.batch + 64,
        max_batch=max(args.batch, args.prompts),
        max_prefill_tokens=args.prompts * args.prompt_len,
        enable_prefix_cache=False))


def prompt(n: int, seed: int) -> list[int]:
    g = torch.Generator().manual_seed(seed)
    return torch.randint(1, VOCAB, (n,), generator=g).tolist()


def prefill_ms(eng, args) -> float:
    from llmlb_amd.backend.sampler import SamplingParams
    times = []
    for it in range(args.warmup + args.steps):
        ids = [prompt(args.prompt_len, 1000 * it + i)
               for i in range(args.prompts)]
        for p in ids:
            eng.submit(p, SamplingParams(max_new_tokens=1))
        torch.cuda.synchronize()
        t0 = time.monotonic()
        while eng.waiting.qsize() or eng.running:
            eng.step()
        torch.cuda.synchronize()
        if it >= args.warmup:
            times.append(time.monotonic() - t0)
    return 1e3 * sum(times) / len(times)


def decode_ms(eng, args) -> float:
    from llmlb_amd.backend.sampler import SamplingParams
    warm = args.warmup + 4
    for i in range(args.batch):
        eng.submit(prompt(args.context, i),
                   SamplingParams(max_new_tokens=warm + args.decode_steps
                                  + 8))
    while (eng.waiting.qsize() or len(eng.running) < args.batch
           or any(not s.out_ids for s in eng.running)):
        eng.step()
    for _ in range(warm):
        eng.step()
    torch.cuda.synchronize()
    t0 = time.monotonic()
    for _ in range(args.decode_steps):
        eng.step()
    torch.cuda.synchronize()
    dt = time.monotonic() - t0
    assert len(eng.running) == args.batch
    for s in list(eng.running):
        eng._retire(s)
    return 1e3 * dt / args.decode_steps


def measure(kind: str, size: str, args) -> dict:
    cfg = CONFIGS[kind](size)
    eng = make_engine(cfg, args)
    out = {"parameters_m": round(sum(
        p.numel() for p in eng.model.parameters()) / 1e6, 1)}
    if args.phase in ("all", "prefill"):
        ms = prefill_ms(eng, args)
        out["prefill_ms"] = round(ms, 3)
        out["prefill_tokens_per_s"] = round(
            args.prompts * args.prompt_len / ms * 1e3)
    if args.phase in ("all", "decode"):
        ms = decode_ms(eng, args)
        out["decode_ms"] = round(ms, 3)
        out["decode_tokens_per_s"] = round(args.batch / ms * 1e3)
    del eng
    torch.cuda.empty_cache()
    return out


def add_arguments(ap) -> None:
    ap.add_argument("--size", default="s,m,l", help="of s, m, l")
    ap.add_argument("--only", default="llama,dibelix,taletar,fidepel,rasodra")
    ap.add_argument("--phase", default="all",
                    choices=("all", "prefill", "decode"))
    ap.add_argument("--prompts", type=int, default=8)
    ap.add_argument("--prompt-len", type=int, default=2048)
    ap.add_argument("--batch", type=int, default=64)
    ap.add_argument("--context", type=int, default=1024)
    ap.add_argument("--decode-steps", type=int, default=64)


def run(args) -> dict:
    with torch.inference_mode():
        sizes = {}
        for size in args.size.split(","):
            sizes[size] = {}
            for kind in args.only.split(","):
                sizes[size][kind] = measure(kind, size, args)
                print(f"[hybrid] {size} {kind} {sizes[size][kind]}",
                      file=sys.stderr, flush=True)
    return {"metric": "hybrid_tokens_per_sec", "dtype": "bf16",
            "data": "synthetic prompts, random weights",
            "config": {"prompts": args.prompts,
                       "prompt_len": args.prompt_len, "batch": args.batch,
                       "context": args.context, "window": WINDOW,
                       "chunk": CHUNK,
                       "layers": {
                           "dibelix": "latent attention, two gated delta "
                                      "layers, shared latents; repeated",
                           "taletar": "differential attention, gated "
                                      "linear attention, Mamba-2, gated "
                                      "linear attention; repeated",
                           "fidepel": "windowed attention and 4 of 16 "
                                      "experts beside a shared one",
                           "rasodra": "chunked attention, mLSTM, latent "
                                      "attention, mLSTM; repeated"}},
            "steps": args.steps, "warmup": args.warmup, "sizes": sizes}


def main(argv=None) -> None:
    ap = argparse.ArgumentParser()
    ap.add_argument("--steps", type=int, default=3)
    ap.add_argument("--warmup", type=int, default=1)
    add_arguments(ap)
    print(json.dumps(run(ap.parse_args(argv))), flush=True)


if __name__ == "__main__":
    main()
