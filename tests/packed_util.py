"""Runs that the tests of packed-batch models share."""
from __future__ import annotations

import json

import torch
from safetensors.torch import save_file

from llmlb_amd.backend.engine import Engine, EngineConfig
from llmlb_amd.backend.kv_cache import HybridCache
from llmlb_amd.backend.ragged import RaggedBatch
from llmlb_amd.models.registry import resolve


def write_model(folder, cfg, w):
    folder.mkdir(parents=True, exist_ok=True)
    (folder / "config.json").write_text(json.dumps(cfg))
    save_file(w, str(folder / "model.safetensors"))
    return folder


def engine(folder, device="cpu", dtype="float32", blocks=64, rows=6,
           max_pos=1024, **kw):
    cfg, _ = resolve(str(folder))
    cfg.max_pos = max_pos
    return Engine(EngineConfig(model=cfg, device=device, dtype=dtype,
                               kv_cache_blocks=blocks, max_batch=rows,
                               weights_path=str(folder), **kw))


def tokens(n, vocab, seed):
    g = torch.Generator().manual_seed(seed)
    return torch.randint(0, vocab, (n,), generator=g).tolist()


def run_cuts(eng, toks, cuts, close=True):
    """All logits of one sequence fed in portions ending at ``cuts``."""
    seq = eng.open_sequence()
    out, at = [], 0
    for c in list(cuts) + [len(toks)]:
        if c > at:
            out.append(eng.run_batch(
                [(seq, toks[at:c], list(range(c - at)))]).cpu().double())
            at = c
    if close:
        eng.close_sequence(seq)
    return torch.cat(out)


def error(got, want):
    """Largest over positions of the rms logit error, relative to the
    spread of the logits."""
    d = got.cpu().double() - want
    return (d.pow(2).mean(-1).sqrt().max() / want.std()).item()


def serve_at_random(eng, reqs, rows, sizes, seed=7, skip=0.25):
    """Run ``reqs`` (token lists) through batches of unequal portions,
    at most ``rows`` of them live; some are left out of a step, and the
    pages and slots of finished ones serve new ones.  Returns every
    request's logits."""
    g = torch.Generator().manual_seed(seed)
    waiting, live = list(range(len(reqs))), {}
    got = {i: [] for i in waiting}
    while waiting or live:
        while waiting and len(live) < rows:
            i = waiting.pop(0)
            live[i] = (eng.open_sequence(), 0)
        work, who = [], []
        for i, (seq, at) in live.items():
            if torch.rand((), generator=g) < skip and len(live) > 1:
                continue
            n = sizes[int(torch.randint(len(sizes), (), generator=g))]
            part = reqs[i][at:at + n]
            work.append((seq, part, list(range(len(part)))))
            who.append((i, len(part)))
        if not work:
            continue
        rows_out = eng.run_batch(work).split([n for _, n in who])
        for (i, n), r in zip(who, rows_out):
            got[i].append(r.double().cpu())
            seq, at = live[i]
            live[i] = (seq, at + n)
            if at + n == len(reqs[i]):
                eng.close_sequence(seq)
                del live[i]
    return {i: torch.cat(r) for i, r in got.items()}


class MixerRun:
    """A mixer with a cache of its own; ``rows`` sequences, pages in a
    shuffled order.  ``step([(row, inputs)])`` runs one packed batch."""

    def __init__(self, mix, rows, max_tokens, seed=0):
        nb = -(-max_tokens // 16)
        g = torch.Generator().manual_seed(seed)
        self.mix, self.dev = mix, mix.device
        spec = mix.cache_spec()
        self.cache = HybridCache([spec], 1 + rows * nb, rows, self.dev,
                                 mix.dtype)
        self.bt = (torch.randperm(rows * nb, generator=g) + 1).to(
            torch.int32).view(rows, nb).to(self.dev)
        self.at = [0] * rows

    def step(self, work):
        order = sorted(range(len(work)), key=lambda i: len(work[i][1]))
        work = [work[i] for i in order]
        runs = [(r, self.at[r], [0] * len(h)) for r, h in work]
        b = RaggedBatch.build(runs, self.bt)
        x = torch.cat([h for _, h in work]).to(self.mix.dtype).to(self.dev)
        y = self.mix(x, b, self.cache, 0).double().cpu()
        out = dict(zip((r for r, _ in work),
                       torch.split(y, [len(h) for _, h in work])))
        for r, h in work:
            self.at[r] += len(h)
        return out

    def cuts(self, row, h, cuts):
        """One sequence in portions ending at ``cuts``."""
        out, at = [], 0
        for c in list(cuts) + [len(h)]:
            if c > at:
                out.append(self.step([(row, h[at:c])])[row])
                at = c
        return torch.cat(out)

    def restart(self, row):
        self.at[row] = 0
