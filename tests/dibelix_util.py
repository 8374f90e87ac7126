"""Small random Dibelix models and mixers for tests.

Configurations are plain dictionaries in the layout of config.json, so
that the oracle and the served model read the same thing.
"""
from __future__ import annotations

import torch

from llmlb_amd.models.mixers import ChannelDelta, LatentAttention
from packed_util import (MixerRun, engine, error, run_cuts,  # noqa: F401
                         serve_at_random, tokens, write_model)


def latent(heads, dim, rot, vdim, rank, window, base=1e4, scale=None,
           kv_from=None):
    m = {"heads": heads, "dim": dim, "rot_dim": rot, "vdim": vdim,
         "kv_rank": rank, "scale": scale or (dim + rot) ** -0.5,
         "mask": {"size": window}, "rot": {"base": base, "dims": rot}}
    if kv_from is not None:
        m["kv_from"] = kv_from
    return {"type": "latent_attention", "mixer": m}


def delta(heads, kv_heads, dim, vdim, taps, low=(12, 20)):
    return {"type": "channel_delta", "low": low, "mixer": {
        "heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim,
        "conv": taps}}


def config(layers, vocab, width, ff, eps=1e-5, softcap=9.0):
    """ff: one size for all layers, or a list with None for 'none'."""
    ffs = ff if isinstance(ff, list) else [ff] * len(layers)
    return {"architecture": "Dibelix", "vocab": vocab, "width": width,
            "norm": {"eps": eps}, "logit_softcap": softcap,
            "layers": [{**ly, "mlp": None if n is None else
                        {"kind": "dense", "ff": n}}
                       for ly, n in zip(layers, ffs)]}


# sizes that fit no vector or tile, a layer without a feed-forward, a
# shared-latent layer with heads and a window of its own
ODD = config([latent(5, 6, 2, 7, 20, 19), delta(3, 1, 10, 5, 2, (7, 9)),
              latent(2, 10, 2, 9, 20, 33, scale=0.4, kv_from=0),
              delta(4, 2, 17, 6, 3, (5, 11))],
             vocab=131, width=52, ff=[70, None, 44, 58], eps=1e-4)
# sizes of the tiled kernels, more than 16 heads, grouped delta heads, a
# second rotation
TILED = config([delta(8, 4, 128, 64, 4, (24, 40)),
                latent(20, 32, 16, 48, 136, 70, base=5e4),
                latent(12, 64, 16, 64, 136, 29, base=5e4, kv_from=1),
                delta(4, 4, 32, 48, 1, (16, 8)),
                latent(16, 24, 32, 40, 88, 41, base=900.0)],
               vocab=320, width=256, ff=208, eps=1e-6, softcap=20.0)
# one layer of each kind, for long runs
PLAIN = config([latent(3, 16, 8, 24, 40, 27), delta(4, 2, 24, 16, 4)],
               vocab=97, width=64, ff=96)


def weights(cfg, seed=0, dtype=torch.bfloat16):
    g = torch.Generator().manual_seed(seed)
    W, V = cfg["width"], cfg["vocab"]
    out = {}

    def rand(name, *shape, std=None):
        out[name] = (torch.randn(*shape, generator=g)
                     * (shape[-1] ** -0.5 if std is None else std)).to(dtype)

    rand("embed", V, W, std=1.0)
    rand("head", V, W)
    rand("final.norm", W, std=0.2)
    for i, ly in enumerate(cfg["layers"]):
        p, m = f"l{i}.mix.", ly["mixer"]
        H = m["heads"]
        rand(f"l{i}.norm1", W, std=0.2)
        if ly["type"] == "latent_attention":
            r = m["kv_rank"]
            rand(p + "q", H * (m["dim"] + m["rot_dim"]), W)
            if "kv_from" not in m:
                rand(p + "dkv", r + m["rot_dim"], W)
                rand(p + "dkv.norm", r, std=0.3)
                out[p + "dkv.norm"] += 1
            rand(p + "uk", H * m["dim"], r)
            rand(p + "uv", H * m["vdim"], r)
            rand(p + "o", W, H * m["vdim"])
        else:
            qk, v, n = m["kv_heads"] * m["dim"], H * m["vdim"], H * m["dim"]
            a, b = ly["low"]
            for name, rows in (("q", qk), ("k", qk), ("v", v)):
                rand(p + name, rows, W)
                rand(p + name + ".conv", rows, m["conv"], std=0.6)
            rand(p + "b", H, W)
            rand(p + "A_log", H, std=0.7)
            rand(p + "norm", m["vdim"], std=0.3)
            out[p + "norm"] += 1
            rand(p + "a1", a, W)
            rand(p + "a2", n, a)
            rand(p + "dt_bias", n, std=1.0)
            out[p + "dt_bias"] -= 2
            rand(p + "g1", b, W)
            rand(p + "g2", v, b)
            rand(p + "o", W, v)
        if ly["mlp"] is not None:
            rand(f"l{i}.norm2", W, std=0.2)
            rand(f"l{i}.mlp.up", ly["mlp"]["ff"], W)
            rand(f"l{i}.mlp.down", W, ly["mlp"]["ff"])
    return out


# -- one mixer alone -------------------------------------------------------

def latent_mixer(m, w, eps, width, device="cpu", dtype=torch.float32,
                 max_pos=1024):
    from llmlb_amd.ops.reference import build_cos_sin_table
    mix = LatentAttention(
        width=width, heads=m["heads"], dim=m["dim"], rot_dim=m["rot_dim"],
        vdim=m["vdim"], kv_rank=m["kv_rank"], scale=m["scale"],
        window=m["mask"]["size"], kv_from=m.get("kv_from"), eps=eps,
        dtype=dtype, device=torch.device(device))
    mix.load({k: w[k] for k in mix.weight_shapes()})
    mix.cos_sin = build_cos_sin_table(max_pos, m["rot_dim"],
                                      m["rot"]["base"]).to(device)
    return mix


def delta_mixer(m, w, eps, width, device="cpu", dtype=torch.float32):
    mix = ChannelDelta(
        width=width, heads=m["heads"], kv_heads=m["kv_heads"],
        dim=m["dim"], vdim=m["vdim"], taps=m["conv"],
        decay_rank=w["a1"].shape[0], gate_rank=w["g1"].shape[0], eps=eps,
        dtype=dtype, device=torch.device(device))
    mix.load({k: w[k] for k in mix.weight_shapes()})
    return mix


def planted_attention(m, width, T, pairs, seed=0, strength=9.0):
    """Weights and inputs of a latent layer in which, for every (i, j),
    query i's score with key j stands out in every head.

    Inputs are random except at the query places, where they are solved
    for: W_q h_i must be ``strength`` times the (rotated) key of j over
    its squared length, rotated back from position i."""
    import dibelix_oracle as O

    g = torch.Generator().manual_seed(seed)
    H, D, R, V, r = (m["heads"], m["dim"], m["rot_dim"], m["vdim"],
                     m["kv_rank"])
    assert width >= H * (D + R)
    w = {"q": torch.randn(H * (D + R), width, generator=g) * width ** -0.5,
         "dkv": torch.randn(r + R, width, generator=g) * width ** -0.5,
         "dkv.norm": 1 + 0.2 * torch.randn(r, generator=g),
         "uk": torch.randn(H * D, r, generator=g) * r ** -0.5,
         "uv": torch.randn(H * V, r, generator=g) * r ** -0.5,
         "o": torch.randn(width, H * V, generator=g) * (H * V) ** -0.5}
    w = {k: t.bfloat16().double() for k, t in w.items()}
    h = torch.randn(T, width, generator=g).bfloat16().double()
    queries = {i for i, _ in pairs}
    assert not queries & {j for _, j in pairs}
    c, kr = O.latent_kv(h, w, "", m, 1e-5)
    k = torch.cat([(c @ w["uk"].T).view(T, H, D),
                   kr[:, None].expand(T, H, R)], -1)
    for i, j in pairs:
        t = k[j] / k[j].pow(2).sum(-1, keepdim=True) * strength / m["scale"]
        # turning by -i undoes the rotation that the layer will apply
        t[:, D:] = O.rotate(t[None, :, D:], torch.tensor([-i]),
                            m["rot"]["base"])[0]
        h[i] = torch.linalg.lstsq(w["q"], t.reshape(-1, 1),
                                  driver="gelsd").solution[:, 0]
    return w, h.bfloat16().double()
