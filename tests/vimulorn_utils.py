"""Small Vimulorn configurations and random weights (checkpoint names, bf16) for the tests."""
from __future__ import annotations

import json
import os

import numpy as np
import torch


def latent(heads, dim, vdim, q_rank, kv_rank, scale=None):
    return {"type": "latent_attention",
            "mixer": dict(heads=heads, dim=dim, vdim=vdim, q_rank=q_rank, kv_rank=kv_rank,
                          scale=dim ** -0.5 if scale is None else scale)}


def delta(heads, kv_heads, dim, vdim, conv):
    return {"type": "channel_delta", "mixer": dict(heads=heads, kv_heads=kv_heads, dim=dim, vdim=vdim, conv=conv)}


def window(heads, kv_heads, dim, vdim, conv, size, scale=None):
    return {"type": "attention",
            "mixer": dict(heads=heads, kv_heads=kv_heads, dim=dim, vdim=vdim, conv=conv, mask={"size": size},
                          scale=dim ** -0.5 if scale is None else scale)}


def mlp(ff, limit):
    return {"kind": "dense", "ff": ff, "limit": limit}


def config(width, vocab, layers, loop=None, eps=1e-5):
    out = {"architecture": "Vimulorn", "width": width, "vocab": vocab, "norm": {"eps": eps},
           "layers": [dict(layer, mlp=ff) for layer, ff in layers]}
    if loop is not None:
        out["loop"] = dict(zip(("start", "stop", "times"), loop))
    return out


# Different sizes, orders and branches; none is a multiple of everything.
CONFIGS = {
    # every mixer, a loop over all of them, grouped heads, sizes that are no multiples of 8
    "mixed": config(100, 213, [(window(4, 2, 20, 12, 4, 9), mlp(75, 1.5)), (delta(4, 2, 12, 20, 3), mlp(50, 3.0)),
                               (latent(3, 20, 28, 18, 44), None), (delta(2, 1, 40, 8, 2), mlp(64, 0.7))],
                    loop=(1, 4, 3), eps=3e-5),
    # no loop, one key/value head, one tap, a window longer than some sequences, layers without feed-forward
    "plain": config(64, 96, [(latent(2, 8, 8, 16, 8, scale=0.5), mlp(32, 4.0)), (window(6, 1, 32, 64, 1, 100), None),
                             (delta(3, 3, 72, 24, 5), None)]),
    # loop from the first layer, longest taps first, a window of one token
    "loop0": config(48, 65, [(delta(2, 2, 16, 16, 4), mlp(40, 2.5)), (window(2, 2, 16, 8, 2, 1), mlp(24, 1.0)),
                             (latent(5, 12, 16, 8, 24), mlp(16, 1.0))], loop=(0, 2, 2), eps=1e-4),
    # heads wider than the matrix-core attention takes, more than 8 query heads per key/value head
    "wide": config(72, 80, [(window(10, 1, 264, 40, 3, 33), mlp(48, 2.0)), (latent(9, 136, 272, 24, 72), None),
                            (delta(2, 1, 200, 136, 3), None)]),
}
RANKS = {"mixed": (10, 6), "plain": (8, 16), "loop0": (24, 9), "wide": (16, 8)}


def weights(cfg, seed=0, ranks=(8, 8), sharp=2.0):
    """Random tensors under their checkpoint names.  sharp: gain of query and key projections."""
    gen = torch.Generator().manual_seed(seed)

    def n(*shape, std=1.0, mean=0.0):
        return (torch.randn(*shape, generator=gen) * std + mean).to(torch.bfloat16)

    def lin(out, inp, gain=1.0):
        return n(out, inp, std=gain * inp ** -0.5)

    t, w = {}, cfg["width"]

    def norm(name):
        t[name] = n(w, std=0.2, mean=1.0)
        t[name + ".b"] = n(w, std=0.1)
        t[name + ".alpha"] = n(1, std=0.1, mean=0.6).reshape(())

    def conv(name, channels, taps):
        c = torch.randn(channels, taps, generator=gen) * 0.4
        c[:, -1] += 1.0
        t[name] = c.to(torch.bfloat16)

    t["embed"], t["head"] = n(cfg["vocab"], w), lin(cfg["vocab"], w)
    norm("final.norm")
    for i, layer in enumerate(cfg["layers"]):
        m, p, H = layer["mixer"], f"l{i}.mix.", layer["mixer"]["heads"]
        dim, vdim = m["dim"], m["vdim"]
        for k in ("norm1", "norm1b"):
            norm(f"l{i}.{k}")
        if layer["type"] == "latent_attention":
            qr, kr = m["q_rank"], m["kv_rank"]
            t[p + "dq"], t[p + "dkv"], t[p + "g"] = lin(qr, w), lin(kr, w), lin(H, w)
            t[p + "dq.norm"], t[p + "dkv.norm"] = n(qr, std=0.2, mean=1.0), n(kr, std=0.2, mean=1.0)
            t[p + "uq"], t[p + "uk"], t[p + "uv"] = lin(H * dim, qr, sharp), lin(H * dim, kr, sharp), lin(H * vdim, kr)
        else:
            G, taps = m["kv_heads"], m["conv"]
            vh = H if layer["type"] == "channel_delta" else G
            qh = G if layer["type"] == "channel_delta" else H
            gain = sharp if layer["type"] == "attention" else 1.0
            for k, rows in (("q", qh * dim), ("k", G * dim), ("v", vh * vdim)):
                t[p + k] = lin(rows, w, 1.0 if k == "v" else gain)
                conv(p + k + ".conv", rows, taps)
            if layer["type"] == "attention":
                t[p + "sink"] = n(H, std=1.0, mean=1.0)
            else:
                ra, rg = ranks
                t[p + "b"], t[p + "a1"], t[p + "g1"] = lin(H, w), lin(ra, w), lin(rg, w)
                t[p + "a2"], t[p + "g2"] = lin(H * dim, ra), lin(H * vdim, rg)
                t[p + "A_log"] = n(H, std=1.0, mean=-2.0)
                t[p + "dt_bias"] = n(H * dim, std=1.0)
                t[p + "norm"] = n(vdim, std=0.2, mean=1.0)
        t[p + "o"] = lin(w, H * vdim, 1.5)
        if layer["mlp"] is not None:
            for k in ("norm2", "norm2b"):
                norm(f"l{i}.{k}")
            ff = layer["mlp"]["ff"]
            t[f"l{i}.mlp.gate"], t[f"l{i}.mlp.up"], t[f"l{i}.mlp.down"] = lin(ff, w, 1.5), lin(ff, w, 1.5), lin(w, ff)
    return t


def as_numpy(t):
    return {k: v.float().numpy().astype(np.float64) for k, v in t.items()}


def save(folder, cfg, t):
    from safetensors.torch import save_file

    with open(os.path.join(folder, "config.json"), "w") as f:
        json.dump(cfg, f)
    save_file({k: v.contiguous() for k, v in t.items()}, os.path.join(folder, "model.safetensors"))


def tokens(cfg, n, seed=0):
    return np.random.default_rng(seed).integers(0, cfg["vocab"], n).tolist()


def spread(got, want):
    """Largest over the rows of rms(difference) / rms(wanted), means taken off."""
    got, want = np.asarray(got, np.float64), np.asarray(want, np.float64)
    d = got - want
    d = d - d.mean(-1, keepdims=True)
    w = want - want.mean(-1, keepdims=True)
    return float((np.sqrt((d ** 2).mean(-1)) / np.sqrt((w ** 2).mean())).max())
