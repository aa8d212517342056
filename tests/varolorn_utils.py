"""Small Varolorn configurations and random weights (checkpoint names, bf16) for the tests."""
from __future__ import annotations

import torch

from tests.vimulorn_utils import as_numpy, save, spread, tokens  # noqa: F401


def attention(heads, kv_heads, dim, vdim, chunk, rows, far, v_mix=True, scale=None):
    """rows: of the table of biases (not in config.json: its size is the tensor's)."""
    return {"type": "attention", "rows": rows,
            "mixer": dict(heads=heads, kv_heads=kv_heads, dim=dim, vdim=vdim, bias_max=far, v_mix=v_mix,
                          mask={"size": chunk}, scale=dim ** -0.5 if scale is None else scale)}


def mamba(heads, groups, vdim, state, conv, norm_groups):
    return {"type": "mamba2", "mixer": dict(heads=heads, groups=groups, vdim=vdim, state=state, conv=conv,
                                            norm_groups=norm_groups)}


def ff(size):
    return {"kind": "dense", "ff": size}


def config(width, vocab, streams, layers, scale=1.0, bigram=(31, 7, 3), eps=1e-5):
    buckets, mul_prev, mul_cur = bigram
    return {"architecture": "Varolorn", "width": width, "vocab": vocab, "streams": streams, "norm": {"eps": eps},
            "embedding": {"scale": scale, "bigram": {"buckets": buckets, "mul_prev": mul_prev, "mul_cur": mul_cur}},
            "layers": [dict({k: v for k, v in layer.items() if k != "rows"}, mlp=mlp) for layer, mlp in layers]}


# Different sizes, orders and branches; few are a multiple of anything.
_LAYERS = {
    # every branch, grouped heads, chunks shorter than a key tile, values mixed across a recurrence and across layers
    # with other heads, a layer that mixes none
    "mixed": [(attention(4, 2, 20, 12, 9, 8, 12), ff(75)), (mamba(4, 2, 20, 12, 4, 2), ff(50)),
              (attention(6, 2, 28, 12, 33, 6, 20), None), (attention(3, 3, 16, 24, 70, 12, 40, v_mix=False), ff(33)),
              (mamba(3, 1, 8, 40, 2, 1), None), (attention(2, 2, 8, 12, 64, 5, 9, scale=0.5), ff(24))],
    # one stream, the recurrence first, one tap, heads that are no multiple of anything, chunks longer than sequences
    "one": [(mamba(3, 3, 10, 8, 1, 3), ff(32)), (attention(2, 1, 32, 64, 200, 32, 100), None),
            (mamba(5, 1, 7, 24, 3, 1), ff(16))],
    # more streams than the fused epilogue takes, five taps, chunks of one token, bias rows that end before the chunk
    "many": [(attention(2, 2, 16, 8, 1, 4, 6), ff(40)), (mamba(6, 2, 12, 72, 5, 4), ff(24)),
             (attention(5, 1, 12, 16, 48, 16, 17, v_mix=False), ff(16)), (attention(5, 1, 12, 16, 127, 2, 3, v_mix=False), None)],
    # heads wider than the matrix-core attention takes, many query heads per key head, norm groups of 256
    "wide": [(attention(10, 1, 264, 40, 50, 10, 30), ff(48)), (mamba(32, 4, 16, 200, 4, 2), None),
             (attention(9, 1, 136, 40, 100, 7, 64), ff(8))],
}
CONFIGS = {
    "mixed": config(100, 213, 3, _LAYERS["mixed"], scale=3.0, eps=3e-5),
    "one": config(64, 96, 1, _LAYERS["one"], bigram=(1, 5, 2)),
    "many": config(48, 65, 5, _LAYERS["many"], scale=0.5, bigram=(1000, 999983, 12345), eps=1e-4),
    "wide": config(72, 80, 4, _LAYERS["wide"], bigram=(64, 1, 0)),
}


def weights(name, seed=0, sharp=1.0):
    """Random tensors under their checkpoint names.  sharp: gain of the query norm."""
    cfg = CONFIGS[name]
    gen = torch.Generator().manual_seed(seed)

    def n(*shape, std=1.0, mean=0.0):
        return (torch.randn(*shape, generator=gen) * std + mean).to(torch.bfloat16)

    def lin(out, inp, gain=1.0):
        return n(out, inp, std=gain * inp ** -0.5)

    t, w, S = {}, cfg["width"], cfg["streams"]

    def hyper(pre):
        t[pre + ".in"], t[pre + ".out"] = n(S, std=0.3, mean=1.0 / S), n(S, std=0.3, mean=0.8)
        t[pre + ".mix"] = (torch.eye(S) * 0.8 + torch.randn(S, S, generator=gen) * 0.2).to(torch.bfloat16)

    t["embed"], t["bigram"] = n(cfg["vocab"], w), n(cfg["embedding"]["bigram"]["buckets"] + 1, w, std=0.7)
    t["final.norm"] = n(w, std=0.2)
    for i, (layer, mlp) in enumerate(_LAYERS[name]):
        m, p, H, vdim = layer["mixer"], f"l{i}.mix.", layer["mixer"]["heads"], layer["mixer"]["vdim"]
        t[f"l{i}.norm1"] = n(w, std=0.2)
        hyper(f"l{i}.hc1")
        if layer["type"] == "attention":
            G, dim = m["kv_heads"], m["dim"]
            for k, rows in (("q", H * dim), ("k", G * dim), ("v", G * vdim)):
                t[p + k], t[p + k + ".b"] = lin(rows, w), n(rows, std=0.3)
            t[p + "q.norm"], t[p + "k.norm"] = n(dim, std=0.3, mean=sharp), n(dim, std=0.3, mean=1.0)
            t[p + "rel"], t[p + "g"] = n(layer["rows"], H), lin(H, w)
            if m["v_mix"]:
                t[p + "vmix"] = n(1, std=0.2, mean=0.4).reshape(())
            t[p + "o.b"] = n(w, std=0.2)
        else:
            inner, bc = H * vdim, m["groups"] * m["state"]
            t[p + "in"] = lin(2 * inner + 2 * bc + H, w)
            conv = torch.randn(inner + 2 * bc, m["conv"], generator=gen) * 0.4
            conv[:, -1] += 1.0
            t[p + "conv"], t[p + "conv.b"] = conv.to(torch.bfloat16), n(inner + 2 * bc, std=0.2)
            t[p + "A_log"], t[p + "dt_bias"], t[p + "D"] = n(H, std=1.0, mean=-0.5), n(H, mean=-2.0), n(H, mean=1.0)
            t[p + "norm"] = n(inner, std=0.2, mean=1.0)
        t[p + "o"] = lin(w, H * vdim)
        if mlp is not None:
            t[f"l{i}.norm2"] = n(w, std=0.2)
            hyper(f"l{i}.hc2")
            size = mlp["ff"]
            t[f"l{i}.mlp.gate"], t[f"l{i}.mlp.up"], t[f"l{i}.mlp.down"] = lin(size, w, 1.5), lin(size, w, 1.5), lin(w, size)
    return t
