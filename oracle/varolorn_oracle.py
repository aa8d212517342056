"""Plain CPU statement of the Varolorn decoder: test infrastructure only.

Varolorn is a decoder whose layers mix tokens by chunk-local attention (a learned bias by distance instead of a
rotation, values mixed with those of an earlier layer, a gate per head) or by a Mamba-2 recurrence, around several
residual streams that every sublayer reads as a weighted sum and writes back through a small matrix.  Tokens are
embedded together with their predecessor.  Everything is written for whole sequences, one token after the other, in
float64 by default; nothing here is shared with the device path.

``params`` maps tensor names to numpy arrays; ``config`` is the parsed config.json.
"""
from __future__ import annotations

import numpy as np


def sigmoid(z):
    return 1.0 / (1.0 + np.exp(-z))


def silu(z):
    return z * sigmoid(z)


def rms(x, eps):
    """x over its root mean square, along the last axis."""
    return x / np.sqrt((x * x).mean(axis=-1, keepdims=True) + eps)


def zero_centred_norm(x, w, eps):
    return rms(x, eps) * (1.0 + w)


def embed(tokens, table, scale, bigram, mul_prev, mul_cur):
    """bigram has one row per bucket and a last one for the first token of a sequence."""
    buckets = bigram.shape[0] - 1
    out = np.zeros((len(tokens), table.shape[1]), dtype=table.dtype)
    for i, t in enumerate(tokens):
        row = buckets if i == 0 else (int(tokens[i - 1]) * mul_prev + int(t) * mul_cur) % buckets
        out[i] = table[t] * scale + bigram[row]
    return out


def distance_bucket(n, rows, far):
    """Row of the bias table for distance n: the first half of the rows one by one, the rest on a logarithmic scale up
    to ``far``.  The logarithmic part counts the steps k with (far / half)^(k / rest) <= n / half in exact integers."""
    half = rows // 2
    if n < half:
        return n
    rest = rows - half
    if far <= half:
        return rows - 1
    k = 0
    while k < rest and (far ** (k + 1)) * half ** rest <= n ** rest * half ** (k + 1):
        k += 1
    return min(rows - 1, half + k)


def biased_attention(q, k, v, scale, table, far, chunk):
    """q (T, H, dim), k (T, G, dim), v (T, G, vdim); table (rows, H).  Query i sees the keys j <= i of its own chunk
    (of all, without a chunk size)."""
    T, H = q.shape[:2]
    rep = H // k.shape[1]
    reach = min(T, chunk) if chunk else T
    bias = np.stack([table[distance_bucket(n, table.shape[0], far)] for n in range(reach)])  # (distance, H)
    out = np.zeros((T, H, v.shape[2]), dtype=q.dtype)
    for i in range(T):
        lo = i // chunk * chunk if chunk else 0
        for h in range(H):
            s = (k[lo:i + 1, h // rep] @ q[i, h]) * scale + bias[i - lo::-1, h]
            p = np.exp(s - s.max())
            out[i, h] = p @ v[lo:i + 1, h // rep] / p.sum()
    return out


def attention(h, p, mixer, eps, v_first=None):
    """p: the mixer's tensors without their prefix; v_first: the values to mix in (None: none).  Returns the output and
    the layer's values before mixing."""
    T, H, G, dim, vdim = h.shape[0], mixer["heads"], mixer["kv_heads"], mixer["dim"], mixer["vdim"]
    q = (h @ p["q"].T + p["q.b"]).reshape(T, H, dim)
    k = (h @ p["k"].T + p["k.b"]).reshape(T, G, dim)
    v = (h @ p["v"].T + p["v.b"]).reshape(T, G, vdim)
    own = v
    if v_first is not None:
        lam = float(np.asarray(p["vmix"]).reshape(()))
        v = (1.0 - lam) * v + lam * v_first
    q, k = rms(q, eps) * p["q.norm"], rms(k, eps) * p["k.norm"]
    o = biased_attention(q, k, v, mixer["scale"], p["rel"], mixer["bias_max"], (mixer.get("mask") or {}).get("size"))
    o = o * sigmoid(h @ p["g"].T)[:, :, None]
    return o.reshape(T, H * vdim) @ p["o"].T + p["o.b"], own


def causal_conv(u, w, b):
    """u (T, channels), w (channels, taps) with the current token's tap last, zeros before the start."""
    T, taps = u.shape[0], w.shape[1]
    y = np.tile(np.asarray(b, dtype=u.dtype), (T, 1))
    for j in range(taps):
        back = taps - 1 - j
        if back < T:
            y[back:] += w[:, j] * u[:T - back]
    return y


def ssd(x, B, C, dt, A, D, S):
    """x (T, H, P), B and C (T, H, N), dt (T, H) step sizes, A (H,) positive rates, S (H, N, P) updated in place."""
    y = np.zeros_like(x)
    for t in range(x.shape[0]):
        for h in range(x.shape[1]):
            S[h] = np.exp(-A[h] * dt[t, h]) * S[h] + dt[t, h] * np.outer(B[t, h], x[t, h])
            y[t, h] = S[h].T @ C[t, h] + D[h] * x[t, h]
    return y


def grouped_norm(y, groups, w, eps):
    T, n = y.shape
    return rms(y.reshape(T, groups, n // groups), eps).reshape(T, n) * w


def mamba2(h, p, mixer, eps):
    T, H, P, N, G = h.shape[0], mixer["heads"], mixer["vdim"], mixer["state"], mixer["groups"]
    inner, bc = H * P, G * N
    u = h @ p["in"].T
    z, xbc, dt = u[:, :inner], u[:, inner:2 * inner + 2 * bc], u[:, 2 * inner + 2 * bc:]
    xbc = silu(causal_conv(xbc, p["conv"], p["conv.b"]))
    x = xbc[:, :inner].reshape(T, H, P)
    per_head = lambda a: np.repeat(a.reshape(T, G, N), H // G, axis=1)  # noqa: E731
    B, C = per_head(xbc[:, inner:inner + bc]), per_head(xbc[:, inner + bc:])
    dt = np.logaddexp(0.0, dt + p["dt_bias"])
    y = ssd(x, B, C, dt, np.exp(p["A_log"]), p["D"], np.zeros((H, N, P), dtype=h.dtype))
    y = y.reshape(T, inner) * silu(z)
    return grouped_norm(y, mixer["norm_groups"], p["norm"], eps) @ p["o"].T


def relu_glu(h, p):
    return (np.maximum(h @ p["gate"].T, 0.0) * (h @ p["up"].T)) @ p["down"].T


def read_streams(streams, hc):
    """streams (s, T, width)"""
    return np.tensordot(hc["in"], streams, axes=1)


def write_streams(streams, hc, y):
    """Every stream becomes a mix of the old ones (matrix indexed [from, to]) and takes its share of y."""
    return np.stack([sum(hc["mix"][s, t] * streams[s] for s in range(len(streams))) + hc["out"][t] * y
                     for t in range(len(streams))])


def _sub(params, prefix):
    return {k[len(prefix):]: v for k, v in params.items() if k.startswith(prefix)}


def forward(config, params, tokens, dtype=np.float64, residuals=None):
    """tokens (T,) -> logits (T, vocab).  ``residuals``: a list that receives the sum of the streams after every layer."""
    P = {k: np.asarray(v).astype(dtype) for k, v in params.items()}
    eps, emb = config["norm"]["eps"], config["embedding"]
    big = emb["bigram"]
    x = embed(tokens, P["embed"], emb["scale"], P["bigram"], big["mul_prev"], big["mul_cur"])
    streams = np.stack([x] * config["streams"])
    v_first = None
    for i, spec in enumerate(config["layers"]):
        p = _sub(P, f"l{i}.")

        def sublayer(q, fn):
            hc = _sub(p, f"hc{q}.")
            return write_streams(streams, hc, fn(zero_centred_norm(read_streams(streams, hc), p[f"norm{q}"], eps)))

        def mix(h):
            nonlocal v_first
            m = _sub(p, "mix.")
            if spec["type"] == "mamba2":
                return mamba2(h, m, spec["mixer"], eps)
            mixes = spec["mixer"].get("v_mix")
            y, own = attention(h, m, spec["mixer"], eps, v_first if mixes else None)
            if mixes and v_first is None:
                v_first = own
            return y

        streams = sublayer(1, mix)
        if spec.get("mlp") is not None:
            streams = sublayer(2, lambda h: relu_glu(h, _sub(p, "mlp.")))
        if residuals is not None:
            residuals.append(streams.sum(axis=0))
    return zero_centred_norm(streams.sum(axis=0), P["final.norm"], eps) @ P["embed"].T
