"""Plain CPU statement of the Vimulorn decoder: test infrastructure only.

Vimulorn is a decoder whose layers mix tokens in one of three ways -- attention over a low-rank latent without
positions, a gated delta rule with a decay per key channel, and sliding-window attention with short convolutions and
a sink -- between dynamic-tanh norms, with a clamped gated feed-forward, and with a stretch of layers that is run
several times.  Everything is written for whole sequences, one token after the other, in float64 by default; nothing
here is shared with the device path.

``params`` maps tensor names to numpy arrays; ``config`` is the parsed config.json.
"""
from __future__ import annotations

import numpy as np


def sigmoid(z):
    return 1.0 / (1.0 + np.exp(-z))


def silu(z):
    return z * sigmoid(z)


def softplus(z):
    return np.logaddexp(0.0, z)


def rms_norm(x, eps, weight=None):
    """x / sqrt(mean(x^2) + eps) over the last axis, then an optional weight."""
    y = x / np.sqrt(np.mean(x * x, axis=-1, keepdims=True) + eps)
    return y if weight is None else y * weight


def dynamic_tanh(x, alpha, weight, bias):
    return np.tanh(alpha * x) * weight + bias


def short_conv(u, w):
    """Causal depthwise convolution.  u: (T, channels), w: (channels, taps); the last tap meets the current token."""
    T, taps = u.shape[0], w.shape[1]
    y = np.zeros_like(u)
    for t in range(T):
        for j in range(taps):
            s = t - (taps - 1) + j
            if s >= 0:
                y[t] += w[:, j] * u[s]
    return y


def unit_norm(x):
    return x / np.sqrt(np.sum(x * x, axis=-1, keepdims=True) + 1e-6)


def softmax_attention(q, k, v, scale, window=None, sink=None):
    """q (T, H, dim), k (T, G, dim), v (T, G, vdim) -> (T, H, vdim).  Query i sees keys j with 0 <= i - j < window
    (any j <= i without a window); sink (H,) adds exp(sink) to the denominator."""
    T, H = q.shape[:2]
    G = k.shape[1]
    out = np.zeros((T, H, v.shape[2]), dtype=q.dtype)
    for i in range(T):
        lo = 0 if window is None else max(0, i - window + 1)
        for h in range(H):
            g = h // (H // G)
            s = (k[lo:i + 1, g] @ q[i, h]) * scale
            m = s.max() if sink is None else max(s.max(), sink[h])
            p = np.exp(s - m)
            den = p.sum() + (0.0 if sink is None else np.exp(sink[h] - m))
            out[i, h] = p @ v[lo:i + 1, g] / den
    return out


def latent_attention(h, p, mixer, eps):
    """p: the mixer's tensors without their prefix."""
    T, H, dim, vdim = h.shape[0], mixer["heads"], mixer["dim"], mixer["vdim"]
    cq = rms_norm(h @ p["dq"].T, eps, p["dq.norm"])
    q = (cq @ p["uq"].T).reshape(T, H, dim)
    c = rms_norm(h @ p["dkv"].T, eps, p["dkv.norm"])
    k = (c @ p["uk"].T).reshape(T, H, dim)
    v = (c @ p["uv"].T).reshape(T, H, vdim)
    o = softmax_attention(q, k, v, mixer["scale"])
    o = o * sigmoid(h @ p["g"].T)[:, :, None]
    return o.reshape(T, -1) @ p["o"].T


def window_attention(h, p, mixer, eps):
    T, H, G, dim, vdim = h.shape[0], mixer["heads"], mixer["kv_heads"], mixer["dim"], mixer["vdim"]
    q = rms_norm(short_conv(h @ p["q"].T, p["q.conv"]).reshape(T, H, dim), eps)
    k = rms_norm(short_conv(h @ p["k"].T, p["k.conv"]).reshape(T, G, dim), eps)
    v = short_conv(h @ p["v"].T, p["v.conv"]).reshape(T, G, vdim)
    o = softmax_attention(q, k, v, mixer["scale"], window=mixer["mask"]["size"], sink=p["sink"])
    return o.reshape(T, -1) @ p["o"].T


def delta_rule(q, k, v, g, beta, S):
    """q, k, g (T, heads, dim), v (T, heads, vdim), beta (T, heads), S (heads, dim, vdim), which is updated in place.
    Returns the read-outs (T, heads, vdim)."""
    T, H = beta.shape
    out = np.zeros(v.shape, dtype=v.dtype)
    for t in range(T):
        for h in range(H):
            S[h] *= g[t, h][:, None]
            u = beta[t, h] * (v[t, h] - S[h].T @ k[t, h])
            S[h] += np.outer(k[t, h], u)
            out[t, h] = S[h].T @ q[t, h]
    return out


def channel_delta(h, p, mixer, eps):
    T, H, G, dim, vdim = h.shape[0], mixer["heads"], mixer["kv_heads"], mixer["dim"], mixer["vdim"]
    rep = H // G
    q = silu(short_conv(h @ p["q"].T, p["q.conv"])).reshape(T, G, dim)
    k = silu(short_conv(h @ p["k"].T, p["k.conv"])).reshape(T, G, dim)
    v = silu(short_conv(h @ p["v"].T, p["v.conv"])).reshape(T, H, vdim)
    q = np.repeat(unit_norm(q) * dim ** -0.5, rep, axis=1)
    k = np.repeat(unit_norm(k), rep, axis=1)
    beta = sigmoid(h @ p["b"].T)
    z = ((h @ p["a1"].T) @ p["a2"].T + p["dt_bias"]).reshape(T, H, dim)
    g = np.exp(-np.exp(p["A_log"])[None, :, None] * softplus(z))
    o = delta_rule(q, k, v, g, beta, np.zeros((H, dim, vdim), dtype=h.dtype))
    o = rms_norm(o, eps, p["norm"])
    o = o * sigmoid((h @ p["g1"].T) @ p["g2"].T).reshape(T, H, vdim)
    return o.reshape(T, -1) @ p["o"].T


MIXERS = {"latent_attention": latent_attention, "channel_delta": channel_delta, "attention": window_attention}


def clamped_glu(h, p, limit):
    g = np.minimum(h @ p["gate"].T, limit)
    u = np.clip(h @ p["up"].T, -limit, limit)
    return (g * sigmoid(1.702 * g) * (u + 1.0)) @ p["down"].T


def _sub(params, prefix):
    return {k[len(prefix):]: v for k, v in params.items() if k.startswith(prefix)}


def layer_runs(config):
    """[(layer, first of a repeated pass)] in the order of execution."""
    n = len(config["layers"])
    loop = config.get("loop")
    if not loop:
        return [(i, False) for i in range(n)]
    a, b, times = loop["start"], loop["stop"], loop["times"]
    runs = [(i, False) for i in range(a)]
    for t in range(times):
        runs += [(i, t > 0 and i == a) for i in range(a, b)]
    return runs + [(i, False) for i in range(b, n)]


def forward(config, params, tokens, dtype=np.float64, residuals=None):
    """tokens (T,) -> logits (T, vocab).  ``residuals``: a list that receives the residual stream after every layer."""
    P = {k: np.asarray(v).astype(dtype) for k, v in params.items()}
    eps = config["norm"]["eps"]

    def norm(x, name):
        return dynamic_tanh(x, P[name + ".alpha"].reshape(()), P[name], P[name + ".b"])

    x0 = P["embed"][np.asarray(tokens)]
    x = x0.copy()
    for i, again in layer_runs(config):
        spec, l = config["layers"][i], f"l{i}."
        if again:
            x = x + x0
        y = MIXERS[spec["type"]](norm(x, l + "norm1"), _sub(P, l + "mix."), spec["mixer"], eps)
        x = x + norm(y, l + "norm1b")
        if spec.get("mlp") is not None:
            y = clamped_glu(norm(x, l + "norm2"), _sub(P, l + "mlp."), spec["mlp"]["limit"])
            x = x + norm(y, l + "norm2b")
        if residuals is not None:
            residuals.append(x.copy())
    return norm(x, "final.norm") @ P["head"].T
