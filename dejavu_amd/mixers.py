"""Token mixers, norm and feed-forward of decoders whose layers differ in how they mix tokens.

  LatentAttention   low-rank latent cache, no positions, one sigmoid gate per head
  WindowAttention   sliding window, short convolutions on q / k / v, RMS-normed q and k, a sink per head
  ChunkAttention    chunks of positions, learned bias by distance, normed q and k, values mixed with those of an
                    earlier layer, one sigmoid gate per head
  ChannelDelta      gated delta rule with a decay per key channel and an fp32 state
  Mamba2            state-space duality: one decay per head and token, an fp32 state, gated norm in groups
  ClampedGLU        gated feed-forward with clamped gate and value
  ReluGLU           gated feed-forward with a relu gate
  DynamicTanh       norm without statistics: tanh(alpha x) w + b
  RMSNorm           x / rms(x) w
  HyperConnection   how a sublayer reads several residual streams and joins them

A mixer's ``forward`` takes the normed rows h (n, width) of the next n tokens of ONE sequence (one token may come as a
``mixer_ops.RmsRow``, whose norm its products apply) and its state dict, moves the state on, and returns what its output
projection is applied to (a tensor, ``mixer_ops.GatedHeads`` or ``mixer_ops.GroupedRow``); the block applies the
projection together with the norm and the residual add that follow it.  One token runs the decode kernels, several
tokens the portion kernels; a prompt may be cut anywhere.

All sizes along vectorised dimensions are padded to multiples of 8 with zeros in the weights (``*_s`` below), which
leaves every result unchanged; means run over the true sizes.
"""
from __future__ import annotations

from typing import Optional

import torch
import torch.nn as nn

from . import mixer_ops as ops
from .mixer_ops import padded


class StepInfo:
    """Where the rows of a call stand: ``pos`` on the host, ``pos_dev`` on the device for captured decode steps.
    ``first_values``: what a layer leaves of its values for later layers of the same call."""

    def __init__(self, pos: int, pos_dev: Optional[torch.Tensor] = None):
        self.pos, self.pos_dev = pos, pos_dev
        self.first_values: Optional[torch.Tensor] = None


def _weight(rows, cols, dtype, device):
    return nn.Parameter(torch.zeros(rows, cols, dtype=dtype, device=device), requires_grad=False)


def _vector(*shape, device):
    return nn.Parameter(torch.zeros(*shape, dtype=torch.float32, device=device), requires_grad=False)


class DynamicTanh(nn.Module):
    def __init__(self, width: int, device=None):
        super().__init__()
        self.weight = _vector(padded(width), device=device)
        self.bias = _vector(padded(width), device=device)
        self.alpha = _vector(1, device=device)
        self._struct, self._stamp = None, None

    def struct(self):
        """The kernels' argument; alpha is read back once per loaded value."""
        stamp = (self.weight.data_ptr(), self.bias.data_ptr(), self.alpha.data_ptr(), self.alpha._version)
        if self._stamp != stamp:
            self._struct = ops.L.DynTanh(w=self.weight.data_ptr(), b=self.bias.data_ptr(), alpha=float(self.alpha.item()))
            self._stamp = stamp
        return self._struct


class RMSNorm(nn.Module):
    def __init__(self, width: int, eps: float, device=None):
        super().__init__()
        self.dim, self.eps = width, float(eps)
        self.weight = _vector(padded(width), device=device)


class HyperConnection(nn.Module):
    """A sublayer among several residual streams: it reads their sum weighted by ``weights``; they become
    x_t <- sum_s mix[s, t] x_s + out[t] y."""

    def __init__(self, streams: int, device=None):
        super().__init__()
        self.weights = _vector(streams, device=device)
        self.out = _vector(streams, device=device)
        self.mix = _vector(streams, streams, device=device)


class ReluGLU(nn.Module):
    """down(max(gate, 0) up); gate and up rows alternate."""

    def __init__(self, width: int, ff: int, dtype=None, device=None):
        super().__init__()
        self.gate_up = _weight(2 * padded(ff), padded(width), dtype, device)
        self.down = _weight(padded(width), padded(ff), dtype, device)

    def forward(self, h):
        return ops.relu_glu(h, self.gate_up)

    @property
    def out_weight(self):
        return self.down


class ClampedGLU(nn.Module):
    """down(g sigmoid(1.702 g) (u + 1)) with g = min(gate, limit), u = clamp(up); gate and up rows alternate."""

    def __init__(self, width: int, ff: int, limit: float, dtype=None, device=None):
        super().__init__()
        self.limit = float(limit)
        self.gate_up = _weight(2 * padded(ff), padded(width), dtype, device)
        self.down = _weight(padded(width), padded(ff), dtype, device)

    def forward(self, h):
        return ops.clamped_glu(h, self.gate_up, self.limit)

    @property
    def out_weight(self):
        return self.down


class LatentAttention(nn.Module):
    def __init__(self, width, heads, dim, vdim, q_rank, kv_rank, scale, eps, dtype=None, device=None):
        super().__init__()
        self.heads, self.dim, self.vdim, self.q_rank, self.kv_rank = heads, dim, vdim, q_rank, kv_rank
        self.dim_s, self.vdim_s, self.q_rank_s, self.kv_rank_s = (padded(x) for x in (dim, vdim, q_rank, kv_rank))
        self.scale, self.eps = float(scale), float(eps)
        # rows: query latent, key/value latent, one gate per head
        self.in_proj = _weight(self.q_rank_s + self.kv_rank_s + padded(heads), padded(width), dtype, device)
        self.q_norm = _vector(self.q_rank_s, device=device)
        self.kv_norm = _vector(self.kv_rank_s, device=device)
        self.q_up = _weight(heads * self.dim_s, self.q_rank_s, dtype, device)
        self.k_up = _weight(heads * self.dim_s, self.kv_rank_s, dtype, device)
        self.v_up = _weight(heads * self.vdim_s, self.kv_rank_s, dtype, device)
        self.out_proj = _weight(padded(width), heads * self.vdim_s, dtype, device)

    @property
    def out_weight(self):
        return self.out_proj

    def new_state(self, max_len: int):
        w = self.in_proj
        return {"latent": torch.zeros(max_len, self.kv_rank_s, dtype=w.dtype, device=w.device)}

    def forward(self, h, state, step: StepInfo):
        n, qs, ks = h.shape[0], self.q_rank_s, self.kv_rank_s
        cache = state["latent"]
        if n == 1:
            p = ops.linear(h, self.in_proj, f32=True)
            side = (p[0, qs:], self.kv_norm, self.kv_rank, cache, step.pos_dev, step.pos)
            q = ops.row_rms_linear(p, self.q_norm, self.q_rank, self.eps, self.q_up, side)
            return ops.latent_attention_row(q, self.k_up, self.v_up, cache, self.heads, self.scale, p[0, qs + ks:],
                                            step.pos_dev, step.pos)
        p = ops.linear(h, self.in_proj)
        end = step.pos + n
        ops.rms_rows(p[:, qs:qs + ks], self.kv_norm, self.kv_rank, self.eps, out=cache[step.pos:end])
        q = ops.linear(ops.rms_rows(p[:, :qs], self.q_norm, self.q_rank, self.eps), self.q_up)
        c = cache[:end]
        k, v = ops.linear(c, self.k_up), ops.linear(c, self.v_up)
        return ops.portion_attention(q, k, v, self.heads, self.heads, self.scale, 0, step.pos, gate=p[:, qs + ks:])


def _rings(tokens: int, k_width: int, v_width: int, like: torch.Tensor) -> dict:
    """Keys and values of the newest ``tokens`` tokens: token j in row j % tokens."""
    new = lambda width: torch.zeros(tokens, width, dtype=like.dtype, device=like.device)  # noqa: E731
    return {"k": new(k_width), "v": new(v_width)}


def _behind_history(ring, first: int, hist: int, n: int):
    """Rows for tokens first .. first + hist + n - 1, the first ``hist`` of them read from the ring."""
    rows = torch.empty(hist + n, ring.shape[1], dtype=ring.dtype, device=ring.device)
    if hist:
        ops.ring_copy(rows[:hist], ring, first, to_ring=False)
    return rows


def _keep_newest(ring, rows, n: int, end: int) -> None:
    """The last of the n newest rows (tokens up to end - 1) go to the ring."""
    keep = min(n, ring.shape[0])
    ops.ring_copy(rows[rows.shape[0] - keep:], ring, end - keep, to_ring=True)


class WindowAttention(nn.Module):
    def __init__(self, width, heads, kv_heads, dim, vdim, taps, window, scale, eps, dtype=None, device=None):
        super().__init__()
        self.heads, self.kv_heads, self.dim, self.vdim, self.taps = heads, kv_heads, dim, vdim, taps
        self.dim_s, self.vdim_s = padded(dim), padded(vdim)
        self.window, self.scale, self.eps = int(window), float(scale), float(eps)
        self.channels = (heads + kv_heads) * self.dim_s + kv_heads * self.vdim_s
        self.in_proj = _weight(self.channels, padded(width), dtype, device)  # rows: q, k, v
        self.conv = _vector(self.channels, taps, device=device)
        self.sink = _vector(heads, device=device)
        self.out_proj = _weight(padded(width), heads * self.vdim_s, dtype, device)

    @property
    def out_weight(self):
        return self.out_proj

    def new_state(self, max_len: int):
        w = self.in_proj
        return dict(_rings(min(self.window, max_len), self.kv_heads * self.dim_s, self.kv_heads * self.vdim_s, w),
                    conv=torch.zeros(self.channels, max(1, self.taps - 1), dtype=torch.float32, device=w.device))

    def forward(self, h, state, step: StepInfo):
        n, H, G, ds, vs = h.shape[0], self.heads, self.kv_heads, self.dim_s, self.vdim_s
        kr, vr = state["k"], state["v"]
        if n == 1:
            row = ops.row_conv(h, self.in_proj, self.conv, state["conv"], silu=False)
            return ops.window_attention_row(row, kr, vr, H, G, self.dim, self.scale, self.eps, self.sink, self.window,
                                            step.pos_dev, step.pos)
        p = ops.linear(h, self.in_proj)
        hist = min(step.pos, self.window - 1)  # earlier tokens that this portion can still see
        q = torch.empty(n, H * ds, dtype=h.dtype, device=h.device)
        k, v = (_behind_history(r, step.pos - hist, hist, n) for r in (kr, vr))
        ops.short_conv(p, self.conv, state["conv"],
                       [(H, ds, self.dim, ops.NORM_RMS, self.eps, 1.0, q),
                        (G, ds, self.dim, ops.NORM_RMS, self.eps, 1.0, k[hist:]),
                        (G, vs, self.vdim, ops.NORM_NONE, 0.0, 1.0, v[hist:])], silu=False)
        ops.conv_state(p, self.channels, self.taps, state["conv"])
        o = ops.portion_attention(q, k, v, H, G, self.scale, step.pos - hist, step.pos, sink=self.sink,
                                  window=self.window)
        for ring, rows in ((kr, k), (vr, v)):
            _keep_newest(ring, rows, n, step.pos + n)
        return o


def distance_buckets(distances: int, rows: int, far: int) -> list:
    """Row of a bias table for the distances 0, 1, ..: the first rows // 2 distances have a row each, the others share
    the rest of the rows on a logarithmic scale that ends at ``far``.  Decided in integers: step k begins at the first
    n with (n / half)^rest >= (far / half)^k."""
    half = rows // 2
    rest = rows - half
    out, k = [], 0
    for n in range(distances):
        if n < half:
            out.append(n)
            continue
        while k < rest and (far <= half or n ** rest * half ** (k + 1) >= far ** (k + 1) * half ** rest):
            k += 1
        out.append(min(rows - 1, half + k))
    return out


def bias_distances(rows: int, far: int, chunk: Optional[int]) -> int:
    """Distances that need an entry of their own: from the last one on the bias stays what it is."""
    own = max(far, rows // 2) + 1
    return min(own, chunk) if chunk else own


class ChunkAttention(nn.Module):
    """values: None, "first" (this layer's values are left for later layers) or "mixed" (the values are mixed with
    the ones left there)."""

    def __init__(self, width, heads, kv_heads, dim, vdim, chunk, scale, bias_rows, bias_max, values, eps, dtype=None,
                 device=None):
        super().__init__()
        self.heads, self.kv_heads, self.dim, self.vdim = heads, kv_heads, dim, vdim
        self.dim_s, self.vdim_s = padded(dim), padded(vdim)
        self.chunk, self.scale, self.eps, self.values = chunk, float(scale), float(eps), values
        # rows: q, k, v, one gate per head
        self.off_k = heads * self.dim_s
        self.off_v = self.off_k + kv_heads * self.dim_s
        self.off_g = self.off_v + kv_heads * self.vdim_s
        rows = self.off_g + padded(heads)
        self.in_proj = _weight(rows, padded(width), dtype, device)
        self.in_bias = nn.Parameter(torch.zeros(rows, dtype=dtype, device=device), requires_grad=False)
        self.q_norm = _vector(self.dim_s, device=device)
        self.k_norm = _vector(self.dim_s, device=device)
        self.rel = _vector(heads, bias_distances(bias_rows, bias_max, chunk), device=device)  # by distance
        self.vmix = _vector(1, device=device)
        self.out_proj = _weight(padded(width), heads * self.vdim_s, dtype, device)
        self.out_bias = nn.Parameter(torch.zeros(padded(width), dtype=dtype, device=device), requires_grad=False)

    @property
    def out_weight(self):
        return self.out_proj

    def new_state(self, max_len: int):
        tokens = min(self.chunk, max_len) if self.chunk else max_len
        return _rings(tokens, self.kv_heads * self.dim_s, self.kv_heads * self.vdim_s, self.in_proj)

    def forward(self, h, state, step: StepInfo):
        n, H, G, ds, vs = h.shape[0], self.heads, self.kv_heads, self.dim_s, self.vdim_s
        kr, vr = state["k"], state["v"]
        p = ops.linear(h, self.in_proj, self.in_bias, f32=n == 1)
        v_own, gate = p[:, self.off_v:self.off_g], p[:, self.off_g:]
        mix = None
        if self.values == "first":
            step.first_values = v_own
        elif self.values == "mixed":
            mix = (step.first_values, self.vmix)
        if n == 1:
            return ops.ring_attention_row(p, kr, vr, H, G, self.dim, self.scale, self.eps, step.pos_dev, step.pos,
                                          chunk=self.chunk, rel=self.rel, q_weight=self.q_norm, k_weight=self.k_norm,
                                          mix_v=mix, gate=gate[0])
        hist = step.pos % self.chunk if self.chunk else step.pos  # earlier tokens that this portion can still see
        q = torch.empty(n, H * ds, dtype=h.dtype, device=h.device)
        k, v = (_behind_history(r, step.pos - hist, hist, n) for r in (kr, vr))
        ops.head_rows(p, [(H, ds, self.dim, (self.q_norm, self.eps), q), (G, ds, self.dim, (self.k_norm, self.eps), k[hist:]),
                          (G, vs, self.vdim, mix, v[hist:])])
        o = ops.portion_attention(q, k, v, H, G, self.scale, step.pos - hist, step.pos, gate=gate, chunk=self.chunk,
                                  rel=self.rel)
        for ring, rows in ((kr, k), (vr, v)):
            _keep_newest(ring, rows, n, step.pos + n)
        return o


class Mamba2(nn.Module):
    out_bias = None

    def __init__(self, width, heads, groups, vdim, state, taps, norm_groups, eps, dtype=None, device=None):
        super().__init__()
        self.heads, self.groups, self.vdim, self.state, self.taps = heads, groups, vdim, state, taps
        self.norm_groups, self.eps = norm_groups, float(eps)
        self.inner, self.state_s = heads * vdim, padded(state)
        self.inner_s = padded(self.inner)  # the heads lie side by side, padding behind the last one
        # rows: x, B, C (these pass the convolution), z, one step size per head
        self.off_b = self.inner_s
        self.off_c = self.off_b + groups * self.state_s
        self.channels = self.off_c + groups * self.state_s
        self.off_z = self.channels
        self.off_dt = self.off_z + self.inner_s
        self.in_proj = _weight(self.off_dt + padded(heads), padded(width), dtype, device)
        self.conv = _vector(self.channels, taps, device=device)
        self.conv_bias = _vector(self.channels, device=device)
        self.A_log = _vector(heads, device=device)
        self.dt_bias = _vector(heads, device=device)
        self.D = _vector(heads, device=device)
        self.norm = _vector(self.inner_s, device=device)
        self.out_proj = _weight(padded(width), self.inner_s, dtype, device)

    @property
    def out_weight(self):
        return self.out_proj

    def new_state(self, max_len: int):
        dev = self.in_proj.device
        return {"S": torch.zeros(self.heads, self.vdim, self.state_s, dtype=torch.float32, device=dev),
                "conv": torch.zeros(self.channels, max(1, self.taps - 1), dtype=torch.float32, device=dev)}

    def forward(self, h, state, step: StepInfo):
        n = h.shape[0]
        rule = (self.A_log, self.dt_bias, self.D, state["S"], self.groups, self.off_b, self.off_c)
        if n == 1:
            row = ops.row_conv(h, self.in_proj, self.conv, state["conv"], silu=True, conv_b=self.conv_bias)
            y = ops.ssd_step(row, *rule, self.off_z, self.off_dt, self.inner_s)
            return ops.GroupedRow(y, self.norm, self.inner, self.norm_groups, self.eps, h.dtype)
        p = ops.linear(h, self.in_proj)
        xbc = ops.ssd_rows(n, self.channels, h.device)
        per = 8 if self.taps <= 4 else self.channels  # channels that the convolution kernel takes together
        ops.short_conv(p, self.conv, state["conv"], [(self.channels // per, per, per, ops.NORM_NONE, 0.0, 1.0, xbc)],
                       silu=True, conv_b=self.conv_bias)
        ops.conv_state(p, self.channels, self.taps, state["conv"])
        y = ops.ssd_scan(xbc, p[:, self.off_dt:self.off_dt + self.heads], *rule, self.inner_s)
        return ops.gated_group_norm(y, p[:, self.off_z:self.off_dt], self.norm, self.inner, self.norm_groups, self.eps)


class ChannelDelta(nn.Module):
    def __init__(self, width, heads, kv_heads, dim, vdim, taps, decay_rank, gate_rank, eps, dtype=None, device=None):
        super().__init__()
        self.heads, self.kv_heads, self.dim, self.vdim, self.taps = heads, kv_heads, dim, vdim, taps
        self.dim_s, self.vdim_s, self.eps = padded(dim), padded(vdim), float(eps)
        ra, rg = padded(decay_rank), padded(gate_rank)
        self.channels = 2 * kv_heads * self.dim_s + heads * self.vdim_s
        # rows: q, k, v, step size per head, latent of the decay, latent of the output gate
        off_k = kv_heads * self.dim_s
        off_b = self.channels
        off_a = off_b + padded(heads)
        self.offsets = (off_k, 2 * off_k, off_b, off_a, off_a + ra)
        self.in_proj = _weight(off_a + ra + rg, padded(width), dtype, device)
        self.conv = _vector(self.channels, taps, device=device)
        self.decay_up = _weight(heads * self.dim_s, ra, dtype, device)
        self.gate_up = _weight(heads * self.vdim_s, rg, dtype, device)
        self.A_log = _vector(heads, device=device)
        self.dt_bias = _vector(heads * self.dim_s, device=device)
        self.norm = _vector(self.vdim_s, device=device)
        self.out_proj = _weight(padded(width), heads * self.vdim_s, dtype, device)

    @property
    def out_weight(self):
        return self.out_proj

    def new_state(self, max_len: int):
        dev = self.in_proj.device
        return {"S": torch.zeros(self.heads, self.vdim_s, self.dim_s, dtype=torch.float32, device=dev),
                "conv": torch.zeros(self.channels, max(1, self.taps - 1), dtype=torch.float32, device=dev)}

    def forward(self, h, state, step: StepInfo):
        n, H, G, ds, vs = h.shape[0], self.heads, self.kv_heads, self.dim_s, self.vdim_s
        off_k, off_v, off_b, off_a, off_g = self.offsets
        if n == 1:
            row = ops.row_conv(h, self.in_proj, self.conv, state["conv"], silu=True)
            o, gate = ops.delta_row(row, self.offsets, H, G, self.dim, self.decay_up, self.gate_up, self.A_log,
                                    self.dt_bias, state["S"])
            return ops.GatedHeads(o, gate, self.norm, self.vdim, self.eps)
        p = ops.linear(h, self.in_proj)
        f32 = dict(dtype=torch.float32, device=h.device)
        q, k, v = torch.empty(n, G * ds, **f32), torch.empty(n, G * ds, **f32), torch.empty(n, H * vs, **f32)
        ops.short_conv(p, self.conv, state["conv"],
                       [(G, ds, self.dim, ops.NORM_UNIT, 0.0, self.dim ** -0.5, q),
                        (G, ds, self.dim, ops.NORM_UNIT, 0.0, 1.0, k),
                        (H, vs, self.vdim, ops.NORM_NONE, 0.0, 1.0, v)], silu=True)
        ops.conv_state(p, self.channels, self.taps, state["conv"])
        z = ops.linear(p[:, off_a:off_g], self.decay_up)
        g, beta = ops.delta_gates(z, p[:, off_b:], self.A_log, self.dt_bias, H)
        o = ops.delta_scan(q, k, v, g, beta, state["S"], H, G)
        return ops.gated_head_norm(o, ops.linear(p[:, off_g:], self.gate_up), self.norm, self.vdim, self.eps)
