"""Token mixers, norm and feed-forward of decoders whose layers differ in how they mix tokens.

  LatentAttention   low-rank latent cache, no positions, one sigmoid gate per head
  WindowAttention   sliding window, short convolutions on q / k / v, RMS-normed q and k, a sink per head
  ChannelDelta      gated delta rule with a decay per key channel and an fp32 state
  ClampedGLU        gated feed-forward with clamped gate and value
  DynamicTanh       norm without statistics: tanh(alpha x) w + b

A mixer's ``forward`` takes the normed rows h (n, width) of the next n tokens of ONE sequence and its state dict, moves
the state on, and returns what its output projection is applied to (a tensor, or ``mixer_ops.GatedHeads``); the block
applies the projection together with the norm and the residual add that follow it.  One token runs the decode
kernels, several tokens the portion kernels; a prompt may be cut anywhere.

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
    """Where the rows of a call stand: ``pos`` on the host, ``pos_dev`` on the device for captured decode steps."""

    def __init__(self, pos: int, pos_dev: Optional[torch.Tensor] = None):
        self.pos, self.pos_dev = pos, pos_dev


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
        cap = min(self.window, max_len)
        return {"k": torch.zeros(cap, self.kv_heads * self.dim_s, dtype=w.dtype, device=w.device),
                "v": torch.zeros(cap, self.kv_heads * self.vdim_s, dtype=w.dtype, device=w.device),
                "conv": torch.zeros(self.channels, max(1, self.taps - 1), dtype=torch.float32, device=w.device)}

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
        k = torch.empty(hist + n, G * ds, dtype=h.dtype, device=h.device)
        v = torch.empty(hist + n, G * vs, dtype=h.dtype, device=h.device)
        if hist:
            ops.ring_copy(k[:hist], kr, step.pos - hist, to_ring=False)
            ops.ring_copy(v[:hist], vr, step.pos - hist, to_ring=False)
        ops.short_conv(p, self.conv, state["conv"],
                       [(H, ds, self.dim, ops.NORM_RMS, self.eps, 1.0, q),
                        (G, ds, self.dim, ops.NORM_RMS, self.eps, 1.0, k[hist:]),
                        (G, vs, self.vdim, ops.NORM_NONE, 0.0, 1.0, v[hist:])], silu=False)
        ops.conv_state(p, self.channels, self.taps, state["conv"])
        o = ops.portion_attention(q, k, v, H, G, self.scale, step.pos - hist, step.pos, sink=self.sink,
                                  window=self.window)
        keep = min(n, kr.shape[0])
        ops.ring_copy(k[hist + n - keep:], kr, step.pos + n - keep, to_ring=True)
        ops.ring_copy(v[hist + n - keep:], vr, step.pos + n - keep, to_ring=True)
        return o


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
