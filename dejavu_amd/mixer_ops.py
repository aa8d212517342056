"""Tensor interface of libdejavu_mixers.so.

Weights and activations are bf16 or fp32 (one type per model); the residual stream, norms, scores and recurrent state
are fp32.  All ops enqueue on ``torch.cuda.current_stream()`` and refuse CPU tensors.  Products: one row goes to the
row kernel, up to ``TILE_MAX_ROWS`` bf16 rows to the matrix-core kernel, both with the operation that follows in the
same launch; longer portions (and several fp32 rows) take the library GEMM and a separate elementwise launch, as the
dense products of long prompts do elsewhere in this package.
"""
from __future__ import annotations

import ctypes
from typing import Optional

import torch
import torch.nn.functional as F

from . import _lib_mixers as L
from ._lib_mixers import check, lib

TILE_MAX_ROWS = 64

_DTYPES = {torch.bfloat16: L.BF16, torch.float32: L.F32}
_ref = ctypes.byref


def padded(size: int) -> int:
    """Sizes along vectorised dimensions are multiples of 8 in memory."""
    return (size + 7) // 8 * 8


def _code(t: torch.Tensor) -> int:
    if not t.is_cuda:
        raise RuntimeError("dejavu_amd ops run on the GPU only; got a CPU tensor (there is no CPU fallback)")
    return _DTYPES[t.dtype]


def _ptr(t: Optional[torch.Tensor]):
    return None if t is None else t.data_ptr()


def _stream() -> int:
    return torch.cuda.current_stream().cuda_stream


def _f32(*tensors):
    for t in tensors:
        assert t is None or (t.dtype == torch.float32 and t.is_cuda and t.is_contiguous()), "fp32 contiguous expected"


class ResidualStream:
    """The fp32 residual rows of a portion; ``start`` is a copy of the embedding output for models that add it again."""

    def __init__(self, x: torch.Tensor, start: Optional[torch.Tensor], dtype: torch.dtype):
        self.x, self.start, self.dtype = x, start, dtype

    def args(self, post, pre, add_start: bool, h: Optional[torch.Tensor]) -> L.Residual:
        r = L.Residual(x=self.x.data_ptr(), x0=self.start.data_ptr() if add_start else None, h=_ptr(h))
        if post is not None:
            r.post = post.struct()
        if pre is not None:
            r.pre = pre.struct()
        return r

    def new_h(self) -> torch.Tensor:
        return torch.empty(self.x.shape, dtype=self.dtype, device=self.x.device)


def embed(tokens: torch.Tensor, weight: torch.Tensor, norm, keep_start: bool):
    """tokens (n,) int64 -> (ResidualStream, norm(x))."""
    code = _code(weight)
    assert tokens.dtype == torch.int64 and tokens.is_cuda and tokens.is_contiguous() and weight.is_contiguous()
    n, width = tokens.numel(), weight.shape[1]
    x = torch.empty(n, width, dtype=torch.float32, device=weight.device)
    stream = ResidualStream(x, torch.empty_like(x) if keep_start else None, weight.dtype)
    h = stream.new_h()
    check(lib.dv_mix_embed(code, _ptr(tokens), weight.shape[0], _ptr(weight), n, width, _ptr(x), _ptr(stream.start),
                           _ref(norm.struct()), _ptr(h), _stream()), "dv_mix_embed")
    return stream, h


def residual(y: Optional[torch.Tensor], stream: ResidualStream, post, pre, add_start: bool = False):
    """x += post(y) (y may be None); x += start; returns pre(x) (None without ``pre``)."""
    h = None if pre is None else stream.new_h()
    assert y is None or (y.is_contiguous() and y.shape == stream.x.shape and y.dtype == stream.dtype)
    n, width = stream.x.shape
    check(lib.dv_mix_residual(_DTYPES[stream.dtype], _ptr(y), n, width, _ref(stream.args(post, pre, add_start, h)),
                              _stream()), "dv_mix_residual")
    return h


def _tiles(x: torch.Tensor) -> bool:
    return x.dtype == torch.bfloat16 and x.shape[0] <= TILE_MAX_ROWS


def _product_ok(x, W):
    assert x.dim() == 2 and W.dim() == 2 and x.dtype == W.dtype and x.shape[1] == W.shape[1], "product shapes"
    assert x.stride(1) == 1 and W.stride(1) == 1
    return _code(W)


class RmsRow:
    """One fp32 row that still has to be RMS-normed and weighted; the products that read it do that themselves."""

    before = L.ROW_RMS

    def __init__(self, u: torch.Tensor, weight: torch.Tensor, dim: int, eps: float, dtype: torch.dtype):
        _f32(u, weight)
        assert u.shape == (1, weight.numel())
        self.u, self.weight, self.dim, self.eps, self.dtype = u, weight, dim, eps, dtype
        self.shape, self.device = u.shape, u.device

    def fill(self, a: L.RowArgs) -> None:
        a.xw, a.norm_dim, a.eps = self.weight.data_ptr(), self.dim, self.eps


class GroupedRow(RmsRow):
    """The same with ``groups`` equal parts of the first ``dim`` entries, each by its own root mean square."""

    before = L.ROW_GROUPS

    def __init__(self, u, weight, dim, groups, eps, dtype):
        super().__init__(u, weight, dim, eps, dtype)
        self.groups = groups

    def fill(self, a: L.RowArgs) -> None:
        a.xw, a.x_dim, a.norm_dim, a.eps = self.weight.data_ptr(), self.dim, self.dim // self.groups, self.eps


def _row_product(x, W):
    """(code, before, arguments) of the product of one row: a tensor in W's type, or an ``RmsRow``."""
    if not isinstance(x, RmsRow):
        return _product_ok(x, W), L.ROW_PLAIN, _row_args(x, W)
    assert x.shape == (1, W.shape[1]) and W.stride(1) == 1 and x.dtype == W.dtype, "product shapes"
    a = _row_args(x.u, W)
    x.fill(a)
    return _code(W), x.before, a


def _row_launch(code, before, after, a) -> None:
    check(lib.dv_mix_linear_row(code, before, after, _ref(a), _stream()), "dv_mix_linear_row")


def _row_args(x, W) -> L.RowArgs:
    return L.RowArgs(x=x.data_ptr(), W=W.data_ptr(), ldw=W.stride(0), M=W.shape[0], K=W.shape[1])


def _tile_args(x, W) -> L.TileArgs:
    return L.TileArgs(x=x.data_ptr(), ldx=x.stride(0), W=W.data_ptr(), ldw=W.stride(0), n=x.shape[0], M=W.shape[0],
                      K=W.shape[1])


def linear(x, W: torch.Tensor, bias: Optional[torch.Tensor] = None, f32: bool = False) -> torch.Tensor:
    """x (n, K) W (M, K)^T + bias -> (n, M) in x's type, or fp32."""
    n, M = x.shape[0], W.shape[0]
    out_t = torch.float32 if f32 else x.dtype
    assert bias is None or (bias.dtype == W.dtype and bias.shape == (M,) and bias.is_contiguous())
    if n == 1:
        code, before, a = _row_product(x, W)
        out = torch.empty(1, M, dtype=out_t, device=x.device)
        a.out, a.bias = out.data_ptr(), _ptr(bias)
        _row_launch(code, before, L.OUT_F32 if f32 else L.OUT_T, a)
        return out
    code = _product_ok(x, W)
    if _tiles(x) or (f32 and code == L.BF16):
        out = torch.empty(n, M, dtype=out_t, device=x.device)
        a = _tile_args(x, W)
        a.out, a.ldo, a.bias = out.data_ptr(), M, _ptr(bias)
        check(lib.dv_mix_linear_tiles(L.OUT_F32 if f32 else L.OUT_T, _ref(a), _stream()), "dv_mix_linear_tiles")
        return out
    return F.linear(x, W, bias)


def gated_unit(x, W: torch.Tensor, act: int, limit: float = 0.0) -> torch.Tensor:
    """W holds gate and up rows alternately; act: GLU_*.  Returns (n, M / 2)."""
    n, M = x.shape[0], W.shape[0]
    y = torch.empty(n, M // 2, dtype=x.dtype, device=x.device)
    if n == 1:
        code, before, a = _row_product(x, W)
        a.out, a.act, a.limit = y.data_ptr(), act, limit
        _row_launch(code, before, L.OUT_GLU, a)
        return y
    code = _product_ok(x, W)
    if _tiles(x):
        a = _tile_args(x, W)
        a.out, a.ldo, a.act, a.limit = y.data_ptr(), M // 2, act, limit
        check(lib.dv_mix_linear_tiles(L.OUT_GLU, _ref(a), _stream()), "dv_mix_linear_tiles")
    else:
        gu = F.linear(x, W)
        check(lib.dv_mix_glu(code, _ptr(gu), y.numel(), act, limit, _ptr(y), _stream()), "dv_mix_glu")
    return y


def clamped_glu(x, W: torch.Tensor, limit: float) -> torch.Tensor:
    return gated_unit(x, W, L.GLU_CLAMPED, limit)


def relu_glu(x, W: torch.Tensor) -> torch.Tensor:
    return gated_unit(x, W, L.GLU_RELU)


def linear_residual(x: torch.Tensor, W: torch.Tensor, stream: ResidualStream, post, pre, add_start: bool = False):
    """``residual(x W^T, ...)``."""
    code = _product_ok(x, W)
    n = x.shape[0]
    assert stream.x.shape == (n, W.shape[0])
    if n != 1 and not _tiles(x):
        return residual(F.linear(x, W), stream, post, pre, add_start)
    h = None if pre is None else stream.new_h()
    if n == 1:
        a = _row_args(x, W)
        a.res = stream.args(post, pre, add_start, h)
        _row_launch(code, L.ROW_PLAIN, L.OUT_RESIDUAL, a)
    else:
        a = _tile_args(x, W)
        a.res = stream.args(post, pre, add_start, h)
        check(lib.dv_mix_linear_tiles(L.OUT_RESIDUAL, _ref(a), _stream()), "dv_mix_linear_tiles")
    return h


class GatedHeads:
    """fp32 head outputs of one token that still have to be RMS-normed per head, weighted and gated."""

    def __init__(self, o, gate, weight, dim, eps):
        _f32(o, gate, weight)
        self.o, self.gate, self.weight, self.dim, self.eps = o, gate, weight, dim, eps

    def linear_residual(self, W, stream, post, pre, add_start=False):
        h = None if pre is None else stream.new_h()
        a = _row_args(self.o, W)
        a.xw, a.gate, a.eps = self.weight.data_ptr(), self.gate.data_ptr(), self.eps
        a.norm_dim, a.head_stride = self.dim, self.weight.numel()
        a.res = stream.args(post, pre, add_start, h)
        assert self.o.numel() == W.shape[1]
        _row_launch(_code(W), L.ROW_HEADS, L.OUT_RESIDUAL, a)
        return h


class StreamRead:
    """How a sublayer reads several residual streams: their sum weighted by ``weights`` (streams,), RMS-normed with
    ``norm`` (weight (width,), dim, eps)."""

    def __init__(self, norm, weights: torch.Tensor):
        self.norm, self.weights = norm, weights


class HyperStream:
    """Several fp32 residual streams of a portion, x (n, streams, width)."""

    def __init__(self, x: torch.Tensor, dtype: torch.dtype):
        _f32(x)
        assert x.dim() == 3 and x.shape[1] <= L.HYPER_MAX, "streams"
        self.x, self.dtype = x, dtype

    def total(self) -> torch.Tensor:
        return self.x.sum(1)

    def _structs(self, read: StreamRead, normed: bool):
        """Arguments, and the row(s) that ``read`` will hold: fp32 before its norm, or normed."""
        n, streams, width = self.x.shape
        norm = read.norm
        assert read.weights.shape == (streams,) and norm.weight.shape == (width,)
        _f32(read.weights, norm.weight)
        r = L.Hyper(x=self.x.data_ptr(), in_=read.weights.data_ptr(), streams=streams, width=width)
        o = L.RmsOut(w=norm.weight.data_ptr(), eps=norm.eps, dim=norm.dim)
        if normed:
            h = torch.empty(n, width, dtype=self.dtype, device=self.x.device)
            o.h = h.data_ptr()
        else:
            u = torch.empty(n, width, dtype=torch.float32, device=self.x.device)
            r.u = u.data_ptr()
            h = RmsRow(u, norm.weight, norm.dim, norm.eps, self.dtype)
        return r, o, h

    def read(self, read: StreamRead):
        """The input of a sublayer: an ``RmsRow`` for one token, the normed rows for several."""
        n = self.x.shape[0]
        r, o, h = self._structs(read, n > 1)
        check(lib.dv_mix_hyper_rows(_DTYPES[self.dtype], None, n, _ref(r), _ref(o), _stream()), "dv_mix_hyper_rows")
        return h

    def update(self, y, W: torch.Tensor, bias: Optional[torch.Tensor], write, read: StreamRead):
        """The sublayer's result y W^T + bias joins the streams through ``write`` (mix (from, to), out); returns
        ``read`` of them."""
        n, streams, width = self.x.shape
        assert y.shape[0] == n and W.shape[0] == width and write.mix.shape == (streams, streams)
        _f32(write.mix, write.out)
        fused = n == 1 and streams <= L.HYPER_ROW_MAX
        r, o, h = self._structs(read, not fused)
        r.mix, r.out = write.mix.data_ptr(), write.out.data_ptr()
        if fused:
            code, before, a = _row_product(y, W)
            a.hyper, a.bias = r, _ptr(bias)
            _row_launch(code, before, L.OUT_HYPER, a)
        else:
            y = linear(y, W, bias)
            check(lib.dv_mix_hyper_rows(_DTYPES[self.dtype], _ptr(y), n, _ref(r), _ref(o), _stream()),
                  "dv_mix_hyper_rows")
        return h


def hyper_embed(tokens: torch.Tensor, table: torch.Tensor, scale: float, bigram: Optional[torch.Tensor], mul_prev: int,
                mul_cur: int, history: torch.Tensor, pos_dev, pos: int, streams: int, read: StreamRead):
    """tokens (n,) int64 at positions pos ..; history (capacity,) int64 holds the sequence's earlier tokens and takes
    these.  Returns (HyperStream, ``read`` of it)."""
    code = _code(table)
    n, width = tokens.numel(), table.shape[1]
    for t in (tokens, history):
        assert t.dtype == torch.int64 and t.is_cuda and t.is_contiguous()
    assert table.is_contiguous() and (bigram is None or (bigram.is_contiguous() and bigram.dtype == table.dtype and
                                                         bigram.shape[1] == width))
    stream = HyperStream(torch.empty(n, streams, width, dtype=torch.float32, device=table.device), table.dtype)
    r, o, h = stream._structs(read, n > 1)
    e = L.EmbedArgs(tokens=tokens.data_ptr(), history=history.data_ptr(), capacity=history.numel(), vocab=table.shape[0],
                    embed=table.data_ptr(), scale=scale, pos_dev=_ptr(pos_dev), pos_host=pos, n=n)
    if bigram is not None:
        e.bigram, e.buckets, e.mul_prev, e.mul_cur = bigram.data_ptr(), bigram.shape[0] - 1, mul_prev, mul_cur
    check(lib.dv_mix_hyper_embed(code, _ref(e), _ref(r), _ref(o), _stream()), "dv_mix_hyper_embed")
    return stream, h


def head_rows(x: torch.Tensor, groups) -> None:
    """x (n, >= channels): the groups' heads one after the other, each group (heads, stride, dim, what, out) with out
    (n, heads * stride); what: (weight, eps) for an RMS norm per head, (other, lambda) for (1 - lambda) x + lambda
    other, None for a copy."""
    a = L.HeadArgs(in_=x.data_ptr(), ldi=x.stride(0), n=x.shape[0])
    for i, (heads, stride, dim, what, out) in enumerate(groups):
        assert out.shape == (x.shape[0], heads * stride) and out.stride(1) == 1 and out.dtype == x.dtype
        g = L.HeadGroup(heads=heads, stride=stride, dim=dim, out=out.data_ptr(), ld=out.stride(0))
        if what is not None and isinstance(what[1], float):
            _f32(what[0])
            g.w, g.eps = what[0].data_ptr(), what[1]
        elif what is not None:
            other, lam = what
            _f32(lam)
            assert other.shape == out.shape and other.dtype == x.dtype and other.stride(1) == 1
            g.other, g.ldo = other.data_ptr(), other.stride(0)
            setattr(g, "lambda", lam.data_ptr())
        a.g[i] = g
    check(lib.dv_mix_head_rows(_code(x), _ref(a), _stream()), "dv_mix_head_rows")


def gated_group_norm(y: torch.Tensor, z: torch.Tensor, weight: torch.Tensor, dim: int, groups: int, eps: float):
    """t = y silu(z); t / rms(t) * weight per group of dim / groups entries.  y fp32 (n, padded), z (n, padded)."""
    _f32(weight)
    n, padded_dim = z.shape
    assert y.shape == z.shape and y.dtype == torch.float32 and y.stride(1) == z.stride(1) == 1
    out = torch.empty(n, padded_dim, dtype=z.dtype, device=z.device)
    check(lib.dv_mix_gated_group_norm(_code(z), _ptr(y), y.stride(0), _ptr(z), z.stride(0), n, dim, groups, padded_dim,
                                      _ptr(weight), eps, _ptr(out), _stream()), "dv_mix_gated_group_norm")
    return out


def row_conv(x, W: torch.Tensor, conv_w: torch.Tensor, conv_state: torch.Tensor, silu: bool,
             conv_b: Optional[torch.Tensor] = None):
    """One token: the product in fp32; its first conv_w.shape[0] values pass the short convolution (state moved on)."""
    _f32(conv_w, conv_state, conv_b)
    code, before, a = _row_product(x, W)
    out = torch.empty(1, W.shape[0], dtype=torch.float32, device=x.device)
    a.out = out.data_ptr()
    a.conv_w, a.conv_b, a.conv_state = conv_w.data_ptr(), _ptr(conv_b), conv_state.data_ptr()
    a.conv_rows, a.taps, a.silu = conv_w.shape[0], conv_w.shape[1], int(silu)
    _row_launch(code, before, L.OUT_CONV, a)
    return out


def row_rms_linear(x, weight, dim, eps, W, side=None):
    """One token: fp32 (x / rms(x) * weight) W^T.  ``side``: (row, weight, dim, out, seq_pos, position), a second row
    that is normed the same way and stored as row ``position`` of ``out``."""
    _f32(x, weight)
    out = torch.empty(1, W.shape[0], dtype=torch.float32, device=x.device)
    a = _row_args(x, W)
    assert weight.numel() == W.shape[1]
    a.xw, a.norm_dim, a.eps, a.out = weight.data_ptr(), dim, eps, out.data_ptr()
    if side is not None:
        row, w, sdim, dst, pos_dev, pos = side
        a.side_x, a.side_w, a.side_dim, a.side_padded = row.data_ptr(), w.data_ptr(), sdim, w.numel()
        a.side_out, a.side_ld, a.pos_dev, a.pos_host = dst.data_ptr(), dst.stride(0), _ptr(pos_dev), pos
    _row_launch(_code(W), L.ROW_RMS, L.OUT_F32, a)
    return out


def rms_rows(x: torch.Tensor, weight: torch.Tensor, dim: int, eps: float, out: Optional[torch.Tensor] = None):
    code = _code(x)
    n = x.shape[0]
    if out is None:
        out = torch.empty(n, weight.numel(), dtype=x.dtype, device=x.device)
    assert out.dtype == x.dtype and x.stride(1) == out.stride(1) == 1 and out.shape == (n, weight.numel())
    check(lib.dv_mix_rms_rows(code, _ptr(x), x.stride(0), n, dim, weight.numel(), _ptr(weight), eps, _ptr(out),
                              out.stride(0), _stream()), "dv_mix_rms_rows")
    return out


def gated_head_norm(o: torch.Tensor, gate: torch.Tensor, weight: torch.Tensor, dim: int, eps: float):
    """o (n, heads, vdim_s) fp32, gate (n, heads * vdim_s) -> (n, heads * vdim_s)."""
    n, heads, vs = o.shape
    y = torch.empty(n, heads * vs, dtype=gate.dtype, device=o.device)
    check(lib.dv_mix_gated_head_norm(_code(gate), _ptr(o), _ptr(gate), gate.stride(0), n, heads, dim, vs, _ptr(weight),
                                     eps, _ptr(y), _stream()), "dv_mix_gated_head_norm")
    return y


NORM_NONE, NORM_RMS, NORM_UNIT = 0, 1, 2


def short_conv(x: torch.Tensor, conv_w: torch.Tensor, state: torch.Tensor, groups, silu: bool,
               conv_b: Optional[torch.Tensor] = None) -> None:
    """x (n, >= channels): the groups' channels one after the other.  groups: (heads, stride, dim, norm, eps, scale,
    out) with out (n, heads * stride), all fp32 or all of x's type.  The state is read, not moved on."""
    _f32(conv_w, conv_b)
    a = L.ConvArgs(in_=x.data_ptr(), ldi=x.stride(0), n=x.shape[0], taps=conv_w.shape[1], silu=int(silu),
                   w=conv_w.data_ptr(), b=_ptr(conv_b), state=state.data_ptr())
    for i, (heads, stride, dim, norm, eps, scale, out) in enumerate(groups):
        assert out.shape == (x.shape[0], heads * stride) and out.stride(1) == 1
        a.g[i] = L.ConvGroup(heads=heads, stride=stride, dim=dim, norm=norm, eps=eps, scale=scale, out=out.data_ptr(),
                             ld=out.stride(0))
    check(lib.dv_mix_short_conv(_code(x), int(groups[0][6].dtype == torch.float32), _ref(a), _stream()),
          "dv_mix_short_conv")


def conv_state(x: torch.Tensor, channels: int, taps: int, state: torch.Tensor) -> None:
    """Moves the state on by the n rows of x."""
    check(lib.dv_mix_conv_state(_code(x), _ptr(x), x.stride(0), x.shape[0], channels, taps, _ptr(state), _stream()),
          "dv_mix_conv_state")


def ring_copy(buf: torch.Tensor, ring: torch.Tensor, first: int, to_ring: bool) -> None:
    """Rows of buf are tokens first, first + 1, ...; ring (cap, width)."""
    assert buf.dtype == ring.dtype and buf.shape[1] == ring.shape[1]
    check(lib.dv_mix_ring_copy(_code(buf), _ptr(buf), buf.stride(0), _ptr(ring), ring.shape[0], ring.stride(0), first,
                               buf.shape[0], buf.shape[1], int(to_ring), _stream()), "dv_mix_ring_copy")


def decode_splits(keys: int) -> int:
    """Workgroups that share the keys of a decode row.  ``keys`` is the most there can be: the value may not depend
    on the position, which captured steps only know on the device."""
    return max(1, min(16, (keys + 63) // 64), min(128, keys // 128))


def _attn_args(q, k, v, n, H, G, dim_s, vdim_s, scale, sink, gate, window, ring, base, pos_dev, pos):
    a = L.AttnArgs(q=q.data_ptr(), ldq=q.stride(0), k=k.data_ptr(), ldk=k.stride(0), k_head=dim_s, v=v.data_ptr(),
                   ldv=v.stride(0), v_head=vdim_s, n=n, H=H, G=G, dim_s=dim_s, vdim_s=vdim_s, scale=scale,
                   sink=_ptr(sink), window=window or 0, ring=ring, base=base, pos_dev=_ptr(pos_dev), pos_host=pos,
                   splits=1)
    if gate is not None:
        a.gate, a.ldg = gate.data_ptr(), gate.stride(0)
    return a


def _mask_args(a, window, chunk, rel) -> None:
    a.window, a.chunk = window or 0, chunk or 0
    if rel is not None:
        _f32(rel)
        assert rel.dim() == 2 and rel.shape[0] == a.H
        a.rel, a.rel_len = rel.data_ptr(), rel.shape[1]


def portion_attention(q, k, v, heads: int, kv_heads: int, scale: float, first_key: int, pos: int, sink=None, gate=None,
                      window=None, chunk=None, rel=None) -> torch.Tensor:
    """Causal attention of a portion: q (n, heads * dim) at positions pos .., k / v (keys, kv_heads * dim / vdim) from
    token ``first_key`` on.  window: the newest so many tokens are seen; chunk: the tokens of the query's own chunk,
    counted from position 0; rel (heads, distances): added to the scaled scores, its last entry beyond.  bf16 on the
    matrix cores, fp32 (and heads wider than 256) row by row."""
    n, dim_s, vdim_s = q.shape[0], q.shape[1] // heads, v.shape[1] // kv_heads
    out = torch.empty(n, heads * vdim_s, dtype=q.dtype, device=q.device)
    a = _attn_args(q, k, v, n, heads, kv_heads, dim_s, vdim_s, scale, sink, gate, window, 0, first_key, None, pos)
    _mask_args(a, window, chunk, rel)
    a.out = out.data_ptr()
    assert gate is None or gate.dtype == q.dtype
    if q.dtype == torch.bfloat16 and dim_s <= 256 and vdim_s <= 256:
        check(lib.dv_mix_attn_tiles(_ref(a), k.shape[0], _stream()), "dv_mix_attn_tiles")
        return out
    step = 32768  # rows per launch
    for i in range(0, n, step):
        a.n, a.pos_host = min(step, n - i), pos + i
        a.q, a.out = q[i:].data_ptr(), out[i:].data_ptr()
        if gate is not None:
            a.gate = gate[i:].data_ptr()
        check(lib.dv_mix_attn_rows(_code(q), 0, _ref(a), _stream()), "dv_mix_attn_rows")
    return out


def ring_attention_row(row, k_ring, v_ring, heads, kv_heads, dim, scale, eps, pos_dev, pos, sink=None, window=None,
                       chunk=None, rel=None, q_weight=None, k_weight=None, mix_v=None, gate=None):
    """One token of attention over rings of keys and values (cap, kv_heads * stride).  row: fp32 (q, k, v); q and k
    are RMS-normed (times their weights), v mixed with ``mix_v`` = (other fp32 values, lambda), this token's k and v
    stored.  gate: fp32 logits (heads,).  Masks and rel as in ``portion_attention``."""
    _f32(row, sink, q_weight, k_weight)
    dim_s, vdim_s, cap = k_ring.shape[1] // kv_heads, v_ring.shape[1] // kv_heads, k_ring.shape[0]
    out = torch.empty(1, heads * vdim_s, dtype=k_ring.dtype, device=row.device)
    a = _attn_args(row, k_ring, v_ring, 1, heads, kv_heads, dim_s, vdim_s, scale, sink, None, window, cap, 0, pos_dev,
                   pos)
    _mask_args(a, window, chunk, rel)
    a.q_w, a.k_w = _ptr(q_weight), _ptr(k_weight)
    if mix_v is not None:
        _f32(*mix_v)
        assert mix_v[0].numel() == kv_heads * vdim_s
        a.other_v = mix_v[0].data_ptr()
        setattr(a, "lambda", mix_v[1].data_ptr())
    if gate is not None:
        _f32(gate)
        a.gate, a.ldg = gate.data_ptr(), heads
    a.out, a.norm_dim, a.eps = out.data_ptr(), dim, eps
    a.fresh_k = row.data_ptr() + 4 * heads * dim_s
    a.fresh_v = row.data_ptr() + 4 * (heads + kv_heads) * dim_s
    a.splits = decode_splits(cap)
    part = None
    if a.splits > 1:
        part = torch.empty(heads * a.splits * (vdim_s + 2), dtype=torch.float32, device=row.device)
        a.part = part.data_ptr()
    check(lib.dv_mix_attn_rows(_code(k_ring), 1, _ref(a), _stream()), "dv_mix_attn_rows")
    return out


def window_attention_row(row, k_ring, v_ring, heads, kv_heads, dim, scale, eps, sink, window, pos_dev, pos):
    return ring_attention_row(row, k_ring, v_ring, heads, kv_heads, dim, scale, eps, pos_dev, pos, sink=sink, window=window)


def latent_attention_row(q, k_up, v_up, cache, heads, scale, gate, pos_dev, pos):
    """One token of latent attention.  q fp32 (1, heads * dim), k_up (heads * dim, rank), v_up (heads * vdim, rank),
    cache (tokens, rank) whose row for this token is there, gate fp32 logits (heads,)."""
    _f32(q)
    rank, dim_s, vdim_s = cache.shape[1], k_up.shape[0] // heads, v_up.shape[0] // heads
    code = _code(cache)
    ql = torch.empty(heads, rank, dtype=torch.float32, device=q.device)
    check(lib.dv_mix_latent_absorb(code, _ptr(q), _ptr(k_up), heads, dim_s, rank, _ptr(ql), _stream()),
          "dv_mix_latent_absorb")
    a = _attn_args(ql.view(1, -1), cache, cache, 1, heads, 1, rank, rank, scale, None, None, None, 0, 0, pos_dev, pos)
    a.gate, a.ldg = gate.data_ptr(), heads
    a.splits = max(2, min(128, (cache.shape[0] + 127) // 128))
    part = torch.empty(heads * a.splits * (rank + 2), dtype=torch.float32, device=q.device)
    a.part = part.data_ptr()
    out = torch.empty(1, heads * vdim_s, dtype=cache.dtype, device=q.device)
    check(lib.dv_mix_latent_attn(code, _ref(a), _ptr(v_up), vdim_s, _ptr(out), _stream()), "dv_mix_latent_attn")
    return out


def delta_gates(z, b, A_log, dt_bias, heads: int):
    """z (n, heads * dim_s) and b (n, >= heads) logits -> decays (n, heads * dim_s), beta (n, heads), fp32."""
    n, dim_s = z.shape[0], z.shape[1] // heads
    g = torch.empty(n, heads * dim_s, dtype=torch.float32, device=z.device)
    beta = torch.empty(n, heads, dtype=torch.float32, device=z.device)
    check(lib.dv_mix_delta_gates(_code(z), _ptr(z), z.stride(0), _ptr(b), b.stride(0), _ptr(A_log), _ptr(dt_bias), n,
                                 heads, dim_s, _ptr(g), _ptr(beta), _stream()), "dv_mix_delta_gates")
    return g, beta


def delta_scan(q, k, v, g, beta, S, heads: int, kv_heads: int) -> torch.Tensor:
    """The gated delta rule over n tokens; S (heads, vdim_s, dim_s) is updated.  Returns (n, heads, vdim_s) fp32."""
    _f32(q, k, v, g, beta, S)
    n, vs, ds = q.shape[0], S.shape[1], S.shape[2]
    o = torch.empty(n, heads, vs, dtype=torch.float32, device=q.device)
    assert q.shape == k.shape == (n, kv_heads * ds) and v.shape == (n, heads * vs) and g.shape == (n, heads * ds)
    tm = torch.empty((min(n, 4096) + 15) // 16 * heads * (49 * ((ds + 63) // 64 * 64) + 512), dtype=torch.float32,
                     device=q.device)
    a = L.DeltaArgs(q=q.data_ptr(), k=k.data_ptr(), v=v.data_ptr(), g=g.data_ptr(), beta=beta.data_ptr(),
                    S=S.data_ptr(), o=o.data_ptr(), tm=tm.data_ptr(), tm_floats=tm.numel(), n=n, heads=heads, kv_heads=kv_heads, dim_s=ds, vdim_s=vs)
    check(lib.dv_mix_delta_scan(_ref(a), _stream()), "dv_mix_delta_scan")
    return o


def delta_row(row, offsets, heads, kv_heads, dim, decay_up, gate_up, A_log, dt_bias, S):
    """One token of the gated delta rule from the fp32 projection row; returns (o, gate), fp32 (heads * vdim_s,)."""
    _f32(row, A_log, dt_bias, S)
    vs, ds = S.shape[1], S.shape[2]
    o = torch.empty(1, heads * vs, dtype=torch.float32, device=row.device)
    gate = torch.empty(heads * vs, dtype=torch.float32, device=row.device)
    off_k, off_v, off_b, off_a, off_g = offsets
    a = L.DeltaStepArgs(p=row.data_ptr(), off_k=off_k, off_v=off_v, off_b=off_b, off_a=off_a, off_g=off_g, heads=heads,
                        kv_heads=kv_heads, dim=dim, dim_s=ds, vdim_s=vs, Wa=decay_up.data_ptr(),
                        Wg=gate_up.data_ptr(), rank_a=decay_up.shape[1], rank_g=gate_up.shape[1],
                        A_log=A_log.data_ptr(), dt_bias=dt_bias.data_ptr(), S=S.data_ptr(), o=o.data_ptr(),
                        gate=gate.data_ptr())
    check(lib.dv_mix_delta_step(_code(decay_up), _ref(a), _stream()), "dv_mix_delta_step")
    return o, gate


SSD_CHUNK = 64


def ssd_rows(n: int, channels: int, device) -> torch.Tensor:
    """(n, channels) fp32 for ``ssd_scan``: zeros follow up to the end of the last chunk."""
    rows = torch.empty((n + SSD_CHUNK - 1) // SSD_CHUNK * SSD_CHUNK, channels, dtype=torch.float32, device=device)
    if rows.shape[0] > n:
        rows[n:].zero_()
    return rows[:n]


def ssd_scan(xbc, dt, A_log, dt_bias, D, S, groups: int, off_b: int, off_c: int, width: int) -> torch.Tensor:
    """The Mamba-2 recurrence over n tokens; xbc fp32 (n, channels) from ``ssd_rows``: x of all heads, B from column off_b and C from
    off_c on; dt (n, heads) logits of the step sizes.  S (heads, vdim, state) is updated.  Returns fp32 (n, width), of
    which the first heads * vdim columns are written."""
    _f32(xbc, A_log, dt_bias, D, S)
    n, (heads, vdim, state) = xbc.shape[0], S.shape
    chunks = (n + SSD_CHUNK - 1) // SSD_CHUNK
    assert xbc.untyped_storage().nbytes() >= 4 * (xbc.storage_offset() + chunks * SSD_CHUNK * xbc.stride(0)), "ssd_rows"
    assert dt.shape == (n, heads) and dt.stride(1) == 1 and heads * vdim <= width
    assert heads * vdim <= off_b and off_b + groups * state <= off_c and off_c + groups * state <= xbc.shape[1]
    y = torch.empty(n, width, dtype=torch.float32, device=xbc.device)
    tm = torch.empty(min(chunks, 64) * heads * 2688, dtype=torch.float32, device=xbc.device)
    a = L.SsdArgs(xbc=xbc.data_ptr(), ld=xbc.stride(0), off_b=off_b, off_c=off_c, dt=dt.data_ptr(), lddt=dt.stride(0),
                  A_log=A_log.data_ptr(), dt_bias=dt_bias.data_ptr(), D=D.data_ptr(), S=S.data_ptr(), y=y.data_ptr(),
                  ldy=width, tm=tm.data_ptr(), tm_floats=tm.numel(), n=n, heads=heads, groups=groups, vdim=vdim,
                  state_s=state)
    check(lib.dv_mix_ssd_scan(_code(dt), _ref(a), _stream()), "dv_mix_ssd_scan")
    return y


def ssd_step(row, A_log, dt_bias, D, S, groups: int, off_b: int, off_c: int, off_z: int, off_dt: int, width: int):
    """One token of it from the fp32 projection row, also multiplied by silu(z).  Returns fp32 (1, width)."""
    _f32(row, A_log, dt_bias, D, S)
    heads, vdim, state = S.shape
    assert heads * vdim <= width and off_dt + heads <= row.shape[1] and off_z + heads * vdim <= row.shape[1]
    assert max(off_b, off_c) + groups * state <= row.shape[1]
    y = torch.empty(1, width, dtype=torch.float32, device=row.device)
    a = L.SsdStepArgs(p=row.data_ptr(), off_b=off_b, off_c=off_c, off_z=off_z, off_dt=off_dt, A_log=A_log.data_ptr(),
                      dt_bias=dt_bias.data_ptr(), D=D.data_ptr(), S=S.data_ptr(), y=y.data_ptr(), heads=heads,
                      groups=groups, vdim=vdim, state_s=state)
    check(lib.dv_mix_ssd_step(_ref(a), _stream()), "dv_mix_ssd_step")
    return y


def greedy_advance(logits, token, position, seq_pos, sequences, out_index, scores=None, score_index=None) -> None:
    """``ops.greedy_advance`` for fp32 logits."""
    _f32(logits)
    assert logits.dim() == 1
    check(lib.dv_mix_greedy_advance(_ptr(logits), logits.numel(), _ptr(token), _ptr(position), _ptr(seq_pos),
                                    _ptr(sequences), sequences.numel(), _ptr(out_index), _ptr(scores),
                                    0 if scores is None else scores.stride(0),
                                    0 if scores is None else scores.shape[0], _ptr(score_index), _stream()),
          "dv_mix_greedy_advance")
