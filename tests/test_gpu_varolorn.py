"""Varolorn on the GPU against the plain float64 statement of the design (oracle/varolorn_oracle.py)."""
import json
import os
import subprocess

import numpy as np
import pytest
import torch

from oracle import varolorn_oracle as O
from tests import varolorn_utils as U
from tests.mixer_utils import DTYPES, LIMIT, OP_LIMIT, close, dev, feed, host

pytestmark = pytest.mark.gpu

ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
# whole models: weighted sums of streams may cancel, which leaves bf16 rounding larger beside the result
MODEL_LIMIT = {torch.float32: 2e-5, torch.bfloat16: 5e-2}
_models = {}


def model_of(name, dtype):
    from dejavu_amd.registry import build_model

    if (name, dtype) not in _models:
        t = U.weights(name)
        _models[name, dtype] = (U.CONFIGS[name], U.as_numpy(t), build_model(U.CONFIGS[name], t, dtype=dtype))
    return _models[name, dtype]


def parts(total, cuts):
    """(first, end) of portions of the sizes in ``cuts``, the last one repeated."""
    at, i = 0, 0
    while at < total:
        n = min(cuts[min(i, len(cuts) - 1)], total - at)
        yield at, at + n
        at, i = at + n, i + 1


def norm_of(width, seed, eps=1e-4):
    from dejavu_amd.mixers import RMSNorm

    m = RMSNorm(width, eps, device="cuda")
    m.weight[:width] = dev(np.random.default_rng(seed).normal(1, 0.3, width))
    w = host(m.weight)[:width]
    return m, lambda x: O.rms(x[..., :width], eps) * w


def connection(streams, seed):
    from dejavu_amd.mixers import HyperConnection

    rng = np.random.default_rng(seed)
    m = HyperConnection(streams, device="cuda")
    m.weights.copy_(dev(rng.normal(size=streams)))
    m.out.copy_(dev(rng.normal(size=streams)))
    m.mix.copy_(dev(rng.normal(size=(streams, streams))))
    return m, {"in": host(m.weights), "out": host(m.out), "mix": host(m.mix)}


def rows_of(h, W):
    """What a sublayer's input amounts to: the product with a matrix."""
    from dejavu_amd import mixer_ops as ops

    return ops.linear(h, W, f32=h.shape[0] == 1)


# ---- mechanisms ---------------------------------------------------------------------------------
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("n,K,M", [(1, 64, 40), (1, 1048, 264), (1, 4104, 16), (1, 5000, 24), (2, 72, 40), (17, 264, 104),
                                   (64, 1032, 200), (65, 96, 40)])
def test_products_with_bias_norm_and_relu_unit(n, K, M, dtype):
    """Biases, the relu-gated unit, and for one token the RMS norm of the row inside the product."""
    from dejavu_amd import mixer_ops as ops

    g = torch.Generator().manual_seed(n * 7 + K)
    x = torch.randn(n, K, generator=g).to(dtype).cuda()
    W = (torch.randn(M, K, generator=g) * K ** -0.5).to(dtype).cuda()
    b = torch.randn(M, generator=g).to(dtype).cuda()
    prod = host(x) @ host(W).T
    close(ops.linear(x, W, b), prod + host(b), OP_LIMIT[dtype], f"product + bias {n}x{K}x{M}")
    if n <= 64 or dtype == torch.bfloat16:
        close(ops.linear(x, W, b, f32=True), prod + host(b), 1e-5, "fp32 result")
    close(ops.relu_glu(x, W), np.maximum(prod[:, 0::2], 0) * prod[:, 1::2], OP_LIMIT[dtype], "relu unit")
    if n == 1:
        norm, f = norm_of(K - 5, 1)
        u = torch.randn(1, K, generator=g).cuda()
        u[:, K - 5:] = 0
        row = ops.RmsRow(u, norm.weight, norm.dim, norm.eps, dtype)
        prod = f(host(u)) @ host(W)[:, :K - 5].T
        close(ops.linear(row, W, b, f32=True), prod + host(b), OP_LIMIT[dtype], "normed row")
        close(ops.relu_glu(row, W), np.maximum(prod[:, 0::2], 0) * prod[:, 1::2], OP_LIMIT[dtype], "normed row, relu unit")


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("streams", [1, 2, 3, 4, 5, 16])
@pytest.mark.parametrize("n,width", [(1, 44), (1, 1500), (2, 44), (33, 264), (70, 1500)])
def test_streams_around_a_sublayer(n, width, streams, dtype):
    """Product, bias, update of all streams from the old ones, the next weighted sum and its norm; then a read alone."""
    from dejavu_amd import mixer_ops as ops

    ws, K = ops.padded(width), 48
    g = torch.Generator().manual_seed(n + streams)
    x = torch.randn(n, streams, ws, generator=g).cuda()
    x[:, :, width:] = 0
    y = torch.randn(n, K, generator=g).to(dtype).cuda()
    W, b = (torch.randn(ws, K, generator=g) * K ** -0.5).to(dtype).cuda(), torch.randn(ws, generator=g).to(dtype).cuda()
    W[width:], b[width:] = 0, 0
    write, wd = connection(streams, 5)
    following, fd = connection(streams, 6)
    norm, f = norm_of(width, 2)
    eye = torch.eye(ws, dtype=dtype, device="cuda")
    for bias in (None, b):
        stream = ops.HyperStream(x.clone(), dtype)
        h = stream.update(y, W, bias, write, ops.StreamRead(norm, following.weights))
        res = host(y) @ host(W).T + (0 if bias is None else host(b))
        want = O.write_streams(host(x).transpose(1, 0, 2), wd, res)
        close(stream.x.reshape(n, -1), want.transpose(1, 0, 2).reshape(n, -1), OP_LIMIT[dtype], "streams")
        read = O.read_streams(want, fd)
        close(rows_of(h, eye)[:, :width], f(read), OP_LIMIT[dtype], "next input")
        assert not rows_of(h, eye)[:, width:].any()
    h = stream.read(ops.StreamRead(norm, write.weights))
    close(rows_of(h, eye)[:, :width], f(O.read_streams(host(stream.x).transpose(1, 0, 2), wd)), OP_LIMIT[dtype], "read")
    close(stream.total(), host(stream.x).sum(1), 1e-6, "sum of the streams")


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("width,streams,buckets", [(44, 3, 31), (1504, 1, 1), (264, 6, 100003)])
def test_embedding_with_the_previous_token(width, streams, buckets, dtype):
    """Whole, in portions and token by token with the position on the device; multipliers beyond 32 bits."""
    from dejavu_amd import mixer_ops as ops

    ws, vocab, T = ops.padded(width), 50, 37
    g = torch.Generator().manual_seed(buckets)
    table, bigram = (torch.randn(r, ws, generator=g).to(dtype).cuda() for r in (vocab, buckets + 1))
    table[:, width:], bigram[:, width:] = 0, 0
    toks = np.random.default_rng(1).integers(0, vocab, T)
    mul = (2 ** 40 + 7, 13)
    want = O.embed(toks.tolist(), host(table)[:, :width], 2.5, host(bigram)[:, :width], *mul)
    norm, f = norm_of(width, 3)
    conn, cd = connection(streams, 4)
    eye = torch.eye(ws, dtype=dtype, device="cuda")
    read = ops.StreamRead(norm, conn.weights)
    for cuts in ([T], [1], [2], [5, 1, 1, 8, 2]):
        history = torch.full((T,), 10 ** 12, dtype=torch.int64, device="cuda")
        xs, hs = [], []
        for lo, hi in parts(T, cuts):
            on_dev = torch.tensor([lo], dtype=torch.int32, device="cuda") if hi - lo == 1 and lo % 2 else None
            stream, h = ops.hyper_embed(torch.tensor(toks[lo:hi], device="cuda"), table, 2.5, bigram, *mul, history,
                                        on_dev, 0 if on_dev is not None else lo, streams, read)
            xs.append(stream.x)
            hs.append(rows_of(h, eye).float())
        x = torch.cat(xs)
        for s in range(streams):
            close(x[:, s, :width], want, 1e-6, f"stream {s}, portions {cuts}")
        close(torch.cat(hs)[:, :width], f(O.read_streams(np.stack([want] * streams), cd)), OP_LIMIT[dtype], "first input")
        assert history.tolist() == toks.tolist()


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("dim,groups", [(30, 2), (96, 3), (44, 44), (512, 2), (1000, 1), (1040, 1), (5120, 1), (8192, 8),
                                        (9216, 36), (774, 3)])
def test_gated_norm_in_groups(dim, groups, dtype):
    """For several rows, and inside the product of one row; the entries behind the last group stay out."""
    from dejavu_amd import mixer_ops as ops

    ps, eps = ops.padded(dim), 1e-4
    rng = np.random.default_rng(dim)
    w = torch.zeros(ps, device="cuda")
    w[:dim] = dev(rng.normal(1, 0.3, dim))
    y = torch.full((5, ps), float("nan"), device="cuda")
    y[:, :dim] = dev(rng.normal(size=(5, dim)) * np.exp(rng.normal(size=(5, 1))))
    z = torch.zeros(5, ps + 16, dtype=dtype, device="cuda")
    z[:, 8:8 + dim] = dev(rng.normal(size=(5, dim)), dtype)
    want = O.grouped_norm(host(y)[:, :dim] * O.silu(host(z)[:, 8:8 + dim]), groups, host(w)[:dim], eps)
    got = ops.gated_group_norm(y, z[:, 8:8 + ps], w, dim, groups, eps)
    close(got[:, :dim], want, OP_LIMIT[dtype], "rows")
    assert not got[:, dim:].any()
    t = (host(y)[:, :dim] * O.silu(host(z)[:, 8:8 + dim]))
    W = torch.randn(24, ps, generator=torch.Generator().manual_seed(1)).mul_(dim ** -0.5).to(dtype).cuda()
    for i in range(2):
        row = torch.full((1, ps), float("nan"), device="cuda")
        row[0, :dim] = dev(t[i])
        got = ops.linear(ops.GroupedRow(row, w, dim, groups, eps, dtype), W)
        close(got, (want[i] @ host(W)[:, :dim].T)[None], OP_LIMIT[dtype], "inside a product")


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("taps", [1, 2, 3, 4, 5])
def test_short_convolution_with_bias(taps, dtype):
    """Eight channels per lane without norms: portions shorter and longer than the taps, token by token, the state."""
    from dejavu_amd import mixer_ops as ops

    rng = np.random.default_rng(taps)
    channels, T = 56, 23
    ut, w, b = dev(rng.normal(size=(T, channels)), dtype), dev(rng.normal(size=(channels, taps))), dev(rng.normal(size=channels))
    want = O.silu(O.causal_conv(host(ut), host(w), host(b)))
    per = 8 if taps <= 4 else channels
    for cuts in ([T], [2], [1, 4, 2, 7, 3]):
        state, got = torch.zeros(channels, max(1, taps - 1), device="cuda"), []
        for lo, hi in parts(T, cuts):
            out = torch.empty(hi - lo, channels, device="cuda")
            ops.short_conv(ut[lo:hi], w, state, [(channels // per, per, per, ops.NORM_NONE, 0.0, 1.0, out)], silu=True,
                           conv_b=b)
            ops.conv_state(ut[lo:hi], channels, taps, state)
            got.append(out)
        close(torch.cat(got), want, 1e-5, f"portions {cuts}")
    W = torch.eye(channels, dtype=dtype, device="cuda")
    state = torch.zeros(channels, max(1, taps - 1), device="cuda")
    close(torch.cat([ops.row_conv(ut[t:t + 1], W, w, state, True, b) for t in range(T)]), want, 1e-5, "token by token")


def ssd_case(T, heads, groups, vdim, state, seed, slow):
    rng = np.random.default_rng(seed)
    x, B, C = rng.normal(size=(T, heads, vdim)), rng.normal(size=(T, groups, state)), rng.normal(size=(T, groups, state))
    logit = rng.normal(size=(T, heads)) - 1.0
    A_log, bias, D = rng.normal(size=heads) * 2 - (4.0 if slow else 0.0), rng.normal(size=heads), rng.normal(size=heads)
    return tuple(host(dev(a)) for a in (x, B, C, logit, A_log, bias, D))


def ssd_rows(x, B, C):
    """Rows x | B | C with the sections padded as the mixer lays them out."""
    T, inner = x.shape[0], x.shape[1] * x.shape[2]
    inner_s, ns = (inner + 7) // 8 * 8, (B.shape[2] + 7) // 8 * 8
    off_b = inner_s
    off_c = off_b + B.shape[1] * ns
    out = np.zeros((T, off_c + B.shape[1] * ns))
    out[:, :inner] = x.reshape(T, -1)
    for at, a in ((off_b, B), (off_c, C)):
        p = np.zeros((T, B.shape[1], ns))
        p[:, :, :B.shape[2]] = a
        out[:, at:at + B.shape[1] * ns] = p.reshape(T, -1)
    return dev(out), off_b, off_c, inner_s, ns


def portion(rows, lo, hi):
    from dejavu_amd import mixer_ops as ops

    out = ops.ssd_rows(hi - lo, rows.shape[1], rows.device)
    out.copy_(rows[lo:hi])
    return out


@pytest.mark.parametrize("heads,groups,vdim,state", [(2, 1, 16, 8), (6, 2, 20, 24), (3, 3, 7, 64), (4, 1, 64, 128), (2, 2, 33, 72),
                                                     (1, 1, 16, 200), (2, 1, 48, 256), (5, 1, 1, 140), (96, 2, 34, 40), (64, 4, 66, 88),
                                                     (192, 3, 6, 136)])
def test_recurrence_of_a_portion_and_of_one_token(heads, groups, vdim, state):
    """Portions of every length around the chunk of 64 with the state carried on, fast and slow decays, then decoding."""
    from dejavu_amd import mixer_ops as ops

    for slow, T in ((False, 150), (True, 150 if heads < 60 else 70)):
        x, B, C, logit, A_log, bias, D = ssd_case(T, heads, groups, vdim, state, vdim + state, slow)
        logit[66, 0] = 40.0  # a head whose state is wiped
        per = lambda a: np.repeat(a, heads // groups, axis=1)  # noqa: E731
        dt = np.logaddexp(0.0, logit + bias)
        rows, off_b, off_c, inner_s, ns = ssd_rows(x, B, C)
        rng = np.random.default_rng(1)
        S0 = host(dev(rng.normal(size=(heads, state, vdim))))
        S = S0.copy()
        want = O.ssd(x, per(B), per(C), dt, np.exp(A_log), D, S)
        rule = (dev(A_log), dev(bias), dev(D))
        start = torch.zeros(heads, vdim, ns, device="cuda")
        start[:, :, :state] = dev(S0.transpose(0, 2, 1))
        cols = torch.zeros(T, heads + 3, device="cuda")
        cols[:, 3:] = dev(logit)
        for cuts in ([T], [2], [1, 63, 64, 3, 1], [65, 64]):
            St = start.clone()
            got = [ops.ssd_scan(portion(rows, lo, hi), cols[lo:hi, 3:], *rule, St, groups, off_b, off_c, inner_s)
                   for lo, hi in parts(T, cuts)]
            close(torch.cat(got)[:, :heads * vdim], want.reshape(T, -1), 1e-5, f"read-outs, portions {cuts}, slow {slow}")
            close(St[:, :, :state].reshape(heads, -1), S.transpose(0, 2, 1).reshape(heads, -1), 1e-5, "state")
            assert not St[:, :, state:].any()
        St, z = start.clone(), host(dev(rng.normal(size=(T, heads * vdim))))
        off_z = rows.shape[1]
        row = torch.cat([rows, torch.zeros(T, inner_s + ops.padded(heads), device="cuda")], 1)
        row[:, off_z:off_z + heads * vdim], row[:, off_z + inner_s:off_z + inner_s + heads] = dev(z), dev(logit)
        got = [ops.ssd_step(row[t:t + 1], *rule, St, groups, off_b, off_c, off_z, off_z + inner_s, inner_s) for t in range(T)]
        close(torch.cat(got)[:, :heads * vdim], want.reshape(T, -1) * O.silu(z), 1e-5, "token by token, gated")
        close(St[:, :, :state].reshape(heads, -1), S.transpose(0, 2, 1).reshape(heads, -1), 1e-5, "state")


def test_recurrence_of_a_long_portion():
    """More tokens than the kernels take at a time, 16-bit step sizes, several heads of a group per workgroup."""
    from dejavu_amd import mixer_ops as ops

    T, heads, groups, vdim, state = 4133, 36, 2, 2, 8
    x, B, C, logit, A_log, bias, D = ssd_case(T, heads, groups, vdim, state, 3, True)
    lt = dev(logit, torch.bfloat16)
    S = np.zeros((heads, state, vdim))
    dt = np.logaddexp(0.0, host(lt) + bias)
    want = np.zeros((T, heads, vdim))
    Bh, Ch = (np.repeat(a, heads // groups, axis=1) for a in (B, C))
    decay = np.exp(-np.exp(A_log) * dt)
    for t in range(T):
        S = decay[t][:, None, None] * S + dt[t][:, None, None] * Bh[t][:, :, None] * x[t][:, None, :]
        want[t] = np.einsum("hnp,hn->hp", S, Ch[t]) + D[:, None] * x[t]
    rows, off_b, off_c, inner_s, ns = ssd_rows(x, B, C)
    St = torch.zeros(heads, vdim, ns, device="cuda")
    got = ops.ssd_scan(portion(rows, 0, T), lt, dev(A_log), dev(bias), dev(D), St, groups, off_b, off_c, inner_s)
    # thousands of products of decays next to 1
    close(got[:, :heads * vdim], want.reshape(T, -1), 5e-5, "read-outs")
    close(St.reshape(heads, -1), S.transpose(0, 2, 1).reshape(heads, -1), 5e-5, "state")


def rel_of(table, far, chunk, T):
    from dejavu_amd.mixers import bias_distances, distance_buckets

    rows = table.shape[0]
    return dev(table[distance_buckets(bias_distances(rows, far, chunk), rows, far)].T.copy())


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("T,H,G,dim,vdim,chunk,rows,far", [
    (150, 4, 2, 24, 40, None, 8, 30), (300, 3, 3, 64, 32, 64, 32, 100), (70, 6, 1, 72, 104, 3, 4, 6),
    (330, 2, 2, 136, 136, 65, 6, 9), (270, 2, 1, 232, 248, 128, 16, 200), (65, 9, 1, 16, 8, 1, 2, 3),
    (90, 2, 1, 264, 40, 20, 5, 9), (400, 1, 1, 56, 64, 300, 10, 40)])
def test_attention_in_chunks_with_a_bias(T, H, G, dim, vdim, chunk, rows, far, dtype):
    """Prompt, portions cut inside chunks, and decoding from rings with norms, mixed values and gates."""
    from dejavu_amd import mixer_ops as ops

    rng = np.random.default_rng(T)
    q, k, v = rng.normal(size=(T, H, dim)) * 2, rng.normal(size=(T, G, dim)), rng.normal(size=(T, G, vdim))
    q, k, v = (host(dev(a, dtype)) for a in (q, k, v))
    table = host(dev(rng.normal(size=(rows, H)) * 2))
    gate = host(dev(rng.normal(size=(T, H)), dtype))
    rel = rel_of(table, far, chunk, T)
    want = O.biased_attention(q, k, v, 0.2, table, far, chunk) * O.sigmoid(gate)[:, :, None]
    qt, kt, vt = (dev(a.reshape(T, -1), dtype) for a in (q, k, v))
    gt = torch.cat([dev(gate, dtype), torch.zeros(T, 16 - H, dtype=dtype, device="cuda")], 1)
    for cuts in ([T], [2, 40, 3, 64, 65]):
        for lo, hi in parts(T, cuts):
            first = lo // chunk * chunk if chunk else 0
            got = ops.portion_attention(qt[lo:hi], kt[first:hi], vt[first:hi], H, G, 0.2, first, lo, gate=gt[lo:hi],
                                        chunk=chunk, rel=rel)
            close(got, want[lo:hi].reshape(hi - lo, -1), OP_LIMIT[dtype], f"rows {lo}..{hi}")
    if dim % 8:
        return
    qw, kw, other, lam = dev(rng.normal(2, 0.3, dim)), dev(rng.normal(1, 0.3, dim)), host(dev(rng.normal(size=v.shape))), 0.3
    kept = [host(dev(a, dtype)) for a in (O.rms(k, 1e-4) * host(kw), 0.7 * v + 0.3 * other)]  # what the rings hold
    want = O.biased_attention(O.rms(q, 1e-4) * host(qw), *kept, 0.2, table, far, chunk) * O.sigmoid(gate)[:, :, None]
    cap = min(chunk or T, T)
    kr, vr = (torch.full((cap, G * d), 1e3, dtype=dtype, device="cuda") for d in (dim, vdim))
    got = []
    for t in range(T):
        row = dev(np.concatenate([a[t].reshape(-1) for a in (q, k, v)]))[None].contiguous()
        on_dev = torch.tensor([t], dtype=torch.int32, device="cuda") if t % 2 else None
        got.append(ops.ring_attention_row(row, kr, vr, H, G, dim, 0.2, 1e-4, on_dev, 0 if t % 2 else t, chunk=chunk, rel=rel,
                                          q_weight=qw, k_weight=kw, gate=dev(gate[t]),
                                          mix_v=(dev(other[t].reshape(-1)), dev([lam]))))
    close(torch.cat(got), want.reshape(T, -1), OP_LIMIT[dtype], "decoded")


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("at,key,chunk", [(127, 64, 64), (128, 127, 64), (128, 64, 64), (191, 128, 64), (99, 90, 10), (100, 99, 10),
                                          (225, 150, 75), (225, 149, 75), (224, 150, 75), (200, 0, None), (64, 63, None),
                                          (5, 5, 6), (6, 5, 6)])
def test_a_single_key_at_the_edge_of_a_chunk(at, key, chunk, dtype):
    """One key takes nearly all the weight of the one query that asks for it, if and only if both lie in one chunk --
    in a prompt, and decoded from a ring that has gone round."""
    from dejavu_amd import mixer_ops as ops

    T, dim, vdim = 230, 16, 8
    rng = np.random.default_rng(at)
    q, k, v = rng.normal(size=(T, 1, dim)) * 0.1, rng.normal(size=(T, 1, dim)) * 0.1, rng.normal(size=(T, 1, vdim))
    k[key, 0], q[at, 0] = 4.0, 4.0
    q, k, v = (host(dev(a, dtype)) for a in (q, k, v))
    table = host(dev(rng.normal(size=(6, 1)) * 0.5))
    want = O.biased_attention(q, k, v, 0.25, table, 40, chunk)
    hit = np.abs(want[at, 0] - v[key, 0]).max() < 0.05
    assert hit == (chunk is None or at // chunk == key // chunk)
    rel = rel_of(table, 40, chunk, T)
    qt, kt, vt = (dev(a.reshape(T, -1), dtype) for a in (q, k, v))
    for lo in (0, at - 1):
        first = lo // chunk * chunk if chunk else 0
        got = ops.portion_attention(qt[lo:], kt[first:], vt[first:], 1, 1, 0.25, first, lo, chunk=chunk, rel=rel)
        close(got, want[lo:].reshape(T - lo, -1), OP_LIMIT[dtype], f"portion from {lo}")
        close(got[at - lo:at - lo + 1], want[at].reshape(1, -1), OP_LIMIT[dtype], "the query")
    cap = min(chunk or T, T)
    kr, vr = (torch.full((cap, d), 1e3, dtype=dtype, device="cuda") for d in (dim, vdim))
    got = [ops.ring_attention_row(torch.cat([qt[t], kt[t], vt[t]]).float()[None].contiguous(), kr, vr, 1, 1, dim, 0.25, 1e-5,
                                  None, t, chunk=chunk, rel=rel) for t in range(T)]
    want = O.biased_attention(O.rms(q, 1e-5), O.rms(k, 1e-5), v, 0.25, table, 40, chunk)  # the decode kernel norms both
    close(torch.cat(got), want.reshape(T, -1), OP_LIMIT[dtype], "decoded")


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("rows,far", [(32, 100), (8, 30), (5, 9)])
def test_every_distance_has_its_bias(rows, far, dtype):
    """Equal keys, a large bias on one row of the table at a time: the weight goes to the distances of that row."""
    from dejavu_amd import mixer_ops as ops

    T = far + 70
    rng = np.random.default_rng(rows)
    v = host(dev(rng.normal(size=(T, 1, 16)), dtype))
    zero = torch.zeros(T, 8, dtype=dtype, device="cuda")
    for hot in range(rows):
        table = np.zeros((rows, 1))
        table[hot] = 12.0
        rel = rel_of(table, far, None, T)
        want = O.biased_attention(np.zeros((T, 1, 8)), np.zeros((T, 1, 8)), v, 1.0, table, far, None)
        vt = dev(v.reshape(T, -1), dtype)
        got = ops.portion_attention(zero, zero, vt, 1, 1, 1.0, 0, 0, rel=rel)
        close(got, want.reshape(T, -1), OP_LIMIT[dtype], f"row {hot}")
        kr, vr = zero.clone(), vt.clone()
        for t in (T - 1, far, far // 2, rows // 2, 0):
            row = torch.cat([zero[t].float(), zero[t].float(), vt[t].float()])[None].contiguous()
            one = ops.ring_attention_row(row, kr, vr, 1, 1, 8, 1.0, 1e-5, None, t, rel=rel)
            close(one, want[t].reshape(1, -1), 2 * OP_LIMIT[dtype], f"row {hot}, decoded at {t}")


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", sorted(U.CONFIGS))
def test_mixers_alone(name, dtype):
    """Every mixer of a configuration: whole prompt, portions, token by token, and a prompt then tokens."""
    from dejavu_amd import mixer_ops as ops
    from dejavu_amd.mixers import StepInfo

    cfg, P, model = model_of(name, dtype)
    T, width, eps = 147, cfg["width"], cfg["norm"]["eps"]
    for i, layer in enumerate(cfg["layers"]):
        mix = model.layers[i].mixer
        rng = np.random.default_rng(i)
        ht = torch.zeros(T, mix.in_proj.shape[1], dtype=dtype, device="cuda")
        ht[:, :width] = dev(rng.normal(size=(T, width)), dtype)
        h, p, first = host(ht)[:, :width], O._sub(P, f"l{i}.mix."), None
        if layer["type"] == "mamba2":
            want = O.mamba2(h, p, layer["mixer"], eps)
        else:
            if mix.values == "mixed":
                first = host(dev(rng.normal(size=(T, mix.kv_heads, mix.vdim)), dtype))
                ft = torch.zeros(T, mix.kv_heads, mix.vdim_s, dtype=dtype, device="cuda")
                ft[:, :, :mix.vdim] = dev(first, dtype)
                ft = ft.view(T, -1)
            want = O.attention(h, p, layer["mixer"], eps, first)[0]
        for cuts in ([T], [2, 3, 2, 62, 8], [1], [128, 1]):
            state, outs = mix.new_state(T), []
            for lo, hi in parts(T, cuts):
                step = StepInfo(lo)
                if first is not None:
                    step.first_values = ft[lo:hi].float() if hi - lo == 1 else ft[lo:hi]
                y = mix(ht[lo:hi], state, step)
                outs.append(ops.linear(y, mix.out_weight, mix.out_bias).float())
            close(torch.cat(outs)[:, :width], want, LIMIT[dtype], f"{name} layer {i} {layer['type']} {cuts}")


# ---- the model ----------------------------------------------------------------------------------
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", sorted(U.CONFIGS))
def test_model_does_not_depend_on_how_a_prompt_is_cut(name, dtype):
    from dejavu_amd.inference import SequencePool

    cfg, P, model = model_of(name, dtype)
    toks = U.tokens(cfg, 140, seed=3)
    residuals = []
    want = O.forward(cfg, P, toks, residuals=residuals)
    pool = SequencePool(141)
    for cuts in ([140], [1], [2], [70, 2, 3, 1, 5, 1], [100, 1], [33, 64, 7]):
        got = feed(model, pool.get("a"), toks, cuts)
        pool.end("a")
        close(got, want, MODEL_LIMIT[dtype], f"{name} portions {cuts}")
    if dtype == torch.float32:
        for cuts in ([140], [139, 1]):
            model.record = []
            feed(model, pool.get("a"), toks, cuts)
            pool.end("a")
            record, model.record = model.record, None
            assert len(record) == len(residuals) * len(cuts)
            for i, w in enumerate(residuals):
                close(torch.cat(record[i::len(residuals)]), w, MODEL_LIMIT[dtype], "sum of the streams")


@pytest.mark.parametrize("dtype", DTYPES)
def test_sequences_side_by_side_and_memory_used_again(dtype):
    """Three unequal sequences fed in turns, each in its own memory, then others in the same memory."""
    from dejavu_amd.inference import SequencePool

    cfg, P, model = model_of("mixed", dtype)
    pool = SequencePool(90)
    for turn in range(2):
        seqs = {n: U.tokens(cfg, ln, seed=10 * turn + ln) for n, ln in (("a", 90), ("b", 37), ("c", 1))}
        want = {n: O.forward(cfg, P, t) for n, t in seqs.items()}
        got, at = {n: [] for n in seqs}, {n: 0 for n in seqs}
        sizes, i = [5, 1, 2, 17, 1, 3], 0
        while any(at[n] < len(seqs[n]) for n in seqs):
            for n in sorted(seqs):
                part = seqs[n][at[n]:at[n] + sizes[i % len(sizes)]]
                i += 1
                if part:
                    got[n].append(feed(model, pool.get(f"{n}{turn}"), part, [len(part)]))
                    at[n] += len(part)
        for n in seqs:
            close(np.concatenate(got[n]), want[n], MODEL_LIMIT[dtype], f"sequence {n}, turn {turn}")
            pool.end(f"{n}{turn}")
    assert len(pool.free) == 3 and not pool.live


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", ["mixed", "one", "many"])
def test_long_decoding_through_generate(name, dtype):
    """Greedy generation, eager and replayed from HIP graphs three times, past several chunks; every score row against
    the oracle fed the same tokens."""
    cfg, P, model = model_of(name, dtype)
    prompt = U.tokens(cfg, 6, seed=9)
    ids, total = torch.tensor([prompt], device="cuda"), 226
    kw = dict(max_length=total, return_dict_in_generate=True, output_scores=True)
    eager = model.generate(ids, **kw)
    want = O.forward(cfg, P, eager.sequences[0].tolist()[:-1])[len(prompt) - 1:]
    close(eager.scores, want, MODEL_LIMIT[dtype], "scores")
    top = np.sort(want, axis=-1)
    clear = top[:, -1] - top[:, -2] > 2 * MODEL_LIMIT[dtype] * np.sqrt((want ** 2).mean())
    assert clear.sum() > 20
    assert (want.argmax(-1) == np.array(eager.sequences[0].tolist()[len(prompt):]))[clear].all()
    for _ in range(3):
        out = model.generate(ids, cg=True, **kw)
        assert torch.equal(out.sequences, eager.sequences) and torch.equal(out.scores, eager.scores)
        other = model.generate(torch.tensor([prompt[::-1]], device="cuda"), **kw)  # eager work in between
        assert not torch.equal(other.scores, eager.scores)
    one = model.generate(ids[:, :1], max_length=20, cg=True, return_dict_in_generate=True, output_scores=True)
    close(one.scores, O.forward(cfg, P, one.sequences[0].tolist()[:-1]), MODEL_LIMIT[dtype], "from one token")


@pytest.mark.parametrize("dtype", ["bfloat16", "float32"])
def test_trace_run_program(tmp_path, dtype):
    """bin/trace_run on a saved model: portions, single tokens, two sequences, one of them in used memory."""
    cfg, t = U.CONFIGS["mixed"], U.weights("mixed", seed=5)
    U.save(tmp_path, cfg, t)
    out = tmp_path / "out"
    out.mkdir()
    a, b = U.tokens(cfg, 40, seed=1), U.tokens(cfg, 25, seed=2)
    steps = [([("a", a[:30], [0, 7, 29])], []), ([("a", a[30:31], [0])], []), ([("a", a[31:], [])], ["a"]),
             ([("b", b[:2], [1])], []), ([("b", b[2:], [22, 3])], ["b"])]
    lines = "".join(json.dumps({"step": i, "end": end, "entries": [{"id": n, "tokens": x, "want": w} for n, x, w in es]})
                    + "\n" for i, (es, end) in enumerate(steps))
    r = subprocess.run([os.path.join(ROOT, "bin", "trace_run"), "--model", str(tmp_path), "--dtype", dtype, "--out",
                        str(out), "--max-tokens", "40"], input=lines, capture_output=True, text=True, timeout=110)
    assert r.returncode == 0, r.stderr[-2000:]
    assert [x for x in r.stdout.splitlines() if x.startswith("done")] == [f"done {i}" for i in range(5)]
    P = U.as_numpy(t)
    la, lb = O.forward(cfg, P, a), O.forward(cfg, P, b)
    read = lambda i: np.fromfile(out / f"{i}.f32", dtype="<f4").reshape(-1, cfg["vocab"])  # noqa: E731
    limit = MODEL_LIMIT[getattr(torch, dtype)]
    close(read(0), la[[0, 7, 29]], limit, "portion")
    close(read(1), la[[30]], limit, "token")
    close(read(3), lb[[1]], limit, "other sequence")
    close(read(4), lb[[24, 5]], limit, "its rest, places in the order asked for")
    assert not (out / "2.f32").exists()
