"""Vimulorn on the GPU against the plain float64 statement of the design (oracle/vimulorn_oracle.py)."""
import json
import os
import subprocess

import numpy as np
import pytest
import torch

from oracle import vimulorn_oracle as V
from tests import vimulorn_utils as U
from tests.mixer_utils import DTYPES, LIMIT, OP_LIMIT, close, dev, feed, host

pytestmark = pytest.mark.gpu

ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
_models = {}


def model_of(name, dtype, seed=0, **kw):
    from dejavu_amd.registry import build_model

    key = (name, dtype, seed, tuple(kw.items()))
    if key not in _models:
        cfg = U.CONFIGS[name]
        t = U.weights(cfg, seed=seed, ranks=U.RANKS[name], **kw)
        _models[key] = (cfg, U.as_numpy(t), build_model(cfg, t, dtype=dtype))
    return _models[key]


# ---- mechanisms ---------------------------------------------------------------------------------
def _norm(width, seed):
    from dejavu_amd.mixers import DynamicTanh

    rng = np.random.default_rng(seed)
    w, b, a = rng.normal(1, 0.2, width), rng.normal(0, 0.2, width), 0.7
    m = DynamicTanh(width, device="cuda")
    m.weight[:width], m.bias[:width], m.alpha[0] = dev(w), dev(b), a
    return m, lambda x: V.dynamic_tanh(x, a, dev(w).cpu().numpy().astype(np.float64), dev(b).cpu().numpy().astype(np.float64))


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("n,K,M", [(1, 64, 40), (1, 1048, 264), (2, 72, 40), (3, 520, 64), (17, 264, 104), (33, 128, 72),
                                   (64, 1032, 200), (65, 96, 40), (150, 64, 48)])
def test_products_and_what_follows_them(n, K, M, dtype):
    """Plain product, clamped gated unit, and norm + residual (+ start) + next norm, for every kind of portion."""
    from dejavu_amd import mixer_ops as ops

    g = torch.Generator().manual_seed(n * 7 + K)
    x = torch.randn(n, K, generator=g).to(dtype).cuda()
    W = (torch.randn(M, K, generator=g) * K ** -0.5).to(dtype).cuda()
    prod = host(x) @ host(W).T
    close(ops.linear(x, W), prod, OP_LIMIT[dtype], f"product {n}x{K}x{M}")
    if n <= 64 or dtype == torch.bfloat16:
        close(ops.linear(x, W, f32=True), prod, 1e-5, "product, fp32 result")
    y = ops.clamped_glu(x, W * 2, 0.75)
    gate, up = np.minimum(2 * prod[:, 0::2], 0.75), np.clip(2 * prod[:, 1::2], -0.75, 0.75)
    close(y, gate * V.sigmoid(1.702 * gate) * (up + 1), OP_LIMIT[dtype], "clamped gated unit")
    (post, f_post), (pre, f_pre) = _norm(M, 1), _norm(M, 2)
    for add_start in (False, True):
        x0 = torch.randn(n, M, generator=g).cuda()
        start = torch.randn(n, M, generator=g).cuda()
        stream = ops.ResidualStream(x0.clone(), start, dtype)
        h = ops.linear_residual(x, W, stream, post, pre, add_start)
        want = host(x0) + f_post(prod) + (host(start) if add_start else 0.0)
        close(stream.x, want, OP_LIMIT[dtype], "residual")
        close(h, f_pre(want), OP_LIMIT[dtype], "next norm")
    assert ops.linear_residual(x, W, stream, post, None) is None


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("taps", [1, 2, 3, 5])
def test_short_convolution_in_portions_and_token_by_token(taps, dtype):
    """Filtered values, head norms and the state, for portions shorter and longer than the taps."""
    from dejavu_amd import mixer_ops as ops

    rng = np.random.default_rng(taps)
    heads, ds, dim, T = (3, 2, 2), (16, 16, 8), (13, 13, 8), 23
    channels = sum(h * d for h, d in zip(heads, ds))
    W = torch.eye(channels, dtype=dtype, device="cuda")
    u = rng.normal(size=(T, channels))
    w = rng.normal(size=(channels, taps))
    at = 0
    for h, s, d in zip(heads, ds, dim):  # padding channels are zero, as the loader leaves them
        for i in range(h):
            w[at + i * s + d:at + (i + 1) * s] = 0
        at += h * s
    ut, wt = dev(u, dtype), dev(w)
    full = V.silu(V.short_conv(host(ut), host(wt)))
    q = full[:, :48].reshape(T, 3, 16)[:, :, :13]
    k = full[:, 48:80].reshape(T, 2, 16)[:, :, :13]
    want = (V.rms_norm(q, 1e-4), V.unit_norm(k) * 0.3, full[:, 80:].reshape(T, 2, 8))
    for cuts in ([T], [2], [1, 4, 2, 7, 3]):
        state = torch.zeros(channels, max(1, taps - 1), device="cuda")
        got, at, i = [[], [], []], 0, 0
        while at < T:
            n = min(cuts[min(i, len(cuts) - 1)], T - at)
            p = ut[at:at + n]
            outs = [torch.empty(n, h * s, device="cuda") for h, s in zip(heads, ds)]
            ops.short_conv(p, wt, state, [(3, 16, 13, ops.NORM_RMS, 1e-4, 1.0, outs[0]),
                                          (2, 16, 13, ops.NORM_UNIT, 0.0, 0.3, outs[1]),
                                          (2, 8, 8, ops.NORM_NONE, 0.0, 1.0, outs[2])], silu=True)
            ops.conv_state(p, channels, taps, state)
            for j in range(3):
                got[j].append(outs[j])
            at, i = at + n, i + 1
        for j, name in enumerate(("rms", "unit", "plain")):
            r = host(torch.cat(got[j])).reshape(T, heads[j], ds[j])
            close(r[:, :, :dim[j]].reshape(T, -1), want[j].reshape(T, -1), 1e-5, f"{name}, portions {cuts}")
            assert not r[:, :, dim[j]:].any()
        if taps > 1:
            np.testing.assert_array_equal(host(state), host(ut)[-(taps - 1):].T)
    state = torch.zeros(channels, max(1, taps - 1), device="cuda")
    rows = [ops.row_conv(ut[t:t + 1], W, wt, state, silu=True) for t in range(T)]
    close(torch.cat(rows), full, 1e-5, "token by token")


def _attention_case(T, H, G, dim, vdim, seed=0, sharp=1.0):
    rng = np.random.default_rng(seed)
    return rng.normal(size=(T, H, dim)) * sharp, rng.normal(size=(T, G, dim)), rng.normal(size=(T, G, vdim))


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("T,H,G,dim,vdim,window", [(150, 4, 2, 24, 40, None), (300, 3, 3, 64, 32, 64), (70, 6, 1, 72, 104, 3),
                                                   (129, 2, 2, 136, 136, 65), (260, 2, 1, 232, 248, 128), (65, 9, 1, 16, 8, 1),
                                                   (90, 2, 1, 264, 40, 20)])
def test_portion_attention(T, H, G, dim, vdim, window, dtype):
    """Windows shorter and longer than a key tile, a sink and a gate, and the same rows in portions with the earlier
    keys in front."""
    from dejavu_amd import mixer_ops as ops

    q, k, v = (host(dev(a, dtype)) for a in _attention_case(T, H, G, dim, vdim, seed=T, sharp=2.0))
    sink, gate = np.linspace(-1, 3, H), host(dev(np.random.default_rng(1).normal(size=(T, H)), dtype))
    want = V.softmax_attention(q, k, v, 0.2, window=window, sink=host(dev(sink))) * V.sigmoid(gate)[:, :, None]
    qt, kt, vt, gt = (dev(a.reshape(T, -1), dtype) for a in (q, k, v, gate))
    gt = torch.cat([gt, torch.zeros(T, 16 - H, dtype=dtype, device="cuda")], 1)
    run = lambda lo, hi, first: ops.portion_attention(  # noqa: E731
        qt[lo:hi], kt[first:hi], vt[first:hi], H, G, 0.2, first, lo, sink=dev(sink), gate=gt[lo:hi], window=window)
    close(run(0, T, 0), want.reshape(T, -1), OP_LIMIT[dtype], "whole")
    lo = 0
    for n in (2, 40, 3, T):
        hi = min(T, lo + n)
        first = 0 if window is None else max(0, lo - window + 1)
        close(run(lo, hi, first), want[lo:hi].reshape(hi - lo, -1), OP_LIMIT[dtype], f"rows {lo}..{hi}")
        lo = hi


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("distance,window", [(39, 40), (40, 40), (63, 64), (64, 64), (127, 128), (128, 128), (200, None), (0, 1)])
def test_a_single_key_at_the_edge_of_a_window(distance, window, dtype):
    """One key takes nearly all the weight of the one query that asks for it, if and only if it is in the window --
    in a prompt, and decoded from a ring that has wrapped around."""
    from dejavu_amd import mixer_ops as ops

    T, dim, vdim = 230, 16, 8
    rng = np.random.default_rng(distance)
    q, k, v = rng.normal(size=(T, 1, dim)) * 0.1, rng.normal(size=(T, 1, dim)) * 0.1, rng.normal(size=(T, 1, vdim))
    at = 225
    k[at - distance, 0], q[at, 0] = 4.0, 4.0
    q, k, v = (host(dev(a, dtype)) for a in (q, k, v))
    want = V.softmax_attention(q, k, v, 0.25, window=window, sink=np.array([1.0]))
    hit = np.abs(want[at, 0] - v[at - distance, 0]).max() < 0.05
    assert hit == (window is None or distance < window)
    qt, kt, vt = (dev(a.reshape(T, -1), dtype) for a in (q, k, v))
    got = ops.portion_attention(qt, kt, vt, 1, 1, 0.25, 0, 0, sink=dev([1.0]), window=window)
    close(got, want.reshape(T, -1), OP_LIMIT[dtype], "prompt")
    close(got[at:at + 1], want[at].reshape(1, -1), OP_LIMIT[dtype], "the query")
    if window is not None:
        cap = min(window, T)
        kr, vr = torch.zeros(cap, dim, dtype=dtype, device="cuda"), torch.zeros(cap, vdim, dtype=dtype, device="cuda")
        rows = []
        for t in range(T):
            row = torch.cat([qt[t], kt[t], vt[t]]).float()[None].contiguous()
            on_dev = torch.tensor([t], dtype=torch.int32, device="cuda") if t % 2 else None
            rows.append(ops_row(row, kr, vr, window, on_dev, 0 if t % 2 else t))
        # the decode kernel norms q and k: the same on the oracle's side
        want = V.softmax_attention(V.rms_norm(q, 1e-5), V.rms_norm(k, 1e-5), v, 0.25, window=window, sink=np.array([1.0]))
        close(torch.cat(rows), want.reshape(T, -1), OP_LIMIT[dtype], "decoded")


def ops_row(row, kr, vr, window, pos_dev, pos):
    from dejavu_amd import mixer_ops as ops

    return ops.window_attention_row(row, kr, vr, 1, 1, kr.shape[1], 0.25, 1e-5, dev([1.0]), window, pos_dev, pos)


@pytest.mark.parametrize("heads,kv_heads,dim,vdim", [(2, 1, 16, 8), (3, 3, 64, 40), (4, 2, 72, 24), (2, 2, 128, 128),
                                                     (2, 1, 136, 16), (1, 1, 200, 16), (1, 1, 256, 32)])
def test_delta_rule_scan(heads, kv_heads, dim, vdim):
    """A portion of every length around the staged sixteen tokens, fast and slow decays, and the state carried on."""
    from dejavu_amd import mixer_ops as ops

    rng = np.random.default_rng(dim)
    T = 70
    q, k = rng.normal(size=(2, T, kv_heads, dim))
    q, k = V.unit_norm(q), V.unit_norm(k)
    v, beta = rng.normal(size=(T, heads, vdim)), V.sigmoid(rng.normal(size=(T, heads)))
    g = np.exp(-np.exp(rng.normal(size=(T, heads, dim)) * 3 - 3))
    g[T // 2, :, 0] = 0.0  # a channel that is wiped
    q, k, v, g, beta = (host(dev(a)) for a in (q, k, v, g, beta))
    S0 = host(dev(rng.normal(size=(heads, dim, vdim))))
    S = S0.copy()
    rep = heads // kv_heads
    want = V.delta_rule(np.repeat(q, rep, 1), np.repeat(k, rep, 1), v, g, beta, S)
    for cuts in ([T], [2], [1, 15, 16, 17, 3]):
        St = dev(S0.transpose(0, 2, 1)).contiguous()
        got, at, i = [], 0, 0
        while at < T:
            n = min(cuts[min(i, len(cuts) - 1)], T - at)
            part = lambda a: dev(a[at:at + n].reshape(n, -1))  # noqa: E731
            got.append(ops.delta_scan(part(q), part(k), part(v), part(g), part(beta), St, heads, kv_heads))
            at, i = at + n, i + 1
        close(torch.cat(got).view(T, -1), want.reshape(T, -1), 1e-5, f"read-outs, portions {cuts}")
        close(St.view(heads, -1), S.transpose(0, 2, 1).reshape(heads, -1), 1e-5, "state")


def test_delta_rule_scan_of_a_long_portion():
    """More tokens than the kernels take at a time."""
    from dejavu_amd import mixer_ops as ops

    rng = np.random.default_rng(8)
    T, dim, vdim = 4133, 8, 8
    q, k = (host(dev(V.unit_norm(rng.normal(size=(T, 1, dim))))) for _ in range(2))
    v, beta = host(dev(rng.normal(size=(T, 1, vdim)))), host(dev(V.sigmoid(rng.normal(size=(T, 1)))))
    g = host(dev(np.exp(-np.exp(rng.normal(size=(T, 1, dim)) - 4))))
    S = np.zeros((1, dim, vdim))
    want = V.delta_rule(q, k, v, g, beta, S)
    St = torch.zeros(1, vdim, dim, device="cuda")
    got = ops.delta_scan(*(dev(a.reshape(T, -1)) for a in (q, k, v, g, beta)), St, 1, 1)
    close(got.view(T, -1), want.reshape(T, -1), 1e-5, "read-outs")
    close(St[0], S[0].T, 1e-5, "state")


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("H,dim,rank,vdim,cap", [(20, 32, 200, 16, 300), (5, 64, 512, 72, 700), (33, 16, 520, 8, 260),
                                                 (80, 8, 64, 8, 16500), (3, 8, 1032, 40, 130)])
def test_latent_decode_at_many_sizes(H, dim, rank, vdim, cap, dtype):
    """Latents of every width the kernels distinguish, many and few heads, positions at the edges of tiles and splits."""
    from dejavu_amd import mixer_ops as ops

    rng = np.random.default_rng(rank)
    c, ku, vu = (host(dev(rng.normal(size=s) * f, dtype)) for s, f in
                 (((cap, rank), 1.0), ((H * dim, rank), (rank * dim) ** -0.5), ((H * vdim, rank), rank ** -0.5)))
    q, gate = host(dev(rng.normal(size=(1, H * dim)) * 3)), host(dev(rng.normal(size=H)))
    ct, kt, vt = dev(c, dtype), dev(ku, dtype), dev(vu, dtype)
    ql = np.einsum("hdr,hd->hr", ku.reshape(H, dim, rank), q.reshape(H, dim))
    for pos in (0, 63, 64, 128, 129, cap - 1):
        s = ql @ c[:pos + 1].T * 0.5
        p = np.exp(s - s.max(-1, keepdims=True))
        lat = (p / p.sum(-1, keepdims=True)) @ c[:pos + 1] * V.sigmoid(gate)[:, None]
        want = np.einsum("hvr,hr->hv", vu.reshape(H, vdim, rank), lat)
        where = torch.tensor([pos], dtype=torch.int32, device="cuda") if pos % 2 else None
        got = ops.latent_attention_row(dev(q), kt, vt, ct, H, 0.5, dev(gate), where, 0 if pos % 2 else pos)
        close(got, want.reshape(1, -1), OP_LIMIT[dtype], f"position {pos}")


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", sorted(U.CONFIGS))
def test_mixers_alone(name, dtype):
    """Every mixer of a configuration: whole prompt, portions, token by token, and a prompt then tokens."""
    from dejavu_amd import mixer_ops as ops
    from dejavu_amd.mixers import StepInfo

    cfg, P, model = model_of(name, dtype)
    T, width = 83, cfg["width"]
    for i, layer in enumerate(cfg["layers"]):
        mix = model.layers[i].mixer
        h = np.random.default_rng(i).normal(size=(T, width))
        ht = torch.zeros(T, mix.in_proj.shape[1], dtype=dtype, device="cuda")
        ht[:, :width] = dev(h, dtype)
        want = V.MIXERS[layer["type"]](host(ht)[:, :width], V._sub(P, f"l{i}.mix."), layer["mixer"], cfg["norm"]["eps"])
        for cuts in ([T], [2, 3, 2, 31, 8], [1], [60, 1]):
            state, outs, at, c = mix.new_state(T), [], 0, 0
            while at < T:
                n = min(cuts[min(c, len(cuts) - 1)], T - at)
                y = mix(ht[at:at + n], state, StepInfo(at))
                if isinstance(y, ops.GatedHeads):
                    o = y.o.view(mix.heads, -1)
                    s = o / (o[:, :mix.vdim].pow(2).mean(-1, keepdim=True) + mix.eps).sqrt()
                    y = (s * y.weight * y.gate.view(mix.heads, -1)).view(1, -1).to(dtype)
                outs.append(y.float() @ mix.out_weight.float().t())
                at, c = at + n, c + 1
            close(torch.cat(outs)[:, :width], want, LIMIT[dtype], f"{name} layer {i} {layer['type']} {cuts}")


# ---- the model ----------------------------------------------------------------------------------
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", sorted(U.CONFIGS))
def test_model_does_not_depend_on_how_a_prompt_is_cut(name, dtype):
    from dejavu_amd.inference import SequencePool

    cfg, P, model = model_of(name, dtype)
    toks = U.tokens(cfg, 140, seed=3)
    residuals = []
    want = V.forward(cfg, P, toks, residuals=residuals)
    pool = SequencePool(141)
    for cuts in ([140], [1], [2], [70, 2, 3, 1, 5, 1], [100, 1], [33, 64, 7]):
        got = feed(model, pool.get("a"), toks, cuts)
        pool.end("a")
        close(got, want, LIMIT[dtype], f"{name} portions {cuts}")
    if dtype == torch.float32:
        model.record = []
        feed(model, pool.get("a"), toks, [140])
        record, model.record = model.record, None
        assert len(record) == len(residuals)
        for r, w in zip(record, residuals):
            close(r, w, LIMIT[dtype], "residual stream")


@pytest.mark.parametrize("dtype", DTYPES)
def test_sequences_side_by_side_and_memory_used_again(dtype):
    """Three unequal sequences fed in turns, each in its own memory, then others in the same memory."""
    from dejavu_amd.inference import SequencePool

    cfg, P, model = model_of("mixed", dtype)
    pool = SequencePool(90)
    for turn in range(2):
        seqs = {n: U.tokens(cfg, ln, seed=10 * turn + ln) for n, ln in (("a", 90), ("b", 37), ("c", 1))}
        want = {n: V.forward(cfg, P, t) for n, t in seqs.items()}
        got = {n: [] for n in seqs}
        at = {n: 0 for n in seqs}
        sizes = [5, 1, 2, 17, 1, 3]
        i = 0
        while any(at[n] < len(seqs[n]) for n in seqs):
            for n in sorted(seqs):
                part = seqs[n][at[n]:at[n] + sizes[i % len(sizes)]]
                i += 1
                if part:
                    got[n].append(feed(model, pool.get(f"{n}{turn}"), part, [len(part)]))
                    at[n] += len(part)
        for n in seqs:
            close(np.concatenate(got[n]), want[n], LIMIT[dtype], f"sequence {n}, turn {turn}")
            pool.end(f"{n}{turn}")
    assert len(pool.free) == 3 and not pool.live


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", ["mixed", "plain"])
def test_long_decoding_through_generate(name, dtype):
    """Greedy generation, eager and replayed from HIP graphs three times, past every window; every score row against
    the oracle fed the same tokens."""
    cfg, P, model = model_of(name, dtype)
    prompt = U.tokens(cfg, 6, seed=9)
    ids, total = torch.tensor([prompt], device="cuda"), 166
    kw = dict(max_length=total, return_dict_in_generate=True, output_scores=True)
    eager = model.generate(ids, **kw)
    want = V.forward(cfg, P, eager.sequences[0].tolist()[:-1])[len(prompt) - 1:]
    close(eager.scores, want, LIMIT[dtype], "scores")
    top = np.sort(want, axis=-1)
    clear = top[:, -1] - top[:, -2] > 4 * LIMIT[dtype] * np.sqrt((want ** 2).mean())
    assert clear.sum() > 20
    assert (want.argmax(-1) == np.array(eager.sequences[0].tolist()[len(prompt):]))[clear].all()
    for _ in range(3):
        out = model.generate(ids, cg=True, **kw)
        assert torch.equal(out.sequences, eager.sequences) and torch.equal(out.scores, eager.scores)
        other = model.generate(torch.tensor([prompt[::-1]], device="cuda"), **kw)  # eager work in between
        assert not torch.equal(other.scores, eager.scores)
    # a prompt of one token, and a new maximum length
    one = model.generate(ids[:, :1], max_length=20, cg=True, return_dict_in_generate=True, output_scores=True)
    close(one.scores, V.forward(cfg, P, one.sequences[0].tolist()[:-1]), LIMIT[dtype], "from one token")


def test_far_key_among_many_in_latent_attention():
    """One key 700 tokens back carries the answer: prompt, small portion and decode step see it."""
    from dejavu_amd import mixer_ops as ops

    T, H, dim, rank = 760, 2, 16, 24
    rng = np.random.default_rng(4)
    c = rng.normal(size=(T, rank)) * 0.2
    c[31] = 1.0
    k_up, v_up = rng.normal(size=(H * dim, rank)) * 0.1, rng.normal(size=(H * 8, rank))
    q = rng.normal(size=(T, H * dim)) * 0.05
    for dtype in DTYPES:
        ct, ku, vu = dev(c, dtype), dev(k_up, dtype), dev(v_up, dtype)
        kh = (host(ct) @ host(ku).T).reshape(T, H, dim)
        q[T - 1] = (kh[31] * 40.0).reshape(-1)
        qh = host(dev(q, dtype)).reshape(T, H, dim)
        vh = (host(ct) @ host(vu).T).reshape(T, H, 8)
        gate = host(dev(rng.normal(size=(T, H)), dtype))
        want = V.softmax_attention(qh, kh, vh, 0.25) * V.sigmoid(gate)[:, :, None]
        assert np.abs(want[-1] - (vh[31] * V.sigmoid(gate[-1])[:, None])).max() < 0.1
        g16 = torch.zeros(T, 8, dtype=dtype, device="cuda")
        g16[:, :H] = dev(gate, dtype)
        k, v = ops.linear(ct, ku), ops.linear(ct, vu)
        qt = dev(qh.reshape(T, -1), dtype)
        for lo in (0, T - 2):
            got = ops.portion_attention(qt[lo:], k, v, H, H, 0.25, 0, lo, gate=g16[lo:])
            close(got[-1:], want[-1].reshape(1, -1), OP_LIMIT[dtype], f"the query, portion from {lo}")
            close(got[:-1], want[lo:-1].reshape(T - lo - 1, -1), LIMIT[dtype], f"portion from {lo}")
        for pos in (T - 1, 0, 127, 128):
            got = ops.latent_attention_row(qt[pos:pos + 1].float().contiguous(), ku, vu, ct, H, 0.25,
                                           g16[pos].float().contiguous(), None, pos)
            close(got, want[pos].reshape(1, -1), OP_LIMIT[dtype], f"decode at {pos}")


@pytest.mark.parametrize("dtype", ["bfloat16", "float32"])
def test_trace_run_program(tmp_path, dtype):
    """bin/trace_run on a saved model: portions, single tokens, two sequences, one of them in used memory."""
    cfg = U.CONFIGS["loop0"]
    t = U.weights(cfg, seed=5, ranks=U.RANKS["loop0"])
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
    la, lb = V.forward(cfg, P, a), V.forward(cfg, P, b)
    read = lambda i: np.fromfile(out / f"{i}.f32", dtype="<f4").reshape(-1, cfg["vocab"])  # noqa: E731
    limit = LIMIT[getattr(torch, dtype)]
    close(read(0), la[[0, 7, 29]], limit, "portion")
    close(read(1), la[[30]], limit, "token")
    close(read(3), lb[[1]], limit, "other sequence")
    close(read(4), lb[[24, 5]], limit, "its rest, places in the order asked for")
    assert not (out / "2.f32").exists()
