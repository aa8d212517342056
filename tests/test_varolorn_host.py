"""Varolorn on the host: the oracle against itself, configuration, tensor names, registry, argument checks."""
import json
import math

import numpy as np
import pytest
import torch

from oracle import varolorn_oracle as O
from tests import varolorn_utils as U


def test_recurrence_of_the_oracle_matches_its_sum():
    """y_t = sum_j (C_t . B_j) dt_j decay(j .. t] x_j + D x_t."""
    rng = np.random.default_rng(0)
    T, H, P, N = 6, 2, 3, 4
    x, B, C = rng.normal(size=(T, H, P)), rng.normal(size=(T, H, N)), rng.normal(size=(T, H, N))
    dt, A, D = rng.uniform(0.1, 1, (T, H)), rng.uniform(0.2, 2, H), rng.normal(size=H)
    S = np.zeros((H, N, P))
    y = O.ssd(x, B, C, dt, A, D, S)
    for h in range(H):
        for t in range(T):
            want = D[h] * x[t, h]
            for j in range(t + 1):
                want = want + (C[t, h] @ B[j, h]) * dt[j, h] * np.exp(-A[h] * dt[j + 1:t + 1, h].sum()) * x[j, h]
            np.testing.assert_allclose(y[t, h], want, atol=1e-12)


@pytest.mark.parametrize("rows,far", [(32, 100), (8, 12), (6, 20), (5, 9), (2, 3), (7, 64), (16, 128), (20, 11), (12, 5)])
def test_distance_buckets(rows, far):
    """Against the logarithm where that is not within rounding of a step, and the two statements of it against each
    other; the last row is reached at ``far`` and kept."""
    from dejavu_amd.mixers import bias_distances, distance_buckets

    half = rows // 2
    got = distance_buckets(3 * far, rows, far)
    for n in range(3 * far):
        assert got[n] == O.distance_bucket(n, rows, far)
        if n < half:
            assert got[n] == n
        elif far > half:
            z = math.log(n / half) / math.log(far / half) * (rows - half)
            if abs(z - round(z)) > 1e-9:
                assert got[n] == min(rows - 1, half + math.floor(z))
    assert all(b == rows - 1 for b in got[max(far, half):])
    last = bias_distances(rows, far, None)
    assert distance_buckets(last, rows, far)[-1] == rows - 1 and bias_distances(rows, far, 4) <= 4


def test_chunks_and_bias_of_the_oracle():
    """A chunk starts with its own first token alone; equal keys are weighted by the bias of their distance."""
    T, chunk = 11, 4
    q, k, v = np.zeros((T, 1, 2)), np.zeros((T, 1, 2)), np.arange(T, dtype=float).reshape(T, 1, 1)
    table = np.array([[0.0], [1.0], [-2.0]])  # distances 0; 1; 2 and 3
    o = O.biased_attention(q, k, v, 1.0, table, 2, chunk)[:, 0, 0]
    assert o[0] == 0 and o[4] == 4 and o[8] == 8
    w = np.exp([-2.0, -2.0, 1.0, 0.0])
    np.testing.assert_allclose(o[7], (w / w.sum()) @ np.arange(4.0, 8.0))


def test_one_stream_is_the_plain_residual():
    rng = np.random.default_rng(3)
    x, y = rng.normal(size=(1, 4, 5)), rng.normal(size=(4, 5))
    hc = {"in": np.ones(1), "out": np.ones(1), "mix": np.ones((1, 1))}
    np.testing.assert_allclose(O.read_streams(x, hc), x[0])
    np.testing.assert_allclose(O.write_streams(x, hc, y)[0], x[0] + y)
    mix = np.array([[1.0, 10.0], [100.0, 1000.0]])  # [from, to]
    two = O.write_streams(np.array([[[1.0]], [[2.0]]]), {"mix": mix, "out": np.array([0.1, 0.2])}, np.array([[1.0]]))
    np.testing.assert_allclose(two[:, 0, 0], [1 + 200 + 0.1, 10 + 2000 + 0.2])


def test_embedding_rows_of_the_oracle():
    table, bigram = np.zeros((4, 1)), np.arange(6.0).reshape(6, 1)
    got = O.embed([3, 1, 2], table, 1.0, bigram, 7, 3)[:, 0]
    np.testing.assert_array_equal(got, [5, (3 * 7 + 1 * 3) % 5, (1 * 7 + 2 * 3) % 5])


def test_sizes_come_from_the_tensors_when_the_configuration_leaves_them_out():
    from dejavu_amd.hybrid import HybridConfig

    cfg = json.loads(json.dumps(U.CONFIGS["mixed"]))
    shapes = {k: tuple(v.shape) for k, v in U.weights("mixed").items()}
    full = HybridConfig.from_dict_streams(cfg, shapes)
    for layer in cfg["layers"]:
        for key in ("heads", "kv_heads", "dim", "vdim", "conv"):
            layer["mixer"].pop(key, None)
        if layer["mlp"]:
            layer["mlp"].pop("ff")
    cfg.pop("width"), cfg.pop("vocab"), cfg["embedding"]["bigram"].pop("buckets")
    conf = HybridConfig.from_dict_streams(cfg, shapes)
    assert conf == full
    assert (conf.width, conf.vocab, conf.streams, conf.embedding.buckets) == (100, 213, 3, 31)
    assert [s.mixer.get("values") for s in conf.layers] == ["first", None, "mixed", None, None, "mixed"]
    assert [s.mixer.get("bias_rows") for s in conf.layers] == [8, None, 6, 12, None, 5]
    with pytest.raises(ValueError, match="unknown mixer"):
        HybridConfig.from_dict_streams(dict(cfg, layers=[{"type": "other", "mixer": {}, "mlp": None}]), shapes)
    with pytest.raises(ValueError, match="unknown feed-forward"):
        bad = dict(cfg["layers"][0], mlp={"kind": "routed"})
        HybridConfig.from_dict_streams(dict(cfg, layers=[bad]), shapes)


@pytest.mark.parametrize("name", sorted(U.CONFIGS))
def test_checkpoint_tensors_fill_the_model(name):
    """The products of the padded weights are those of the originals, padding is zero, tables and norms are expanded."""
    from dejavu_amd.registry import build_model

    cfg, t = U.CONFIGS[name], U.weights(name)
    m = build_model(cfg, t, device="cpu", dtype=torch.float32)
    assert m.lm_head is m.embeddings
    w = cfg["width"]
    torch.testing.assert_close(m.final_norm.weight[:w], 1 + t["final.norm"].float())
    assert not m.final_norm.weight[w:].any() and m.bigram.shape[0] == cfg["embedding"]["bigram"]["buckets"] + 1
    x = torch.randn(3, w)
    for i, layer in enumerate(cfg["layers"]):
        blk, p, c = m.layers[i], f"l{i}.mix.", layer["mixer"]
        mix = blk.mixer
        torch.testing.assert_close(blk.hyper1.mix, t[f"l{i}.hc1.mix"].float())
        torch.testing.assert_close(blk.hyper1.weights, t[f"l{i}.hc1.in"].float())
        h = torch.zeros(3, mix.in_proj.shape[1])
        h[:, :w] = x
        rows = h @ mix.in_proj.t()
        if layer["type"] == "attention":
            rows = rows + mix.in_bias
            for n, at, heads, dim, stride in (("q", 0, c["heads"], c["dim"], mix.dim_s),
                                              ("k", mix.off_k, c["kv_heads"], c["dim"], mix.dim_s),
                                              ("v", mix.off_v, c["kv_heads"], c["vdim"], mix.vdim_s)):
                got = rows[:, at:at + heads * stride].view(3, heads, stride)
                want = x @ t[p + n].float().t() + t[p + n + ".b"].float()
                torch.testing.assert_close(got[:, :, :dim].reshape(3, -1), want)
                assert not got[:, :, dim:].any()
            torch.testing.assert_close(rows[:, mix.off_g:mix.off_g + c["heads"]], x @ t[p + "g"].float().t())
            table = t[p + "rel"].float()
            for n in (0, 1, c["bias_max"] // 2, mix.rel.shape[1] - 1):
                if n < mix.rel.shape[1]:
                    torch.testing.assert_close(mix.rel[:, n], table[O.distance_bucket(n, table.shape[0], c["bias_max"])])
        else:
            inner, bc = c["heads"] * c["vdim"], c["groups"] * c["state"]
            want = x @ t[p + "in"].float().t()
            torch.testing.assert_close(rows[:, mix.off_z:mix.off_z + inner], want[:, :inner])
            torch.testing.assert_close(rows[:, :inner], want[:, inner:2 * inner])
            for at, src in ((mix.off_b, 2 * inner), (mix.off_c, 2 * inner + bc)):
                got = rows[:, at:at + c["groups"] * mix.state_s].view(3, c["groups"], mix.state_s)
                torch.testing.assert_close(got[:, :, :c["state"]].reshape(3, -1), want[:, src:src + bc])
                assert not got[:, :, c["state"]:].any()
            torch.testing.assert_close(rows[:, mix.off_dt:mix.off_dt + c["heads"]], want[:, -c["heads"]:])
            torch.testing.assert_close(mix.conv_bias[mix.off_c:mix.off_c + c["state"]],
                                       t[p + "conv.b"].float()[inner + bc:inner + bc + c["state"]])
    with pytest.raises(ValueError, match="unexpected"):
        build_model(cfg, dict(t, extra=torch.zeros(3)), device="cpu", dtype=torch.float32)
    with pytest.raises((KeyError, ValueError)):
        build_model(cfg, {k: v for k, v in t.items() if k != "l0.hc1.mix"}, device="cpu", dtype=torch.float32)


def test_registry_and_state():
    from dejavu_amd import registry
    from dejavu_amd.inference import SequencePool

    name, family = registry.family_of({"architecture": "Varolorn"})
    assert name == "Varolorn" and family.takes_portions and family.dtypes == (torch.bfloat16, torch.float32)
    m = registry.build_model(U.CONFIGS["mixed"], U.weights("mixed"), device="cpu", dtype=torch.float32)
    params = SequencePool(50).get("a")
    states = m._states(params)
    assert [sorted(s) for s in states] == [["k", "v"], ["S", "conv"], ["k", "v"], ["k", "v"], ["S", "conv"], ["k", "v"]]
    assert [s["k"].shape[0] for s in states if "k" in s] == [9, 33, 50, 50]  # a chunk, or all there can be
    assert m._history(params) is m._history(params) and m._history(params).shape == (50,)
    states[1]["S"].fill_(1.0)
    params.restart()
    assert not states[1]["S"].any()


def test_host_side_argument_checks():
    """Bad sizes and null pointers are refused before anything is launched."""
    import ctypes

    from dejavu_amd import _lib_mixers as L

    ref, A = ctypes.byref, 0x1000
    row = L.RowArgs(x=A, W=A, ldw=64, M=64, K=64, out=A)
    assert L.lib.dv_mix_linear_row(0, L.ROW_PLAIN, L.OUT_HYPER, ref(row), None) == -1   # no streams
    row.hyper = L.Hyper(x=A, mix=A, out=A, in_=A, u=A, streams=5, width=64)
    assert L.lib.dv_mix_linear_row(0, L.ROW_PLAIN, L.OUT_HYPER, ref(row), None) == -1   # more than the epilogue takes
    row.hyper.streams, row.hyper.width = 2, 32
    assert L.lib.dv_mix_linear_row(0, L.ROW_PLAIN, L.OUT_HYPER, ref(row), None) == -1   # not as wide as the product
    row.xw, row.x_dim, row.norm_dim = A, 60, 25
    assert L.lib.dv_mix_linear_row(0, L.ROW_GROUPS, L.OUT_T, ref(row), None) == -1      # groups do not divide
    row.norm_dim, row.xw = 64, A + 4
    assert L.lib.dv_mix_linear_row(0, L.ROW_RMS, L.OUT_F32, ref(row), None) == -3       # misaligned weight
    row = L.RowArgs(x=A, W=A, ldw=64, M=64, K=64, out=A, bias=A)
    assert L.lib.dv_mix_linear_row(0, L.ROW_PLAIN, L.OUT_GLU, ref(row), None) == -1     # no bias there
    hy, norm = L.Hyper(x=A, in_=A, streams=17, width=64), L.RmsOut(w=A, eps=1e-5, dim=64, h=A)
    assert L.lib.dv_mix_hyper_rows(0, None, 2, ref(hy), ref(norm), None) == -1          # too many streams
    hy.streams = 2
    assert L.lib.dv_mix_hyper_rows(0, A, 2, ref(hy), ref(norm), None) == -1             # no matrix
    norm.dim = 65
    assert L.lib.dv_mix_hyper_rows(0, None, 2, ref(hy), ref(norm), None) == -1          # norm wider than the row
    norm.dim = 64
    e = L.EmbedArgs(tokens=A, history=A, capacity=4, vocab=9, embed=A, pos_host=3, n=2)
    assert L.lib.dv_mix_hyper_embed(0, ref(e), ref(hy), ref(norm), None) == -1          # past the history
    at = L.AttnArgs(q=A, ldq=64, k=A, ldk=64, k_head=64, v=A, ldv=64, v_head=64, n=1, H=1, G=1, dim_s=64, vdim_s=64,
                    out=A, splits=1, window=3, chunk=3)
    assert L.lib.dv_mix_attn_rows(0, 0, ref(at), None) == -1                            # window and chunk
    at.window, at.rel = 0, A
    assert L.lib.dv_mix_attn_rows(0, 0, ref(at), None) == -1                            # a table without entries
    s = L.SsdArgs(xbc=A, ld=64, off_b=16, off_c=32, dt=A, lddt=8, A_log=A, dt_bias=A, D=A, S=A, y=A, ldy=16, tm=A, n=3,
                  heads=3, groups=2, vdim=5, state_s=8)
    assert L.lib.dv_mix_ssd_scan(0, ref(s), None) == -1                                 # groups do not divide
    s.groups = 3
    assert L.lib.dv_mix_ssd_scan(0, ref(s), None) == -4                                 # scratch too small
    s.state_s = 264
    assert L.lib.dv_mix_ssd_scan(0, ref(s), None) == -2
    assert L.lib.dv_mix_glu(0, A, 64, 2, 0.0, A, None) == -1                            # unknown unit
    assert L.lib.dv_mix_gated_group_norm(0, A, 16, A, 16, 2, 15, 2, 16, A, 1e-5, A, None) == -1
    h = L.HeadArgs(in_=A, ldi=16, n=1)
    h.g[0] = L.HeadGroup(heads=1, stride=16, dim=16, other=A, ldo=16, out=A, ld=16)
    assert L.lib.dv_mix_head_rows(0, ref(h), None) == -1                                # nothing to mix by
