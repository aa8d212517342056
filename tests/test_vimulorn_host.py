"""Vimulorn on the host: the oracle against itself, configuration, tensor names, registry, trace and memory pool."""
import io
import json
import os
import re
import types

import numpy as np
import pytest
import torch

from oracle import vimulorn_oracle as V
from tests import vimulorn_utils as U

ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))


def test_delta_rule_matches_the_matrix_form():
    """One head without decay and with beta 1: S is S (I - k k^T) + k v^T for a unit key."""
    rng = np.random.default_rng(0)
    q, k, v = rng.normal(size=(3, 5, 1, 4))
    k /= np.linalg.norm(k, axis=-1, keepdims=True)
    S = np.zeros((1, 4, 4))
    out = V.delta_rule(q, k, v, np.ones((5, 1, 4)), np.ones((5, 1)), S)
    M = np.zeros((4, 4))
    for t in range(5):
        M = M - np.outer(k[t, 0], k[t, 0] @ M) + np.outer(k[t, 0], v[t, 0])
        np.testing.assert_allclose(out[t, 0], q[t, 0] @ M, atol=1e-12)
    np.testing.assert_allclose(k[4, 0] @ M, v[4, 0], atol=1e-12)  # the newest pair is recalled exactly


def test_window_and_sink_of_the_oracle():
    """The key just inside a window takes the weight, the one just outside does not; the sink takes weight."""
    T, W = 12, 4
    q = np.ones((T, 1, 1))
    k, v = np.zeros((T, 1, 1)), np.arange(T, dtype=float).reshape(T, 1, 1)
    k[5] = 60.0
    o = V.softmax_attention(q, k, v, 1.0, window=W)[:, 0, 0]
    assert abs(o[5 + W - 1] - 5) < 1e-9 and abs(o[5 + W] - np.mean(np.arange(6, 10))) < 1e-9
    s = V.softmax_attention(q, np.zeros((T, 1, 1)), np.ones((T, 1, 1)), 1.0, window=W, sink=np.array([0.0]))[:, 0, 0]
    np.testing.assert_allclose(s, [1 / 2, 2 / 3, 3 / 4] + [4 / 5] * (T - 3))


def test_oracle_short_conv_is_causal():
    u, w = np.arange(8.0).reshape(4, 2), np.array([[1.0, 10.0, 100.0], [0.0, 0.0, 1.0]])
    y = V.short_conv(u, w)
    np.testing.assert_allclose(y[:, 1], u[:, 1])
    np.testing.assert_allclose(y[:, 0], [0, 200, 420, 642])


def test_layer_runs():
    from dejavu_amd.hybrid import HybridConfig

    for name, cfg in U.CONFIGS.items():
        t = U.weights(cfg, ranks=U.RANKS[name])
        conf = HybridConfig.from_dict(cfg, {k: tuple(v.shape) for k, v in t.items()})
        assert conf.runs() == V.layer_runs(cfg)
    cfg = U.CONFIGS["mixed"]
    assert V.layer_runs(cfg) == [(0, False), (1, False), (2, False), (3, False), (1, True), (2, False), (3, False),
                                 (1, True), (2, False), (3, False)]


def test_sizes_come_from_the_tensors_when_the_configuration_leaves_them_out():
    from dejavu_amd.hybrid import HybridConfig

    cfg = json.loads(json.dumps(U.CONFIGS["mixed"]))
    shapes = {k: tuple(v.shape) for k, v in U.weights(cfg, ranks=(10, 6)).items()}
    for layer in cfg["layers"]:
        for key in ("q_rank", "kv_rank", "conv"):
            layer["mixer"].pop(key, None)
        if layer["mlp"]:
            layer["mlp"].pop("ff")
    cfg.pop("width"), cfg.pop("vocab")
    conf = HybridConfig.from_dict(cfg, shapes)
    assert (conf.width, conf.vocab) == (100, 213)
    assert [s.mixer.get("conv") for s in conf.layers] == [4, 3, None, 2]
    assert (conf.layers[2].mixer["q_rank"], conf.layers[2].mixer["kv_rank"]) == (18, 44)
    assert (conf.layers[1].mixer["decay_rank"], conf.layers[1].mixer["gate_rank"]) == (10, 6)
    assert conf.layers[0].mlp["ff"] == 75 and conf.layers[2].mlp is None
    with pytest.raises(ValueError, match="unknown mixer"):
        HybridConfig.from_dict(dict(cfg, layers=[{"type": "other", "mixer": {}, "mlp": None}]), shapes)


@pytest.mark.parametrize("name", sorted(U.CONFIGS))
def test_checkpoint_tensors_fill_the_model(name):
    """Every parameter is filled, padding is zero, and the products of the padded weights are those of the originals."""
    from dejavu_amd.registry import build_model

    cfg = U.CONFIGS[name]
    t = U.weights(cfg, ranks=U.RANKS[name])
    m = build_model(cfg, t, device="cpu", dtype=torch.float32)
    total = sum(v.float().abs().sum().item() for v in t.values())
    held = sum(p.abs().sum().item() for p in m.parameters())
    assert abs(total - held) < 1e-3 * total
    assert len(m.runs) == len(V.layer_runs(cfg)) and m.keeps_start == any(a for _, a in V.layer_runs(cfg))
    x = torch.randn(3, cfg["width"])
    for i, layer in enumerate(cfg["layers"]):
        mix, p = m.layers[i].mixer, f"l{i}.mix."
        h = torch.zeros(3, mix.in_proj.shape[1])
        h[:, :cfg["width"]] = x
        rows = h @ mix.in_proj.t()
        if layer["type"] == "latent_attention":
            torch.testing.assert_close(rows[:, :mix.q_rank], x @ t[p + "dq"].float().t())
            torch.testing.assert_close(rows[:, mix.q_rank_s:mix.q_rank_s + mix.kv_rank], x @ t[p + "dkv"].float().t())
            torch.testing.assert_close(rows[:, mix.q_rank_s + mix.kv_rank_s:][:, :mix.heads], x @ t[p + "g"].float().t())
        else:
            qh = mix.kv_heads if layer["type"] == "channel_delta" else mix.heads
            got = rows[:, :qh * mix.dim_s].view(3, qh, mix.dim_s)
            torch.testing.assert_close(got[:, :, :mix.dim].reshape(3, -1), x @ t[p + "q"].float().t())
            assert not got[:, :, mix.dim:].any()
    bad = dict(t, extra=torch.zeros(3))
    with pytest.raises(ValueError, match="unexpected"):
        build_model(cfg, bad, device="cpu", dtype=torch.float32)
    bad = {k: v for k, v in t.items() if k != "final.norm.b"}
    with pytest.raises((KeyError, ValueError)):
        build_model(cfg, bad, device="cpu", dtype=torch.float32)


def test_registry():
    from dejavu_amd import registry

    assert registry.family_of({"architecture": "Vimulorn"})[1].takes_portions
    assert registry.family_of({"architectures": ["OPTForCausalLM"]})[0] == "OPTForCausalLM"
    with pytest.raises(ValueError, match="no model family"):
        registry.family_of({"architectures": ["Nothing"]})
    cfg = U.CONFIGS["plain"]
    with pytest.raises(ValueError, match="runs in"):
        registry.build_model(cfg, U.weights(cfg), device="cpu", dtype=torch.float16)
    opt = registry.FAMILIES["OPTForCausalLM"].read_config(
        dict(hidden_size=64, ffn_dim=128, num_attention_heads=4, num_hidden_layers=2, vocab_size=50,
             max_position_embeddings=32, mlp_K=24, att_K=[2, 3]), {})
    assert (opt.n_inner, opt.mlp_K, opt.att_K, opt.hidden_size) == (128, 24, [2, 3], 64)


def test_sequence_pool_gives_memory_back():
    from dejavu_amd.inference import SequencePool

    pool = SequencePool(10)
    a = pool.get("a")
    assert pool.get("a") is a and a.max_sequence_len == 10
    a.sequence_len_offset = 7
    a.key_value_memory_dict[0] = {"S": torch.ones(2), "conv": torch.ones(2), "latent": torch.ones(2)}
    a.key_value_memory_dict[1] = (torch.ones(1), torch.ones(1))
    b = pool.get("b")
    assert b is not a
    pool.end("a")
    pool.end("nobody")
    c = pool.get("c")  # the same memory, as new: states are zero, caches are left as they are
    assert c is a and c.sequence_len_offset == 0
    s = c.key_value_memory_dict[0]
    assert not s["S"].any() and not s["conv"].any() and s["latent"].all()


def test_trace_steps(tmp_path):
    """Files, lines and life of the sequences, with a model that answers from its tokens and position."""
    from dejavu_amd import trace
    from dejavu_amd.inference import SequencePool

    def model(ids, inference_params, rows):
        pos = inference_params.sequence_len_offset
        if not rows:
            return types.SimpleNamespace(logits=None)
        return types.SimpleNamespace(logits=torch.tensor([[[pos + r, int(ids[0, r])] for r in rows]]))

    steps = [{"step": 0, "entries": [{"id": "a", "tokens": [4, 5, 6], "want": [0, 2]}], "end": []},
             {"step": 1, "entries": [{"id": "a", "tokens": [7], "want": []}], "end": []},
             {"step": 2, "entries": [{"id": "b", "tokens": [9, 8], "want": [1]}, {"id": "a", "tokens": [3], "want": [0]}],
              "end": ["a", "b"]},
             {"step": 3, "entries": [{"id": "a", "tokens": [2], "want": [0]}], "end": ["a"]}]
    said = []
    trace.run(model, io.StringIO("\n".join(json.dumps(s) for s in steps) + "\n\n"), str(tmp_path), SequencePool(8),
              device="cpu", emit=said.append)
    assert said == [f"done {i}" for i in range(4)]
    read = lambda i: np.fromfile(tmp_path / f"{i}.f32", dtype="<f4").reshape(-1, 2).tolist()  # noqa: E731
    assert read(0) == [[0, 4], [2, 6]] and read(2) == [[1, 8], [4, 3]] and read(3) == [[0, 2]]
    assert not (tmp_path / "1.f32").exists()


def test_header_and_binding_agree():
    from dejavu_amd import _lib_mixers

    text = open(os.path.join(ROOT, "include", "dejavu_mixers.h")).read()
    text = re.sub(r"/\*.*?\*/", "", text, flags=re.S)
    names = set(re.findall(r"\bDV_API\s+[\w\s\*]+?\b(dv_\w+)\s*\(", text))
    assert names == set(_lib_mixers.SIGNATURES)
    for body, c_name in re.findall(r"typedef struct \{(.*?)\}\s*(\w+);", text, flags=re.S):
        fields = []
        for decl in body.split(";"):
            decl = decl.strip()
            if decl:
                names = re.sub(r"^(const\s+)?\w+\s*\**\s*", "", decl, count=1)
                fields += [re.sub(r"[\s\*]|\[.*", "", n) for n in names.split(",")]
        py = getattr(_lib_mixers, c_name[2:])
        assert [n.rstrip("_") for n, *_ in py._fields_] == fields, c_name


def test_host_side_argument_checks():
    """Bad sizes and null pointers are refused before anything is launched."""
    import ctypes

    from dejavu_amd import _lib_mixers as L

    ref, A = ctypes.byref, 0x1000
    row = L.RowArgs(x=A, W=A, ldw=64, M=4, K=60, out=A)
    assert L.lib.dv_mix_linear_row(0, 0, 0, ref(row), None) == -3            # K % 8
    row.K = 64
    assert L.lib.dv_mix_linear_row(2, 0, 0, ref(row), None) == -1            # element type
    assert L.lib.dv_mix_linear_row(0, 1, 0, ref(row), None) == -1            # norm weight missing
    assert L.lib.dv_mix_linear_row(0, 0, 3, ref(row), None) == -1            # residual missing
    assert L.lib.dv_mix_linear_tiles(0, ref(L.TileArgs(x=A + 2, ldx=64, W=A, ldw=64, n=2, M=4, K=64, out=A, ldo=4)), None) == -3
    at = L.AttnArgs(q=A, ldq=64, k=A, ldk=64, k_head=64, v=A, ldv=64, v_head=64, n=3, H=1, G=1, dim_s=64, vdim_s=64,
                    out=A, splits=1)
    assert L.lib.dv_mix_attn_tiles(ref(at), 2, None) == -1                   # fewer keys than queries
    at.H, at.G = 3, 2
    assert L.lib.dv_mix_attn_rows(0, 0, ref(at), None) == -1                 # heads do not divide
    assert L.lib.dv_mix_ring_copy(0, A, 64, A, 4, 64, 0, 5, 64, 1, None) == -1  # more rows than the ring has
    d = L.DeltaArgs(q=A, k=A, v=A, g=A, beta=A, S=A, o=A, tm=A, n=2, heads=2, kv_heads=1, dim_s=264, vdim_s=8)
    assert L.lib.dv_mix_delta_scan(ref(d), None) == -2
    d.dim_s, d.tm_floats = 64, 100
    assert L.lib.dv_mix_delta_scan(ref(d), None) == -4                       # scratch too small
    with pytest.raises(RuntimeError, match="no CPU fallback"):
        from dejavu_amd import mixer_ops
        mixer_ops.linear(torch.zeros(1, 8), torch.zeros(8, 8))
