"""Synthetic, seeded inputs for the sparse decode layer at the benchmark shapes.

Distributions (all stored fp16, drawn in fp32 from one seeded generator in a
fixed order): x, residual ~ N(0, 1); fc1 / fc2 / Wqkv / out_proj weights
~ N(0, 0.02); fc1 bias ~ N(-0.1, 0.02); every other bias 0; predictor
weights ~ N(0, 0.05); KV cache ~ N(0, 1).
"""
from __future__ import annotations

import torch

# d, ffn, heads H, head_dim hd, predictor rank r, active neurons K, active heads Hk, KV length S
CONFIGS = {
    "opt-125m": dict(d=768, ffn=3072, H=12, hd=64, r=128, K=1024, Hk=4, S=128),
    "opt-6.7b": dict(d=4096, ffn=16384, H=32, hd=128, r=1000, K=4096, Hk=16, S=512),
    "opt-13b": dict(d=5120, ffn=20480, H=40, hd=128, r=1000, K=2048, Hk=16, S=384),
    "opt-66b": dict(d=9216, ffn=36864, H=72, hd=128, r=1000, K=4096, Hk=24, S=1024),
    "opt-175b": dict(d=12288, ffn=49152, H=96, hd=128, r=1000, K=4096, Hk=32, S=2048),
}


def _normal(gen, shape, mean, std, device):
    t = torch.empty(shape, dtype=torch.float32, device=device)
    t.normal_(mean, std, generator=gen)
    return t.to(torch.float16)


def make_mlp(cfg: dict, batch: int = 1, device="cpu", seed: int = 0) -> dict:
    """Tensors of one sparse MLP block + its predictor (fc2 stored transposed)."""
    d, ffn, r = cfg["d"], cfg["ffn"], cfg["r"]
    gen = torch.Generator(device=device)
    gen.manual_seed(seed)
    t = {}
    t["x2"] = _normal(gen, (batch, d), 0.0, 1.0, device)
    t["residual"] = _normal(gen, (batch, d), 0.0, 1.0, device)
    t["W1"] = _normal(gen, (ffn, d), 0.0, 0.02, device)
    t["b1"] = _normal(gen, (ffn,), -0.1, 0.02, device)
    t["W2t"] = _normal(gen, (ffn, d), 0.0, 0.02, device)  # fc2.weight.t().contiguous()
    t["b2"] = torch.zeros(d, dtype=torch.float16, device=device)
    t["mlp_Wa"] = _normal(gen, (r, d), 0.0, 0.05, device)
    t["mlp_Wb"] = _normal(gen, (ffn, r), 0.0, 0.05, device)
    t["K"] = cfg["K"]
    return t


def make_layer(cfg: dict, batch: int = 1, device="cpu", seed: int = 0) -> dict:
    """Tensors of one full sparse decode layer (MLP + head-sparse attention)."""
    d, H, hd, r, S = cfg["d"], cfg["H"], cfg["hd"], cfg["r"], cfg["S"]
    t = make_mlp(cfg, batch, device, seed)
    gen = torch.Generator(device=device)
    gen.manual_seed(seed + 1)
    t["x"] = _normal(gen, (batch, d), 0.0, 1.0, device)
    t["Wqkv"] = _normal(gen, (3, H, hd, d), 0.0, 0.02, device)
    t["bqkv"] = torch.zeros(3, H, hd, dtype=torch.float16, device=device)
    t["Wout_t"] = _normal(gen, (H * hd, d), 0.0, 0.02, device)  # out_proj.weight.t().contiguous()
    t["bout"] = torch.zeros(d, dtype=torch.float16, device=device)
    t["att_Wa"] = _normal(gen, (r, d), 0.0, 0.05, device)
    t["att_Wb"] = _normal(gen, (H, r), 0.0, 0.05, device)
    # plain (B, H, S, hd) K and V; the packed key layout is derived where needed
    t["k_cache_bhsd"] = _normal(gen, (batch, H, S, hd), 0.0, 1.0, device)
    t["v_cache"] = _normal(gen, (batch, H, S, hd), 0.0, 1.0, device)
    t["Hk"] = cfg["Hk"]
    t["S"] = S
    return t


def pack_k_cache(k_bhsd: torch.Tensor) -> torch.Tensor:
    """(B, H, S, hd) -> (B, H, hd/8, S, 8), the packed key-cache layout."""
    B, H, S, hd = k_bhsd.shape
    return k_bhsd.view(B, H, S, hd // 8, 8).permute(0, 1, 3, 2, 4).contiguous()


# Vimulorn decoders with the layer sizes of real models: [latent attention, delta rule, windowed attention] twice, the
# second three run twice (nine layer runs)
def vimulorn_config(width: int, ff: int, heads: int, q_rank: int, kv_rank: int, window: int, vocab: int = 32768) -> dict:
    hd = 128
    mlp = {"kind": "dense", "ff": ff, "limit": 7.0}
    trio = [
        {"type": "latent_attention", "mlp": mlp,
         "mixer": dict(heads=heads, dim=hd, vdim=hd, q_rank=q_rank, kv_rank=kv_rank, scale=hd ** -0.5)},
        {"type": "channel_delta", "mlp": mlp,
         "mixer": dict(heads=heads, kv_heads=heads // 2, dim=hd, vdim=hd, conv=4, decay_rank=hd, gate_rank=hd)},
        {"type": "attention", "mlp": mlp,
         "mixer": dict(heads=heads, kv_heads=heads // 4, dim=hd, vdim=hd, conv=4, mask={"size": window},
                       scale=hd ** -0.5)}]
    return {"architecture": "Vimulorn", "width": width, "vocab": vocab, "norm": {"eps": 1e-5}, "layers": trio * 2,
            "loop": {"start": 3, "stop": 6, "times": 2}}


VIMULORN_CONFIGS = {
    "vimulorn-4k": vimulorn_config(4096, 11008, 32, 1536, 512, 1024),
    "vimulorn-2k": vimulorn_config(2048, 5632, 16, 768, 256, 512),
}


# Varolorn decoders of the same width, depth and feed-forward: [chunk attention, Mamba-2, Mamba-2] three times
def varolorn_config(width: int, ff: int, heads: int, chunk: int, streams: int = 4, vocab: int = 32768) -> dict:
    hd, inner = 128, 2 * width
    mlp = {"kind": "dense", "ff": ff}
    attention = {"type": "attention", "mlp": mlp,
                 "mixer": dict(heads=heads, kv_heads=heads // 4, dim=hd, vdim=hd, bias_max=128, bias_rows=32, v_mix=True,
                               mask={"size": chunk}, scale=hd ** -0.5)}
    mamba = {"type": "mamba2", "mlp": mlp,
             "mixer": dict(heads=inner // 64, groups=8, vdim=64, state=128, conv=4, norm_groups=8)}
    return {"architecture": "Varolorn", "width": width, "vocab": vocab, "norm": {"eps": 1e-5}, "streams": streams,
            "embedding": {"scale": width ** 0.5, "bigram": {"buckets": 65521, "mul_prev": 8191, "mul_cur": 31}},
            "layers": [attention, mamba, mamba] * 3}


VAROLORN_CONFIGS = {
    "varolorn-4k": varolorn_config(4096, 11008, 32, 2048),
    "varolorn-2k": varolorn_config(2048, 5632, 16, 1024),
}


@torch.no_grad()
def init_varolorn_synthetic(model, seed: int = 0) -> None:
    """Seeded random weights in place: matrices ~ N(0, 1 / columns), norm weights and D 1, streams read evenly and kept
    as they are, everything else small."""
    dev = next(model.parameters()).device
    gen = torch.Generator(device=dev)
    gen.manual_seed(seed)
    for name, p in model.named_parameters():
        leaf = name.rsplit(".", 1)[-1]
        if leaf in ("weight", "norm", "q_norm", "k_norm", "D", "out"):
            p.fill_(1.0)
        elif leaf == "weights":
            p.fill_(1.0 / p.numel())
        elif leaf == "mix":
            p.copy_(torch.eye(p.shape[0], device=dev))
        elif leaf in ("A_log", "dt_bias"):
            p.fill_(-1.0)
        else:
            tmp = torch.empty(p.shape, dtype=torch.float32, device=dev)
            p.copy_(tmp.normal_(0.0, p.shape[-1] ** -0.5 if p.dim() == 2 else 0.1, generator=gen))


@torch.no_grad()
def init_vimulorn_synthetic(model, seed: int = 0) -> None:
    """Seeded random weights in place: matrices ~ N(0, 1 / columns), norm weights 1, everything else small."""
    dev = next(model.parameters()).device
    gen = torch.Generator(device=dev)
    gen.manual_seed(seed)
    for name, p in model.named_parameters():
        tmp = torch.empty(p.shape, dtype=torch.float32, device=dev)
        leaf = name.rsplit(".", 1)[-1]
        if leaf in ("weight", "norm", "q_norm", "kv_norm"):
            tmp.fill_(1.0)
        elif leaf == "alpha":
            tmp.fill_(0.5)
        elif leaf == "A_log":
            tmp.fill_(-2.0)
        else:
            tmp.normal_(0.0, p.shape[-1] ** -0.5 if p.dim() == 2 else 0.1, generator=gen)
        p.copy_(tmp)
