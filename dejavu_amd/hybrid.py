"""Decoders whose layers differ in how they mix tokens (latent attention, gated delta rule, windowed attention).

``Vimulorn`` is the family that is registered: sandwich dynamic-tanh norms (before and after every sublayer), a
clamped gated feed-forward, and optionally a stretch of layers that runs several times with the same weights, where
every pass but the first adds the embedding output again and every pass keeps its own cache or state.

A layer is: h -> mixer -> output projection (with norm, residual add and the next norm behind it) -> feed-forward ->
down projection (likewise).  No norm has a launch of its own.
"""
from __future__ import annotations

from dataclasses import dataclass
from typing import Dict, List, Optional, Tuple

import torch
import torch.nn as nn

from . import mixer_ops as ops
from .generation import CausalLMOutput, GreedyDecoding
from .inference import InferenceParams
from .mixer_ops import padded
from .mixers import ChannelDelta, ClampedGLU, DynamicTanh, LatentAttention, StepInfo, WindowAttention


@dataclass
class LayerSpec:
    """One layer: the kind of mixer with its sizes, and the feed-forward (None: the layer has none)."""

    type: str
    mixer: dict
    mlp: Optional[dict] = None


@dataclass
class HybridConfig:
    width: int
    vocab: int
    layers: List[LayerSpec]
    norm_eps: float = 1e-5
    loop: Optional[Tuple[int, int, int]] = None  # layers start .. stop - 1 run `times` times

    @classmethod
    def from_dict(cls, config: dict, shapes: Optional[Dict[str, tuple]] = None) -> "HybridConfig":
        """config: parsed config.json; shapes: tensor name -> shape of the checkpoint, the source of every size that
        config.json leaves out (the ranks of the low-rank projections)."""
        shapes = shapes or {}

        def rows(name, default=None):
            return shapes[name][0] if name in shapes else default

        layers = []
        for i, entry in enumerate(config["layers"]):
            kind, mix, mlp, pre = entry["type"], dict(entry["mixer"]), entry.get("mlp"), f"l{i}.mix."
            if kind == "latent_attention":
                for key, name in (("q_rank", "dq"), ("kv_rank", "dkv")):
                    mix.setdefault(key, rows(pre + name))
            elif kind == "channel_delta":
                for key, name in (("decay_rank", "a1"), ("gate_rank", "g1")):
                    if pre + name in shapes:
                        mix[key] = rows(pre + name)
            elif kind != "attention":
                raise ValueError(f"layer {i}: unknown mixer {kind!r}")
            if kind in ("channel_delta", "attention") and pre + "q.conv" in shapes:
                mix["conv"] = max(shapes[pre + t + ".conv"][1] for t in "qkv")
            if mlp is not None:
                if mlp.get("kind", "dense") != "dense":
                    raise ValueError(f"layer {i}: unknown feed-forward {mlp['kind']!r}")
                mlp = dict(mlp)
                mlp.setdefault("ff", rows(f"l{i}.mlp.gate"))
            layers.append(LayerSpec(kind, mix, mlp))
        loop = config.get("loop")
        if loop:
            loop = (int(loop["start"]), int(loop["stop"]), int(loop["times"]))
            assert 0 <= loop[0] <= loop[1] <= len(layers) and loop[2] >= 1, "loop bounds"
        return cls(width=config.get("width", shapes.get("embed", (0, 0))[1]),
                   vocab=config.get("vocab", shapes.get("embed", (0, 0))[0]), layers=layers,
                   norm_eps=float(config["norm"]["eps"]), loop=loop or None)

    def runs(self) -> List[Tuple[int, bool]]:
        """(layer, does it start a repeated pass) in the order of execution."""
        order = list(range(len(self.layers)))
        if not self.loop:
            return [(i, False) for i in order]
        start, stop, times = self.loop
        if start == stop:
            return [(i, False) for i in order]
        body = [(i, t > 0 and i == start) for t in range(times) for i in range(start, stop)]
        return [(i, False) for i in order[:start]] + body + [(i, False) for i in order[stop:]]


def create_mixer(spec: LayerSpec, width: int, eps: float, dtype=None, device=None) -> nn.Module:
    m = spec.mixer
    kw = dict(eps=eps, dtype=dtype, device=device)
    if spec.type == "latent_attention":
        return LatentAttention(width, m["heads"], m["dim"], m["vdim"], m["q_rank"], m["kv_rank"], m["scale"], **kw)
    if spec.type == "channel_delta":
        return ChannelDelta(width, m["heads"], m["kv_heads"], m["dim"], m["vdim"], m["conv"], m["decay_rank"],
                            m["gate_rank"], **kw)
    if spec.type == "attention":
        return WindowAttention(width, m["heads"], m["kv_heads"], m["dim"], m["vdim"], m["conv"], m["mask"]["size"],
                               m["scale"], **kw)
    raise ValueError(f"unknown mixer {spec.type!r}")


class HybridBlock(nn.Module):
    def __init__(self, spec: LayerSpec, width: int, eps: float, dtype=None, device=None):
        super().__init__()
        self.norm1 = DynamicTanh(width, device=device)
        self.mixer = create_mixer(spec, width, eps, dtype=dtype, device=device)
        self.norm1b = DynamicTanh(width, device=device)
        self.mlp = None
        if spec.mlp is not None:
            self.norm2 = DynamicTanh(width, device=device)
            self.mlp = ClampedGLU(width, spec.mlp["ff"], spec.mlp["limit"], dtype=dtype, device=device)
            self.norm2b = DynamicTanh(width, device=device)

    def forward(self, h, stream: ops.ResidualStream, state: dict, step: StepInfo, pre, add_start: bool = False):
        """h: norm1 of the stream.  Adds both sublayers to the stream (then, with ``add_start``, the stream's start
        once more) and returns ``pre`` of it, the input of whatever comes next (None without ``pre``)."""
        y = self.mixer(h, state, step)
        last = self.mlp is None
        after = (self.norm1b, pre, add_start) if last else (self.norm1b, self.norm2, False)
        if isinstance(y, ops.GatedHeads):
            h = y.linear_residual(self.mixer.out_weight, stream, *after)
        else:
            h = ops.linear_residual(y, self.mixer.out_weight, stream, *after)
        if last:
            return h
        return ops.linear_residual(self.mlp(h), self.mlp.out_weight, stream, self.norm2b, pre, add_start)


class HybridLMHeadModel(GreedyDecoding, nn.Module):
    decode_period = 8  # steps per captured graph

    def __init__(self, config: HybridConfig, device=None, dtype=torch.bfloat16):
        super().__init__()
        assert dtype in (torch.bfloat16, torch.float32), "weights and activations in bf16 or fp32"
        self.config = config
        width = padded(config.width)
        self.embeddings = nn.Parameter(torch.zeros(config.vocab, width, dtype=dtype, device=device), requires_grad=False)
        self.layers = nn.ModuleList([HybridBlock(s, config.width, config.norm_eps, dtype=dtype, device=device)
                                     for s in config.layers])
        self.final_norm = DynamicTanh(config.width, device=device)
        self.lm_head = nn.Parameter(torch.zeros(config.vocab, width, dtype=dtype, device=device), requires_grad=False)
        self.runs = config.runs()
        self.keeps_start = any(again for _, again in self.runs)
        # when a list, every forward appends the residual stream after every layer run
        self.record = None

    def _states(self, inference_params: InferenceParams) -> List[dict]:
        """One cache or state per layer RUN, created on first use."""
        memory = inference_params.key_value_memory_dict
        for key, (i, _) in enumerate(self.runs):
            if key not in memory:
                memory[key] = self.layers[i].mixer.new_state(inference_params.max_sequence_len)
        return [memory[key] for key in range(len(self.runs))]

    @torch.no_grad()
    def forward(self, input_ids, position_ids=None, inference_params=None, last_token_only=False, rows=None):
        """input_ids (1, n): the next n tokens of the sequence whose state ``inference_params`` holds, at position
        ``sequence_len_offset`` (``lengths_per_sample``, when set, holds it on the device for one-token steps).  The
        caller moves the offset on.  Returns CausalLMOutput(logits (1, rows, vocab) fp32) of all tokens, the last one,
        or the places in ``rows``; None for an empty ``rows``."""
        assert input_ids.dim() == 2 and input_ids.shape[0] == 1, "one sequence per call"
        n = input_ids.shape[1]
        ip = inference_params
        if ip is None:
            ip = InferenceParams(max_sequence_len=n, max_batch_size=1)
        pos = ip.sequence_len_offset
        assert pos + n <= ip.max_sequence_len, "the sequence does not fit its memory"
        step = StepInfo(pos, ip.lengths_per_sample if n == 1 else None)
        states = self._states(ip)
        stream, h = ops.embed(input_ids.reshape(-1), self.embeddings, self.layers[self.runs[0][0]].norm1,
                              self.keeps_start)
        for key, (i, _) in enumerate(self.runs):
            if key + 1 < len(self.runs):
                following, again = self.runs[key + 1]
                pre = self.layers[following].norm1
            else:
                pre, again = self.final_norm, False
            if self.record is None:
                h = self.layers[i](h, stream, states[key], step, pre, again)
            else:
                self.layers[i](h, stream, states[key], step, None)
                self.record.append(stream.x[:, :self.config.width].clone())
                h = ops.residual(None, stream, None, pre, again)
        if rows is not None:
            if len(rows) == 0:
                return CausalLMOutput(logits=None)
            if list(rows) != list(range(n)):
                h = h[torch.as_tensor(rows, device=h.device)]
        elif last_token_only:
            h = h[-1:]
        return CausalLMOutput(logits=ops.linear(h, self.lm_head, f32=True)[None])

    # ---- generation -----------------------------------------------------------------
    def vocab_rows(self):
        return self.config.vocab

    def step_graph_key(self, position_in_period):
        return 0  # every decode step is alike

    def advance(self, logits_row, cache):
        ops.greedy_advance(logits_row, cache.token, cache.position, cache.seq_pos, cache.sequences, cache.out_index,
                           cache.scores, cache.score_index)
