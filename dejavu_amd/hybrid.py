"""Decoders whose layers differ in how they mix tokens (attention of several kinds, recurrences).

Two families are registered.  ``Vimulorn``: one residual stream between sandwich dynamic-tanh norms (before and after
every sublayer), a clamped gated feed-forward, and optionally a stretch of layers that runs several times with the same
weights, where every pass but the first adds the embedding output again and every pass keeps its own cache or state.
``Varolorn``: several residual streams that every sublayer reads as a weighted sum and joins through a matrix, RMS norms
before the sublayers, a relu-gated feed-forward, an embedding of every token with its predecessor, and a head that is
the embedding table.

A layer is: h -> mixer -> output projection (with what the residual does and the next norm behind it) -> feed-forward ->
down projection (likewise).  At decode no norm has a launch of its own.
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
from .mixers import (ChannelDelta, ChunkAttention, ClampedGLU, DynamicTanh, HyperConnection, LatentAttention, Mamba2,
                     ReluGLU, RMSNorm, StepInfo, WindowAttention)


@dataclass
class LayerSpec:
    """One layer: the kind of mixer with its sizes, and the feed-forward (None: the layer has none)."""

    type: str
    mixer: dict
    mlp: Optional[dict] = None


@dataclass
class EmbeddingSpec:
    """embed[token] scale + bigram[(previous mul_prev + token mul_cur) mod buckets]; buckets 0: no second table."""

    scale: float = 1.0
    buckets: int = 0
    mul_prev: int = 0
    mul_cur: int = 0


@dataclass
class HybridConfig:
    width: int
    vocab: int
    layers: List[LayerSpec]
    norm_eps: float = 1e-5
    loop: Optional[Tuple[int, int, int]] = None  # layers start .. stop - 1 run `times` times
    streams: Optional[int] = None                # None: one stream and sandwich norms; else that many, pre-norm
    embedding: Optional[EmbeddingSpec] = None    # of models with streams; their head is the embedding table

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

    @classmethod
    def from_dict_streams(cls, config: dict, shapes: Optional[Dict[str, tuple]] = None) -> "HybridConfig":
        """The same for models with several residual streams (Varolorn)."""
        shapes = shapes or {}

        def size(name, axis=0):
            return shapes[name][axis] if name in shapes else None

        layers, values = [], "first"
        for i, entry in enumerate(config["layers"]):
            kind, mix, mlp, pre = entry["type"], dict(entry["mixer"]), entry.get("mlp"), f"l{i}.mix."
            if kind == "attention":
                kind = "chunk_attention"
                mix.setdefault("heads", size(pre + "g"))
                mix.setdefault("dim", size(pre + "q.norm"))
                if pre + "k" in shapes:
                    mix.setdefault("kv_heads", size(pre + "k") // mix["dim"])
                    mix.setdefault("vdim", size(pre + "v") // mix["kv_heads"])
                    mix["bias_rows"] = size(pre + "rel")
                mix["chunk"] = (mix.get("mask") or {}).get("size")
                mix["bias_max"] = int(mix["bias_max"])
                mix["values"] = None
                if mix.get("v_mix"):  # the first layer that says so is the source of the others
                    mix["values"], values = values, "mixed"
            elif kind == "mamba2":
                mix.setdefault("heads", size(pre + "A_log"))
                mix.setdefault("conv", size(pre + "conv", 1))
                if pre + "o" in shapes:
                    mix.setdefault("vdim", size(pre + "o", 1) // mix["heads"])
            else:
                raise ValueError(f"layer {i}: unknown mixer {kind!r}")
            if mlp is not None:
                if mlp.get("kind", "dense") != "dense":
                    raise ValueError(f"layer {i}: unknown feed-forward {mlp['kind']!r}")
                mlp = dict(mlp)
                mlp.setdefault("ff", size(f"l{i}.mlp.gate"))
            layers.append(LayerSpec(kind, mix, mlp))
        emb = config.get("embedding") or {}
        big = emb.get("bigram")
        spec = EmbeddingSpec(scale=float(emb.get("scale", 1.0)))
        if big:
            buckets = big.get("buckets", (size("bigram") or 1) - 1)
            spec = EmbeddingSpec(spec.scale, int(buckets), int(big["mul_prev"]), int(big["mul_cur"]))
        return cls(width=config.get("width", size("embed", 1)), vocab=config.get("vocab", size("embed")), layers=layers,
                   norm_eps=float(config["norm"]["eps"]), streams=int(config.get("streams", 1)), embedding=spec)

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
    if spec.type == "chunk_attention":
        return ChunkAttention(width, m["heads"], m["kv_heads"], m["dim"], m["vdim"], m["chunk"], m["scale"],
                              m["bias_rows"], m["bias_max"], m["values"], **kw)
    if spec.type == "mamba2":
        return Mamba2(width, m["heads"], m["groups"], m["vdim"], m["state"], m["conv"], m["norm_groups"], **kw)
    raise ValueError(f"unknown mixer {spec.type!r}")


class HybridBlock(nn.Module):
    """One residual stream, a norm before and after every sublayer."""

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

    @property
    def entry(self):
        """What makes the layer's input of the residual."""
        return self.norm1

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


class StreamsBlock(nn.Module):
    """Several residual streams, a norm before every sublayer."""

    def __init__(self, spec: LayerSpec, width: int, eps: float, streams: int, dtype=None, device=None):
        super().__init__()
        self.norm1, self.hyper1 = RMSNorm(width, eps, device=device), HyperConnection(streams, device=device)
        self.mixer = create_mixer(spec, width, eps, dtype=dtype, device=device)
        self.mlp = None
        if spec.mlp is not None:
            self.norm2, self.hyper2 = RMSNorm(width, eps, device=device), HyperConnection(streams, device=device)
            self.mlp = ReluGLU(width, spec.mlp["ff"], dtype=dtype, device=device)

    @property
    def entry(self):
        return ops.StreamRead(self.norm1, self.hyper1.weights)

    def forward(self, h, stream: ops.HyperStream, state: dict, step: StepInfo, following, add_start: bool = False):
        """h: this layer's ``entry`` of the streams.  Both sublayers join the streams; returns ``following`` of them."""
        assert not add_start
        middle = following if self.mlp is None else ops.StreamRead(self.norm2, self.hyper2.weights)
        h = stream.update(self.mixer(h, state, step), self.mixer.out_weight, self.mixer.out_bias, self.hyper1, middle)
        if self.mlp is None:
            return h
        return stream.update(self.mlp(h), self.mlp.out_weight, None, self.hyper2, following)


class HybridLMHeadModel(GreedyDecoding, nn.Module):
    decode_period = 8  # steps per captured graph

    def __init__(self, config: HybridConfig, device=None, dtype=torch.bfloat16):
        super().__init__()
        assert dtype in (torch.bfloat16, torch.float32), "weights and activations in bf16 or fp32"
        self.config = config
        width = padded(config.width)

        def table(rows):
            return nn.Parameter(torch.zeros(rows, width, dtype=dtype, device=device), requires_grad=False)

        kw = dict(dtype=dtype, device=device)
        self.embeddings = table(config.vocab)
        if config.streams is None:
            self.layers = nn.ModuleList([HybridBlock(s, config.width, config.norm_eps, **kw) for s in config.layers])
            self.final_norm = DynamicTanh(config.width, device=device)
            self.lm_head = table(config.vocab)
        else:
            assert config.loop is None, "one stream only"
            self.bigram = table(config.embedding.buckets + 1) if config.embedding.buckets else None
            self.layers = nn.ModuleList([StreamsBlock(s, config.width, config.norm_eps, config.streams, **kw)
                                         for s in config.layers])
            self.final_norm = RMSNorm(config.width, config.norm_eps, device=device)
            self.register_buffer("_ones", torch.ones(config.streams, device=device), persistent=False)
            self.lm_head = self.embeddings
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

    def _history(self, inference_params: InferenceParams) -> torch.Tensor:
        """The sequence's tokens by position (an embedding reads the one before a portion)."""
        state = inference_params.key_value_memory_dict.setdefault("embedding", {})
        if "tokens" not in state:
            state["tokens"] = torch.zeros(inference_params.max_sequence_len, dtype=torch.long,
                                          device=self.embeddings.device)
        return state["tokens"]

    def _exit(self):
        """What makes the head's input of the residual."""
        return self.final_norm if self.config.streams is None else ops.StreamRead(self.final_norm, self._ones)

    def _embed(self, tokens, ip: InferenceParams, step: StepInfo):
        first = self.layers[self.runs[0][0]].entry
        if self.config.streams is None:
            return ops.embed(tokens, self.embeddings, first, self.keeps_start)
        e = self.config.embedding
        return ops.hyper_embed(tokens, self.embeddings, e.scale, self.bigram, e.mul_prev, e.mul_cur, self._history(ip),
                               step.pos_dev, step.pos, self.config.streams, first)

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
        stream, h = self._embed(input_ids.reshape(-1), ip, step)
        for key, (i, _) in enumerate(self.runs):
            if key + 1 < len(self.runs):
                following, again = self.runs[key + 1]
                pre = self.layers[following].entry
            else:
                pre, again = self._exit(), False
            if self.record is None:
                h = self.layers[i](h, stream, states[key], step, pre, again)
            elif self.config.streams is None:
                self.layers[i](h, stream, states[key], step, None)
                self.record.append(stream.x[:, :self.config.width].clone())
                h = ops.residual(None, stream, None, pre, again)
            else:
                h = self.layers[i](h, stream, states[key], step, pre)
                self.record.append(stream.total()[:, :self.config.width])
        if rows is not None:
            if len(rows) == 0:
                return CausalLMOutput(logits=None)
            if list(rows) != list(range(n)):
                h = h[torch.as_tensor(rows, device=h.device)]
        elif last_token_only and n > 1:
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
