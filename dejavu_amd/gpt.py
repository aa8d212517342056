"""Decoder-only model around the sparse blocks, and greedy generation.

Mirrors the data flow of the reference's model wrapper
(Dejavu/src/models/gpt_dejavu.py:168-380 create_mixer_cls / create_mlp_cls /
create_block, :462-623 GPTModel, :626-700 GPTLMHeadModel): embeddings, blocks
that hand their predictions (``next_mlp_sp_logit``, ``next_att_idx``) to the next
block, a final add + LayerNorm and an lm_head tied to the word embeddings.  The
first block receives no prediction and therefore runs dense, as in the
reference.

``generate`` is the shared greedy loop (generation.py); a decode step's host-side state is the position inside the
16-token back-fill window, so a captured period is one window.
"""
from __future__ import annotations

import math
from dataclasses import dataclass, field
from functools import partial
from typing import List, Optional

import torch
import torch.nn as nn
import torch.nn.functional as F

from . import modules as dv_modules
from . import fused_layer, ops
from .block import BlockDejavu, BlockMlpAttSparse
from .generation import (CausalLMOutput, GreedyDecoding,  # noqa: F401
                         GreedySearchDecoderOnlyOutput)
from .modules import ParallelFusedMLPDejavu, ParallelMHADejavu, ParallelMHASparseAttMlp, decode_linear


@dataclass
class SparseGPTConfig:
    """The fields of the reference's GPT2Config (+ sparsity attributes set in
    Dejavu/benchmarks/benchmark_generation_opt_dejavu.py:77-105) that the model reads."""

    hidden_size: int
    num_attention_heads: int
    num_hidden_layers: int
    vocab_size: int
    n_inner: Optional[int] = None
    max_position_embeddings: int = 2048
    layer_norm_epsilon: float = 1e-5
    activation_function: str = "relu"
    scale_attn_weights: bool = True
    scale_attn_by_inverse_layer_idx: bool = False
    initializer_range: float = 0.02
    pad_vocab_size_multiple: int = 1
    mlp_sparse: bool = True
    mlp_K: int = 0
    mlp_sp_dim: int = 1000
    att_sparse: bool = True
    att_K: List[int] = field(default_factory=lambda: [0, 0])
    att_sp_dim: int = 1000

    @property
    def n_embd(self):
        return self.hidden_size


def create_mixer_cls(config, layer_idx=None, process_group=None, device=None, dtype=None):
    """Dejavu/src/models/gpt_dejavu.py:168-255."""
    head_dim = getattr(config, "head_dim", config.hidden_size // config.num_attention_heads)
    softmax_scale = 1.0 if not config.scale_attn_weights else head_dim ** (-0.5)
    if config.scale_attn_by_inverse_layer_idx:
        assert layer_idx is not None
        softmax_scale /= float(layer_idx + 1)
    common = dict(num_heads=config.num_attention_heads, process_group=process_group, softmax_scale=softmax_scale,
                  causal=True, layer_idx=layer_idx, sequence_parallel=False, device=device, dtype=dtype)
    if getattr(config, "att_sparse", False):
        att_ks = config.att_K
        # the last third of the layers uses att_K[0], the others att_K[1]
        l1 = int(0.35 * config.num_hidden_layers)
        l2 = int(0.65 * config.num_hidden_layers)
        att_k = att_ks[0] if (l1 <= layer_idx and layer_idx >= l2) else att_ks[1]
        sp_kwargs = {"embed_dim": config.hidden_size, "low_rank_dim": config.att_sp_dim,
                     "out_dim": config.num_attention_heads, "K": att_k}
        return partial(ParallelMHASparseAttMlp, sp_kwargs=sp_kwargs, **common)
    return partial(ParallelMHADejavu, **common)


def create_mlp_cls(config, layer_idx=None, process_group=None, device=None, dtype=None):
    """Dejavu/src/models/gpt_dejavu.py:257-331 (sparse MLP case)."""
    inner_dim = config.n_inner if config.n_inner is not None else 4 * config.hidden_size
    assert getattr(config, "mlp_sparse", False), "this model is built around the sparse MLP"
    assert config.activation_function in ["relu", "gelu_approx", "gelu_new", "gelu_fast"]
    activation = "relu" if config.activation_function == "relu" else "gelu_approx"
    sp_kwargs = {"embed_dim": config.hidden_size, "low_rank_dim": config.mlp_sp_dim, "out_dim": inner_dim,
                 "K": config.mlp_K}
    return partial(ParallelFusedMLPDejavu, hidden_features=inner_dim, sp_kwargs=sp_kwargs, activation=activation,
                   layer_idx=layer_idx, process_group=process_group, sequence_parallel=False, device=device,
                   dtype=dtype)


def create_block(config, layer_idx=None, process_group=None, device=None, dtype=None):
    """Dejavu/src/models/gpt_dejavu.py:333-380."""
    mixer_cls = create_mixer_cls(config, layer_idx, process_group=process_group, device=device, dtype=dtype)
    mlp_cls = create_mlp_cls(config, layer_idx, process_group=process_group, device=device, dtype=dtype)
    norm_cls = partial(nn.LayerNorm, eps=config.layer_norm_epsilon, device=device, dtype=dtype)
    if getattr(config, "att_sparse", False):
        block = BlockMlpAttSparse(config.hidden_size, mixer_cls, mlp_cls, norm_cls=norm_cls, prenorm=True)
    else:
        block = BlockDejavu(config.hidden_size, mixer_cls, mlp_cls, norm_cls=norm_cls, prenorm=True)
    block.layer_idx = layer_idx
    return block


class GPT2Embeddings(nn.Module):
    """Word + learned position embeddings (what the reference takes from
    flash_attn.modules.embedding, gpt_dejavu.py:489-496)."""

    def __init__(self, embed_dim, vocab_size, max_position_embeddings, device=None, dtype=None):
        super().__init__()
        self.word_embeddings = nn.Embedding(vocab_size, embed_dim, device=device, dtype=dtype)
        self.max_position_embeddings = max_position_embeddings
        self.position_embeddings = nn.Embedding(max_position_embeddings, embed_dim, device=device, dtype=dtype)

    def forward(self, input_ids, position_ids=None):
        """input_ids: (B, s); position_ids: (B, s) or None for 0..s-1."""
        embeddings = self.word_embeddings(input_ids)
        if position_ids is None:
            position_ids = torch.arange(input_ids.shape[1], dtype=torch.long, device=input_ids.device)
        return embeddings + self.position_embeddings(position_ids)


class GPTModel(nn.Module):
    def __init__(self, config, process_group=None, device=None, dtype=None):
        super().__init__()
        assert process_group is None, "this build runs the model on one GPU"
        self.config = config
        pad = getattr(config, "pad_vocab_size_multiple", 1)
        vocab_size = math.ceil(config.vocab_size / pad) * pad
        self.embeddings = GPT2Embeddings(config.hidden_size, vocab_size, config.max_position_embeddings,
                                         device=device, dtype=dtype)
        self.layers = nn.ModuleList([create_block(config, layer_idx=i, device=device, dtype=dtype)
                                     for i in range(config.num_hidden_layers)])
        self.ln_f = nn.LayerNorm(config.hidden_size, eps=config.layer_norm_epsilon, device=device, dtype=dtype)
        # every block's hidden_states go straight into the next add + LayerNorm (the next block's, or ln_f):
        # at a batched decode step the split reduction of fc2 runs in that launch
        for layer in self.layers:
            if hasattr(layer, "defer_mlp_reduce"):
                layer.defer_mlp_reduce = True
        self.sparse = bool(getattr(config, "mlp_sparse", False) or getattr(config, "att_sparse", False))
        self.att_sparse = bool(getattr(config, "att_sparse", False))
        # when a list, every decode forward appends, per block, the lookahead inputs it
        # consumed: (head_idx, mlp_sp_logit) clones (None for the first block)
        self.record = None
        # when a list (together with `record`), every decode forward also appends, per block, the MLP
        # neurons the block selected (None for a block without a selection)
        self.record_mlp_idx = None
        # False: every block through its own forward (one fused call per block)
        self.chain_layers = True

    def forward(self, input_ids, position_ids=None, inference_params=None):
        """Dejavu/src/models/gpt_dejavu.py:552-623."""
        hidden_states = self.embeddings(input_ids, position_ids=position_ids)
        residual = None
        mixer_kwargs = {}
        if inference_params is not None:
            mixer_kwargs["inference_params"] = inference_params
        # attention idx & mlp logit are passed on to the next layer
        next_mlp_sp_logit = None
        next_att_idx = None
        # Consecutive head-sparse decode steps go through ONE call (fused_layer.LayerChain: the launch
        # that ends a block also prepares the next one).  Not while recording: the record clones each
        # block's inputs when the block is reached, and a chain only enqueues them at its end.
        chain = None
        chaining = (self.chain_layers and self.att_sparse and self.record is None and input_ids.shape[1] == 1
                    and input_ids.shape[0] == 1)
        for layer in self.layers:
            if self.record is not None and input_ids.shape[1] == 1:
                dv_modules.join_side_stream()  # the predictions of the block before may be pending on the side stream
                self.record.append((None if next_att_idx is None else next_att_idx.clone(),
                                    None if next_mlp_sp_logit is None else next_mlp_sp_logit.clone()))
            if chaining and getattr(layer, "use_fused_layer", False) and fused_layer.eligible(
                    layer, hidden_states, residual, next_att_idx, next_mlp_sp_logit, inference_params):
                if chain is None:
                    chain = fused_layer.LayerChain()
                    outs = chain.add(layer, next_att_idx, next_mlp_sp_logit, inference_params, hidden_states, residual)
                else:
                    outs = chain.add(layer, next_att_idx, next_mlp_sp_logit, inference_params)
                hidden_states, residual, next_mlp_sp_logit, next_att_idx = outs[0], outs[1], outs[2].view(-1), outs[3]
                continue
            if chain is not None:
                chain.run()
                chain = None
            if self.att_sparse:
                hidden_states, residual, next_mlp_sp_logit, next_att_idx = layer(
                    hidden_states, residual, head_idx=next_att_idx, mlp_sp_logit=next_mlp_sp_logit,
                    mixer_kwargs=mixer_kwargs)
            else:
                hidden_states, residual, next_mlp_sp_logit = layer(
                    hidden_states, residual, mlp_sp_logit=next_mlp_sp_logit, mixer_kwargs=mixer_kwargs)
            if self.record is not None and self.record_mlp_idx is not None and input_ids.shape[1] == 1:
                idx = getattr(layer, "last_mlp_idx", None)
                self.record_mlp_idx.append(None if idx is None else idx.clone())
        if chain is not None:
            chain.run()
        if hidden_states.is_cuda and hidden_states.dtype == torch.float16:
            hidden_states, _ = ops.add_layer_norm(hidden_states, residual, self.ln_f.weight, self.ln_f.bias,
                                                  self.ln_f.eps)
        else:
            residual = hidden_states + residual if residual is not None else hidden_states
            hidden_states = self.ln_f(residual.to(dtype=self.ln_f.weight.dtype))
        return hidden_states


class GPTLMHeadModel(GreedyDecoding, nn.Module):
    decode_period = ParallelMHASparseAttMlp.WINDOW
    decode_warm_steps = ParallelMHASparseAttMlp.WINDOW

    def __init__(self, config, process_group=None, device=None, dtype=None):
        super().__init__()
        assert process_group is None, "this build runs the model on one GPU"
        self.config = config
        self.transformer = GPTModel(config, device=device, dtype=dtype)
        pad = getattr(config, "pad_vocab_size_multiple", 1)
        vocab_size = math.ceil(config.vocab_size / pad) * pad
        self.lm_head = nn.Linear(config.hidden_size, vocab_size, bias=False, device=device, dtype=dtype)
        self.tie_weights()

    def tie_weights(self):
        self.lm_head.weight = self.transformer.embeddings.word_embeddings.weight

    def forward(self, input_ids, position_ids=None, inference_params=None, last_token_only=False):
        """Returns CausalLMOutput(logits (B, s, vocab)).  ``last_token_only`` computes
        the logits of the final position only (all that generation reads)."""
        hidden_states = self.transformer(input_ids, position_ids=position_ids, inference_params=inference_params)
        if last_token_only:
            hidden_states = hidden_states[:, -1:]
        return CausalLMOutput(logits=decode_linear(self.lm_head, hidden_states.contiguous()))

    # ---- generation ---------------------------------------------------------------
    def _sparse_mixers(self):
        return [layer.mixer for layer in self.transformer.layers if isinstance(layer.mixer, ParallelMHASparseAttMlp)]

    def max_positions(self):
        return self.transformer.embeddings.max_position_embeddings

    def vocab_rows(self):
        return self.lm_head.weight.shape[0]

    @property
    def score_dtype(self):
        return self.lm_head.weight.dtype

    def advance(self, logits_row, cache):
        ops.greedy_advance(logits_row, cache.token, cache.position, cache.seq_pos, cache.sequences, cache.out_index,
                           cache.scores, cache.score_index)

    def host_state(self):
        return [m.counter for m in self._sparse_mixers()]

    def set_host_state(self, state):
        for m, v in zip(self._sparse_mixers(), state):
            m.counter = v

    def end_of_step(self):
        dv_modules.join_side_stream()
