"""Greedy generation, shared by the model families (batch 1).

``GreedyDecoding`` restates the greedy loop the reference reaches through ``model.generate`` (flash-attention v0.2.8
``flash_attn/utils/generation.py``, call site Dejavu/benchmarks/benchmark_generation_opt_dejavu.py:187-196).  With
``cg=True`` a decode step (all layers, head, argmax and the bookkeeping of token / position / sequence length) is
replayed from HIP graphs: the values that change from token to token live in device buffers, and what a step depends
on beside them (host state such as the position inside a back-fill window) selects the graph: one graph holds a whole
period of steps, and single-step graphs serve the tokens before the first and after the last whole period.
"""
from __future__ import annotations

from collections import namedtuple
from typing import Optional

import torch

from .inference import InferenceParams

CausalLMOutput = namedtuple("CausalLMOutput", ["logits"])
GreedySearchDecoderOnlyOutput = namedtuple("GreedySearchDecoderOnlyOutput", ["sequences", "scores"])


class DecodingCache:
    """Buffers and graphs of a generation session (batch 1), kept on the model between
    ``generate`` calls of the same maximum length."""

    def __init__(self, max_length, device):
        self.max_length = max_length
        self.inference_params = InferenceParams(max_sequence_len=max_length, max_batch_size=1)
        # device-resident per-token state
        self.token = torch.zeros(1, 1, dtype=torch.long, device=device)
        self.position = torch.zeros(1, 1, dtype=torch.long, device=device)
        self.seq_pos = torch.zeros(1, dtype=torch.int32, device=device)  # == lengths_per_sample
        self.out_index = torch.zeros(1, dtype=torch.long, device=device)    # column of `sequences` to write
        self.score_index = torch.zeros(1, dtype=torch.long, device=device)  # row of `scores` to write
        self.sequences = torch.zeros(1, max_length, dtype=torch.long, device=device)
        self.scores = None
        self.graphs = {}
        self.host_state_after = {}


class GreedyDecoding:
    """Mixin: ``generate`` on top of ``forward(input_ids, position_ids, inference_params, last_token_only)``."""

    decode_period = 1     # decode steps after which the host state repeats; captured as one graph
    decode_warm_steps = 1  # eager steps before the first capture (they create what later steps reuse)
    score_dtype = torch.float32
    _decoding_cache: Optional[DecodingCache] = None

    # ---- what a family defines ------------------------------------------------------
    def max_positions(self) -> Optional[int]:
        """Longest sequence the model's positions allow (None: no limit)."""
        return None

    def vocab_rows(self) -> int:
        raise NotImplementedError

    def advance(self, logits_row, cache: DecodingCache) -> None:
        """Argmax and the device bookkeeping of one token, in one launch."""
        raise NotImplementedError

    def step_graph_key(self, position_in_period: int):
        """Steps with the same key may be replayed from the same single-step graph."""
        return position_in_period

    def host_state(self):
        """Host state that a decode step moves on (kept beside its graph)."""
        return None

    def set_host_state(self, state) -> None:
        pass

    def end_of_step(self) -> None:
        """Joins work that a step left on other streams (before a capture ends)."""

    # ---- the loop -------------------------------------------------------------------
    def _decode_step(self, cache: DecodingCache, vocab_size: Optional[int]):
        """One token: forward at the device-resident position, argmax, bookkeeping.
        Everything is enqueued; nothing is read back."""
        logits = self(cache.token, position_ids=cache.position, inference_params=cache.inference_params).logits[:, -1]
        if vocab_size is not None:
            logits = logits[..., :vocab_size]
        self.advance(logits[0].contiguous(), cache)

    def _replay(self, cache, key, steps, vocab_size):
        ip = cache.inference_params
        if key not in cache.graphs:
            offset = ip.sequence_len_offset
            g = torch.cuda.CUDAGraph()
            with torch.cuda.graph(g):
                for _ in range(steps):
                    self._decode_step(cache, vocab_size)
                    self.end_of_step()
                    ip.sequence_len_offset += 1
            ip.sequence_len_offset = offset
            cache.graphs[key] = g
            cache.host_state_after[key] = self.host_state()
        cache.graphs[key].replay()
        self.set_host_state(cache.host_state_after[key])

    @torch.no_grad()
    def generate(self, input_ids, max_length, top_k=1, top_p=0.0, temperature=1.0, fused_ft_kernel=True, cg=False,
                 vocab_size=None, return_dict_in_generate=False, output_scores=False, timing=False, **kwargs):
        """Greedy decoding of ``max_length - input_ids.shape[1]`` tokens (batch 1).

        Returns the (1, max_length) sequences, or GreedySearchDecoderOnlyOutput(sequences,
        scores) with ``return_dict_in_generate``; scores is a (new tokens, vocab) tensor
        when ``output_scores``."""
        assert top_k == 1 and top_p == 0.0, "greedy decoding only"
        assert fused_ft_kernel, "the decode kernels work on the packed cache layouts"
        batch_size, seqlen_og = input_ids.shape
        assert batch_size == 1, "one sequence: the layers keep one window / state"
        limit = self.max_positions()
        assert seqlen_og < max_length and (limit is None or max_length <= limit)
        device = input_ids.device
        cache = self._decoding_cache
        if cache is None or cache.max_length != max_length:
            cache = self._decoding_cache = DecodingCache(max_length, device)
        n_new = max_length - seqlen_og
        vocab = self.vocab_rows() if vocab_size is None else vocab_size
        if output_scores and (cache.scores is None or cache.scores.shape != (max_length, vocab)):
            # sized for the longest run so that captured steps do not depend on the prompt length
            cache.scores = torch.zeros(max_length, vocab, dtype=self.score_dtype, device=device)
            cache.graphs.clear()
        elif not output_scores and cache.scores is not None:
            cache.scores = None
            cache.graphs.clear()
        if getattr(cache, "graph_key", None) != (vocab_size, bool(output_scores)):
            cache.graphs.clear()  # captured steps hold the logits slice and the score buffer of their run
            cache.graph_key = (vocab_size, bool(output_scores))
        ip = cache.inference_params

        # prompt: fills the caches
        ip.restart()
        logits = self(input_ids, inference_params=ip, last_token_only=True).logits[:, -1]
        if vocab_size is not None:
            logits = logits[..., :vocab_size]
        cache.sequences[:, :seqlen_og] = input_ids
        next_token = logits.argmax(dim=-1, keepdim=True)
        cache.token.copy_(next_token)
        cache.sequences[:, seqlen_og:seqlen_og + 1] = next_token
        if cache.scores is not None:
            cache.scores[0] = logits[0]
        cache.position.fill_(seqlen_og)
        cache.seq_pos.fill_(seqlen_og)
        cache.out_index.fill_(seqlen_og + 1)
        cache.score_index.fill_(1)
        ip.sequence_len_offset = seqlen_og
        ip.lengths_per_sample = cache.seq_pos

        period, warm = self.decode_period, self.decode_warm_steps
        total = n_new - 1
        step = 0
        while step < total:
            c = step % period  # position inside the period (back-fill window: every sparse mixer's counter)
            key = self.step_graph_key(c)
            count = 1
            if cg and c == 0 and total - step >= period and (step >= warm or "window" in cache.graphs):
                # A whole period is one graph: the gap between two graph launches is paid once per period instead
                # of once per token.  Nothing in it depends on the host: token, position and sequence length live
                # on the device.
                self._replay(cache, "window", period, vocab_size)
                count = period
            elif cg and (step >= warm or key in cache.graphs):
                # captured once such a step has run eagerly; later generations replay from their first decode step on
                self._replay(cache, key, 1, vocab_size)
            else:
                self._decode_step(cache, vocab_size)
            ip.sequence_len_offset += count
            step += count
        sequences = cache.sequences.clone()
        if return_dict_in_generate:
            return GreedySearchDecoderOnlyOutput(sequences=sequences,
                                                 scores=None if cache.scores is None else cache.scores[:n_new].clone())
        return sequences
