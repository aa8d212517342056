"""Decode-time state of a sequence, shared by the layers of a model."""
from __future__ import annotations

from dataclasses import dataclass, field
from typing import Dict, List, Optional

import torch


@dataclass
class InferenceParams:
    """Decode-time state shared by the layers (same fields as the
    ``inference_params`` object the reference's modules read).

    ``key_value_memory_dict`` holds what a layer keeps of a sequence, under the key the layer chooses: (k_cache,
    v_cache) of the OPT layers; a dict of tensors for layers whose state is not only keys and values.  In such a dict
    the names in ``zeroed`` start a sequence as zeros; the others (caches) are only read where they were written."""

    max_sequence_len: int
    max_batch_size: int
    sequence_len_offset: int = 0
    batch_size_offset: int = 0
    key_value_memory_dict: dict = field(default_factory=dict)
    fused_ft_kernel: bool = True
    lengths_per_sample: Optional[torch.Tensor] = None
    zeroed: tuple = ("conv", "S")

    def restart(self) -> None:
        """Position 0 of a new sequence in the same memory."""
        self.sequence_len_offset = 0
        self.lengths_per_sample = None
        for state in self.key_value_memory_dict.values():
            if isinstance(state, dict):
                for name in self.zeroed:
                    if name in state:
                        state[name].zero_()


class SequencePool:
    """Memory of live sequences by name: taken when a name is first seen, given back when it ends and then used
    again by the next new name."""

    def __init__(self, max_sequence_len: int):
        self.max_sequence_len = max_sequence_len
        self.live: Dict[str, InferenceParams] = {}
        self.free: List[InferenceParams] = []

    def get(self, name: str) -> InferenceParams:
        if name not in self.live:
            params = self.free.pop() if self.free else InferenceParams(self.max_sequence_len, max_batch_size=1)
            params.restart()
            self.live[name] = params
        return self.live[name]

    def end(self, name: str) -> None:
        params = self.live.pop(name, None)
        if params is not None:
            self.free.append(params)
