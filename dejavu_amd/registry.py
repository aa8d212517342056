"""Model families by the architecture that a checkpoint's config.json names.

    model = load_model("folder")              # config.json + model.safetensors (or pytorch_model.bin)
    model.generate(ids, max_length=..., cg=True)

A family says how its configuration is read, which class runs it, how checkpoint tensors map to the class's
parameters, which element types it runs in, and which kernel library it needs.
"""
from __future__ import annotations

import json
import os
from dataclasses import dataclass
from typing import Callable, Dict, Optional, Tuple

import torch

from . import build


@dataclass(frozen=True)
class Family:
    libraries: Tuple[str, ...]
    dtypes: Tuple[torch.dtype, ...]   # the first one is the default
    read_config: Callable             # (config dict, {tensor: shape}) -> configuration
    model_class: Callable             # () -> class
    remap: Callable                   # (state dict, configuration) -> the class's state dict
    takes_portions: bool              # prompts may arrive in portions (several tokens at any position)


def _vimulorn_config(config, shapes):
    from .hybrid import HybridConfig

    return HybridConfig.from_dict(config, shapes)


def _hybrid_class():
    from .hybrid import HybridLMHeadModel

    return HybridLMHeadModel


def _vimulorn_remap(state_dict, config):
    from .loaders import remap_state_dict_vimulorn

    return remap_state_dict_vimulorn(state_dict, config)


def _varolorn_config(config, shapes):
    from .hybrid import HybridConfig

    return HybridConfig.from_dict_streams(config, shapes)


def _varolorn_remap(state_dict, config):
    from .loaders import remap_state_dict_varolorn

    return remap_state_dict_varolorn(state_dict, config)


def _opt_config(config, shapes):
    """HuggingFace OPT fields; the sparsity sizes come under the names SparseGPTConfig has (absent: no selection,
    every neuron and head)."""
    from .gpt import SparseGPTConfig

    if not config.get("do_layer_norm_before", True) or config.get("word_embed_proj_dim", config["hidden_size"]) != \
            config["hidden_size"]:
        raise ValueError("OPT variants with post-norm or projected embeddings are not built")
    ffn, heads = config["ffn_dim"], config["num_attention_heads"]
    return SparseGPTConfig(
        hidden_size=config["hidden_size"], num_attention_heads=heads, num_hidden_layers=config["num_hidden_layers"],
        vocab_size=config["vocab_size"], n_inner=ffn, max_position_embeddings=config["max_position_embeddings"],
        activation_function=config.get("activation_function", "relu"),
        pad_vocab_size_multiple=config.get("pad_vocab_size_multiple", 8), mlp_K=config.get("mlp_K", ffn),
        mlp_sp_dim=config.get("mlp_sp_dim", 1000), att_K=list(config.get("att_K", [heads, heads])),
        att_sp_dim=config.get("att_sp_dim", 1000))


def _opt_class():
    from .gpt import GPTLMHeadModel

    return GPTLMHeadModel


def _opt_remap(state_dict, config):
    from .loaders import remap_state_dict_opt

    return remap_state_dict_opt(state_dict, config)


FAMILIES: Dict[str, Family] = {
    "Vimulorn": Family((build.MIXERS_LIB_NAME,), (torch.bfloat16, torch.float32), _vimulorn_config, _hybrid_class,
                       _vimulorn_remap, takes_portions=True),
    "Varolorn": Family((build.MIXERS_LIB_NAME,), (torch.bfloat16, torch.float32), _varolorn_config, _hybrid_class,
                       _varolorn_remap, takes_portions=True),
    "OPTForCausalLM": Family((build.LIB_NAME,), (torch.float16,), _opt_config, _opt_class, _opt_remap,
                             takes_portions=False),
}


def read_config_file(folder: str) -> dict:
    with open(os.path.join(folder, "config.json")) as f:
        return json.load(f)


def family_of(config: dict) -> Tuple[str, Family]:
    names = [config.get("architecture")] + list(config.get("architectures") or [])
    for name in names:
        if name in FAMILIES:
            return name, FAMILIES[name]
    raise ValueError(f"no model family for {[n for n in names if n]}; known: {sorted(FAMILIES)}")


def build_model(config: dict, state_dict, device="cuda", dtype: Optional[torch.dtype] = None):
    """Model of a parsed config.json with the tensors of ``state_dict`` (checkpoint names)."""
    name, family = family_of(config)
    dtype = family.dtypes[0] if dtype is None else dtype
    if dtype not in family.dtypes:
        raise ValueError(f"{name} runs in {family.dtypes}, not {dtype}")
    conf = family.read_config(config, {k: tuple(v.shape) for k, v in state_dict.items()})
    model = family.model_class()(conf, device=device, dtype=dtype)
    missing, unexpected = model.load_state_dict(family.remap(state_dict, conf), strict=False)
    # sparsity predictors may be trained and loaded separately
    missing = [k for k in missing if ".sp." not in k]
    if missing or unexpected:
        raise ValueError(f"checkpoint does not fit {name}: missing {missing[:4]}, unexpected {unexpected[:4]}")
    return model.eval()


def load_model(folder: str, device="cuda", dtype: Optional[torch.dtype] = None):
    """Reads config.json and the weights of a folder; kernels are compiled first if they are not there."""
    from .loaders import load_checkpoint_folder

    config = read_config_file(folder)
    for lib in family_of(config)[1].libraries:
        build.ensure_built(lib)
    return build_model(config, load_checkpoint_folder(folder), device=device, dtype=dtype)
