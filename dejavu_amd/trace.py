"""Replays given tokens through a model, step by step, and writes logits (``bin/trace_run``).

Steps come as JSON lines on standard input:

    {"step": 0, "entries": [{"id": "s1", "tokens": [11, 4, 250, 9], "want": [3]}], "end": []}

An entry brings the next tokens of a sequence (a new id starts one) and the places among them whose logits are wanted.
``OUT/<step>.f32`` gets those logits, little-endian fp32 [wanted, vocab], in the order of the entries and of ``want``;
``done <step>`` on standard output follows every step.  Sequences in ``end`` are finished: their memory is used again.
The forward pass, state and kernels are the ones ``generate`` uses.
"""
from __future__ import annotations

import argparse
import json
import os
import sys

import numpy as np


def run(model, lines, out_dir: str, pool, device="cuda", emit=None) -> None:
    """lines: iterable of JSON texts; emit: called with each line of output."""
    import torch

    emit = emit or (lambda text: print(text, flush=True))
    for line in lines:
        if not line.strip():
            continue
        step = json.loads(line)
        wanted = []
        for entry in step["entries"]:
            tokens, want = entry["tokens"], list(entry.get("want") or [])
            params = pool.get(entry["id"])
            if tokens:
                ids = torch.tensor([tokens], dtype=torch.long, device=device)
                logits = model(ids, inference_params=params, rows=want).logits
                params.sequence_len_offset += len(tokens)
                if want:
                    wanted.append(logits[0].float().cpu().numpy())
        if wanted:
            np.concatenate(wanted).astype("<f4").tofile(os.path.join(out_dir, f"{step['step']}.f32"))
        for name in step.get("end") or []:
            pool.end(name)
        emit(f"done {step['step']}")


def main(argv=None) -> int:
    ap = argparse.ArgumentParser(prog="trace_run", description=__doc__.split("\n", 1)[0])
    ap.add_argument("--model", required=True, help="folder with config.json and model.safetensors")
    ap.add_argument("--dtype", default="bfloat16", choices=["bfloat16", "float32"])
    ap.add_argument("--out", required=True, help="folder for the logits")
    ap.add_argument("--max-tokens", type=int, required=True, help="most tokens that live sequences hold at any time")
    args = ap.parse_args(argv)

    import torch

    from .inference import SequencePool
    from .registry import family_of, load_model, read_config_file

    name, family = family_of(read_config_file(args.model))
    dtype = getattr(torch, args.dtype)
    if dtype not in family.dtypes or not family.takes_portions:
        print(f"{name} does not run given tokens in {args.dtype}", file=sys.stderr)
        return 2
    model = load_model(args.model, device="cuda", dtype=dtype)
    os.makedirs(args.out, exist_ok=True)
    run(model, sys.stdin, args.out, SequencePool(max(1, args.max_tokens)))
    return 0
