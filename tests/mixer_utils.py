"""What the GPU tests of the mixer families share: tensors to and from the device, limits, feeding a model in portions."""
from __future__ import annotations

import numpy as np
import torch

from tests.vimulorn_utils import spread

DTYPES = [torch.float32, torch.bfloat16]
# largest rms difference of a row over the rms of the rows: fp32 rounding; bf16 operands and activations
LIMIT = {torch.float32: 2e-5, torch.bfloat16: 3e-2}
# a single mechanism on its own
OP_LIMIT = {torch.float32: 1e-5, torch.bfloat16: 1.5e-2}


def dev(a, dtype=torch.float32):
    return torch.as_tensor(np.asarray(a), dtype=torch.float32).to(dtype).cuda()


def host(t):
    return t.detach().float().cpu().numpy().astype(np.float64)


def close(got, want, limit, what):
    s = spread(host(got) if torch.is_tensor(got) else got, want)
    print(f"{what}: {s:.2e} (limit {limit:.0e})", flush=True)
    assert s <= limit, what


def feed(model, params, tokens, cuts):
    """Logits of all tokens, given in portions of the sizes in ``cuts`` (the last one repeated)."""
    out, at, i = [], 0, 0
    while at < len(tokens):
        n = min(cuts[min(i, len(cuts) - 1)], len(tokens) - at)
        ids = torch.tensor([tokens[at:at + n]], device="cuda")
        out.append(model(ids, inference_params=params).logits[0])
        params.sequence_len_offset += n
        at, i = at + n, i + 1
    return host(torch.cat(out))
