"""ctypes binding of libdejavu_mixers.so (the C ABI declared in include/dejavu_mixers.h)."""
from __future__ import annotations

import ctypes
import os

from ._binding import DejavuHipError, load_library

LIB_PATH = os.path.join(os.path.dirname(os.path.abspath(__file__)), "libdejavu_mixers.so")

BF16, F32 = 0, 1
ROW_PLAIN, ROW_RMS, ROW_HEADS, ROW_GROUPS = 0, 1, 2, 3
OUT_F32, OUT_T, OUT_GLU, OUT_RESIDUAL, OUT_CONV, OUT_HYPER = 0, 1, 2, 3, 4, 5
GLU_CLAMPED, GLU_RELU = 0, 1
HYPER_MAX, HYPER_ROW_MAX = 16, 4

_i = ctypes.c_int
_l = ctypes.c_int64
_p = ctypes.c_void_p
_f = ctypes.c_float


def _struct(name, *fields):
    return type(name, (ctypes.Structure,), {"_fields_": list(fields)})


# Mirrors of the structs in the header (same field order).
DynTanh = _struct("DynTanh", ("w", _p), ("b", _p), ("alpha", _f))
Residual = _struct("Residual", ("x", _p), ("x0", _p), ("h", _p), ("post", DynTanh), ("pre", DynTanh))
Hyper = _struct("Hyper", ("x", _p), ("mix", _p), ("out", _p), ("in_", _p), ("u", _p), ("streams", _i), ("width", _i))
RmsOut = _struct("RmsOut", ("w", _p), ("eps", _f), ("dim", _i), ("h", _p))
RowArgs = _struct("RowArgs", ("x", _p), ("W", _p), ("ldw", _l), ("M", _i), ("K", _i), ("xw", _p), ("gate", _p),
                  ("eps", _f), ("norm_dim", _i), ("head_stride", _i), ("x_dim", _i), ("bias", _p), ("out", _p),
                  ("act", _i), ("limit", _f), ("res", Residual), ("hyper", Hyper), ("conv_w", _p), ("conv_b", _p),
                  ("conv_state", _p), ("conv_rows", _i), ("taps", _i), ("silu", _i),
                  ("side_x", _p), ("side_w", _p), ("side_out", _p), ("side_ld", _l), ("side_dim", _i),
                  ("side_padded", _i), ("pos_dev", _p), ("pos_host", _i))
TileArgs = _struct("TileArgs", ("x", _p), ("ldx", _l), ("W", _p), ("ldw", _l), ("n", _i), ("M", _i), ("K", _i),
                   ("bias", _p), ("out", _p), ("ldo", _l), ("act", _i), ("limit", _f), ("res", Residual))
ConvGroup = _struct("ConvGroup", ("heads", _i), ("stride", _i), ("dim", _i), ("norm", _i), ("eps", _f), ("scale", _f),
                    ("out", _p), ("ld", _l))
ConvArgs = _struct("ConvArgs", ("in_", _p), ("ldi", _l), ("n", _i), ("taps", _i), ("silu", _i), ("w", _p),
                   ("b", _p), ("state", _p), ("g", ConvGroup * 3))
HeadGroup = _struct("HeadGroup", ("heads", _i), ("stride", _i), ("dim", _i), ("w", _p), ("eps", _f), ("other", _p),
                    ("ldo", _l), ("lambda", _p), ("out", _p), ("ld", _l))
HeadArgs = _struct("HeadArgs", ("in_", _p), ("ldi", _l), ("n", _i), ("g", HeadGroup * 3))
AttnArgs = _struct("AttnArgs", ("q", _p), ("ldq", _l), ("k", _p), ("ldk", _l), ("k_head", _l), ("v", _p), ("ldv", _l),
                   ("v_head", _l), ("n", _i), ("H", _i), ("G", _i), ("dim_s", _i), ("vdim_s", _i), ("scale", _f),
                   ("sink", _p), ("gate", _p), ("ldg", _l), ("window", _i), ("chunk", _i),
                   ("rel", _p), ("rel_len", _i), ("ring", _i), ("base", _i),
                   ("pos_dev", _p), ("pos_host", _i), ("out", _p), ("part", _p), ("splits", _i), ("fresh_k", _p),
                   ("fresh_v", _p), ("norm_dim", _i), ("eps", _f), ("q_w", _p), ("k_w", _p), ("other_v", _p),
                   ("lambda", _p))
DeltaArgs = _struct("DeltaArgs", ("q", _p), ("k", _p), ("v", _p), ("g", _p), ("beta", _p), ("S", _p), ("o", _p),
                    ("tm", _p), ("tm_floats", _l), ("n", _i), ("heads", _i), ("kv_heads", _i), ("dim_s", _i), ("vdim_s", _i))
DeltaStepArgs = _struct("DeltaStepArgs", ("p", _p), ("off_k", _i), ("off_v", _i), ("off_b", _i), ("off_a", _i),
                        ("off_g", _i), ("heads", _i), ("kv_heads", _i), ("dim", _i), ("dim_s", _i), ("vdim_s", _i),
                        ("Wa", _p), ("Wg", _p), ("rank_a", _i), ("rank_g", _i), ("A_log", _p), ("dt_bias", _p),
                        ("S", _p), ("o", _p), ("gate", _p))
SsdArgs = _struct("SsdArgs", ("xbc", _p), ("ld", _l), ("off_b", _i), ("off_c", _i), ("dt", _p), ("lddt", _l),
                  ("A_log", _p), ("dt_bias", _p), ("D", _p), ("S", _p), ("y", _p), ("ldy", _l), ("tm", _p),
                  ("tm_floats", _l), ("n", _i), ("heads", _i), ("groups", _i), ("vdim", _i), ("state_s", _i))
SsdStepArgs = _struct("SsdStepArgs", ("p", _p), ("off_b", _i), ("off_c", _i), ("off_z", _i), ("off_dt", _i),
                      ("A_log", _p), ("dt_bias", _p), ("D", _p), ("S", _p), ("y", _p), ("heads", _i), ("groups", _i),
                      ("vdim", _i), ("state_s", _i))
EmbedArgs = _struct("EmbedArgs", ("tokens", _p), ("history", _p), ("capacity", _l), ("vocab", _l), ("embed", _p),
                    ("scale", _f), ("bigram", _p), ("buckets", _l), ("mul_prev", _l), ("mul_cur", _l), ("pos_dev", _p),
                    ("pos_host", _i), ("n", _i))

_P = ctypes.POINTER
# name -> (restype, argtypes); one entry per prototype in include/dejavu_mixers.h
SIGNATURES = {
    "dv_mix_embed": (_i, [_i, _p, _l, _p, _i, _i, _p, _p, _P(DynTanh), _p, _p]),
    "dv_mix_residual": (_i, [_i, _p, _l, _i, _P(Residual), _p]),
    "dv_mix_glu": (_i, [_i, _p, _l, _i, _f, _p, _p]),
    "dv_mix_hyper_embed": (_i, [_i, _P(EmbedArgs), _P(Hyper), _P(RmsOut), _p]),
    "dv_mix_hyper_rows": (_i, [_i, _p, _i, _P(Hyper), _P(RmsOut), _p]),
    "dv_mix_head_rows": (_i, [_i, _P(HeadArgs), _p]),
    "dv_mix_gated_group_norm": (_i, [_i, _p, _l, _p, _l, _l, _i, _i, _i, _p, _f, _p, _p]),
    "dv_mix_rms_rows": (_i, [_i, _p, _l, _l, _i, _i, _p, _f, _p, _l, _p]),
    "dv_mix_gated_head_norm": (_i, [_i, _p, _p, _l, _l, _i, _i, _i, _p, _f, _p, _p]),
    "dv_mix_linear_row": (_i, [_i, _i, _i, _P(RowArgs), _p]),
    "dv_mix_linear_tiles": (_i, [_i, _P(TileArgs), _p]),
    "dv_mix_short_conv": (_i, [_i, _i, _P(ConvArgs), _p]),
    "dv_mix_conv_state": (_i, [_i, _p, _l, _i, _i, _i, _p, _p]),
    "dv_mix_ring_copy": (_i, [_i, _p, _l, _p, _i, _l, _i, _i, _i, _i, _p]),
    "dv_mix_attn_rows": (_i, [_i, _i, _P(AttnArgs), _p]),
    "dv_mix_attn_tiles": (_i, [_P(AttnArgs), _i, _p]),
    "dv_mix_latent_absorb": (_i, [_i, _p, _p, _i, _i, _i, _p, _p]),
    "dv_mix_latent_attn": (_i, [_i, _P(AttnArgs), _p, _i, _p, _p]),
    "dv_mix_delta_gates": (_i, [_i, _p, _l, _p, _l, _p, _p, _i, _i, _i, _p, _p, _p]),
    "dv_mix_delta_scan": (_i, [_P(DeltaArgs), _p]),
    "dv_mix_delta_step": (_i, [_i, _P(DeltaStepArgs), _p]),
    "dv_mix_ssd_scan": (_i, [_i, _P(SsdArgs), _p]),
    "dv_mix_ssd_step": (_i, [_P(SsdStepArgs), _p]),
    "dv_mix_greedy_advance": (_i, [_p, _i, _p, _p, _p, _p, _l, _p, _p, _l, _l, _p, _p]),
}

lib = load_library(LIB_PATH, SIGNATURES)

_ERRORS = {-1: "invalid argument", -2: "shape not supported", -3: "misaligned pointer or size",
           -4: "workspace missing or too small", -5: "launch rejected"}


def check(code: int, what: str) -> None:
    if code != 0:
        raise DejavuHipError(f"{what}: {_ERRORS.get(code, 'error')} (code {code})")
