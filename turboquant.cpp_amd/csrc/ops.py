"""Python face of the HIP kernels: one function per kernel, on torch tensors that live on the GPU.

Every function checks on the host that shapes, types and strides are what its kernel and launch
grid assume before anything is launched, and raises :class:`KernelError` with the kernel's name
otherwise.  There is no other implementation behind these functions: without a GPU, or without
the compiled library, they raise.
"""
from __future__ import annotations

import ctypes
import dataclasses
import math
import os
import re
import struct

import torch

from . import build as _build


class KernelError(RuntimeError):
    pass


ACT_DTYPES = {"float32": torch.float32, "bfloat16": torch.bfloat16}
# activations of the gate in a gated pair of products: the lines of gates.def, numbered as the kernels number them
with open(os.path.join(os.path.dirname(os.path.abspath(__file__)), "gates.def"), encoding="utf-8") as _f:
    GATES = {name: i for i, name in enumerate(re.findall(r"^TQ_GATE\((\w+),", _f.read(), re.M))}
_WTYPE = {torch.float32: 0, torch.bfloat16: 1}
_LIBS: dict[str, ctypes.CDLL] = {}

_c_int, _c_i64, _c_f32, _c_ptr = ctypes.c_int, ctypes.c_int64, ctypes.c_float, ctypes.c_void_p

_SIGNATURES = {
    "tq_embed": [_c_ptr, _c_ptr, _c_int, _c_ptr, _c_int, _c_int, _c_f32, _c_ptr],
    "tq_softcap": [_c_ptr, _c_i64, _c_f32, _c_ptr],
    "tq_scale_softcap": [_c_ptr, _c_i64, _c_f32, _c_f32, _c_ptr],
    "tq_move_rows": [_c_ptr, _c_ptr, _c_ptr, _c_int, _c_i64, _c_int, _c_ptr],
    "tq_gated_act": [_c_ptr, _c_i64, _c_ptr, _c_int, _c_int, _c_int, _c_ptr],
    "tq_head_rmsnorm": [_c_ptr, _c_ptr, _c_ptr, _c_int, _c_f32, _c_int, _c_int, _c_int, _c_int, _c_int, _c_ptr],
    "tq_add_rmsnorm": [_c_ptr, _c_ptr, _c_int, _c_i64, _c_ptr, _c_ptr, _c_ptr, _c_int, _c_ptr, _c_ptr, _c_int, _c_f32,
                       _c_ptr, _c_int, _c_ptr, _c_ptr, _c_int, _c_ptr],
    "tq_rope_kv_write": [_c_ptr, _c_ptr, _c_int, _c_ptr, _c_ptr, _c_ptr, _c_int, _c_ptr, _c_int, _c_int, _c_ptr, _c_ptr, _c_ptr,
                         _c_int, _c_i64, _c_int, _c_int, _c_int, _c_int, _c_int, _c_ptr, _c_ptr, _c_ptr, _c_int, _c_int,
                         _c_ptr],
    "tq_moe_combine": [_c_ptr, _c_ptr, _c_ptr, _c_int, _c_ptr, _c_int, _c_i64, _c_ptr, _c_ptr, _c_int, _c_int, _c_ptr],
    "tq_gemm_generic": [_c_ptr, _c_i64, _c_ptr, _c_int, _c_ptr, _c_ptr, _c_int, _c_i64, _c_ptr, _c_ptr, _c_ptr, _c_int,
                        _c_ptr, _c_i64, _c_int, _c_int, _c_int, _c_int, _c_int, _c_int, _c_ptr],
    "tq_attention_generic": [_c_ptr, _c_ptr, _c_ptr, _c_ptr, _c_ptr, _c_ptr, _c_int, _c_int, _c_i64, _c_int, _c_int,
                             _c_int, _c_int, _c_int, _c_f32, _c_ptr, _c_ptr],
    "tq_router_topk": [_c_ptr, _c_ptr, _c_ptr, _c_int, _c_int, _c_int, _c_int, _c_ptr, _c_ptr, _c_ptr, _c_ptr, _c_int, _c_int,
                       _c_ptr],
    "tq_moe_align": [_c_ptr, _c_int, _c_int, _c_int, _c_int, _c_int, _c_ptr, _c_ptr, _c_ptr, _c_ptr, _c_ptr],
    "tq_route": [_c_ptr, _c_ptr, _c_ptr, _c_int, _c_int, _c_int, _c_int, _c_ptr, _c_ptr, _c_ptr, _c_ptr, _c_int, _c_int,
                 _c_ptr, _c_ptr, _c_ptr, _c_ptr, _c_int, _c_int, _c_ptr],
    "tq_argmax": [_c_ptr, _c_int, _c_int, _c_ptr, _c_ptr],
    "tq_nll": [_c_ptr, _c_int, _c_int, _c_ptr, _c_ptr, _c_ptr],
    "tq_probs_half": [_c_ptr, _c_int, _c_int, _c_ptr, _c_ptr, _c_ptr, _c_ptr],
    "tq_rep_penalty": [_c_ptr, _c_int, _c_int, _c_ptr, _c_int, _c_ptr, _c_f32, _c_ptr],
    "tq_sample_topp_scratch": [_c_int],
    "tq_embed_pos": [_c_ptr, _c_ptr, _c_ptr, _c_ptr, _c_int, _c_ptr, _c_int, _c_int, _c_f32, _c_ptr],
    "tq_add_normed_rmsnorm": [_c_ptr, _c_ptr, _c_int, _c_i64, _c_ptr, _c_ptr, _c_ptr, _c_int, _c_ptr, _c_ptr, _c_f32, _c_ptr,
                              _c_int, _c_f32, _c_ptr, _c_int, _c_ptr, _c_ptr, _c_int, _c_ptr],
    "tq_add_normed_rmsnorm_shift": [_c_ptr, _c_ptr, _c_int, _c_i64, _c_ptr, _c_ptr, _c_ptr, _c_int, _c_ptr, _c_ptr, _c_f32, _c_ptr,
                                    _c_int, _c_f32, _c_ptr, _c_int, _c_ptr, _c_ptr, _c_int, _c_ptr, _c_ptr, _c_ptr, _c_ptr],
    "tq_attention_generic_mod": [_c_ptr, _c_ptr, _c_ptr, _c_ptr, _c_ptr, _c_ptr, _c_int, _c_int, _c_i64, _c_int, _c_int,
                                 _c_int, _c_int, _c_int, _c_f32, _c_f32, _c_ptr, _c_ptr, _c_int, _c_ptr, _c_ptr, _c_ptr],
    "tq_attention_generic_sig": [_c_ptr, _c_ptr, _c_ptr, _c_ptr, _c_ptr, _c_ptr, _c_int, _c_int, _c_i64, _c_int, _c_int,
                                 _c_int, _c_int, _c_int, _c_f32, _c_f32, _c_ptr, _c_ptr, _c_int, _c_ptr, _c_ptr, _c_int, _c_ptr,
                                 _c_ptr],
    "tq_route_scored": [_c_ptr, _c_ptr, _c_ptr, _c_int, _c_int, _c_int, _c_int, _c_ptr, _c_ptr, _c_ptr, _c_ptr, _c_int, _c_int,
                        _c_ptr, _c_ptr, _c_ptr, _c_ptr, _c_int, _c_int, _c_ptr],
    "tq_token_shift": [_c_ptr, _c_ptr, _c_int, _c_ptr, _c_ptr, _c_ptr, _c_int, _c_ptr, _c_int, _c_int, _c_ptr],
    "tq_value_norm_mix": [_c_ptr, _c_i64, _c_int, _c_int, _c_int, _c_f32, _c_ptr, _c_i64, _c_int, _c_ptr, _c_int, _c_int,
                          _c_ptr],
    "tq_attn_prep_kv_write": [_c_ptr, _c_i64, _c_ptr, _c_ptr, _c_ptr, _c_int, _c_ptr, _c_int, _c_int, _c_f32, _c_ptr, _c_ptr, _c_int,
                              _c_f32, _c_int, _c_f32, _c_int, _c_ptr, _c_i64, _c_int, _c_ptr, _c_ptr, _c_ptr, _c_ptr, _c_int, _c_i64,
                              _c_int, _c_int, _c_int, _c_int, _c_int, _c_ptr, _c_ptr, _c_ptr, _c_int, _c_int, _c_ptr],
    "tq_act_rows": [_c_ptr, _c_i64, _c_ptr, _c_i64, _c_ptr, _c_int, _c_int, _c_int, _c_ptr],
    "tq_gate_rows": [_c_ptr, _c_ptr, _c_i64, _c_ptr, _c_int, _c_int, _c_int, _c_ptr],
    "tq_latent_norm": [_c_ptr, _c_i64, _c_ptr, _c_int, _c_f32, _c_ptr, _c_i64, _c_int, _c_int, _c_int, _c_int, _c_ptr],
    "tq_head_gemm": [_c_ptr, _c_int, _c_i64, _c_ptr, _c_int, _c_ptr, _c_int, _c_i64, _c_ptr, _c_i64, _c_int, _c_int, _c_int,
                     _c_int, _c_int, _c_ptr],
    "tq_delta_prep_h": [_c_ptr, _c_ptr, _c_ptr, _c_i64, _c_ptr, _c_ptr, _c_ptr, _c_int, _c_int, _c_int, _c_int, _c_int, _c_ptr,
                        _c_ptr, _c_ptr, _c_ptr, _c_ptr, _c_int, _c_ptr],
    "tq_delta_scan_h": [_c_ptr, _c_ptr, _c_ptr, _c_ptr, _c_ptr, _c_ptr, _c_ptr, _c_ptr, _c_i64, _c_int, _c_int, _c_int, _c_int,
                        _c_int, _c_int, _c_int, _c_ptr, _c_ptr],
    "tq_delta_out_h": [_c_ptr, _c_ptr, _c_f32, _c_ptr, _c_int, _c_ptr, _c_ptr, _c_ptr, _c_i64, _c_int, _c_int, _c_int, _c_int,
                       _c_int, _c_int, _c_int, _c_ptr, _c_ptr],
    "tq_delta_decode_h": [_c_ptr, _c_ptr, _c_ptr, _c_ptr, _c_ptr, _c_ptr, _c_ptr, _c_f32, _c_ptr, _c_int, _c_ptr, _c_ptr, _c_ptr,
                          _c_i64, _c_int, _c_int, _c_int, _c_int, _c_int, _c_int, _c_ptr, _c_ptr],
    "tq_router_topk_grouped": [_c_ptr, _c_ptr, _c_ptr, _c_int, _c_int, _c_int, _c_int, _c_int, _c_int, _c_ptr, _c_ptr, _c_ptr,
                               _c_ptr, _c_int, _c_int, _c_ptr],
    "tq_route_grouped": [_c_ptr, _c_ptr, _c_ptr, _c_int, _c_int, _c_int, _c_int, _c_int, _c_int, _c_ptr, _c_ptr, _c_ptr, _c_ptr,
                         _c_int, _c_int, _c_ptr, _c_ptr, _c_ptr, _c_ptr, _c_int, _c_int, _c_ptr],
    "tq_delta_state_floats": [_c_int, _c_int, _c_int, _c_int, _c_int],
    "tq_delta_prep": [_c_ptr, _c_ptr, _c_ptr, _c_i64, _c_ptr, _c_int, _c_int, _c_int, _c_int, _c_int, _c_int, _c_int, _c_ptr,
                      _c_ptr, _c_ptr, _c_ptr, _c_ptr, _c_int, _c_ptr],
    "tq_delta_scan": [_c_ptr, _c_ptr, _c_ptr, _c_ptr, _c_ptr, _c_ptr, _c_ptr, _c_ptr, _c_ptr, _c_ptr, _c_i64, _c_int, _c_int,
                      _c_int, _c_int, _c_int, _c_int, _c_int, _c_ptr, _c_ptr],
    "tq_delta_decode": [_c_ptr, _c_ptr, _c_ptr, _c_ptr, _c_ptr, _c_ptr, _c_int, _c_ptr, _c_ptr, _c_ptr, _c_f32, _c_ptr, _c_ptr,
                        _c_ptr, _c_ptr, _c_i64, _c_int, _c_int, _c_int, _c_int, _c_int, _c_int, _c_int, _c_int, _c_ptr, _c_ptr],
    "tq_delta_out": [_c_ptr, _c_ptr, _c_ptr, _c_f32, _c_ptr, _c_ptr, _c_ptr, _c_ptr, _c_i64, _c_int, _c_int, _c_int, _c_int,
                     _c_int, _c_int, _c_int, _c_int, _c_int, _c_ptr, _c_ptr],
    "tq_sample_topp": [_c_ptr, _c_int, _c_int, _c_f32, _c_f32, _c_ptr, _c_ptr, _c_ptr, _c_ptr, _c_ptr],
    "tq_set_pair_limit": [_c_f32],
    "tq_add_terms_rmsnorm": [_c_ptr, _c_ptr, _c_ptr, _c_ptr, _c_int, _c_i64, _c_ptr, _c_ptr, _c_ptr, _c_ptr, _c_int, _c_ptr, _c_int,
                             _c_f32, _c_ptr, _c_int, _c_ptr, _c_ptr, _c_int, _c_ptr],
    "tq_router_topk_sigmoid": [_c_ptr, _c_ptr, _c_ptr, _c_ptr, _c_int, _c_int, _c_int, _c_int, _c_int, _c_int, _c_f32, _c_ptr,
                               _c_ptr, _c_ptr, _c_ptr, _c_int, _c_int, _c_ptr],
    "tq_route_sigmoid": [_c_ptr, _c_ptr, _c_ptr, _c_ptr, _c_int, _c_int, _c_int, _c_int, _c_int, _c_int, _c_f32, _c_ptr, _c_ptr,
                         _c_ptr, _c_ptr, _c_int, _c_int, _c_ptr, _c_ptr, _c_ptr, _c_ptr, _c_int, _c_int, _c_ptr],
    "tq_mm_scan": [_c_ptr, _c_i64, _c_ptr, _c_f32, _c_ptr, _c_ptr, _c_ptr, _c_i64, _c_int, _c_int, _c_int, _c_int, _c_ptr, _c_ptr,
                   _c_ptr, _c_ptr],
    "tq_mm_chunked": [_c_ptr, _c_i64, _c_ptr, _c_f32, _c_ptr, _c_ptr, _c_ptr, _c_i64, _c_int, _c_int, _c_int, _c_int, _c_int,
                      _c_ptr, _c_ptr, _c_int, _c_ptr, _c_ptr, _c_ptr],
    "tq_mm_out": [_c_ptr, _c_ptr, _c_ptr, _c_i64, _c_ptr, _c_int, _c_f32, _c_ptr, _c_i64, _c_int, _c_int, _c_int, _c_ptr, _c_ptr, _c_ptr,
                  _c_i64, _c_i64, _c_ptr],
    "tq_mm_decode": [_c_ptr, _c_i64, _c_ptr, _c_f32, _c_ptr, _c_ptr, _c_i64, _c_int, _c_int, _c_int, _c_int, _c_ptr, _c_int,
                     _c_f32, _c_ptr, _c_i64, _c_ptr, _c_ptr, _c_ptr, _c_int, _c_ptr, _c_ptr, _c_ptr, _c_int, _c_i64, _c_int,
                     _c_int, _c_int, _c_ptr],
    "tq_router_topk_weighted": [_c_ptr, _c_ptr, _c_ptr, _c_ptr, _c_int, _c_int, _c_int, _c_int, _c_int, _c_f32, _c_ptr, _c_ptr,
                                _c_ptr, _c_ptr, _c_int, _c_int, _c_ptr],
    "tq_route_weighted": [_c_ptr, _c_ptr, _c_ptr, _c_ptr, _c_int, _c_int, _c_int, _c_int, _c_int, _c_f32, _c_ptr, _c_ptr, _c_ptr,
                          _c_ptr, _c_int, _c_int, _c_ptr, _c_ptr, _c_ptr, _c_ptr, _c_int, _c_int, _c_ptr],
    "tq_add_norm": [_c_ptr, _c_ptr, _c_int, _c_i64, _c_ptr, _c_ptr, _c_ptr, _c_int, _c_ptr, _c_int, _c_ptr, _c_ptr, _c_f32,
                    _c_int, _c_ptr, _c_ptr, _c_f32, _c_int, _c_ptr, _c_int, _c_ptr, _c_ptr, _c_int, _c_ptr],
    "tq_token_gate": [_c_ptr, _c_int, _c_ptr, _c_ptr, _c_int, _c_i64, _c_int, _c_ptr, _c_int, _c_int, _c_ptr],
    "tq_token_gate_product": [_c_ptr, _c_i64, _c_ptr, _c_ptr, _c_ptr, _c_int, _c_i64, _c_int, _c_ptr, _c_int, _c_int, _c_int, _c_ptr],
    "tq_row_norm_kv_write": [_c_ptr, _c_i64, _c_ptr, _c_ptr, _c_ptr, _c_int, _c_ptr, _c_int, _c_int, _c_f32, _c_ptr, _c_ptr,
                             _c_int, _c_f32, _c_int, _c_int, _c_int, _c_ptr, _c_ptr, _c_ptr, _c_int, _c_i64, _c_int, _c_int,
                             _c_int, _c_int, _c_int, _c_ptr, _c_ptr, _c_ptr, _c_int, _c_int, _c_ptr],
    "tq_diff_prep_kv_write": [_c_ptr, _c_i64, _c_ptr, _c_ptr, _c_ptr, _c_int, _c_ptr, _c_ptr, _c_int, _c_f32, _c_int, _c_f32,
                              _c_f32, _c_ptr, _c_ptr, _c_ptr, _c_int, _c_i64, _c_int, _c_int, _c_int, _c_int, _c_int, _c_int,
                              _c_ptr, _c_ptr, _c_ptr, _c_int, _c_int, _c_ptr],
    "tq_diff_combine": [_c_ptr, _c_f32, _c_f32, _c_int, _c_f32, _c_ptr, _c_i64, _c_ptr, _c_int, _c_int, _c_int, _c_ptr],
    "tq_ssd_prep": [_c_ptr, _c_i64, _c_ptr, _c_ptr, _c_i64, _c_ptr, _c_ptr, _c_ptr, _c_int, _c_int, _c_int, _c_int, _c_int,
                    _c_ptr, _c_ptr, _c_int, _c_ptr],
    "tq_ssd_scan": [_c_ptr, _c_ptr, _c_ptr, _c_ptr, _c_ptr, _c_ptr, _c_ptr, _c_i64, _c_int, _c_int, _c_int, _c_int, _c_int,
                    _c_int, _c_ptr, _c_ptr],
    "tq_ssd_chunked": [_c_ptr, _c_ptr, _c_ptr, _c_ptr, _c_ptr, _c_ptr, _c_ptr, _c_i64, _c_int, _c_int, _c_int, _c_int, _c_int,
                       _c_int, _c_int, _c_ptr, _c_ptr, _c_int, _c_ptr, _c_ptr],
    "tq_ssd_decode": [_c_ptr, _c_i64, _c_ptr, _c_ptr, _c_i64, _c_ptr, _c_ptr, _c_ptr, _c_ptr, _c_ptr, _c_int, _c_int, _c_int,
                      _c_int, _c_int, _c_int, _c_ptr, _c_ptr],
    "tq_ssd_out": [_c_ptr, _c_ptr, _c_i64, _c_ptr, _c_int, _c_f32, _c_int, _c_ptr, _c_ptr, _c_ptr, _c_i64, _c_int, _c_int,
                   _c_int, _c_int, _c_int, _c_int, _c_int, _c_ptr, _c_ptr],
    "tq_gate_heads": [_c_ptr, _c_ptr, _c_i64, _c_ptr, _c_int, _c_int, _c_int, _c_int, _c_ptr],
    "tq_lead_norm": [_c_ptr, _c_i64, _c_ptr, _c_int, _c_f32, _c_ptr, _c_int, _c_i64, _c_int, _c_int, _c_int, _c_int, _c_int,
                     _c_ptr],
    "tq_rope_kv_write_ex": [_c_ptr, _c_i64, _c_ptr, _c_int, _c_ptr, _c_ptr, _c_ptr, _c_int, _c_ptr, _c_int, _c_int, _c_f32,
                            _c_f32, _c_int, _c_ptr, _c_ptr, _c_ptr, _c_int, _c_i64, _c_int, _c_int, _c_int, _c_int, _c_int,
                            _c_ptr, _c_ptr, _c_ptr, _c_int, _c_int, _c_ptr],
    "tq_router_topk_biased": [_c_ptr, _c_ptr, _c_ptr, _c_ptr, _c_int, _c_int, _c_int, _c_int, _c_int, _c_int, _c_ptr, _c_ptr,
                              _c_ptr, _c_ptr, _c_int, _c_int, _c_ptr],
    "tq_route_biased": [_c_ptr, _c_ptr, _c_ptr, _c_ptr, _c_int, _c_int, _c_int, _c_int, _c_int, _c_int, _c_ptr, _c_ptr, _c_ptr,
                        _c_ptr, _c_int, _c_int, _c_ptr, _c_ptr, _c_ptr, _c_ptr, _c_int, _c_int, _c_ptr],
    "tq_lightning_scan": [_c_ptr, _c_i64, _c_ptr, _c_ptr, _c_ptr, _c_ptr, _c_i64, _c_int, _c_int, _c_int, _c_int, _c_ptr,
                          _c_ptr],
    "tq_lightning_chunked": [_c_ptr, _c_i64, _c_ptr, _c_ptr, _c_ptr, _c_ptr, _c_i64, _c_int, _c_int, _c_int, _c_int, _c_int,
                             _c_ptr, _c_int, _c_ptr, _c_ptr],
    "tq_lightning_out": [_c_ptr, _c_ptr, _c_i64, _c_ptr, _c_int, _c_f32, _c_ptr, _c_int, _c_int, _c_ptr],
}
# entry points that only one of the two libraries has
_OPTIONAL = {
    "tq_gemm_f32": [_c_ptr, _c_i64, _c_ptr, _c_int, _c_ptr, _c_ptr, _c_i64, _c_ptr, _c_ptr, _c_ptr, _c_int,
                    _c_ptr, _c_i64, _c_int, _c_int, _c_int, _c_int, _c_int, _c_ptr, _c_int, _c_ptr],
    "tq_gemm_f32_runs": [_c_int, _c_int, _c_int, _c_int],
    "tq_attention_f32_scratch": [_c_int, _c_int, _c_int, _c_int],
    "tq_attention_f32": [_c_ptr, _c_ptr, _c_ptr, _c_ptr, _c_int, _c_ptr, _c_ptr, _c_ptr, _c_int, _c_i64, _c_int, _c_int,
                         _c_int, _c_int, _c_int, _c_f32, _c_ptr, _c_ptr, _c_int, _c_int, _c_int, _c_ptr],
    "tq_gemm_mfma": [_c_ptr, _c_i64, _c_ptr, _c_int, _c_ptr, _c_ptr, _c_i64, _c_ptr, _c_ptr, _c_ptr, _c_int,
                     _c_ptr, _c_i64, _c_int, _c_int, _c_int, _c_int, _c_int, _c_int, _c_int, _c_ptr],
    "tq_gemm_mfma_splits": [_c_int, _c_int, _c_int],
    "tq_gemm_mfma_pair_splits": [_c_int, _c_int, _c_int, _c_int, _c_int, _c_int],
    "tq_gemm_mfma_pair": [_c_ptr, _c_ptr, _c_int, _c_ptr],
    "tq_qkv_rope_write": [_c_ptr, _c_i64, _c_ptr, _c_ptr, _c_int, _c_int, _c_int, _c_ptr, _c_ptr, _c_ptr, _c_int, _c_ptr,
                          _c_ptr, _c_ptr, _c_ptr, _c_int, _c_i64, _c_int, _c_int, _c_int, _c_ptr],
    "tq_probe_stream": [_c_ptr, _c_i64, _c_int, ctypes.c_uint, _c_ptr, _c_ptr],
    "tq_probe_mfma": [_c_int, _c_int, _c_int, ctypes.c_uint, _c_ptr, _c_ptr],
    "tq_attention_decode_scratch": [_c_int, _c_int, _c_int, _c_int],
    "tq_attention_f32_mod": [_c_ptr, _c_ptr, _c_ptr, _c_ptr, _c_int, _c_ptr, _c_ptr, _c_ptr, _c_int, _c_i64, _c_int, _c_int,
                             _c_int, _c_int, _c_int, _c_f32, _c_f32, _c_ptr, _c_ptr, _c_int, _c_ptr, _c_ptr, _c_ptr, _c_int,
                             _c_int, _c_int, _c_ptr],
    "tq_attention_f32_sig": [_c_ptr, _c_ptr, _c_ptr, _c_ptr, _c_int, _c_ptr, _c_ptr, _c_ptr, _c_int, _c_i64, _c_int, _c_int,
                             _c_int, _c_int, _c_int, _c_f32, _c_f32, _c_ptr, _c_ptr, _c_int, _c_ptr, _c_ptr, _c_int, _c_ptr,
                             _c_ptr, _c_int, _c_int, _c_int, _c_ptr],
    "tq_attention_mfma_sig": [_c_ptr, _c_ptr, _c_ptr, _c_ptr, _c_int, _c_ptr, _c_ptr, _c_ptr, _c_int, _c_i64, _c_int,
                              _c_int, _c_int, _c_int, _c_int, _c_f32, _c_f32, _c_ptr, _c_ptr, _c_int, _c_ptr, _c_ptr,
                              _c_ptr, _c_int, _c_int, _c_int, _c_int, _c_ptr, _c_i64, _c_ptr, _c_int, _c_ptr],
    "tq_attention_mfma_ld": [_c_ptr, _c_ptr, _c_ptr, _c_ptr, _c_int, _c_ptr, _c_ptr, _c_ptr, _c_int, _c_i64, _c_int,
                             _c_int, _c_int, _c_int, _c_int, _c_f32, _c_f32, _c_ptr, _c_ptr, _c_int, _c_ptr, _c_ptr,
                             _c_ptr, _c_int, _c_int, _c_int, _c_int, _c_ptr, _c_i64, _c_ptr, _c_int, _c_i64, _c_ptr],
    "tq_attention_mfma_diff": [_c_ptr, _c_ptr, _c_ptr, _c_ptr, _c_int, _c_ptr, _c_ptr, _c_ptr, _c_int, _c_i64, _c_int, _c_int,
                               _c_int, _c_int, _c_f32, _c_f32, _c_f32, _c_int, _c_f32, _c_ptr, _c_i64, _c_ptr, _c_ptr, _c_int,
                               _c_int, _c_int, _c_ptr],
    "tq_attention_mfma_mod": [_c_ptr, _c_ptr, _c_ptr, _c_ptr, _c_int, _c_ptr, _c_ptr, _c_ptr, _c_int, _c_i64, _c_int, _c_int,
                              _c_int, _c_int, _c_int, _c_f32, _c_f32, _c_ptr, _c_ptr, _c_int, _c_ptr, _c_ptr, _c_ptr, _c_int,
                              _c_int, _c_int, _c_ptr],
    "tq_attention_mfma": [_c_ptr, _c_ptr, _c_ptr, _c_ptr, _c_int, _c_ptr, _c_ptr, _c_ptr, _c_int, _c_i64, _c_int, _c_int,
                          _c_int, _c_int, _c_int, _c_f32, _c_ptr, _c_ptr, _c_int, _c_int, _c_int, _c_ptr],
    "tq_attention_mfma_ex": [_c_ptr, _c_ptr, _c_ptr, _c_ptr, _c_int, _c_ptr, _c_ptr, _c_ptr, _c_int, _c_i64, _c_int,
                             _c_int, _c_int, _c_int, _c_int, _c_f32, _c_f32, _c_ptr, _c_ptr, _c_int, _c_ptr, _c_ptr,
                             _c_ptr, _c_int, _c_int, _c_int, _c_int, _c_ptr, _c_i64, _c_ptr],
}


def dtype_name(dtype) -> str:
    if isinstance(dtype, str):
        if dtype in ("float32", "f32", "fp32"):
            return "float32"
        if dtype in ("bfloat16", "bf16"):
            return "bfloat16"
    elif dtype == torch.float32:
        return "float32"
    elif dtype == torch.bfloat16:
        return "bfloat16"
    raise KernelError(f"no kernels for activation type {dtype!r}: float32 and bfloat16 are built")


def library(dtype) -> ctypes.CDLL:
    """The compiled kernels for one activation type; builds them at the first call if they are not there."""
    name = dtype_name(dtype)
    lib = _LIBS.get(name)
    if lib is not None:
        return lib
    if not torch.cuda.is_available():
        raise KernelError("no GPU is visible: the kernels of this library run on gfx950 only and have no CPU form")
    path = _build.find_library(name) or _build.build(name)
    try:
        lib = ctypes.CDLL(path)
    except OSError as e:
        raise KernelError(f"cannot load the kernel library {path}: {e}") from e
    for fn, sig in _SIGNATURES.items():
        f = getattr(lib, fn)
        f.argtypes, f.restype = sig, _c_int
    for fn, sig in _OPTIONAL.items():
        if hasattr(lib, fn):
            f = getattr(lib, fn)
            f.argtypes, f.restype = sig, _c_int
    lib.tq_sample_topp_scratch.restype = _c_i64
    lib.tq_delta_state_floats.restype = _c_i64
    for fn in ("tq_attention_decode_scratch", "tq_attention_f32_scratch"):
        if hasattr(lib, fn):
            getattr(lib, fn).restype = _c_i64
    _LIBS[name] = lib
    return lib


_raw_stream = getattr(torch._C, "_cuda_getCurrentRawStream", None) or (lambda dev: torch.cuda.current_stream(dev).cuda_stream)


def has_kernel(dtype, name: str) -> bool:
    return hasattr(library(dtype), name)


def _stream() -> int:
    """The current stream's handle (the raw call: building a stream object for every launch cost 5 us of the host's
    time, a fifth of what a launch took)."""
    return _raw_stream(torch.cuda.current_device())


def _ptr(t: torch.Tensor | None) -> int | None:
    return None if t is None else t.data_ptr()


def _need(cond: bool, kernel: str, what) -> None:
    """``what``: the message, or a function that makes it (so that a check that holds formats nothing)."""
    if not cond:
        raise KernelError(f"{kernel}: {what() if callable(what) else what}")


def _check(t: torch.Tensor, kernel: str, name: str, dtype=None, shape=None) -> None:
    if not (isinstance(t, torch.Tensor) and t.is_cuda):
        raise KernelError(f"{kernel}: {name} must be a GPU tensor")
    if not t.is_contiguous():
        raise KernelError(f"{kernel}: {name} must be contiguous, has strides {t.stride()}")
    if dtype is not None and not (t.dtype in dtype if type(dtype) in (tuple, list) else t.dtype == dtype):
        raise KernelError(f"{kernel}: {name} must be {dtype}, is {t.dtype}")
    if shape is not None and tuple(t.shape) != tuple(shape):
        raise KernelError(f"{kernel}: {name} must have shape {tuple(shape)}, has {tuple(t.shape)}")


# Timing by kind of work, as the reference's --profile has it (/root/reference/src/engine/tq_transformer.c:60-93,
# :2995-3020: matmul, moe, attn and the rest): while a profile is open, an event is recorded behind every launch, and
# the time between two events is put down to the kernel between them (the step must run on one stream).
_PROFILE: list | None = None
_KIND = {"gemm": "matmul", "gemm_mfma": "matmul", "gemm_f32": "matmul", "gemm_pair": "matmul", "qkv_rope_write": "matmul",
         "gated_act": "matmul", "attention": "attn", "attention_mfma": "attn", "attention_f32": "attn",
         "router_topk": "moe", "route": "moe", "moe_align": "moe", "moe_combine": "moe",
         "delta_prep": "attn", "delta_scan": "attn", "delta_out": "attn", "delta_decode": "attn",
         "head_gemm": "matmul", "latent_norm": "attn", "gate_rows": "attn", "gate_heads": "attn",
         "mm_scan": "attn", "mm_chunked": "attn", "mm_out": "attn", "mm_decode": "attn",
         "lightning_scan": "attn", "lightning_chunked": "attn", "lightning_out": "attn",
         "ssd_prep": "attn", "ssd_scan": "attn", "ssd_chunked": "attn", "ssd_decode": "attn", "ssd_out": "attn",
         "row_norm_kv_write": "attn", "diff_prep_kv_write": "attn", "diff_combine": "attn"}


def profile_begin() -> None:
    global _PROFILE
    e = torch.cuda.Event(enable_timing=True)
    e.record()
    _PROFILE = [(None, e)]


def profile_end() -> dict:
    """Milliseconds per kind since ``profile_begin`` ("matmul", "moe", "attn", "other"), "total", and "kernels":
    name -> [launches, milliseconds]."""
    global _PROFILE
    marks, _PROFILE = _PROFILE or [], None
    torch.cuda.synchronize()
    out = {"matmul": 0.0, "moe": 0.0, "attn": 0.0, "other": 0.0}
    kernels: dict[str, list] = {}
    for (_, before), ((kind, name), after) in zip(marks, marks[1:]):
        ms = before.elapsed_time(after)
        out[kind] += ms
        row = kernels.setdefault(name, [0, 0.0])
        row[0] += 1
        row[1] += ms
    out["total"] = sum(out.values())
    out["kernels"] = kernels
    return out


def _mark(kind: str, name: str = "vendor product") -> None:
    e = torch.cuda.Event(enable_timing=True)
    e.record()
    _PROFILE.append(((kind, name), e))


def _run(kernel: str, code: int, kind: str | None = None) -> None:
    if code == 0:
        if _PROFILE is not None:
            kind = kind or _KIND.get(kernel, "other")
            _mark(kind, kernel + (" (experts)" if kind == "moe" and kernel.startswith("gemm") else ""))
        return
    if code == -1:
        raise KernelError(f"{kernel}: arguments rejected by the launcher")
    if code == -2:
        raise KernelError(f"{kernel}: size not supported by this kernel")
    raise KernelError(f"{kernel}: HIP error {code} at launch")


# ------------------------------------------------------------------ row-wise kernels
def embed(tokens: torch.Tensor, table: torch.Tensor, act, scale: float = 1.0, pos_table: torch.Tensor | None = None,
          positions: torch.Tensor | None = None) -> torch.Tensor:
    """x[t] = table[tokens[t]] (times ``scale``) as float32 [T, H]; with ``pos_table`` [P, H] and ``positions`` [T],
    plus pos_table[positions[t]] (a learned vector per position; positions beyond the table are the caller's to refuse)."""
    k = "embed"
    _check(tokens, k, "tokens", torch.int32)
    _need(tokens.dim() == 1 and table.dim() == 2, k, "tokens [T], table [V, H]")
    _check(table, k, "table", tuple(_WTYPE))
    T, (V, H) = tokens.numel(), table.shape
    x = torch.empty((T, H), dtype=torch.float32, device=table.device)
    if pos_table is not None:
        _check(pos_table, k, "pos_table", table.dtype)
        _need(pos_table.dim() == 2 and pos_table.shape[1] == H, k, lambda: f"pos_table must be [P, {H}]")
        _check(positions, k, "positions", torch.int32, (T,))
        _run(k, library(act).tq_embed_pos(_ptr(tokens), _ptr(positions), _ptr(table), _ptr(pos_table), _WTYPE[table.dtype],
                                          _ptr(x), T, H, float(scale), _stream()))
        return x
    _run(k, library(act).tq_embed(_ptr(tokens), _ptr(table), _WTYPE[table.dtype], _ptr(x), T, H, float(scale), _stream()))
    return x


def softcap(logits: torch.Tensor, cap: float | None, act, scale: float = 1.0) -> torch.Tensor:
    """logits <- cap * tanh(logits / cap), in place; with ``scale``, of the logits times it (``cap`` None: that alone)."""
    k = "softcap"
    _check(logits, k, "logits", torch.float32)
    if scale != 1.0 or cap is None:
        _need(cap is None or cap > 0, k, "the cap must be positive")
        _run(k, library(act).tq_scale_softcap(_ptr(logits), logits.numel(), float(scale), float(cap or 0.0), _stream()))
        return logits
    _need(cap > 0, k, "the cap must be positive")
    _run(k, library(act).tq_softcap(_ptr(logits), logits.numel(), float(cap), _stream()))
    return logits


def gather_rows(src: torch.Tensor, index: torch.Tensor, act) -> torch.Tensor:
    """``src[index]`` along the first dimension (``index`` int32 on the device): the rows of a step's sequences out of
    a tensor that has a row per slot."""
    k = "gather_rows"
    _check(src, k, "src")
    _check(index, k, "index", torch.int32)
    _need(index.dim() == 1 and src.dim() >= 1, k, "index must be [n], src [rows, ...]")
    row_bytes = (src.numel() // max(src.shape[0], 1)) * src.element_size()
    out = torch.empty((index.numel(), *src.shape[1:]), dtype=src.dtype, device=src.device)
    _run(k, library(act).tq_move_rows(_ptr(src), _ptr(index), _ptr(out), index.numel(), row_bytes, 0, _stream()))
    return out


def scatter_rows(dst: torch.Tensor, index: torch.Tensor, rows: torch.Tensor, act) -> None:
    """``dst[index] = rows`` along the first dimension; every index at most once."""
    k = "scatter_rows"
    _check(dst, k, "dst")
    _check(index, k, "index", torch.int32)
    _check(rows, k, "rows", dst.dtype, (index.numel(), *dst.shape[1:]))
    row_bytes = (dst.numel() // max(dst.shape[0], 1)) * dst.element_size()
    _run(k, library(act).tq_move_rows(_ptr(rows), _ptr(index), _ptr(dst), index.numel(), row_bytes, 1, _stream()))


@dataclasses.dataclass
class GatheredSum:
    """A part's output that nobody has summed yet:
    ``out[t] = sum_j weights[t, j] * y[pair_slot[t, j]] + gate[t] * sum_s dense[s, t]`` (j ascending; ``dense``
    and ``gate`` may be None).  The next norm adds it into the residual stream in the pass that normalises;
    ``materialize`` gives it as a float32 [1, T, H] tensor to whoever needs it earlier."""
    y: torch.Tensor                      # float32 [rows, H]
    pair_slot: torch.Tensor              # int32 [T, k]
    weights: torch.Tensor                # float32 [T, k]
    dense: torch.Tensor | None = None    # float32 [S, T, H]
    gate: torch.Tensor | None = None     # float32 [T]

    def materialize(self, act) -> torch.Tensor:
        return moe_combine(self.y, self.pair_slot, self.weights, self.dense, self.gate, act)


@dataclasses.dataclass
class NormedDelta:
    """A part's output that joins the residual stream only after a norm of its own:
    ``x += rmsnorm(inner, eps) * weight``, or with ``bias`` ``x += layernorm(inner, eps) * weight + bias``, ``inner`` being
    float32 partial sums [S, T, H] or a GatheredSum.  The next norm does both in one pass; ``materialize`` gives the normed
    tensor [1, T, H] to whoever needs it earlier."""
    inner: object
    weight: torch.Tensor
    eps: float
    bias: torch.Tensor | None = None

    def materialize(self, act) -> torch.Tensor:
        ref = self.inner.y if isinstance(self.inner, GatheredSum) else self.inner
        T = self.inner.pair_slot.shape[0] if isinstance(self.inner, GatheredSum) else ref.shape[1]
        x = torch.zeros((T, ref.shape[-1]), dtype=torch.float32, device=ref.device)
        add_rmsnorm(x, self, None, 0.0, act, want_act=False)
        return x[None]


@dataclasses.dataclass
class Terms:
    """What several parts that ran side by side leave for the residual stream, not yet summed:
    ``vector + sum_j weights[t, j] * y[pair_slot[t, j]] + sum_g coef_g * sum_s delta_g[s, t]``, ``parts`` being (coef, delta
    float32 [S, T, H]) pairs, ``gathered`` a GatheredSum without a gate (or None) and ``vector`` float32 [H] or None.  The
    next norm adds it all in the pass that normalises; ``materialize`` gives it as a float32 [1, T, H] tensor."""
    parts: list
    gathered: GatheredSum | None = None
    vector: torch.Tensor | None = None

    @staticmethod
    def of(*terms, vector: torch.Tensor | None = None) -> "Terms":
        """From (coef, what a part returned) pairs: partial sums, a GatheredSum, other Terms, or None."""
        out = Terms([], None, vector)
        for coef, t in terms:
            if t is None:
                continue
            if isinstance(t, Terms):
                _need(coef == 1.0 and (t.vector is None or out.vector is None), "terms", "terms within terms come unscaled, with one vector")
                out.parts += t.parts
                out.vector = t.vector if t.vector is not None else out.vector
                t, dense, gate = t.gathered, None, None
                if t is None:
                    continue
            elif isinstance(t, GatheredSum):
                dense, gate = t.dense, t.gate
                t = GatheredSum(t.y, t.pair_slot, t.weights)
            else:
                out.parts.append((float(coef), t))
                continue
            _need(coef == 1.0 and gate is None and out.gathered is None, "terms",
                  "one sum over experts, unscaled and without a gate, goes with other terms")
            out.gathered = t
            if dense is not None:
                out.parts.append((1.0, dense))
        return out

    def materialize(self, act) -> torch.Tensor:
        ref = self.parts[0][1] if self.parts else self.gathered.y if self.gathered is not None else self.vector[None]
        T = ref.shape[1] if self.parts else self.gathered.pair_slot.shape[0] if self.gathered is not None else 1
        x = torch.zeros((T, ref.shape[-1]), dtype=torch.float32, device=ref.device)
        add_rmsnorm(x, self, None, 0.0, act, want_act=False)
        return x[None]


def _add_terms_rmsnorm(x, terms: Terms, weight, eps: float, act, rows, want_act: bool, want_f32: bool):
    k = "add_terms_rmsnorm"
    T, H = x.shape
    _need(len(terms.parts) <= 4, k, lambda: f"{len(terms.parts)} parts are beyond the 4 this kernel takes")
    n = len(terms.parts)
    for _, d in terms.parts:
        _check(d, k, "a part", torch.float32)
        _need(d.dim() == 3 and tuple(d.shape[1:]) == (T, H), k, lambda: f"a part must be [S, {T}, {H}], is {tuple(d.shape)}")
    _need(sum(d.shape[0] for _, d in terms.parts) <= 128, k, "more partial sums than the 128 this kernel takes")
    y = pair_slot = weights = None
    topk = 0
    if terms.gathered is not None:
        y, pair_slot, weights = terms.gathered.y, terms.gathered.pair_slot, terms.gathered.weights
        _check(y, k, "y", torch.float32)
        _need(y.dim() == 2 and y.shape[1] == H, k, lambda: f"y must be [rows, {H}]")
        _check(pair_slot, k, "pair_slot", torch.int32)
        topk = pair_slot.shape[1]
        _need(pair_slot.shape[0] == T and 1 <= topk <= 64, k, lambda: f"pair_slot must be [{T}, 1..64]")
        _check(weights, k, "weights", torch.float32, (T, topk))
    if terms.vector is not None:
        _check(terms.vector, k, "vector", torch.float32, (H,))
    R = T
    if rows is not None:
        _check(rows, k, "rows", torch.int32)
        R = rows.numel()
    if weight is not None:
        _check(weight, k, "weight", tuple(_WTYPE), (H,))
    else:
        _need(rows is None, k, "without a weight all rows are summed")
        want_act = want_f32 = False
    out = torch.empty((R, H), dtype=ACT_DTYPES[dtype_name(act)], device=x.device) if want_act else None
    out32 = torch.empty((R, H), dtype=torch.float32, device=x.device) if want_f32 else None
    deltas = (ctypes.c_int64 * max(n, 1))(*[_ptr(d) for _, d in terms.parts])
    sums = (ctypes.c_int * max(n, 1))(*[d.shape[0] for _, d in terms.parts])
    coefs = (ctypes.c_float * max(n, 1))(*[c for c, _ in terms.parts])
    _run("add_rmsnorm", library(act).tq_add_terms_rmsnorm(
        _ptr(x), deltas, sums, coefs, n, T * H, _ptr(terms.vector), _ptr(y), _ptr(pair_slot), _ptr(weights), topk, _ptr(weight),
        _WTYPE[weight.dtype] if weight is not None else 0, float(eps), _ptr(rows), R, _ptr(out), _ptr(out32), H, _stream()))
    return out, out32


def _add_norm(x, delta, weight, bias, eps: float, act, rows, want_act: bool, want_f32: bool, stream: bool):
    """``add_rmsnorm`` where what is added, or what is returned, passes a layer norm."""
    k = "add_norm"
    T, H = x.shape
    if isinstance(delta, Terms):
        delta = delta.materialize(act)
    post = delta if isinstance(delta, NormedDelta) else None
    inner = post.inner if post is not None else delta
    y = pair_slot = weights = gate = None
    topk = 0
    if isinstance(inner, GatheredSum):
        y, pair_slot, weights, gate, inner = inner.y, inner.pair_slot, inner.weights, inner.gate, inner.dense
        _check(y, k, "y", torch.float32)
        _need(y.dim() == 2 and y.shape[1] == H, k, lambda: f"y must be [rows, {H}]")
        _check(pair_slot, k, "pair_slot", torch.int32)
        topk = pair_slot.shape[1]
        _need(pair_slot.shape[0] == T and 1 <= topk <= 64, k, lambda: f"pair_slot must be [{T}, 1..64]")
        _check(weights, k, "weights", torch.float32, (T, topk))
        if gate is not None:
            _check(gate, k, "gate", torch.float32, (T,))
    S = 0
    if inner is not None:
        _check(inner, k, "delta", torch.float32)
        _need(inner.dim() == 3 and tuple(inner.shape[1:]) == (T, H), k, lambda: f"delta must be [S, {T}, {H}], is {tuple(inner.shape)}")
        S = inner.shape[0]
    wtype = None
    for name, t in (("the added part's norm weight", post.weight if post is not None else None),
                    ("the added part's norm bias", post.bias if post is not None else None), ("weight", weight), ("bias", bias)):
        if t is not None:
            _check(t, k, name, tuple(_WTYPE), (H,))
            _need(wtype in (None, t.dtype), k, "the norms' weights and biases must have one type")
            wtype = t.dtype
    R = T
    if rows is not None:
        _check(rows, k, "rows", torch.int32)
        _need(rows.dim() == 1 and weight is not None, k, "rows must be [R], and picks rows of what is normed")
        R = rows.numel()
    if weight is None:
        _need(bias is None, k, "a bias goes with a weight")
        want_act, want_f32 = stream and dtype_name(act) != "float32", False
    out = torch.empty((R, H), dtype=ACT_DTYPES[dtype_name(act)], device=x.device) if want_act else None
    out32 = torch.empty((R, H), dtype=torch.float32, device=x.device) if want_f32 else None
    _run("add_rmsnorm", library(act).tq_add_norm(
        _ptr(x), _ptr(inner), S, T * H, _ptr(y), _ptr(pair_slot), _ptr(weights), topk, _ptr(gate),
        0 if post is None else 1 if post.bias is None else 2, _ptr(post.weight) if post is not None else None,
        _ptr(post.bias) if post is not None else None, float(post.eps) if post is not None else 0.0,
        0 if weight is None else 1 if bias is None else 2, _ptr(weight), _ptr(bias), float(eps),
        _WTYPE[wtype] if wtype is not None else 0, _ptr(rows), R, _ptr(out), _ptr(out32), H, _stream()))
    return (x if stream and out is None else out), out32


def add_rmsnorm(x: torch.Tensor, delta, weight: torch.Tensor | None, eps: float, act,
                rows: torch.Tensor | None = None, want_act: bool = True, want_f32: bool = False, stream: bool = False,
                shift: tuple | None = None, bias: torch.Tensor | None = None):
    """x += delta (in place, unless ``rows`` picks rows), where delta is None, float32 partial sums [S, T, H] added
    one after the other, a GatheredSum, Terms, or a NormedDelta around partial sums or a GatheredSum (then what is added is its RMS norm); returns
    rmsnorm(x) * weight as (activation-typed or None, float32 or None), one row per entry of ``rows`` (all rows if
    None).  ``weight`` None (with a NormedDelta only): the stream is summed and nothing is returned.  ``stream`` (with
    ``weight`` None, and delta None or a NormedDelta): the summed stream itself is returned in the activation type, for
    a part that reads the stream un-normed (on the float32 library that is ``x``, which the next sum changes).
    ``shift`` (with ``stream`` behind a NormedDelta, in a step of one token per sequence): (weight float32 [H], state float32
    [slots, H], slots int32 [T]); what is returned is the summed row blended with the row that the sequence's slot keeps,
    ``a + (state[slot] - a) * weight``, and the slot then keeps the summed row: ``token_shift`` without a launch of its own.
    ``bias`` (with ``weight``): what is returned is the layer norm of x (the mean taken off), times ``weight``, plus ``bias``."""
    k = "add_rmsnorm"
    _check(x, k, "x", torch.float32)
    _need(x.dim() == 2, k, "x must be [T, H]")
    T, H = x.shape
    post = None
    if bias is not None or (isinstance(delta, NormedDelta) and delta.bias is not None):
        _need(shift is None, k, "a shift does not ride behind a layer norm")
        return _add_norm(x, delta, weight, bias, eps, act, rows, want_act, want_f32, stream)
    if isinstance(delta, Terms):
        _need(not stream and shift is None, k, "the sum of several parts is normed, or only summed")
        return _add_terms_rmsnorm(x, delta, weight, eps, act, rows, want_act, want_f32)
    if stream:
        _need(weight is None and rows is None and (delta is None or isinstance(delta, NormedDelta)), k,
              "the stream itself is returned for all rows, behind nothing or a normed part")
        if delta is None:
            return (x if dtype_name(act) == "float32" else act_rows(x, None, None, act)), None
    if isinstance(delta, NormedDelta):
        post, delta = delta, delta.inner
        _check(post.weight, k, "the added part's norm weight", tuple(_WTYPE), (H,))
        _need(delta is not None, k, "a normed part needs something to norm")
    if weight is None:
        _need(post is not None and rows is None, k, "without a weight only a normed part can be summed, into all rows")
        want_act, want_f32 = stream and (dtype_name(act) != "float32" or shift is not None), False
    else:
        _check(weight, k, "weight", tuple(_WTYPE), (H,))
        _need(post is None or post.weight.dtype == weight.dtype, k, "the two norms' weights must have one type")
    shift_args = (None, None, None)
    if shift is not None:
        _need(stream and post is not None and post.weight.dtype == torch.float32, k,
              "a shift rides behind the sum of a normed part whose norm weights are float32")
        sw, sstate, sslots = shift
        _check(sw, k, "shift weight", torch.float32, (H,))
        _check(sstate, k, "shift state", torch.float32)
        _need(sstate.dim() == 2 and sstate.shape[1] == H, k, lambda: f"shift state must be [slots, {H}]")
        _check(sslots, k, "shift slots", torch.int32, (T,))
        shift_args = (_ptr(sw), _ptr(sstate), _ptr(sslots))
    y = pair_slot = weights = gate = None
    topk = 0
    if isinstance(delta, GatheredSum):
        y, pair_slot, weights, gate, delta = delta.y, delta.pair_slot, delta.weights, delta.gate, delta.dense
        _check(y, k, "y", torch.float32)
        _need(y.dim() == 2 and y.shape[1] == H, k, lambda: f"y must be [rows, {H}]")
        _check(pair_slot, k, "pair_slot", torch.int32)
        _need(pair_slot.dim() == 2 and pair_slot.shape[0] == T, k, lambda: f"pair_slot must be [{T}, k]")
        topk = pair_slot.shape[1]
        _need(1 <= topk <= 64, k, lambda: f"{topk} experts per token is beyond the 64 this kernel takes")
        _check(weights, k, "weights", torch.float32, (T, topk))
        if gate is not None:
            _check(gate, k, "gate", torch.float32, (T,))
    S, stride = 0, 0
    if delta is not None:
        _check(delta, k, "delta", torch.float32)
        _need(delta.dim() == 3 and tuple(delta.shape[1:]) == (T, H), k, lambda: f"delta must be [S, {T}, {H}], is {tuple(delta.shape)}")
        S, stride = delta.shape[0], T * H
    R = T
    if rows is not None:
        _check(rows, k, "rows", torch.int32)
        _need(rows.dim() == 1, k, "rows must be [R]")
        R = rows.numel()
    adt = ACT_DTYPES[dtype_name(act)]
    out = torch.empty((R, H), dtype=adt, device=x.device) if want_act else None
    out32 = torch.empty((R, H), dtype=torch.float32, device=x.device) if want_f32 else None
    if post is not None:
        _run(k, library(act).tq_add_normed_rmsnorm_shift(_ptr(x), _ptr(delta), S, stride, _ptr(y), _ptr(pair_slot), _ptr(weights),
                                                         topk, _ptr(gate), _ptr(post.weight), float(post.eps), _ptr(weight),
                                                         _WTYPE[post.weight.dtype], float(eps), _ptr(rows), R, _ptr(out),
                                                         _ptr(out32), H, *shift_args, _stream()))
        return (x if stream and out is None else out), out32
    _run(k, library(act).tq_add_rmsnorm(_ptr(x), _ptr(delta), S, stride, _ptr(y), _ptr(pair_slot), _ptr(weights), topk,
                                        _ptr(gate), _ptr(weight), _WTYPE[weight.dtype], float(eps), _ptr(rows), R,
                                        _ptr(out), _ptr(out32), H, _stream()))
    return out, out32


def head_rmsnorm(qkv: torch.Tensor, q_weight: torch.Tensor | None, k_weight: torch.Tensor | None, eps: float,
                 num_heads: int, num_kv_heads: int, head_dim: int, act, norm_dim: int | None = None) -> torch.Tensor:
    """RMS norm of every query head (weights ``q_weight`` [hd]) and key head (``k_weight``) of the float32 rows
    ``qkv`` [T, (nh + 2 nkv) * hd], in place; None leaves those heads alone.  ``norm_dim``: the values a head really
    has, where heads are laid out wider (zeros behind them, in the rows and in the weights): the mean is over these.
    Returns ``qkv``."""
    k = "head_rmsnorm"
    _check(qkv, k, "qkv", torch.float32)
    _need(qkv.dim() == 2 and qkv.shape[1] == (num_heads + 2 * num_kv_heads) * head_dim, k,
          lambda: f"qkv must be [T, {(num_heads + 2 * num_kv_heads) * head_dim}]")
    wtype = None
    for name, w in (("q_weight", q_weight), ("k_weight", k_weight)):
        if w is not None:
            _check(w, k, name, tuple(_WTYPE), (head_dim,))
            _need(wtype in (None, w.dtype), k, "q_weight and k_weight must have one type")
            wtype = w.dtype
    if wtype is not None:
        _run(k, library(act).tq_head_rmsnorm(_ptr(qkv), _ptr(q_weight), _ptr(k_weight), _WTYPE[wtype], float(eps),
                                             qkv.shape[0], num_heads, num_kv_heads, head_dim,
                                             head_dim if norm_dim is None else int(norm_dim), _stream()))
    return qkv


def rope_kv_write(qkv: torch.Tensor, positions: torch.Tensor, seq_of_token: torch.Tensor, block_table: torch.Tensor,
                  inv_freq: torch.Tensor, pairing: int, rotary_dim: int, k_pages: torch.Tensor | None,
                  v_pages: torch.Tensor | None, layer_offset: int, page_size: int, page_stride: int,
                  num_heads: int, num_kv_heads: int, head_dim: int, act, runs: dict | None = None,
                  bias: torch.Tensor | None = None, amplitude: float = 1.0, norm_eps: float | None = None,
                  norm_dim: int | None = None) -> torch.Tensor:
    """Rotates queries and keys, returns the queries [T, nh*hd] and writes keys and values into the pages.
    ``bias`` [width] is added to ``qkv`` as it is read, for a product that left its bias out.  ``qkv`` may be the first
    columns of the rows of a wider tensor.  ``amplitude``: a factor on every sine and cosine.  ``norm_eps``: behind the
    rotation every query and key head is divided by its root mean square over its first ``norm_dim`` values (all of the
    head by default; heads laid out wider hold zeros behind them), without weights.
    ``k_pages``/``v_pages`` are the flat page pools of the cache group (None: nothing is written, for a
    layer that reads another layer's cache); ``layer_offset`` is the layer's offset inside a page.  ``runs``
    (as for ``attention``) describes the tokens as one run of consecutive positions per sequence; with it the
    values of whole prompts are written by tiles."""
    k = "rope_kv_write"
    T = positions.numel()
    width = (num_heads + 2 * num_kv_heads) * head_dim
    _need(isinstance(qkv, torch.Tensor) and qkv.is_cuda and qkv.dtype == torch.float32 and tuple(qkv.shape) == (T, width)
          and qkv.stride(1) == 1 and qkv.stride(0) >= width, k,
          lambda: f"qkv must be float32 [{T}, {width}] on the GPU with unit stride along its rows")
    _need(k_pages is None or head_dim % 4 != 0 or (qkv.stride(0) % 4 == 0 and qkv.data_ptr() % 16 == 0), k,
          "rows of qkv must start at multiples of 16 bytes")
    if bias is not None:
        _check(bias, k, "bias", tuple(_WTYPE), (width,))
    _need(norm_eps is None or (norm_eps > 0 and rotary_dim <= 512), k, "a norm behind the rotation needs a positive eps and at most 512 rotated values")
    _check(positions, k, "positions", torch.int32, (T,))
    _check(seq_of_token, k, "seq_of_token", torch.int32, (T,))
    _check(block_table, k, "block_table", torch.int32)
    _need(block_table.dim() == 2, k, "block_table must be [B, pages]")
    _check(inv_freq, k, "inv_freq", torch.float32)
    _need(inv_freq.numel() * 2 == rotary_dim or rotary_dim == 0, k, lambda: f"inv_freq must hold rotary_dim/2 = {rotary_dim // 2} entries")
    adt = ACT_DTYPES[dtype_name(act)]
    q = torch.empty((T, num_heads * head_dim), dtype=adt, device=qkv.device)
    write = k_pages is not None
    kp = vp = None
    if write:
        _check(k_pages, k, "k_pages", adt)
        _check(v_pages, k, "v_pages", adt)
        _need(layer_offset + num_kv_heads * page_size * head_dim <= page_stride, k, "layer does not fit in a page")
        esz = k_pages.element_size()
        kp, vp = k_pages.data_ptr() + layer_offset * esz, v_pages.data_ptr() + layer_offset * esz
    cu = slots = start = None
    B = max_new = 0
    if runs is not None and write and not runs["decode"]:
        B = runs["slots"].numel()
        cu, slots, start, max_new = runs["cu_seqlens"], runs["slots"], runs["start"], int(runs["max_new"])
        _check(cu, k, "cu_seqlens", torch.int32, (B + 1,))
        _check(slots, k, "slots", torch.int32, (B,))
        _check(start, k, "start", torch.int32, (B,))
        _need(int(runs["max_end"]) <= block_table.shape[1] * page_size, k, "positions reach beyond the page table")
    _run(k, library(act).tq_rope_kv_write_ex(_ptr(qkv), qkv.stride(0), _ptr(bias), _WTYPE[bias.dtype] if bias is not None else 0,
                                             _ptr(positions), _ptr(seq_of_token), _ptr(block_table),
                                             block_table.shape[1], _ptr(inv_freq), pairing, rotary_dim, float(amplitude),
                                             float(norm_eps or 0.0), int(norm_dim or head_dim), _ptr(q), kp, vp,
                                             page_size, page_stride, T, num_heads, num_kv_heads, head_dim, int(write),
                                             _ptr(cu), _ptr(slots), _ptr(start), B, max_new, _stream()))
    return q


_ZERO_ANGLES: dict = {}


def _zero_angles(device, n: int) -> torch.Tensor:
    key = (str(device), n)
    if key not in _ZERO_ANGLES:
        _ZERO_ANGLES[key] = torch.zeros((n,), dtype=torch.float32, device=device)
    return _ZERO_ANGLES[key]


def qkv_rope_write(a: torch.Tensor, qkv_weight: torch.Tensor, qkv_bias: torch.Tensor | None, positions: torch.Tensor,
                   seq_of_token: torch.Tensor, block_table: torch.Tensor, inv_freq: torch.Tensor, pairing: int,
                   rotary_dim: int, k_pages: torch.Tensor | None, v_pages: torch.Tensor | None, layer_offset: int,
                   page_size: int, page_stride: int, num_heads: int, num_kv_heads: int, head_dim: int, act,
                   runs: dict | None = None) -> torch.Tensor:
    """``gemm(a, qkv_weight, bias=qkv_bias)`` followed by ``rope_kv_write``: the queries [T, nh*hd], keys and
    values in their pages.  Up to 16 tokens in bfloat16, with heads rotated whole in "half" pairing, take one
    launch (the product's workgroups rotate and store what they have summed); anything else is the two calls."""
    k = "qkv_rope_write"
    lib = library(act)
    T, K = a.shape
    if (rotary_dim == 0 and T <= 16 and head_dim % 32 == 0 and hasattr(lib, "tq_qkv_rope_write")
            and _use_mfma(act, a, qkv_weight, K)):
        # no rotation at all: angles of zero turn nothing (cosine 1, sine 0: a * 1 - b * 0 is a to the bit), so the
        # one launch whose workgroups rotate and store what they have summed serves such a mixer as well
        inv_freq, pairing, rotary_dim = _zero_angles(a.device, head_dim // 2), 0, head_dim
    fused = (hasattr(lib, "tq_qkv_rope_write") and T <= 16 and pairing == 0 and rotary_dim == head_dim
             and head_dim % 32 == 0 and _use_mfma(act, a, qkv_weight, K)
             and (qkv_bias is None or qkv_bias.dtype in _WTYPE))
    if not fused:
        # the vendor library's product has no bias of its own that costs nothing: the rotation adds it as it reads
        late = qkv_bias is not None and a.dim() == 2 and _vendor_product(act, a, qkv_weight, T, K)
        qkv = gemm(a, qkv_weight, act, bias=None if late else qkv_bias)
        return rope_kv_write(qkv, positions, seq_of_token, block_table, inv_freq, pairing, rotary_dim, k_pages, v_pages,
                             layer_offset, page_size, page_stride, num_heads, num_kv_heads, head_dim, act, runs=runs,
                             bias=qkv_bias if late else None)
    adt = ACT_DTYPES[dtype_name(act)]
    width = (num_heads + 2 * num_kv_heads) * head_dim
    _check(a, k, "a", adt)
    _need(a.stride(1) == 1, k, "a must have unit stride along its rows")
    _check(qkv_weight, k, "qkv_weight", torch.bfloat16, (width, K))
    if qkv_bias is not None:
        _check(qkv_bias, k, "qkv_bias", tuple(_WTYPE), (width,))
    _check(positions, k, "positions", torch.int32, (T,))
    _check(seq_of_token, k, "seq_of_token", torch.int32, (T,))
    _check(block_table, k, "block_table", torch.int32)
    _need(block_table.dim() == 2, k, "block_table must be [B, pages]")
    _check(inv_freq, k, "inv_freq", torch.float32, (head_dim // 2,))
    q = torch.empty((T, num_heads * head_dim), dtype=adt, device=a.device)
    kp = vp = None
    if k_pages is not None:
        _check(k_pages, k, "k_pages", adt)
        _check(v_pages, k, "v_pages", adt)
        _need(layer_offset + num_kv_heads * page_size * head_dim <= page_stride, k, "layer does not fit in a page")
        esz = k_pages.element_size()
        kp, vp = k_pages.data_ptr() + layer_offset * esz, v_pages.data_ptr() + layer_offset * esz
    _run(k, lib.tq_qkv_rope_write(_ptr(a), a.stride(0), _ptr(qkv_weight), _ptr(qkv_bias),
                                  _WTYPE[qkv_bias.dtype] if qkv_bias is not None else 0, T, K, _ptr(positions),
                                  _ptr(seq_of_token), _ptr(block_table), block_table.shape[1], _ptr(inv_freq), _ptr(q),
                                  kp, vp, page_size, page_stride, num_heads, num_kv_heads, head_dim, _stream()))
    return q


def moe_combine(y: torch.Tensor, pair_slot: torch.Tensor, weights: torch.Tensor, shared: torch.Tensor | None,
                shared_gate: torch.Tensor | None, act) -> torch.Tensor:
    """out[t] = sum_j weights[t, j] * y[pair_slot[t, j]] + shared_gate[t] * sum_s shared[s, t]; float32 [1, T, H]."""
    k = "moe_combine"
    _check(y, k, "y", torch.float32)
    T, topk = pair_slot.shape
    H = y.shape[1]
    _check(pair_slot, k, "pair_slot", torch.int32)
    _check(weights, k, "weights", torch.float32, (T, topk))
    S, stride = 0, 0
    if shared is not None:
        _check(shared, k, "shared", torch.float32)
        _need(shared.dim() == 3 and tuple(shared.shape[1:]) == (T, H), k, lambda: f"shared must be [S, {T}, {H}]")
        S, stride = shared.shape[0], T * H
    if shared_gate is not None:
        _check(shared_gate, k, "shared_gate", torch.float32, (T,))
    out = torch.empty((1, T, H), dtype=torch.float32, device=y.device)
    _run(k, library(act).tq_moe_combine(_ptr(y), _ptr(pair_slot), _ptr(weights), topk, _ptr(shared), S, stride,
                                        _ptr(shared_gate), _ptr(out), T, H, _stream()))
    return out


# ------------------------------------------------------------------ matrix products
def _use_mfma(act, a: torch.Tensor, w: torch.Tensor, K: int) -> bool:
    return (dtype_name(act) == "bfloat16" and w.dtype == torch.bfloat16 and K % 8 == 0
            and has_kernel(act, "tq_gemm_mfma"))


EXPERT_16_UPTO, EXPERT_32_UPTO = 5, 10
# Rows per expert on average from which the row order's unit is 128 and 256: never, since units of 64 taken two at a
# time do better wherever the taller units did (see expert_tile_rows); tests lower them to run those kernels.
EXPERT_128_FROM = EXPERT_256_FROM = 1 << 30
TILE_PAIRS = 1024            # added to tile_rows 64: two units of one expert per workgroup (TQ_TILE_PAIRS)
EXPERT_PAIRS_FROM = 48       # rows per expert on average from which units of 64 are taken two at a time


def expert_tile_rows(n_pairs: int, num_experts: int, act, a: torch.Tensor, w: torch.Tensor,
                     w_behind: torch.Tensor | None = None) -> int:
    """Rows per tile (the padding unit of the row order) that suit a product over experts, by the pairs per expert on
    average.  Up to 5: 16, the streaming kernel, which passes an expert's matrices once per 16 of its rows.  Up to 10,
    where the bfloat16 matrix-core product runs: 32, the same kernel with two row tiles and two column tiles to a wave.
    Beyond: tiles of 64 rows.  Where the borders lie depends on how evenly the router deals: with tokens dealt evenly
    (60 experts of 1,408 x 2,048, 4 per token, both products) units of 16 are best up to 8 rows per expert by 3 to 6 %,
    units of 32 from 10 to 24 by 9 to 13 % (202 us at 16 rows per expert against 270 and 233), tiles of 64 rows beyond;
    with a router of random weights, which gives some experts three times the rows of others, units of 32 are best up
    to 6 rows per expert (64 experts, 8 per token: up to 12) and tiles of 64 rows win by 10 to 18 % from 12 on, since a
    crowded expert's matrices pass the streaming kernel once per unit.  The borders here lose at most 6 % either way (a replayed decode step of 64 sequences, 4.3 rows per expert, is 2 %
    faster with units of 16 than of 32).
    Without the matrix-core product 16 up to 12.  Units of 128 and 256 rows (EXPERT_128_FROM, EXPERT_256_FROM) are
    not chosen: they were 8 to 17 % faster than single tiles of 64 rows from 256 rows per expert on, but units of 64
    taken two at a time (expert_product_rows) are faster than either (60 experts of 1,408 x 2,048, both products:
    396 us against 448 at 205 rows per expert, 492 against 565 at 273, 841 against 949 at 546; 64 experts of
    2,560 x 3,584 at 1,650 rows each: a prompt step of 425 ms against 436 with units of 256)."""
    # (``w_behind``: the matrices of the product that follows on the same row order, over another k: the units that only
    # the matrix-core product takes are chosen where both products run there)
    mfma = _use_mfma(act, a, w, a.shape[1]) and (w_behind is None or _use_mfma(act, a, w_behind, w_behind.shape[-1]))
    if n_pairs <= (EXPERT_16_UPTO if mfma else 12) * num_experts:
        return 16
    if mfma and n_pairs <= EXPERT_32_UPTO * num_experts:
        return 32
    if mfma and n_pairs >= EXPERT_128_FROM * num_experts:
        return 256 if n_pairs >= EXPERT_256_FROM * num_experts else 128
    return 64


def expert_product_rows(unit: int, n_pairs: int, num_experts: int) -> int:
    """The ``tile_rows`` that a product over experts is called with when the row order has units of ``unit`` rows: from
    48 rows per expert on average, units of 64 two at a time (measured on 60 experts of 1,408 x 2,048, four per
    token, both products together: 251 us against 286 at 68 rows per expert, 260 against 307 at 102, 346 against 360
    at 137; level below; a prompt step of 24 layers: 10.3 ms against 10.9 at 1,024 tokens, 15.8 against 17.0 at
    2,048, 22.3 against 23.7 at 3,072; where the border lies, by such steps: 9.42 ms against 9.73 at 55 rows per
    expert and 9.75 against 10.22 at 60, which already gives many experts a second unit, level at 43 and 47, 7.97
    against 7.81 at 34)."""
    if unit == 64 and n_pairs >= EXPERT_PAIRS_FROM * num_experts:
        return 64 + TILE_PAIRS
    return unit


def _gemm_problem(k: str, a, w, act, bias, w2, out_act, a_rows, tile_group, n_tiles, tile_rows, gather):
    """Checks one product's operands; returns (M, N, K, tile_rows, group stride)."""
    adt = ACT_DTYPES[dtype_name(act)]
    _check(a, k, "a", adt)
    _need(a.dim() == 2, k, "a must be [M, K]")
    K = a.shape[1]
    _check(w, k, "w", tuple(_WTYPE))
    grouped = tile_group is not None
    if grouped:
        _need(w.dim() == 3 and w.shape[2] == K, k, lambda: f"grouped w must be [G, N, {K}], is {tuple(w.shape)}")
        _need(a_rows is not None and n_tiles is not None and tile_rows in (16, 32, 64, 128, 256, 64 + TILE_PAIRS), k,
              "grouped product needs a_rows, n_tiles and tile_rows of 16, 64, 128 or 256")
        if not _use_mfma(act, a, w, a.shape[1]):
            _need(tile_rows % TILE_PAIRS in (16, 64), k, "tiles of 32, 128 and 256 rows are for the bfloat16 matrix-core product")
            tile_rows %= TILE_PAIRS      # pairs of units are that product's too: the others take unit by unit
        _check(a_rows, k, "a_rows", torch.int32)
        _check(tile_group, k, "tile_group", torch.int32)
        _check(n_tiles, k, "n_tiles", torch.int32)
        M = a_rows.numel()
        unit = tile_rows % TILE_PAIRS
        _need(M % unit == 0 and tile_group.numel() >= M // unit, k, "a_rows must hold whole tiles, each with a group")
        _need(tile_rows == unit or (tile_group.numel() >= 2 * (M // unit) and n_tiles.numel() >= 2), k,
              "pairs of tiles need the items behind the row tiles (tile_group [2 M / 64], n_tiles [2])")
        N = w.shape[1]
        gstride = N * K
    else:
        _need(w.dim() == 2 and w.shape[1] == K, k, lambda: f"w must be [N, {K}], is {tuple(w.shape)}")
        N = w.shape[0]
        M = a.shape[0] if a_rows is None else a_rows.numel()
        if a_rows is not None:
            _check(a_rows, k, "a_rows", torch.int32)
        gstride = 0
        if tile_rows is None:
            tile_rows = 16 if M <= 32 else 64
    if w2 is not None:
        _check(w2, k, "w2", w.dtype, tuple(w.shape))
    if bias is not None:
        _check(bias, k, "bias", tuple(_WTYPE), (N,))
    return M, N, K, tile_rows, gstride


# Plain bfloat16 products of many rows may go through the vendor's matrix library (hipBLASLt behind torch.mm), as the
# reference's engine hands its plain products to a BLAS where it has one
# (/root/reference/src/engine/tq_ops.c:296-305): measured on gfx950 it is 25 to 35 % faster than the tile kernel here
# from 512 rows on ([2048, 2048] x [6144, 2048]: 48 against 63 us; 13,199 rows: 282 against 401), slower or equal
# below and where k is long and the rows are not many ([4096, 20480] x [3584, 20480]: 724 against 687 us).  A call
# into the library costs the host twice what a launch here costs, and a step of 512 to 767 rows is as long on the
# host as on the chip (24 layers of 512 tokens: 9.7 ms through the library, 7.9 without), so it starts at 768 rows.
# TQ_PLAIN_PRODUCTS=own keeps every product in this library's kernels.  Products over experts, gated pairs whose
# matrices lie apart, products with a bias that nothing behind them can add, products of few rows, decode steps,
# steps under graph capture and the 32-bit path never leave them.
VENDOR_MIN_ROWS = 768
_VENDOR = os.environ.get("TQ_PLAIN_PRODUCTS", "vendor") != "own"


class own_products:
    """``with own_products(True):`` keeps every product inside in this library's kernels: what a decode step runs
    eagerly must be what its capture will replay, however many sequences it has."""

    def __init__(self, on: bool = True):
        self.on = on

    def __enter__(self):
        global _VENDOR
        self.before = _VENDOR
        if self.on:
            _VENDOR = False

    def __exit__(self, *exc):
        global _VENDOR
        _VENDOR = self.before


def _vendor_product(act, a, w, M: int, K: int) -> bool:
    return (_VENDOR and M >= VENDOR_MIN_ROWS and (K < 16384 or M >= 8192) and dtype_name(act) == "bfloat16"
            and w.dtype == torch.bfloat16 and a.stride(1) == 1 and w.is_contiguous()
            and not torch.cuda.is_current_stream_capturing())


def _vendor_gemm(a, w, out_act: bool) -> torch.Tensor:
    """a w^T by the vendor library: sums in float32, stored as bfloat16 or float32.  It adds no bias: its product
    with one takes a pass more over the result (77 against 48 us), so a product with a bias stays here unless the
    caller has a kernel behind it that adds the bias on its way."""
    out = torch.mm(a, w.t()) if out_act else torch.mm(a, w.t(), out_dtype=torch.float32)
    if _PROFILE is not None:
        _mark("matmul")
    return out


VENDOR_GATED_ROWS = 4096      # rows of a gated pair that go through the vendor library at a time


def side_by_side(first: torch.Tensor, second: torch.Tensor) -> tuple[torch.Tensor, torch.Tensor]:
    """The two matrices of a gated pair in one piece of memory, the second right behind the first: so laid, ``gemm``
    may hand a pair of many rows to the vendor library as one product over both."""
    both = torch.cat([first, second])
    return both[:first.shape[0]], both[first.shape[0]:]


def _behind(w: torch.Tensor, w2: torch.Tensor) -> bool:
    return (w2.is_contiguous() and w2.untyped_storage().data_ptr() == w.untyped_storage().data_ptr()
            and w2.data_ptr() == w.data_ptr() + w.numel() * w.element_size())


def _vendor_gated(a, w, N: int, K: int, gate: int, act) -> torch.Tensor:
    """f(a w^T) * (a w2^T) with w2 behind w: one product of the vendor library over both matrices into float32, a
    few thousand rows at a time, and the gate's activation in a pass of its own."""
    both = torch.as_strided(w, (2 * N, K), (K, 1))
    M = a.shape[0]
    out = torch.empty((M, N), dtype=ACT_DTYPES[dtype_name(act)], device=a.device)
    lib = library(act)
    for r in range(0, M, VENDOR_GATED_ROWS):
        rows = min(VENDOR_GATED_ROWS, M - r)
        gu = torch.mm(a[r:r + rows], both.t(), out_dtype=torch.float32)
        if _PROFILE is not None:
            _mark("matmul")
        _run("gated_act", lib.tq_gated_act(_ptr(gu), 2 * N, _ptr(out[r:]), rows, N, gate, _stream()))
    return out


def _gate_code(k: str, activation: str) -> int:
    _need(activation in GATES, k, lambda: f"unknown activation {activation!r}; known: {', '.join(sorted(GATES))}")
    return GATES[activation]


def _use_f32(act, a: torch.Tensor, w: torch.Tensor, K: int, gstride: int) -> bool:
    """The float matrix-core product takes float operands whose rows start at multiples of 16 bytes."""
    return (dtype_name(act) == "float32" and w.dtype == torch.float32 and a.dtype == torch.float32 and K % 4 == 0
            and a.stride(0) % 4 == 0 and gstride % 4 == 0 and a.data_ptr() % 16 == 0 and w.data_ptr() % 16 == 0
            and has_kernel(act, "tq_gemm_f32"))


def gemm(a: torch.Tensor, w: torch.Tensor, act, bias: torch.Tensor | None = None, w2: torch.Tensor | None = None,
         out_act: bool = False, a_rows: torch.Tensor | None = None, tile_group: torch.Tensor | None = None,
         n_tiles: torch.Tensor | None = None, tile_rows: int | None = None, gather: bool = True,
         partial_sums: bool = False, activation: str = "silu", act_alone: bool = False,
         pair_limit: float | None = None) -> torch.Tensor:
    """out[m, n] = sum_k a[row(m), k] * w[g, n, k]  (+ bias[n]);  with ``w2``: f(a w^T) * (a w2^T), f being the
    ``activation`` (a name of GATES); with ``pair_limit`` L beside it: f(min(a w^T, L)) * (clamp(a w2^T, -L, L) + 1).  ``act_alone`` (a plain product, no ``w2``): f of the product, in the
    activation type: in the product's own epilogue where this library's matrix-core kernel runs it, else in a launch
    of its own behind it.

    ``a`` [M, K] activations.  ``w`` [N, K], or [G, N, K] with ``tile_group`` naming the matrix of each tile of
    ``tile_rows`` output rows and ``a_rows`` [P] the row of ``a`` behind each output row (-1: none; with
    ``gather`` false a live output row m reads row m of ``a``).
    Output is float32 unless ``out_act``.  Sums run over k in ascending order whatever M is.
    ``partial_sums`` (plain products into float32 only): the result is [S, M, N], S >= 1 partial sums over runs of
    k that the caller adds up in order, as the next norm does with a part's output; the kernel chooses S.
    """
    k = "gemm"
    if pair_limit is not None:
        # the launchers read the limit as they fill their argument blocks; from there on it is a kernel argument
        _need(w2 is not None and pair_limit > 0, k, "a limit is for gated pairs and positive")
        lib = library(act)
        lib.tq_set_pair_limit(float(pair_limit))
        try:
            return gemm(a, w, act, bias=bias, w2=w2, out_act=out_act, a_rows=a_rows, tile_group=tile_group, n_tiles=n_tiles,
                        tile_rows=tile_rows, gather=gather, partial_sums=partial_sums, activation=activation)
        finally:
            lib.tq_set_pair_limit(0.0)
    adt = ACT_DTYPES[dtype_name(act)]
    grouped = tile_group is not None
    M, N, K, tile_rows, gstride = _gemm_problem(k, a, w, act, bias, w2, out_act, a_rows, tile_group, n_tiles, tile_rows,
                                                gather)
    if partial_sums:
        _need(w2 is None and not out_act and not grouped and a_rows is None, k,
              "partial sums are for plain products into float32")
    lib = library(act)
    gate = _gate_code(k, activation)
    if act_alone and (grouped or a_rows is not None):
        # a product over experts whose result passes an activation: in the matrix-core product's own epilogue, else behind it
        _need(w2 is None and not partial_sums and out_act, k, "an activation alone leaves its result in the activation type")
        if _use_mfma(act, a, w, K) and (bias is None or bias.dtype in _WTYPE):
            out = torch.empty((M, N), dtype=adt, device=a.device)
            _run("gemm_mfma", lib.tq_gemm_mfma(_ptr(a), a.stride(0), _ptr(a_rows), int(gather), _ptr(w), None, gstride,
                                               _ptr(tile_group), _ptr(n_tiles), _ptr(bias),
                                               _WTYPE[bias.dtype] if bias is not None else 0, _ptr(out), N, 1, M, N, K,
                                               tile_rows, 1, gate + 256, _stream()), "moe" if grouped else None)
            return out
        return act_rows(gemm(a, w, act, bias=bias, a_rows=a_rows, tile_group=tile_group, n_tiles=n_tiles, tile_rows=tile_rows,
                             gather=gather), None, activation, act)
    if act_alone:
        _need(w2 is None and not partial_sums and not grouped and a_rows is None, k, "an activation alone is for plain products")
        if (dtype_name(act) == "bfloat16" and not (bias is None and _vendor_product(act, a, w, M, K))
                and _use_mfma(act, a, w, K) and (bias is None or bias.dtype in _WTYPE)):
            out = torch.empty((M, N), dtype=adt, device=a.device)
            _run("gemm_mfma", lib.tq_gemm_mfma(_ptr(a), a.stride(0), None, 1, _ptr(w), None, gstride, None, None, _ptr(bias),
                                               _WTYPE[bias.dtype] if bias is not None else 0, _ptr(out), N, 1, M, N, K,
                                               tile_rows, 1, gate + 256, _stream()))
            return out
        return act_rows(gemm(a, w, act, bias=bias), None, activation, act)
    if not grouped and a_rows is None and bias is None and _vendor_product(act, a, w, M, K):
        if w2 is None:
            out = _vendor_gemm(a, w, out_act)
            return out[None] if partial_sums else out
        if out_act and _behind(w, w2):
            return _vendor_gated(a, w, N, K, gate, act)
    if _use_mfma(act, a, w, K) and (bias is None or bias.dtype in _WTYPE):
        splits = lib.tq_gemm_mfma_splits(M, N, K) if partial_sums else 1
        out = torch.empty((splits, M, N) if partial_sums else (M, N), dtype=adt if out_act else torch.float32,
                          device=a.device)
        _run("gemm_mfma", lib.tq_gemm_mfma(_ptr(a), a.stride(0), _ptr(a_rows), int(gather), _ptr(w), _ptr(w2), gstride,
                                           _ptr(tile_group), _ptr(n_tiles), _ptr(bias),
                                           _WTYPE[bias.dtype] if bias is not None else 0, _ptr(out), N, int(out_act),
                                           M, N, K, tile_rows, splits, gate, _stream()), "moe" if grouped else None)
        return out
    if _use_f32(act, a, w, K, gstride) and (w2 is None or w2.data_ptr() % 16 == 0):
        # a narrow matrix times few rows is cut into runs of k: they come back apart if the caller adds them up
        # anyway, else they pass through scratch memory and a second kernel
        runs = lib.tq_gemm_f32_runs(M, N, K, int(grouped or a_rows is not None))
        out = torch.empty((runs, M, N) if partial_sums else (M, N), dtype=torch.float32, device=a.device)
        scratch = None
        if runs > 1 and not partial_sums:
            scratch = torch.empty((runs * (2 if w2 is not None else 1), M, N), dtype=torch.float32, device=a.device)
        _run("gemm_f32", lib.tq_gemm_f32(_ptr(a), a.stride(0), _ptr(a_rows), int(gather), _ptr(w), _ptr(w2), gstride,
                                         _ptr(tile_group), _ptr(n_tiles), _ptr(bias),
                                         _WTYPE[bias.dtype] if bias is not None else 0, _ptr(out), N, M, N, K, tile_rows,
                                         gate, _ptr(scratch), int(partial_sums and runs > 1), _stream()),
             "moe" if grouped else None)
        return out
    out = torch.empty((1, M, N) if partial_sums else (M, N), dtype=adt if out_act else torch.float32, device=a.device)
    _run(k, lib.tq_gemm_generic(_ptr(a), a.stride(0), _ptr(a_rows), int(gather), _ptr(w), _ptr(w2), _WTYPE[w.dtype], gstride,
                                _ptr(tile_group), _ptr(n_tiles), _ptr(bias),
                                _WTYPE[bias.dtype] if bias is not None else 0, _ptr(out), N, int(out_act), M, N, K,
                                tile_rows, gate, _stream()), "moe" if grouped else None)
    return out


def gemm_pair(first: dict, second: dict, act) -> tuple[torch.Tensor, torch.Tensor]:
    """Two products that do not depend on each other; ``first`` and ``second`` hold the arguments of ``gemm``
    (``partial_sums`` only in the second).  Products of few rows of the same kind (both gated or both plain, into
    the same type) go out in one launch, so that the smaller one costs no launch of its own; anything else is two
    calls."""
    k = "gemm_pair"
    keys = ("bias", "w2", "out_act", "a_rows", "tile_group", "n_tiles", "tile_rows", "gather", "partial_sums", "activation",
            "pair_limit")
    probs = []
    _need(not first.get("partial_sums", False), k, "only the second product may leave partial sums")
    for p in (first, second):
        full = {"bias": None, "w2": None, "out_act": False, "a_rows": None, "tile_group": None, "n_tiles": None,
                "tile_rows": None, "gather": True, "partial_sums": False, "activation": "silu", "pair_limit": None}
        _need(set(p) <= set(full) | {"a", "w"}, k, lambda: f"unknown arguments {sorted(set(p) - set(full) - {'a', 'w'})}")
        full.update(p)
        _need(full["pair_limit"] is None or (full["w2"] is not None and full["pair_limit"] > 0), k,
              "a limit is for gated pairs and positive")
        probs.append(full)
    lib = library(act) if dtype_name(act) == "bfloat16" else None
    fused = lib is not None and hasattr(lib, "tq_gemm_mfma_pair")
    dims = []
    for p in probs:
        M, N, K, tile_rows, gstride = _gemm_problem(k, p["a"], p["w"], act, p["bias"], p["w2"], p["out_act"], p["a_rows"],
                                                    p["tile_group"], p["n_tiles"], p["tile_rows"], p["gather"])
        dims.append((M, N, K, tile_rows, gstride))
        few = (p["tile_group"] is not None and tile_rows == 16) or (p["tile_group"] is None and M <= 16)
        fused = fused and few and _use_mfma(act, p["a"], p["w"], K) and (p["bias"] is None or p["bias"].dtype in _WTYPE)
    fused = fused and (probs[0]["w2"] is None) == (probs[1]["w2"] is None) and probs[0]["out_act"] == probs[1]["out_act"]
    if not fused:
        return tuple(gemm(p["a"], p["w"], act, **{n: p[n] for n in keys}) for p in probs)
    adt = ACT_DTYPES[dtype_name(act)]
    outs, descs = [], []
    splits = 1
    if probs[1]["partial_sums"]:
        p2 = probs[1]
        _need(p2["w2"] is None and not p2["out_act"] and p2["tile_group"] is None and p2["a_rows"] is None, k,
              "partial sums are for plain products into float32")
        splits = lib.tq_gemm_mfma_pair_splits(dims[0][1], dims[0][2], int(probs[0]["tile_group"] is not None),
                                              dims[1][1], dims[1][2], 0)
    for p, (M, N, K, tile_rows, gstride) in zip(probs, dims):
        shape = (splits, M, N) if p["partial_sums"] else (M, N)
        out = torch.empty(shape, dtype=adt if p["out_act"] else torch.float32, device=p["a"].device)
        outs.append(out)
        vals = [_ptr(p["a"]), p["a"].stride(0), _ptr(p["a_rows"]), int(p["gather"]), _ptr(p["w"]), _ptr(p["w2"]), gstride,
                _ptr(p["tile_group"]), _ptr(p["n_tiles"]), _ptr(p["bias"]),
                _WTYPE[p["bias"].dtype] if p["bias"] is not None else 0, _ptr(out), N, int(p["out_act"]), M, N, K, tile_rows,
                _gate_code(k, p["activation"]), struct.unpack("<I", struct.pack("<f", p["pair_limit"] or 0.0))[0]]
        descs.append((ctypes.c_int64 * 20)(*[0 if v is None else int(v) for v in vals]))
    _run(k, lib.tq_gemm_mfma_pair(descs[0], descs[1], splits, _stream()),
         "moe" if any(p["tile_group"] is not None for p in probs) else None)
    return outs[0], outs[1]


# ------------------------------------------------------------------ attention
def attention(q: torch.Tensor, k_pages: torch.Tensor, v_pages: torch.Tensor, layer_offset: int,
              positions: torch.Tensor, seq_of_token: torch.Tensor, block_table: torch.Tensor, page_size: int,
              page_stride: int, num_heads: int, num_kv_heads: int, head_dim: int, window: int | None,
              scale: float, act, runs: dict | None = None, softcap: float | None = None,
              distance_bias: tuple[torch.Tensor, torch.Tensor] | None = None, chunk: int | None = None,
              sink: torch.Tensor | None = None, value_width: int | None = None,
              head_gate: torch.Tensor | None = None, sigmoid_bias: torch.Tensor | None = None,
              keep_first: int = 0, out: torch.Tensor | None = None) -> torch.Tensor:
    """Each token attends to its sequence's cached positions up to its own; returns [T, nh*hd].

    ``out`` (bfloat16 only, see ``attention_writes_into``): where the result goes, columns of a wider matrix.

    ``value_width``: a head's value rows hold zeros behind their first ``value_width`` numbers (keys wider than values, both
    laid out at the keys' width); the output is zero there, and a kernel may leave those dimensions out.
    ``head_gate`` float32 [T, nh] (rows may be runs of columns of a wider tensor): head h's output of token t is multiplied by
    sigmoid(head_gate[t, h]), in the kernel that normalises the output where it knows how, else by ``gate_heads`` behind it.

    ``softcap`` c: a scaled score s becomes c tanh(s / c).  ``distance_bias`` (r1, r2), float32 [nh] each: then
    r1[h] ln(1 + r2[h] (i - j)) is taken off the score of query position i and key position j.  ``chunk`` n: position i
    sees j only if i // n == j // n, beside j <= i and the window.  ``sink`` float32 [nh]: the softmax's denominator of
    head h also holds exp(sink[h]), a score without key and value that is neither scaled nor capped and counts once.
    ``sigmoid_bias`` float32 [nh]: no softmax; the weight of a visible key is sigmoid(score + sigmoid_bias[h]) and the
    weights are not normalised over the keys.  ``keep_first`` n: the sequence's first n positions stay visible to every
    later token, whatever the window.

    ``seq_of_token`` gives each token's row of ``block_table`` (its slot).  ``runs`` describes the same tokens
    as runs of consecutive positions, one per sequence, for the kernels that work on tiles of tokens:
    ``cu_seqlens`` [B+1], ``slots`` [B], ``start`` [B] (device, int32) and the host numbers ``max_new``,
    ``max_end`` and ``decode`` (every sequence brings one token).  Without it the token-by-token kernel runs."""
    k = "attention"
    adt = ACT_DTYPES[dtype_name(act)]
    T = positions.numel()
    _check(q, k, "q", adt, (T, num_heads * head_dim))
    _check(k_pages, k, "k_pages", adt)
    _check(v_pages, k, "v_pages", adt)
    _check(positions, k, "positions", torch.int32, (T,))
    _check(seq_of_token, k, "seq_of_token", torch.int32, (T,))
    _check(block_table, k, "block_table", torch.int32)
    _need(block_table.dim() == 2, k, "block_table must be [B, pages]")
    _need(num_heads % num_kv_heads == 0, k, "heads must be a multiple of kv heads")
    _need(head_dim <= 512, k, lambda: f"head size {head_dim} is beyond the 512 this kernel takes")
    _need(layer_offset + num_kv_heads * page_size * head_dim <= page_stride, k, "layer does not fit in a page")
    _need(value_width is None or 1 <= value_width <= head_dim, k, "the values' width lies within the head")
    _need(head_gate is None or (isinstance(head_gate, torch.Tensor) and head_gate.is_cuda and head_gate.dtype == torch.float32
                                and tuple(head_gate.shape) == (T, num_heads) and head_gate.stride(1) == 1), k,
          lambda: f"head_gate must be float32 [{T}, {num_heads}] on the GPU with unit stride along its rows")
    into = out is not None
    if into:
        _need(out.is_cuda and out.dtype == adt and tuple(out.shape) == tuple(q.shape) and out.stride(1) == 1
              and out.stride(0) % 8 == 0 and out.data_ptr() % 16 == 0, k, "out must be columns of a matrix of the activation type, 16 bytes aligned")
    else:
        out = torch.empty_like(q)
    esz = k_pages.element_size()
    lib = library(act)
    cap = float(softcap or 0.0)
    _need(cap >= 0 and (chunk is None or chunk >= 1), k, "softcap and chunk must be positive")
    r1 = r2 = None
    if distance_bias is not None:
        r1, r2 = distance_bias
        _check(r1, k, "r1", torch.float32, (num_heads,))
        _check(r2, k, "r2", torch.float32, (num_heads,))
    if sink is not None:
        _check(sink, k, "sink", torch.float32, (num_heads,))
    if sigmoid_bias is not None:
        _check(sigmoid_bias, k, "sigmoid_bias", torch.float32, (num_heads,))
        _need(sink is None, k, "sigmoid weights have no denominator for a sink to join")
    _need(keep_first >= 0, k, "keep_first counts positions")
    mod = (cap, _ptr(r1), _ptr(r2), int(chunk or 0), _ptr(sink))
    sig = (_ptr(sigmoid_bias), int(keep_first))
    if (runs is not None and dtype_name(act) == "bfloat16" and hasattr(lib, "tq_attention_mfma")
            and head_dim % 16 == 0 and head_dim <= 512 and page_size % 64 == 0 and page_stride % 8 == 0 and scale > 0
            and ((sigmoid_bias is None and keep_first == 0) or hasattr(lib, "tq_attention_mfma_sig"))):
        B = runs["slots"].numel()
        _check(runs["cu_seqlens"], k, "cu_seqlens", torch.int32, (B + 1,))
        _check(runs["slots"], k, "slots", torch.int32, (B,))
        _check(runs["start"], k, "start", torch.int32, (B,))
        _need(runs["max_end"] <= block_table.shape[1] * page_size, k, "positions reach beyond the page table")
        partial = None
        if runs["decode"]:
            _need(T == B, k, "decoding brings one token per sequence")
            partial = torch.empty((lib.tq_attention_decode_scratch(B, num_heads, head_dim, int(runs["max_end"])),),
                                  dtype=torch.float32, device=q.device)
        plain = sigmoid_bias is None and keep_first == 0 and not into
        _run("attention_mfma", (lib.tq_attention_mfma_ex if plain else lib.tq_attention_mfma_ld if into else lib.tq_attention_mfma_sig)(
            _ptr(q), k_pages.data_ptr() + layer_offset * esz, v_pages.data_ptr() + layer_offset * esz,
            _ptr(block_table), block_table.shape[1], _ptr(runs["cu_seqlens"]), _ptr(runs["slots"]), _ptr(runs["start"]),
            page_size, page_stride, B, num_heads, num_kv_heads, head_dim, int(window or 0), float(scale), *mod, _ptr(out),
            _ptr(partial), int(bool(runs["decode"])), int(runs["max_new"]), int(runs["max_end"]), int(value_width or 0),
            _ptr(head_gate), head_gate.stride(0) if head_gate is not None else 0, *(() if plain else sig), *((out.stride(0),) if into else ()), _stream()))
        return out
    _need(not into, k, "only the bfloat16 matrix-core kernels write into columns of a wider matrix")
    if (runs is not None and dtype_name(act) == "float32" and hasattr(lib, "tq_attention_f32") and head_dim % 4 == 0
            and head_dim <= 256 and page_size % 64 == 0 and page_stride % 4 == 0 and layer_offset % 4 == 0):
        B = runs["slots"].numel()
        _check(runs["cu_seqlens"], k, "cu_seqlens", torch.int32, (B + 1,))
        _check(runs["slots"], k, "slots", torch.int32, (B,))
        _check(runs["start"], k, "start", torch.int32, (B,))
        _need(runs["max_end"] <= block_table.shape[1] * page_size, k, "positions reach beyond the page table")
        partial = None
        if runs["decode"]:
            _need(T == B, k, "decoding brings one token per sequence")
            partial = torch.empty((lib.tq_attention_f32_scratch(B, num_heads, head_dim, int(runs["max_end"])),),
                                  dtype=torch.float32, device=q.device)
        _run("attention_f32", lib.tq_attention_f32_sig(
            _ptr(q), k_pages.data_ptr() + layer_offset * esz, v_pages.data_ptr() + layer_offset * esz,
            _ptr(block_table), block_table.shape[1], _ptr(runs["cu_seqlens"]), _ptr(runs["slots"]), _ptr(runs["start"]),
            page_size, page_stride, B, num_heads, num_kv_heads, head_dim, int(window or 0), float(scale), *mod, *sig, _ptr(out),
            _ptr(partial), int(bool(runs["decode"])), int(runs["max_new"]), int(runs["max_end"]), _stream()))
        return out if head_gate is None else gate_heads(out, head_gate, num_heads, "sigmoid", act)
    _run(k, lib.tq_attention_generic_sig(_ptr(q), k_pages.data_ptr() + layer_offset * esz,
                                         v_pages.data_ptr() + layer_offset * esz, _ptr(positions),
                                         _ptr(seq_of_token), _ptr(block_table), block_table.shape[1], page_size,
                                         page_stride, T, num_heads, num_kv_heads, head_dim, int(window or 0),
                                         float(scale), *mod, *sig, _ptr(out), _stream()))
    return out if head_gate is None else gate_heads(out, head_gate, num_heads, "sigmoid", act)


def attention_writes_into(act, head_dim: int, scale: float) -> bool:
    """Whether ``attention`` takes ``out``: heads and scale that the bfloat16 matrix-core kernels run (with pages of whole tiles)."""
    return dtype_name(act) == "bfloat16" and head_dim % 16 == 0 and head_dim <= 512 and scale > 0


# ------------------------------------------------------------------ routing
def _expert_groups(k: str, E: int, top_k: int, groups, pairs: bool = False) -> tuple[int, int]:
    """(count, keep) of a choice within the best ``keep`` of ``count`` equal groups of neighbouring experts."""
    if groups is None:
        return 1, 1
    count, keep = int(groups[0]), int(groups[1])
    _need(1 <= count <= 256 and E % count == 0 and 1 <= keep <= count and top_k <= keep * (E // count), k,
          lambda: f"{count} groups of which {keep} are kept do not fit {E} experts with {top_k} per token")
    if keep == count or (keep >= top_k and not pairs):
        # nothing is ever left out: the best top_k experts lie in at most top_k groups, each of which has a better best
        # expert than any group without one of them, so all of these groups are among the kept
        return 1, 1
    return count, keep


def router_topk(x32: torch.Tensor, router: torch.Tensor, shared_scale: torch.Tensor | None, top_k: int,
                renormalize: bool, act, groups: tuple[int, int] | None = None, bias: torch.Tensor | None = None,
                sigmoid: bool = False, weight_scale: float = 1.0, pair_groups: bool = False):
    """ids int32 [T, k], weights float32 [T, k], and sigmoid(x . shared_scale) float32 [T] (or None).
    ``groups`` (count, keep): only experts of the ``keep`` groups with the largest best score can be chosen.
    ``bias`` float32 [E]: added to the experts' logits before the choice.
    ``sigmoid``: no softmax; an expert's score is the sigmoid of its logit, and the weights are the chosen scores over (their
    sum + 1e-20), times ``weight_scale`` (``renormalize`` true says so too).  ``weight_scale`` without it: the softmax over the
    chosen logits (``renormalize`` true) times that.  ``pair_groups`` (with ``sigmoid``): a group's score is the
    sum of its two largest scores instead of its largest."""
    k = "router_topk"
    T, H, E, ids, weights, gate, logits = _router_outputs(k, x32, router, shared_scale, top_k)
    count, keep = _expert_groups(k, E, top_k, groups, pair_groups)
    if bias is not None:
        _check(bias, k, "bias", torch.float32, (E,))
    _need(sigmoid or not pair_groups, k, "groups by their two best go with sigmoid scores")
    _need(not (sigmoid or weight_scale != 1.0) or renormalize, k, "sigmoid scores, and weights with a scale, are renormalised over the chosen")
    if sigmoid:
        _run(k, library(act).tq_router_topk_sigmoid(_ptr(x32), _ptr(router), _ptr(shared_scale), _ptr(bias), _WTYPE[router.dtype],
                                                    E, top_k, count, keep, int(pair_groups), float(weight_scale), _ptr(ids),
                                                    _ptr(weights), _ptr(gate), _ptr(logits), T, H, _stream()))
        return ids, weights, gate
    if weight_scale != 1.0:
        _run(k, library(act).tq_router_topk_weighted(_ptr(x32), _ptr(router), _ptr(shared_scale), _ptr(bias), _WTYPE[router.dtype],
                                                     E, top_k, count, keep, float(weight_scale), _ptr(ids), _ptr(weights),
                                                     _ptr(gate), _ptr(logits), T, H, _stream()))
        return ids, weights, gate
    _run(k, library(act).tq_router_topk_biased(_ptr(x32), _ptr(router), _ptr(shared_scale), _ptr(bias), _WTYPE[router.dtype], E,
                                               top_k, int(bool(renormalize)), count, keep, _ptr(ids), _ptr(weights), _ptr(gate),
                                               _ptr(logits), T, H, _stream()))
    return ids, weights, gate


def _router_outputs(k: str, x32: torch.Tensor, router: torch.Tensor, shared_scale: torch.Tensor | None, top_k: int):
    _check(x32, k, "x", torch.float32)
    _need(x32.dim() == 2, k, "x must be [T, H]")
    T, H = x32.shape
    _check(router, k, "router", tuple(_WTYPE))
    _need(router.dim() == 2 and router.shape[1] == H, k, lambda: f"router must be [E, {H}]")
    E = router.shape[0]
    _need(1 <= top_k <= min(E, 64), k, lambda: f"top_k {top_k} must be within 1..min(E, 64)")
    if shared_scale is not None:
        _check(shared_scale, k, "shared_scale", router.dtype)
        _need(shared_scale.numel() == H, k, lambda: f"shared_scale must hold {H} values")
    ids = torch.empty((T, top_k), dtype=torch.int32, device=x32.device)
    weights = torch.empty((T, top_k), dtype=torch.float32, device=x32.device)
    gate = torch.empty((T,), dtype=torch.float32, device=x32.device) if shared_scale is not None else None
    logits = torch.empty((T, E + (1 if shared_scale is not None else 0)), dtype=torch.float32, device=x32.device)
    return T, H, E, ids, weights, gate, logits


def _align_outputs(T: int, topk: int, num_experts: int, unit: int, dev):
    n_pairs = T * topk
    # every expert with at least one pair wastes at most unit-1 rows
    cap = n_pairs + min(num_experts, n_pairs) * (unit - 1)
    cap = (cap + unit - 1) // unit * unit
    sorted_token = torch.empty((cap,), dtype=torch.int32, device=dev)
    pair_slot = torch.empty((T, topk), dtype=torch.int32, device=dev)
    tile_expert = torch.empty((2 * (cap // unit),), dtype=torch.int32, device=dev)      # row tiles, then items of two
    n_tiles = torch.empty((2,), dtype=torch.int32, device=dev)
    return cap, sorted_token, pair_slot, tile_expert, n_tiles


def route(x32: torch.Tensor, router: torch.Tensor, shared_scale: torch.Tensor | None, top_k: int, renormalize: bool,
          unit: int, act, groups: tuple[int, int] | None = None, bias: torch.Tensor | None = None,
          correction: torch.Tensor | None = None, identity: int = 0, sigmoid: bool = False, weight_scale: float = 1.0,
          pair_groups: bool = False):
    """``router_topk`` followed by ``moe_align`` in one call: (ids, weights, gate, sorted_token, pair_slot,
    tile_expert, n_tiles), with the same results; a handful of tokens takes one kernel less.

    ``correction`` float32 [E] (with ``renormalize`` false and neither groups, bias nor shared gate): the softmax runs over
    all E rows of the router, the choice is by score + correction and the weights are the scores themselves.  ``identity`` n
    (with ``correction``): the router's last n rows are experts without matrices whose output is their input; their pairs
    get ``pair_slot`` -1 and no rows in the order, and ``gate`` [T] is the sum of each token's weights for them.
    ``sigmoid``, ``weight_scale``, ``pair_groups``: as for ``router_topk``."""
    k = "route"
    T, H, E, ids, weights, gate, logits = _router_outputs(k, x32, router, shared_scale, top_k)
    _need(unit in (16, 32, 64, 128, 256), k, "unit must be 16, 32, 64, 128 or 256")
    if correction is not None:
        _need(not renormalize and groups is None and bias is None and shared_scale is None and 0 <= identity < E, k,
              "a choice by corrected scores goes with plain softmax weights over all experts, of which some are real")
        _check(correction, k, "correction", torch.float32, (E,))
        if identity:
            gate = torch.empty((T,), dtype=torch.float32, device=x32.device)
        cap, sorted_token, pair_slot, tile_expert, n_tiles = _align_outputs(T, top_k, E, unit, x32.device)
        _run(k, library(act).tq_route_scored(_ptr(x32), _ptr(router), _ptr(correction), _WTYPE[router.dtype], E, E - identity,
                                             top_k, _ptr(ids), _ptr(weights), _ptr(gate), _ptr(logits), unit, cap,
                                             _ptr(sorted_token), _ptr(pair_slot), _ptr(tile_expert), _ptr(n_tiles), T, H,
                                             _stream()))
        return ids, weights, gate, sorted_token, pair_slot, tile_expert, n_tiles
    _need(identity == 0, k, "experts that are the identity come with a choice by corrected scores")
    count, keep = _expert_groups(k, E, top_k, groups, pair_groups)
    if bias is not None:
        _check(bias, k, "bias", torch.float32, (E,))
    _need(sigmoid or not pair_groups, k, "groups by their two best go with sigmoid scores")
    _need(not (sigmoid or weight_scale != 1.0) or renormalize, k, "sigmoid scores, and weights with a scale, are renormalised over the chosen")
    cap, sorted_token, pair_slot, tile_expert, n_tiles = _align_outputs(T, top_k, E, unit, x32.device)
    if sigmoid:
        _run(k, library(act).tq_route_sigmoid(_ptr(x32), _ptr(router), _ptr(shared_scale), _ptr(bias), _WTYPE[router.dtype], E,
                                              top_k, count, keep, int(pair_groups), float(weight_scale), _ptr(ids), _ptr(weights),
                                              _ptr(gate), _ptr(logits), unit, cap, _ptr(sorted_token), _ptr(pair_slot),
                                              _ptr(tile_expert), _ptr(n_tiles), T, H, _stream()))
        return ids, weights, gate, sorted_token, pair_slot, tile_expert, n_tiles
    if weight_scale != 1.0:
        _run(k, library(act).tq_route_weighted(_ptr(x32), _ptr(router), _ptr(shared_scale), _ptr(bias), _WTYPE[router.dtype], E,
                                               top_k, count, keep, float(weight_scale), _ptr(ids), _ptr(weights), _ptr(gate),
                                               _ptr(logits), unit, cap, _ptr(sorted_token), _ptr(pair_slot), _ptr(tile_expert),
                                               _ptr(n_tiles), T, H, _stream()))
        return ids, weights, gate, sorted_token, pair_slot, tile_expert, n_tiles
    _run(k, library(act).tq_route_biased(_ptr(x32), _ptr(router), _ptr(shared_scale), _ptr(bias), _WTYPE[router.dtype], E, top_k,
                                         int(bool(renormalize)), count, keep, _ptr(ids), _ptr(weights), _ptr(gate),
                                         _ptr(logits), unit, cap, _ptr(sorted_token), _ptr(pair_slot), _ptr(tile_expert),
                                         _ptr(n_tiles), T, H, _stream()))
    return ids, weights, gate, sorted_token, pair_slot, tile_expert, n_tiles


def moe_align(ids: torch.Tensor, num_experts: int, unit: int, act):
    """Orders the (token, expert) pairs by expert.  Returns sorted_token [cap], pair_slot [T, k],
    tile_expert [cap/unit], n_tiles [1]; each expert's rows start at a multiple of ``unit``."""
    k = "moe_align"
    _check(ids, k, "ids", torch.int32)
    T, topk = ids.shape
    n_pairs = T * topk
    cap, sorted_token, pair_slot, tile_expert, n_tiles = _align_outputs(T, topk, num_experts, unit, ids.device)
    _run(k, library(act).tq_moe_align(_ptr(ids), n_pairs, num_experts, topk, unit, cap, _ptr(sorted_token),
                                      _ptr(pair_slot), _ptr(tile_expert), _ptr(n_tiles), _stream()))
    return sorted_token, pair_slot, tile_expert, n_tiles


# ------------------------------------------------------------------ the gated delta rule
@dataclasses.dataclass(frozen=True)
class DeltaDims:
    """Sizes of a delta-rule mixer: heads, q/k heads, key width, value width, convolution taps, and the ranks of the
    decay's and the gate's first products."""
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    taps: int
    rank_a: int
    rank_g: int
    head_decay: bool = False      # one decay per head from a projection of its own, a full gate; no ranks

    @property
    def channels(self) -> int:
        return 2 * self.kv_heads * self.dim + self.heads * self.vdim

    @property
    def projections(self) -> int:
        if self.head_decay:        # q | k | v | b (H) | a (H) | gate (H V)
            return self.channels + 2 * self.heads + self.heads * self.vdim
        return self.channels + self.heads + self.rank_a + self.rank_g

    @property
    def state_floats(self) -> int:
        return self.heads * self.dim * self.vdim + self.channels * (self.taps - 1)

    def sizes(self):
        return self.heads, self.kv_heads, self.dim, self.vdim, self.taps


def _delta_state(k: str, state: torch.Tensor, dims: DeltaDims) -> int:
    _check(state, k, "state", torch.float32)
    _need(state.dim() == 2 and state.shape[1] >= dims.state_floats, k,
          lambda: f"state must be [slots, >= {dims.state_floats}], is {tuple(state.shape)}")
    _need(dims.heads % dims.kv_heads == 0 and 1 <= dims.dim <= 256 and 1 <= dims.taps <= 64, k,
          "heads must be a multiple of kv heads, the key width at most 256, the taps at most 64")
    return state.shape[1]


def delta_prep(proj: torch.Tensor, slot_of_token: torch.Tensor, state: torch.Tensor, conv_w: torch.Tensor,
               dims: DeltaDims, act):
    """From the float32 projections [T, q | k | v | b | a1 | g1] of a step's tokens: q and k after convolution, silu
    and scaling to unit length (q also by dim^-1/2) [T, G*dim], v after convolution and silu [T, H*vdim],
    beta = sigmoid(b) [T, H], all float32, and the low-rank activations [T, rank_a + rank_g] in the activation type.
    The convolution's inputs before a token's run are read from ``state`` [slots, floats]; nothing is written there."""
    k = "delta_prep"
    T = slot_of_token.numel()
    _check(proj, k, "proj", torch.float32, (T, dims.projections))
    _check(slot_of_token, k, "slot_of_token", torch.int32, (T,))
    stride = _delta_state(k, state, dims)
    _check(conv_w, k, "conv_w", torch.float32, (dims.channels, dims.taps))
    dev, f32 = proj.device, torch.float32
    G, D, H, V = dims.kv_heads, dims.dim, dims.heads, dims.vdim
    qn = torch.empty((T, G * D), dtype=f32, device=dev)
    kn = torch.empty((T, G * D), dtype=f32, device=dev)
    vc = torch.empty((T, H * V), dtype=f32, device=dev)
    beta = torch.empty((T, H), dtype=f32, device=dev)
    low = torch.empty((T, dims.rank_a + dims.rank_g), dtype=ACT_DTYPES[dtype_name(act)], device=dev)
    _run(k, library(act).tq_delta_prep(_ptr(proj), _ptr(slot_of_token), _ptr(state), stride, _ptr(conv_w), *dims.sizes(),
                                       dims.rank_a, dims.rank_g, _ptr(qn), _ptr(kn), _ptr(vc), _ptr(beta), _ptr(low), T,
                                       _stream()))
    return qn, kn, vc, beta, low


def delta_scan(qn: torch.Tensor, kn: torch.Tensor, vc: torch.Tensor, beta: torch.Tensor, ag: torch.Tensor,
               a_log: torch.Tensor, dt_bias: torch.Tensor, runs: dict, state: torch.Tensor, dims: DeltaDims, act):
    """The recurrence over each sequence's run of tokens, in order, from and into its row of ``state``:
    S <- diag(g) S; u = beta (v - S^T k); S <- S + k u^T; o = S^T q, with g = exp(-exp(a_log) softplus(a + dt_bias))
    from the first H*dim columns of ``ag`` [T, H*dim + H*vdim] (which a step of many tokens overwrites with those g).
    Returns o, float32 [T, H*vdim]."""
    k = "delta_scan"
    T = qn.shape[0]
    G, D, H, V = dims.kv_heads, dims.dim, dims.heads, dims.vdim
    for name, t, w in (("qn", qn, G * D), ("kn", kn, G * D), ("vc", vc, H * V), ("beta", beta, H), ("ag", ag, H * D + H * V)):
        _check(t, k, name, torch.float32, (T, w))
    _check(a_log, k, "a_log", torch.float32, (H,))
    _check(dt_bias, k, "dt_bias", torch.float32, (H * D,))
    stride = _delta_state(k, state, dims)
    B = runs["slots"].numel()
    _check(runs["cu_seqlens"], k, "cu_seqlens", torch.int32, (B + 1,))
    _check(runs["slots"], k, "slots", torch.int32, (B,))
    o = torch.empty((T, H * V), dtype=torch.float32, device=qn.device)
    _run(k, library(act).tq_delta_scan(_ptr(qn), _ptr(kn), _ptr(vc), _ptr(beta), _ptr(ag), _ptr(a_log), _ptr(dt_bias),
                                       _ptr(runs["cu_seqlens"]), _ptr(runs["slots"]), _ptr(state), stride, *dims.sizes(), T, B,
                                       _ptr(o), _stream()))
    return o


def delta_out(o: torch.Tensor, ag: torch.Tensor, norm_w: torch.Tensor, eps: float, proj: torch.Tensor, runs: dict,
              state: torch.Tensor, dims: DeltaDims, act) -> torch.Tensor:
    """Every head's read-out divided by its root mean square, times ``norm_w`` [vdim], times the sigmoid of the gate
    (the last H*vdim columns of ``ag``), in the activation type [T, H*vdim]; and the convolution's part of every
    sequence's state brought to the end of its run."""
    k = "delta_out"
    T = o.shape[0]
    H, D, V = dims.heads, dims.dim, dims.vdim
    _check(o, k, "o", torch.float32, (T, H * V))
    _check(ag, k, "ag", torch.float32, (T, H * D + H * V))
    _check(norm_w, k, "norm_w", torch.float32, (V,))
    _check(proj, k, "proj", torch.float32, (T, dims.projections))
    stride = _delta_state(k, state, dims)
    B = runs["slots"].numel()
    _check(runs["cu_seqlens"], k, "cu_seqlens", torch.int32, (B + 1,))
    _check(runs["slots"], k, "slots", torch.int32, (B,))
    out = torch.empty((T, H * V), dtype=ACT_DTYPES[dtype_name(act)], device=o.device)
    _run(k, library(act).tq_delta_out(_ptr(o), _ptr(ag), _ptr(norm_w), float(eps), _ptr(proj), _ptr(runs["cu_seqlens"]),
                                      _ptr(runs["slots"]), _ptr(state), stride, *dims.sizes(), dims.rank_a, dims.rank_g, T,
                                      B, _ptr(out), _stream()))
    return out


def delta_decode_fits(dims: DeltaDims) -> bool:
    """Whether a head's lanes (16 key channels of a value channel each) fit the one workgroup of ``delta_decode``."""
    nseg = 1
    while nseg * 16 < dims.dim:
        nseg *= 2
    return -(-nseg * dims.vdim // 64) * 64 <= 1024


def delta_decode(qn: torch.Tensor, kn: torch.Tensor, vc: torch.Tensor, beta: torch.Tensor, low: torch.Tensor,
                 low_weight: torch.Tensor, a_log: torch.Tensor, dt_bias: torch.Tensor, norm_w: torch.Tensor, eps: float,
                 proj: torch.Tensor, runs: dict, state: torch.Tensor, dims: DeltaDims, act) -> torch.Tensor:
    """A decode step (one token per sequence) from ``delta_prep``'s outputs to the mixer's output [T, H*vdim] in the
    activation type, in one launch: what the product over ``low_weight`` (the block-diagonal matrix of both second
    low-rank products, [H*dim + H*vdim, rank_a + rank_g]), ``delta_scan`` and ``delta_out`` do in three (a row of that
    product is summed by four lanes, each over every fourth element of the rank)."""
    k = "delta_decode"
    T = qn.shape[0]
    G, D, H, V = dims.kv_heads, dims.dim, dims.heads, dims.vdim
    R = dims.rank_a + dims.rank_g
    for name, t, w in (("qn", qn, G * D), ("kn", kn, G * D), ("vc", vc, H * V), ("beta", beta, H)):
        _check(t, k, name, torch.float32, (T, w))
    _check(low, k, "low", ACT_DTYPES[dtype_name(act)], (T, R))
    _check(low_weight, k, "low_weight", tuple(_WTYPE), (H * D + H * V, R))
    _check(a_log, k, "a_log", torch.float32, (H,))
    _check(dt_bias, k, "dt_bias", torch.float32, (H * D,))
    _check(norm_w, k, "norm_w", torch.float32, (V,))
    _check(proj, k, "proj", torch.float32, (T, dims.projections))
    stride = _delta_state(k, state, dims)
    B = runs["slots"].numel()
    _need(T == B and runs["decode"], k, "a decode step brings one token per sequence")
    _need(delta_decode_fits(dims), k, "a head's lanes do not fit one workgroup")
    _check(runs["cu_seqlens"], k, "cu_seqlens", torch.int32, (B + 1,))
    _check(runs["slots"], k, "slots", torch.int32, (B,))
    out = torch.empty((T, H * V), dtype=ACT_DTYPES[dtype_name(act)], device=qn.device)
    _run(k, library(act).tq_delta_decode(_ptr(qn), _ptr(kn), _ptr(vc), _ptr(beta), _ptr(low), _ptr(low_weight),
                                         _WTYPE[low_weight.dtype], _ptr(a_log), _ptr(dt_bias), _ptr(norm_w), float(eps),
                                         _ptr(proj), _ptr(runs["cu_seqlens"]), _ptr(runs["slots"]), _ptr(state), stride,
                                         *dims.sizes(), dims.rank_a, dims.rank_g, B, _ptr(out), _stream()))
    return out


def _delta_runs(k: str, runs: dict):
    B = runs["slots"].numel()
    _check(runs["cu_seqlens"], k, "cu_seqlens", torch.int32, (B + 1,))
    _check(runs["slots"], k, "slots", torch.int32, (B,))
    return B


def delta_prep_h(proj: torch.Tensor, slot_of_token: torch.Tensor, state: torch.Tensor, conv_w: torch.Tensor,
                 a_log: torch.Tensor, dt_bias: torch.Tensor, dims: DeltaDims, act):
    """The form of ``delta_prep`` with one decay per head: from the float32 projections [T, q | k | v | b | a | gate]
    q, k, v and beta as there, and dec = exp(-exp(a_log[h]) softplus(a + dt_bias[h])), float32 [T, H]."""
    k = "delta_prep"
    T = slot_of_token.numel()
    _need(dims.head_decay, k, "the sizes must be those of the form with a decay per head")
    _check(proj, k, "proj", torch.float32, (T, dims.projections))
    _check(slot_of_token, k, "slot_of_token", torch.int32, (T,))
    stride = _delta_state(k, state, dims)
    _check(conv_w, k, "conv_w", torch.float32, (dims.channels, dims.taps))
    G, D, H, V = dims.kv_heads, dims.dim, dims.heads, dims.vdim
    _check(a_log, k, "a_log", torch.float32, (H,))
    _check(dt_bias, k, "dt_bias", torch.float32, (H,))
    dev, f32 = proj.device, torch.float32
    qn = torch.empty((T, G * D), dtype=f32, device=dev)
    kn = torch.empty((T, G * D), dtype=f32, device=dev)
    vc = torch.empty((T, H * V), dtype=f32, device=dev)
    beta = torch.empty((T, H), dtype=f32, device=dev)
    dec = torch.empty((T, H), dtype=f32, device=dev)
    _run(k, library(act).tq_delta_prep_h(_ptr(proj), _ptr(slot_of_token), _ptr(state), stride, _ptr(conv_w), _ptr(a_log),
                                         _ptr(dt_bias), *dims.sizes(), _ptr(qn), _ptr(kn), _ptr(vc), _ptr(beta), _ptr(dec), T,
                                         _stream()))
    return qn, kn, vc, beta, dec


def delta_scan_h(qn: torch.Tensor, kn: torch.Tensor, vc: torch.Tensor, beta: torch.Tensor, dec: torch.Tensor, runs: dict,
                 state: torch.Tensor, dims: DeltaDims, act) -> torch.Tensor:
    """The recurrence of ``delta_scan`` with the whole state of a head decaying by dec[t, h] before token t's write."""
    k = "delta_scan"
    T = qn.shape[0]
    G, D, H, V = dims.kv_heads, dims.dim, dims.heads, dims.vdim
    for name, t, w in (("qn", qn, G * D), ("kn", kn, G * D), ("vc", vc, H * V), ("beta", beta, H), ("dec", dec, H)):
        _check(t, k, name, torch.float32, (T, w))
    stride = _delta_state(k, state, dims)
    B = _delta_runs(k, runs)
    o = torch.empty((T, H * V), dtype=torch.float32, device=qn.device)
    _run(k, library(act).tq_delta_scan_h(_ptr(qn), _ptr(kn), _ptr(vc), _ptr(beta), _ptr(dec), _ptr(runs["cu_seqlens"]),
                                         _ptr(runs["slots"]), _ptr(state), stride, *dims.sizes(), T, B, _ptr(o), _stream()))
    return o


def delta_out_h(o: torch.Tensor, norm_w: torch.Tensor, eps: float, proj: torch.Tensor, gate: str, runs: dict,
                state: torch.Tensor, dims: DeltaDims, act) -> torch.Tensor:
    """As ``delta_out``, the gate being activation ``gate`` (a name of GATES) of the last H*vdim columns of ``proj``."""
    k = "delta_out"
    T = o.shape[0]
    H, V = dims.heads, dims.vdim
    _check(o, k, "o", torch.float32, (T, H * V))
    _check(norm_w, k, "norm_w", torch.float32, (V,))
    _check(proj, k, "proj", torch.float32, (T, dims.projections))
    stride = _delta_state(k, state, dims)
    B = _delta_runs(k, runs)
    out = torch.empty((T, H * V), dtype=ACT_DTYPES[dtype_name(act)], device=o.device)
    _run(k, library(act).tq_delta_out_h(_ptr(o), _ptr(norm_w), float(eps), _ptr(proj), _gate_code(k, gate),
                                        _ptr(runs["cu_seqlens"]), _ptr(runs["slots"]), _ptr(state), stride, *dims.sizes(), T, B,
                                        _ptr(out), _stream()))
    return out


def delta_decode_h(qn: torch.Tensor, kn: torch.Tensor, vc: torch.Tensor, beta: torch.Tensor, a_log: torch.Tensor,
                   dt_bias: torch.Tensor, norm_w: torch.Tensor, eps: float, proj: torch.Tensor, gate: str, runs: dict,
                   state: torch.Tensor, dims: DeltaDims, act) -> torch.Tensor:
    """A decode step of the form with a decay per head, from ``delta_prep_h``'s outputs to the mixer's output
    [T, H*vdim] in the activation type, in one launch."""
    k = "delta_decode"
    T = qn.shape[0]
    G, D, H, V = dims.kv_heads, dims.dim, dims.heads, dims.vdim
    for name, t, w in (("qn", qn, G * D), ("kn", kn, G * D), ("vc", vc, H * V), ("beta", beta, H)):
        _check(t, k, name, torch.float32, (T, w))
    _check(a_log, k, "a_log", torch.float32, (H,))
    _check(dt_bias, k, "dt_bias", torch.float32, (H,))
    _check(norm_w, k, "norm_w", torch.float32, (V,))
    _check(proj, k, "proj", torch.float32, (T, dims.projections))
    stride = _delta_state(k, state, dims)
    B = _delta_runs(k, runs)
    _need(T == B and runs["decode"], k, "a decode step brings one token per sequence")
    _need(delta_decode_fits(dims), k, "a head's lanes do not fit one workgroup")
    out = torch.empty((T, H * V), dtype=ACT_DTYPES[dtype_name(act)], device=qn.device)
    _run(k, library(act).tq_delta_decode_h(_ptr(qn), _ptr(kn), _ptr(vc), _ptr(beta), _ptr(a_log), _ptr(dt_bias), _ptr(norm_w),
                                           float(eps), _ptr(proj), _gate_code(k, gate), _ptr(runs["cu_seqlens"]),
                                           _ptr(runs["slots"]), _ptr(state), stride, *dims.sizes(), B, _ptr(out), _stream()))
    return out


# ------------------------------------------------------------------ products per head, and what goes with them
def act_rows(g: torch.Tensor, u: torch.Tensor | None, activation: str | None, act) -> torch.Tensor:
    """f(g) * u in the activation type, row by row: ``g`` and ``u`` float32 [M, N] whose rows may be runs of columns
    of wider tensors (unit stride along a row); ``u`` None: f(g) alone; ``activation`` None: no f (with ``u`` None
    that is a change of type)."""
    k = "act_rows"
    for name, t in (("g", g), ("u", u)):
        if t is not None:
            _need(isinstance(t, torch.Tensor) and t.is_cuda and t.dtype == torch.float32 and t.dim() == 2 and t.stride(1) == 1,
                  k, lambda: f"{name} must be float32 [M, N] on the GPU with unit stride along its rows")
    M, N = g.shape
    _need(u is None or tuple(u.shape) == (M, N), k, "g and u must have one shape")
    out = torch.empty((M, N), dtype=ACT_DTYPES[dtype_name(act)], device=g.device)
    code = -1 if activation is None else _gate_code(k, activation)
    _run(k, library(act).tq_act_rows(_ptr(g), g.stride(0), _ptr(u), u.stride(0) if u is not None else 0, _ptr(out), M, N,
                                     code, _stream()))
    return out


def gate_rows(o: torch.Tensor, gate: torch.Tensor, activation: str, act) -> torch.Tensor:
    """o * f(gate), in place: ``o`` [M, N] contiguous in the activation type, ``gate`` float32 [M, N] whose rows may be
    runs of columns of a wider tensor, f an activation of GATES."""
    k = "gate_rows"
    _check(o, k, "o", ACT_DTYPES[dtype_name(act)])
    M, N = o.shape
    _need(isinstance(gate, torch.Tensor) and gate.is_cuda and gate.dtype == torch.float32 and tuple(gate.shape) == (M, N)
          and gate.stride(1) == 1, k, lambda: f"gate must be float32 [{M}, {N}] on the GPU with unit stride along its rows")
    _run(k, library(act).tq_gate_rows(_ptr(o), _ptr(gate), gate.stride(0), _ptr(o), M, N, _gate_code(k, activation), _stream()))
    return o


def token_shift(x: torch.Tensor, weight: torch.Tensor, state: torch.Tensor, runs: dict, act) -> torch.Tensor:
    """out[t] = x[t] + (x[t-1] - x[t]) * weight in the activation type, x[t-1] being the row of the sequence's token before:
    the step's own row, or for a run's first token the row that ``state`` [slots, H] keeps for the sequence's slot (zeros
    for a new sequence); afterwards the slot keeps the run's last row of ``x``.  ``runs`` as for ``attention``."""
    k = "token_shift"
    _check(x, k, "x", torch.float32)
    _need(x.dim() == 2, k, "x must be [T, H]")
    T, H = x.shape
    _check(weight, k, "weight", tuple(_WTYPE), (H,))
    _check(state, k, "state", torch.float32)
    _need(state.dim() == 2 and state.shape[1] == H, k, lambda: f"state must be [slots, {H}]")
    B = runs["slots"].numel()
    _check(runs["cu_seqlens"], k, "cu_seqlens", torch.int32, (B + 1,))
    _check(runs["slots"], k, "slots", torch.int32, (B,))
    out = torch.empty((T, H), dtype=ACT_DTYPES[dtype_name(act)], device=x.device)
    _run(k, library(act).tq_token_shift(_ptr(x), _ptr(weight), _WTYPE[weight.dtype], _ptr(state), _ptr(runs["cu_seqlens"]),
                                        _ptr(runs["slots"]), B, _ptr(out), T, H, _stream()))
    return out


def value_norm_mix(v: torch.Tensor, num_heads: int, head_dim: int, value_dim: int, eps: float, act,
                   first: torch.Tensor | None = None, first_head_dim: int | None = None,
                   mix: torch.Tensor | None = None) -> torch.Tensor:
    """Every value head of the float32 rows ``v`` [T, num_heads * head_dim] (columns of a wider tensor, a head's first
    ``value_dim`` numbers its values) divided by its root mean square over them, in place, without weights; with ``first``
    (another layer's values of the same tokens, so normed, laid out alike at ``first_head_dim`` a head) each then becomes
    (1 - mix) v + mix first, ``mix`` a tensor of one number.  Returns ``v``."""
    k = "value_norm_mix"
    T = v.shape[0]
    _need(v.is_cuda and v.dtype == torch.float32 and v.dim() == 2 and v.shape[1] == num_heads * head_dim and v.stride(1) == 1,
          k, lambda: f"v must be float32 [T, {num_heads * head_dim}] on the GPU with unit stride along its rows")
    _need(1 <= value_dim <= head_dim and eps >= 0, k, "the values lie within the head, and eps is positive (0: no norm)")
    fhd = 0
    if first is not None:
        fhd = int(first_head_dim or head_dim)
        _need(first.is_cuda and first.dtype == torch.float32 and first.dim() == 2 and first.shape[0] == T
              and first.shape[1] == num_heads * fhd and first.stride(1) == 1 and value_dim <= fhd, k,
              lambda: f"first must be float32 [{T}, {num_heads * fhd}] on the GPU with unit stride along its rows")
        _check(mix, k, "mix", tuple(_WTYPE))
        _need(mix.numel() == 1, k, "mix is one number")
    _run(k, library(act).tq_value_norm_mix(_ptr(v), v.stride(0), head_dim, value_dim, num_heads, float(eps), _ptr(first),
                                           first.stride(0) if first is not None else 0, fhd, _ptr(mix),
                                           _WTYPE[mix.dtype] if first is not None else 0, T, _stream()))
    return v


def attn_prep_kv_write(qkv: torch.Tensor, positions: torch.Tensor, seq_of_token: torch.Tensor, block_table: torch.Tensor,
                       inv_freq: torch.Tensor, pairing: int, rotary_dim: int, k_pages: torch.Tensor | None,
                       v_pages: torch.Tensor | None, layer_offset: int, page_size: int, page_stride: int, num_heads: int,
                       num_kv_heads: int, head_dim: int, act, runs: dict | None = None, amplitude: float = 1.0,
                       q_weight: torch.Tensor | None = None, k_weight: torch.Tensor | None = None, qk_eps: float = 0.0,
                       norm_dim: int | None = None, value_eps: float = 0.0, value_dim: int | None = None,
                       first: torch.Tensor | None = None, first_head_dim: int | None = None,
                       mix: torch.Tensor | None = None) -> torch.Tensor:
    """``head_rmsnorm``, ``value_norm_mix`` and ``rope_kv_write`` in one launch: every query and key head of the float32
    rows ``qkv`` normed with its weights (``qk_eps`` > 0), every value head brought to unit root mean square over its first
    ``value_dim`` numbers (``value_eps`` > 0) and mixed with ``first`` (as in ``value_norm_mix``), queries and keys rotated,
    keys and values written into the pages; returns the queries.  The values are also written back into ``qkv`` as the
    cache holds them.  ``qkv`` holds every product's bias already."""
    k = "attn_prep_kv_write"
    T = positions.numel()
    width = (num_heads + 2 * num_kv_heads) * head_dim
    _need(isinstance(qkv, torch.Tensor) and qkv.is_cuda and qkv.dtype == torch.float32 and tuple(qkv.shape) == (T, width)
          and qkv.stride(1) == 1 and qkv.stride(0) >= width, k,
          lambda: f"qkv must be float32 [{T}, {width}] on the GPU with unit stride along its rows")
    _check(positions, k, "positions", torch.int32, (T,))
    _check(seq_of_token, k, "seq_of_token", torch.int32, (T,))
    _check(block_table, k, "block_table", torch.int32)
    _need(block_table.dim() == 2, k, "block_table must be [B, pages]")
    _check(inv_freq, k, "inv_freq", torch.float32)
    _need(inv_freq.numel() * 2 == rotary_dim or rotary_dim == 0, k, lambda: f"inv_freq must hold rotary_dim/2 = {rotary_dim // 2} entries")
    _need(rotary_dim <= 512 and qk_eps >= 0 and value_eps >= 0, k, "at most 512 rotated values; eps of 0 or more")
    wtype = None
    for name, w in (("q_weight", q_weight), ("k_weight", k_weight), ("mix", mix)):
        if w is not None:
            _check(w, k, name, tuple(_WTYPE), (1,) if name == "mix" else (head_dim,))
            _need(wtype in (None, w.dtype), k, "the norms' weights and the mix must have one type")
            wtype = w.dtype
    vd = int(value_dim or head_dim)
    fhd = 0
    if first is not None:
        fhd = int(first_head_dim or head_dim)
        _need(first.is_cuda and first.dtype == torch.float32 and first.dim() == 2 and first.shape[0] == T
              and first.shape[1] == num_kv_heads * fhd and first.stride(1) == 1 and vd <= fhd and mix is not None, k,
              lambda: f"first must be float32 [{T}, {num_kv_heads * fhd}] on the GPU with unit stride along its rows, with a mix")
    adt = ACT_DTYPES[dtype_name(act)]
    q = torch.empty((T, num_heads * head_dim), dtype=adt, device=qkv.device)
    write = k_pages is not None
    kp = vp = None
    if write:
        _check(k_pages, k, "k_pages", adt)
        _check(v_pages, k, "v_pages", adt)
        _need(layer_offset + num_kv_heads * page_size * head_dim <= page_stride, k, "layer does not fit in a page")
        esz = k_pages.element_size()
        kp, vp = k_pages.data_ptr() + layer_offset * esz, v_pages.data_ptr() + layer_offset * esz
    cu = slots = start = None
    B = max_new = 0
    if runs is not None and write and not runs["decode"]:
        B = runs["slots"].numel()
        cu, slots, start, max_new = runs["cu_seqlens"], runs["slots"], runs["start"], int(runs["max_new"])
        _check(cu, k, "cu_seqlens", torch.int32, (B + 1,))
        _check(slots, k, "slots", torch.int32, (B,))
        _check(start, k, "start", torch.int32, (B,))
        _need(int(runs["max_end"]) <= block_table.shape[1] * page_size, k, "positions reach beyond the page table")
    _run(k, library(act).tq_attn_prep_kv_write(
        _ptr(qkv), qkv.stride(0), _ptr(positions), _ptr(seq_of_token), _ptr(block_table), block_table.shape[1], _ptr(inv_freq),
        pairing, rotary_dim, float(amplitude), _ptr(q_weight), _ptr(k_weight), _WTYPE[wtype] if wtype is not None else 0,
        float(qk_eps), int(norm_dim or head_dim), float(value_eps), vd, _ptr(first), first.stride(0) if first is not None else 0,
        fhd, _ptr(mix), _ptr(q), kp, vp, page_size, page_stride, T, num_heads, num_kv_heads, head_dim, int(write), _ptr(cu),
        _ptr(slots), _ptr(start), B, max_new, _stream()))
    return q


def latent_norm(src: torch.Tensor, weight: torch.Tensor, eps: float, out: torch.Tensor, copies: int, width: int, act) -> None:
    """RMS norm of the rows of ``src`` (float32 [T, R], a run of columns of a wider tensor allowed) with ``weight`` [R],
    written ``copies`` times side by side into the rows of ``out`` (float32 [T, copies * width], likewise), each copy
    padded with zeros to ``width`` columns."""
    k = "latent_norm"
    for name, t in (("src", src), ("out", out)):
        _need(isinstance(t, torch.Tensor) and t.is_cuda and t.dtype == torch.float32 and t.dim() == 2 and t.stride(1) == 1,
              k, lambda: f"{name} must be float32 [T, n] on the GPU with unit stride along its rows")
    T, R = src.shape
    _check(weight, k, "weight", tuple(_WTYPE), (R,))
    _need(width >= R and copies >= 1 and tuple(out.shape) == (T, copies * width), k,
          lambda: f"out must be [{T}, {copies * width}], is {tuple(out.shape)}")
    _run(k, library(act).tq_latent_norm(_ptr(src), src.stride(0), _ptr(weight), _WTYPE[weight.dtype], float(eps), _ptr(out),
                                        out.stride(0), copies, R, width, T, _stream()))


def head_gemm(a: torch.Tensor, w: torch.Tensor, act, out: torch.Tensor | None = None, out_act: bool = False,
              gate: torch.Tensor | None = None, activation: str = "sigmoid") -> torch.Tensor:
    """A product per head: out[t, h*N + n] = sum_k a[t, h*K + k] * w[h, n, k], ``w`` [H, N, K].  ``a`` [T, H*K] is
    float32 or of the activation type, ``out`` [T, H*N] float32 (or the activation type with ``out_act``); both may be
    runs of columns of wider tensors, and ``out`` may be given.  ``gate`` float32 [T, H*N]: the result is multiplied
    by ``activation`` (a name of GATES) of it."""
    k = "head_gemm"
    adt = ACT_DTYPES[dtype_name(act)]
    _need(isinstance(w, torch.Tensor) and w.is_cuda and w.dim() == 3 and w.is_contiguous() and w.dtype in _WTYPE, k,
          "w must be a contiguous [H, N, K] matrix on the GPU")
    H, N, K = w.shape
    _need(isinstance(a, torch.Tensor) and a.is_cuda and a.dim() == 2 and a.shape[1] == H * K and a.stride(1) == 1
          and a.dtype in (torch.float32, adt), k, lambda: f"a must be [T, {H * K}] float32 or {adt} with unit stride along its rows")
    T = a.shape[0]
    odt = adt if out_act else torch.float32
    if out is None:
        out = torch.empty((T, H * N), dtype=odt, device=a.device)
    _need(out.is_cuda and out.dtype == odt and tuple(out.shape) == (T, H * N) and out.stride(1) == 1, k,
          lambda: f"out must be [{T}, {H * N}] {odt} with unit stride along its rows")
    if gate is not None:
        _need(gate.is_cuda and gate.dtype == torch.float32 and tuple(gate.shape) == (T, H * N) and gate.stride(1) == 1, k,
              lambda: f"gate must be float32 [{T}, {H * N}] with unit stride along its rows")
    _run(k, library(act).tq_head_gemm(_ptr(a), _WTYPE[a.dtype], a.stride(0), _ptr(w), _WTYPE[w.dtype], _ptr(out), int(out_act),
                                      out.stride(0), _ptr(gate), gate.stride(0) if gate is not None else 0,
                                      _gate_code(k, activation), T, H, N, K, _stream()))
    return out


def gate_heads(o: torch.Tensor, gate: torch.Tensor, num_heads: int, activation: str, act) -> torch.Tensor:
    """o[:, h * hd : (h + 1) * hd] *= f(gate[:, h]), in place: one number per head and token gates the head's whole output.
    ``o`` [M, heads * hd] contiguous in the activation type, ``gate`` float32 [M, heads] whose rows may be runs of
    columns of a wider tensor."""
    k = "gate_heads"
    _check(o, k, "o", ACT_DTYPES[dtype_name(act)])
    M, N = o.shape
    _need(num_heads >= 1 and N % num_heads == 0, k, lambda: f"{N} columns are not {num_heads} heads")
    _need(isinstance(gate, torch.Tensor) and gate.is_cuda and gate.dtype == torch.float32 and tuple(gate.shape) == (M, num_heads)
          and gate.stride(1) == 1, k, lambda: f"gate must be float32 [{M}, {num_heads}] on the GPU with unit stride along its rows")
    _run(k, library(act).tq_gate_heads(_ptr(o), _ptr(gate), gate.stride(0), _ptr(o), M, num_heads, N // num_heads,
                                       _gate_code(k, activation), _stream()))
    return o


def lead_norm(src: torch.Tensor, rank: int, weight: torch.Tensor, eps: float, copies: int, width: int, act,
              out: torch.Tensor | None = None, out_act: bool = False) -> torch.Tensor:
    """Rows ``src`` (float32 [T, rank + lead], a run of columns of a wider tensor allowed): the first ``rank`` columns
    are RMS-normed with ``weight`` [rank], the ``lead`` columns behind them pass as they are; every copy in ``out``
    [T, copies * width] holds the lead first, then the normed columns, then zeros up to ``width``.  ``out`` is float32, or
    of the activation type with ``out_act``."""
    k = "lead_norm"
    _need(isinstance(src, torch.Tensor) and src.is_cuda and src.dtype == torch.float32 and src.dim() == 2 and src.stride(1) == 1,
          k, "src must be float32 [T, n] on the GPU with unit stride along its rows")
    T, lead = src.shape[0], src.shape[1] - rank
    _need(rank >= 1 and lead >= 0 and width >= rank + lead and copies >= 1, k, "rank, lead and width do not fit")
    _check(weight, k, "weight", tuple(_WTYPE), (rank,))
    odt = ACT_DTYPES[dtype_name(act)] if out_act else torch.float32
    if out is None:
        out = torch.empty((T, copies * width), dtype=odt, device=src.device)
    _need(out.is_cuda and out.dtype == odt and tuple(out.shape) == (T, copies * width) and out.stride(1) == 1, k,
          lambda: f"out must be [{T}, {copies * width}] {odt} with unit stride along its rows")
    _run(k, library(act).tq_lead_norm(_ptr(src), src.stride(0), _ptr(weight), _WTYPE[weight.dtype], float(eps), _ptr(out),
                                      int(out_act), out.stride(0), copies, rank, lead, width, T, _stream()))
    return out


# ------------------------------------------------------------------ linear attention with a decay per head
def lightning_scan(proj: torch.Tensor, decay: torch.Tensor, runs: dict, state: torch.Tensor, num_heads: int, head_dim: int,
                   value_dim: int, act) -> torch.Tensor:
    """The recurrence S <- decay_h S + k v^T, o = S^T q over the step's runs of tokens, from and into the sequences' rows
    of ``state`` (float32 [slots, heads * dim * vdim]); ``proj`` float32 [T, >= 2 H D + 2 H V] holds q | k | v | gate
    before their silu.  Returns o float32 [T, H * V]."""
    k = "lightning_scan"
    H, D, V = num_heads, head_dim, value_dim
    _need(isinstance(proj, torch.Tensor) and proj.is_cuda and proj.dtype == torch.float32 and proj.dim() == 2
          and proj.stride(1) == 1 and proj.shape[1] >= 2 * H * D + 2 * H * V, k,
          lambda: f"proj must be float32 [T, >= {2 * H * D + 2 * H * V}] on the GPU with unit stride along its rows")
    _check(decay, k, "decay", torch.float32, (H,))
    _check(state, k, "state", torch.float32)
    _need(state.dim() == 2 and state.shape[1] == H * D * V, k, lambda: f"state must be [slots, {H * D * V}]")
    _need(D <= 256, k, lambda: f"a key width of {D} is beyond the 256 this kernel takes")
    B = runs["slots"].numel()
    _check(runs["cu_seqlens"], k, "cu_seqlens", torch.int32, (B + 1,))
    _check(runs["slots"], k, "slots", torch.int32, (B,))
    T = proj.shape[0]
    o = torch.empty((T, H * V), dtype=torch.float32, device=proj.device)
    _run(k, library(act).tq_lightning_scan(_ptr(proj), proj.stride(0), _ptr(decay), _ptr(runs["cu_seqlens"]), _ptr(runs["slots"]),
                                           _ptr(state), state.stride(0), B, H, D, V, _ptr(o), _stream()))
    return o


LIGHTNING_CHUNK = 64           # tokens of a chunk of the chunked recurrence


def lightning_chunked(proj: torch.Tensor, decay: torch.Tensor, runs: dict, state: torch.Tensor, num_heads: int, head_dim: int,
                      value_dim: int, act) -> torch.Tensor:
    """``lightning_scan`` for steps with long runs: the same function over chunks of 64 tokens on the matrix cores, in
    float32 on both libraries (three launches: every chunk's own sum of k v^T, the states before the chunks, every
    chunk's read-outs).  ``runs`` also names ``max_new``, the longest run.  Its sums are ordered by the chunks, which start
    at the first token that the step brings: results agree with ``lightning_scan`` to rounding."""
    k = "lightning_chunked"
    H, D, V = num_heads, head_dim, value_dim
    _need(isinstance(proj, torch.Tensor) and proj.is_cuda and proj.dtype == torch.float32 and proj.dim() == 2
          and proj.stride(1) == 1 and proj.shape[1] >= 2 * H * D + 2 * H * V, k,
          lambda: f"proj must be float32 [T, >= {2 * H * D + 2 * H * V}] on the GPU with unit stride along its rows")
    _check(decay, k, "decay", torch.float32, (H,))
    _check(state, k, "state", torch.float32)
    _need(state.dim() == 2 and state.shape[1] == H * D * V, k, lambda: f"state must be [slots, {H * D * V}]")
    _need(D <= 256, k, lambda: f"a key width of {D} is beyond the 256 this kernel takes")
    B = runs["slots"].numel()
    _check(runs["cu_seqlens"], k, "cu_seqlens", torch.int32, (B + 1,))
    _check(runs["slots"], k, "slots", torch.int32, (B,))
    T, max_new = proj.shape[0], int(runs["max_new"])
    _need(1 <= max_new <= T, k, lambda: f"the longest run has {max_new} of {T} tokens")
    chunks = T // LIGHTNING_CHUNK + B
    scratch = torch.empty((chunks, H * D * V), dtype=torch.float32, device=proj.device)
    o = torch.empty((T, H * V), dtype=torch.float32, device=proj.device)
    _run(k, library(act).tq_lightning_chunked(_ptr(proj), proj.stride(0), _ptr(decay), _ptr(runs["cu_seqlens"]), _ptr(runs["slots"]),
                                              _ptr(state), state.stride(0), B, H, D, V, max_new, _ptr(scratch), chunks, _ptr(o),
                                              _stream()))
    return o


def lightning_out(o: torch.Tensor, gate: torch.Tensor, weight: torch.Tensor, eps: float, act) -> torch.Tensor:
    """rmsnorm(o) * weight * sigmoid(gate) in the activation type, the norm over a token's whole row (all heads together):
    ``o`` float32 [T, N] contiguous, ``gate`` float32 [T, N] whose rows may be runs of columns of a wider tensor."""
    k = "lightning_out"
    _check(o, k, "o", torch.float32)
    T, N = o.shape
    _need(isinstance(gate, torch.Tensor) and gate.is_cuda and gate.dtype == torch.float32 and tuple(gate.shape) == (T, N)
          and gate.stride(1) == 1, k, lambda: f"gate must be float32 [{T}, {N}] on the GPU with unit stride along its rows")
    _check(weight, k, "weight", tuple(_WTYPE), (N,))
    out = torch.empty((T, N), dtype=ACT_DTYPES[dtype_name(act)], device=o.device)
    _run(k, library(act).tq_lightning_out(_ptr(o), _ptr(gate), gate.stride(0), _ptr(weight), _WTYPE[weight.dtype], float(eps),
                                          _ptr(out), T, N, _stream()))
    return out


# ------------------------------------------------------------------ a matrix memory with exponential gates
@dataclasses.dataclass(frozen=True)
class MemoryDims:
    """Heads, key width and value width of a matrix memory, and the cap of its gates."""
    heads: int
    dim: int
    vdim: int
    cap: float

    @property
    def projections(self) -> int:
        """Numbers of a token's row of projections: q | k | v | gate | input gate | forget gate."""
        return 2 * self.heads * (self.dim + self.vdim + 1)

    @property
    def m_offset(self) -> int:
        return self.heads * (self.dim * self.vdim + self.dim)

    @property
    def state_floats(self) -> int:
        """Floats of a sequence's row of state: S [heads][dim][vdim], n [heads][dim], m [heads], filled up to a multiple of 4."""
        return -(-(self.m_offset + self.heads) // 4) * 4


def _memory_args(k: str, proj: torch.Tensor, bias: torch.Tensor, runs: dict, state: torch.Tensor, d: MemoryDims) -> int:
    _need(isinstance(proj, torch.Tensor) and proj.is_cuda and proj.dtype == torch.float32 and proj.dim() == 2
          and proj.stride(1) == 1 and proj.shape[1] >= d.projections, k,
          lambda: f"proj must be float32 [T, >= {d.projections}] on the GPU with unit stride along its rows")
    _check(bias, k, "bias", torch.float32, (2 * d.heads,))
    _check(state, k, "state", torch.float32)
    _need(state.dim() == 2 and state.shape[1] == d.state_floats, k, lambda: f"state must be [slots, {d.state_floats}]")
    B = runs["slots"].numel()
    _check(runs["cu_seqlens"], k, "cu_seqlens", torch.int32, (B + 1,))
    _check(runs["slots"], k, "slots", torch.int32, (B,))
    return B


def _memory_rows(k: str, out: torch.Tensor | None, T: int, N: int, act, device) -> torch.Tensor:
    adt = ACT_DTYPES[dtype_name(act)]
    if out is None:
        return torch.empty((T, N), dtype=adt, device=device)
    _need(out.is_cuda and out.dtype == adt and tuple(out.shape) == (T, N) and out.stride(1) == 1 and out.stride(0) >= N, k,
          lambda: f"out must be [{T}, {N}] of the activation type with unit stride along its rows")
    return out


def mm_scan(proj: torch.Tensor, bias: torch.Tensor, runs: dict, state: torch.Tensor, dims: MemoryDims, act):
    """The memory's recurrence over the step's runs of tokens, in order, from and into the sequences' rows of ``state``;
    ``proj`` float32 [T, >= dims.projections] holds q | k | v | gate | raw input gate | raw forget gate, ``bias`` float32
    [2 heads] the two gates' biases.  Returns (numerators [T, heads * vdim], denominators [T, heads], running maxima
    [T, heads]), float32; the rows' own running maxima are for ``mm_out`` to write."""
    k = "mm_scan"
    B = _memory_args(k, proj, bias, runs, state, dims)
    _need(dims.dim <= 1024, k, lambda: f"a key width of {dims.dim} is beyond the 1,024 this kernel takes")
    T, dev = proj.shape[0], proj.device
    num = torch.empty((T, dims.heads * dims.vdim), dtype=torch.float32, device=dev)
    den = torch.empty((T, dims.heads), dtype=torch.float32, device=dev)
    mrow = torch.empty((T, dims.heads), dtype=torch.float32, device=dev)
    _run(k, library(act).tq_mm_scan(_ptr(proj), proj.stride(0), _ptr(bias), dims.cap, _ptr(runs["cu_seqlens"]), _ptr(runs["slots"]),
                                    _ptr(state), state.stride(0), B, dims.heads, dims.dim, dims.vdim, _ptr(num), _ptr(den),
                                    _ptr(mrow), _stream()))
    return num, den, mrow


def mm_chunked(proj: torch.Tensor, bias: torch.Tensor, runs: dict, state: torch.Tensor, dims: MemoryDims, act):
    """``mm_scan`` for steps with long runs: the same sums over chunks of 64 tokens on the matrix cores, in float32 on both
    libraries (three launches), key widths of up to 256.  ``runs`` also names ``max_new``, the longest run.  Returns
    (numerators, denominators); the rows of state are complete."""
    k = "mm_chunked"
    B = _memory_args(k, proj, bias, runs, state, dims)
    _need(dims.dim <= 256, k, lambda: f"a key width of {dims.dim} is beyond the 256 this kernel takes")
    T, dev, max_new = proj.shape[0], proj.device, int(runs["max_new"])
    _need(1 <= max_new <= T, k, lambda: f"the longest run has {max_new} of {T} tokens")
    chunks = T // LIGHTNING_CHUNK + B
    scratch = torch.empty((chunks, dims.m_offset), dtype=torch.float32, device=dev)
    scal = torch.empty((chunks, dims.heads, 3), dtype=torch.float64, device=dev)
    num = torch.empty((T, dims.heads * dims.vdim), dtype=torch.float32, device=dev)
    den = torch.empty((T, dims.heads), dtype=torch.float32, device=dev)
    _run(k, library(act).tq_mm_chunked(_ptr(proj), proj.stride(0), _ptr(bias), dims.cap, _ptr(runs["cu_seqlens"]),
                                       _ptr(runs["slots"]), _ptr(state), state.stride(0), B, dims.heads, dims.dim, dims.vdim,
                                       max_new, _ptr(scratch), _ptr(scal), chunks, _ptr(num), _ptr(den), _stream()))
    return num, den


def mm_out(num: torch.Tensor, den: torch.Tensor, gate: torch.Tensor, weight: torch.Tensor, eps: float, dims: MemoryDims, act,
           mrow: torch.Tensor | None = None, slot_of_token: torch.Tensor | None = None, state: torch.Tensor | None = None,
           out: torch.Tensor | None = None):
    """Every head's read-out num / den divided by its root mean square, times ``weight`` [heads * vdim] and sigmoid(gate), in the
    activation type [T, heads * vdim].  ``mrow`` (from ``mm_scan``) with ``slot_of_token`` and ``state``: the running maxima of
    every run's last token go into the rows of state.  ``out``: where the result goes, columns of a wider matrix."""
    k = "mm_out"
    T, N = num.shape
    _check(num, k, "num", torch.float32, (T, dims.heads * dims.vdim))
    _check(den, k, "den", torch.float32, (T, dims.heads))
    _need(isinstance(gate, torch.Tensor) and gate.is_cuda and gate.dtype == torch.float32 and tuple(gate.shape) == (T, N)
          and gate.stride(1) == 1, k, lambda: f"gate must be float32 [{T}, {N}] on the GPU with unit stride along its rows")
    _check(weight, k, "weight", tuple(_WTYPE), (N,))
    if mrow is not None:
        _check(mrow, k, "mrow", torch.float32, (T, dims.heads))
        _check(slot_of_token, k, "slot_of_token", torch.int32, (T,))
        _check(state, k, "state", torch.float32)
        _need(state.dim() == 2 and state.shape[1] == dims.state_floats, k, lambda: f"state must be [slots, {dims.state_floats}]")
    out = _memory_rows(k, out, T, N, act, num.device)
    _run(k, library(act).tq_mm_out(_ptr(num), _ptr(den), _ptr(gate), gate.stride(0), _ptr(weight), _WTYPE[weight.dtype], float(eps),
                                   _ptr(out), out.stride(0), T, dims.heads, dims.vdim, _ptr(mrow), _ptr(slot_of_token),
                                   _ptr(state) if mrow is not None else None, state.stride(0) if mrow is not None else 0,
                                   dims.m_offset, _stream()))
    return out


def mm_decode_fits(proj: torch.Tensor, dims: MemoryDims) -> bool:
    """Whether ``mm_decode`` takes these sizes (rows that start at multiples of 16 bytes, whole groups of four channels)."""
    return (dims.vdim % 4 == 0 and dims.vdim <= 1024 and dims.dim <= 1024 and (2 * dims.heads * dims.dim) % 4 == 0
            and proj.stride(0) % 4 == 0 and proj.data_ptr() % 16 == 0)


@dataclasses.dataclass
class KVWrite:
    """Queries, keys and values of a decode step that a launch lays out beside its own work: ``qkv`` float32 [B, (nh + 2 nkv) *
    hd], columns of the matrix whose other columns the launch reads; ``q`` [B, nh * hd] gets the queries, the pages get keys and
    values as ``rope_kv_write`` writes them without a rotation."""
    qkv: torch.Tensor
    positions: torch.Tensor
    block_table: torch.Tensor
    k_pages: torch.Tensor
    v_pages: torch.Tensor
    layer_offset: int
    page_size: int
    page_stride: int
    num_heads: int
    num_kv_heads: int
    head_dim: int
    q: torch.Tensor


def mm_decode(proj: torch.Tensor, bias: torch.Tensor, runs: dict, state: torch.Tensor, weight: torch.Tensor, eps: float,
              dims: MemoryDims, act, out: torch.Tensor | None = None, kv_write: KVWrite | None = None) -> torch.Tensor:
    """``mm_scan`` and ``mm_out`` of a step of one token per sequence, in one launch, which also does ``kv_write``."""
    k = "mm_decode"
    B = _memory_args(k, proj, bias, runs, state, dims)
    _need(proj.shape[0] == B, k, "decoding brings one token per sequence")
    N = dims.heads * dims.vdim
    _check(weight, k, "weight", tuple(_WTYPE), (N,))
    out = _memory_rows(k, out, B, N, act, proj.device)
    extra = (None, None, None, 0, None, None, None, 0, 0, 0, 0, 0)
    if kv_write is not None:
        w, adt = kv_write, ACT_DTYPES[dtype_name(act)]
        width = (w.num_heads + 2 * w.num_kv_heads) * w.head_dim
        _need(w.qkv.is_cuda and w.qkv.dtype == torch.float32 and tuple(w.qkv.shape) == (B, width) and w.qkv.stride(1) == 1
              and w.qkv.stride(0) == proj.stride(0), k, lambda: f"qkv must be float32 [{B}, {width}], columns of proj's matrix")
        _check(w.positions, k, "positions", torch.int32, (B,))
        _check(w.block_table, k, "block_table", torch.int32)
        _check(w.k_pages, k, "k_pages", adt)
        _check(w.v_pages, k, "v_pages", adt)
        _check(w.q, k, "q", adt, (B, w.num_heads * w.head_dim))
        _need(w.block_table.dim() == 2 and w.layer_offset + w.num_kv_heads * w.page_size * w.head_dim <= w.page_stride, k,
              "layer does not fit in a page")
        esz = w.k_pages.element_size()
        extra = (_ptr(w.qkv), _ptr(w.positions), _ptr(w.block_table), w.block_table.shape[1], _ptr(w.q),
                 w.k_pages.data_ptr() + w.layer_offset * esz, w.v_pages.data_ptr() + w.layer_offset * esz, w.page_size,
                 w.page_stride, w.num_heads, w.num_kv_heads, w.head_dim)
    _run(k, library(act).tq_mm_decode(_ptr(proj), proj.stride(0), _ptr(bias), dims.cap, _ptr(runs["slots"]), _ptr(state),
                                      state.stride(0), B, dims.heads, dims.dim, dims.vdim, _ptr(weight), _WTYPE[weight.dtype],
                                      float(eps), _ptr(out), out.stride(0), *extra, _stream()))
    return out


# ------------------------------------------------------------------ a token's own vector as a factor
def token_gate(p: torch.Tensor, tokens: torch.Tensor, table: torch.Tensor, activation: str, act) -> torch.Tensor:
    """f(sum_s p[s, t]) * table[tokens[t]] in the activation type: ``p`` float32 [S, T, N] partial sums, ``table`` [V, N], whose
    rows may be runs of columns of a wider table."""
    k = "token_gate"
    _check(p, k, "p", torch.float32)
    _need(p.dim() == 3, k, "p must be [S, T, N]")
    S, T, N = p.shape
    _check(tokens, k, "tokens", torch.int32, (T,))
    _need(isinstance(table, torch.Tensor) and table.is_cuda and table.dtype in _WTYPE and table.dim() == 2 and table.shape[1] == N
          and table.stride(1) == 1, k, lambda: f"table must be [V, {N}] on the GPU with unit stride along its rows")
    out = torch.empty((T, N), dtype=ACT_DTYPES[dtype_name(act)], device=p.device)
    _run(k, library(act).tq_token_gate(_ptr(p), S, _ptr(tokens), _ptr(table), _WTYPE[table.dtype], table.stride(0),
                                       _gate_code(k, activation), _ptr(out), T, N, _stream()))
    return out


def token_gate_product(a: torch.Tensor, w: torch.Tensor, tokens: torch.Tensor, table: torch.Tensor, activation: str, act) -> torch.Tensor:
    """``token_gate`` of the product a w^T (``w`` [N, K]): one launch for up to 16 tokens, else two."""
    k = "token_gate_product"
    adt = ACT_DTYPES[dtype_name(act)]
    T, K = a.shape
    if (T > 16 or w.dtype != adt or a.dtype != adt or K % (16 // adt.itemsize) or a.stride(0) % (16 // adt.itemsize)
            or a.data_ptr() % 16 or w.data_ptr() % 16):
        return token_gate(gemm(a, w, act, partial_sums=True), tokens, table, activation, act)
    _need(a.is_cuda and a.stride(1) == 1, k, "a must be on the GPU with unit stride along its rows")
    _check(w, k, "w", adt)
    N = w.shape[0]
    _need(w.dim() == 2 and w.shape[1] == K, k, lambda: f"w must be [N, {K}]")
    _check(tokens, k, "tokens", torch.int32, (T,))
    _need(isinstance(table, torch.Tensor) and table.is_cuda and table.dtype in _WTYPE and table.dim() == 2 and table.shape[1] == N
          and table.stride(1) == 1, k, lambda: f"table must be [V, {N}] on the GPU with unit stride along its rows")
    out = torch.empty((T, N), dtype=adt, device=a.device)
    _run(k, library(act).tq_token_gate_product(_ptr(a), a.stride(0), _ptr(w), _ptr(tokens), _ptr(table), _WTYPE[table.dtype],
                                               table.stride(0), _gate_code(k, activation), _ptr(out), T, N, K, _stream()))
    return out


# ------------------------------------------------------------------ between a product and its attention
def _kv_places(k: str, k_pages, v_pages, layer_offset: int, page_size: int, page_stride: int, num_kv_heads: int, head_dim: int,
               block_table, runs, adt):
    """What a launch that writes keys and values is told: pool addresses, and the runs of a step that brings more than a token
    per sequence (cu_seqlens, slots, start, number of runs, longest run)."""
    _check(k_pages, k, "k_pages", adt)
    _check(v_pages, k, "v_pages", adt)
    _need(layer_offset + num_kv_heads * page_size * head_dim <= page_stride, k, "layer does not fit in a page")
    esz = k_pages.element_size()
    places = (k_pages.data_ptr() + layer_offset * esz, v_pages.data_ptr() + layer_offset * esz)
    if runs is None or runs["decode"]:
        return places, (None, None, None, 0, 0)
    B = runs["slots"].numel()
    _check(runs["cu_seqlens"], k, "cu_seqlens", torch.int32, (B + 1,))
    _check(runs["slots"], k, "slots", torch.int32, (B,))
    _check(runs["start"], k, "start", torch.int32, (B,))
    _need(int(runs["max_end"]) <= block_table.shape[1] * page_size, k, "positions reach beyond the page table")
    return places, (_ptr(runs["cu_seqlens"]), _ptr(runs["slots"]), _ptr(runs["start"]), B, int(runs["max_new"]))


def _qkv_rows(k: str, qkv, T: int, width: int, head_dim: int) -> None:
    _need(isinstance(qkv, torch.Tensor) and qkv.is_cuda and qkv.dtype == torch.float32 and qkv.dim() == 2
          and tuple(qkv.shape) == (T, width) and qkv.stride(1) == 1 and qkv.stride(0) >= width, k,
          lambda: f"qkv must be float32 [{T}, {width}] on the GPU with unit stride along its rows")
    _need(head_dim % 4 != 0 or (qkv.stride(0) % 4 == 0 and qkv.data_ptr() % 16 == 0), k,
          "rows of qkv must start at multiples of 16 bytes")


def row_norm_kv_write(qkv: torch.Tensor, positions: torch.Tensor, seq_of_token: torch.Tensor, block_table: torch.Tensor,
                      inv_freq: torch.Tensor, pairing: int, rotary_dim: int, k_pages: torch.Tensor | None,
                      v_pages: torch.Tensor | None, layer_offset: int, page_size: int, page_stride: int, num_heads: int,
                      num_kv_heads: int, head_dim: int, act, q_weight: torch.Tensor, k_weight: torch.Tensor | None, eps: float,
                      q_dim: int, k_dim: int, values_are_keys: bool = False, runs: dict | None = None,
                      amplitude: float = 1.0) -> torch.Tensor:
    """Between the product and the attention where queries and keys are normed over all their heads together: q over all of
    its numbers (``q_dim`` of them count; heads laid out wider hold zeros) with ``q_weight`` [nh * hd], k alike, then the
    rotation; keys and values go to the pages, the queries [T, nh * hd] are returned.  ``qkv`` float32 [T, q | k | v]; with
    ``values_are_keys`` [T, q | k], and the values are the keys as they stand there.  ``k_pages`` None: [T, q], nothing is written."""
    k = "row_norm_kv_write"
    T = positions.numel()
    write = k_pages is not None
    _qkv_rows(k, qkv, T, (num_heads + (0 if not write else num_kv_heads * (1 if values_are_keys else 2))) * head_dim, head_dim)
    _check(positions, k, "positions", torch.int32, (T,))
    _check(seq_of_token, k, "seq_of_token", torch.int32, (T,))
    _check(block_table, k, "block_table", torch.int32)
    _need(block_table.dim() == 2, k, "block_table must be [B, pages]")
    _check(inv_freq, k, "inv_freq", torch.float32)
    _need(inv_freq.numel() * 2 == rotary_dim or rotary_dim == 0, k, lambda: f"inv_freq must hold rotary_dim/2 = {rotary_dim // 2} entries")
    _check(q_weight, k, "q_weight", tuple(_WTYPE), (num_heads * head_dim,))
    if write:
        _check(k_weight, k, "k_weight", q_weight.dtype, (num_kv_heads * head_dim,))
    adt = ACT_DTYPES[dtype_name(act)]
    q = torch.empty((T, num_heads * head_dim), dtype=adt, device=qkv.device)
    places, tiles = (None, None), (None, None, None, 0, 0)
    if write:
        places, tiles = _kv_places(k, k_pages, v_pages, layer_offset, page_size, page_stride, num_kv_heads, head_dim, block_table,
                                   runs, adt)
    _run(k, library(act).tq_row_norm_kv_write(
        _ptr(qkv), qkv.stride(0), _ptr(positions), _ptr(seq_of_token), _ptr(block_table), block_table.shape[1], _ptr(inv_freq),
        pairing, rotary_dim, float(amplitude), _ptr(q_weight), _ptr(k_weight) if write else None, _WTYPE[q_weight.dtype],
        float(eps), int(q_dim), int(k_dim), num_heads if values_are_keys else num_heads + num_kv_heads, _ptr(q), *places, page_size,
        page_stride, T, num_heads, num_kv_heads if write else 0, head_dim, int(write), *tiles, _stream()))
    return q


def diff_prep_kv_write(qkv: torch.Tensor, positions: torch.Tensor, seq_of_token: torch.Tensor, block_table: torch.Tensor,
                       k_pages: torch.Tensor | None, v_pages: torch.Tensor | None, layer_offset: int, page_size: int,
                       page_stride: int, num_heads: int, num_kv_heads: int, head_dim: int, act, q_weight: torch.Tensor,
                       k_weight: torch.Tensor | None, eps: float, norm_dim: int, temperature: tuple[float, float] | None = None,
                       expand: bool = True, runs: dict | None = None) -> torch.Tensor:
    """Between the product and a differential attention: ``qkv`` float32 [T, q | k | v], heads of ``head_dim`` numbers, a query
    or key head being its two maps of head_dim / 2 one behind the other (``norm_dim`` of each count, zeros behind them).  Every
    map is RMS-normed with ``q_weight`` / ``k_weight`` [head_dim / 2], queries are multiplied by
    1 + coef ln(floor((position + 1) / every) + 1), ``temperature`` being (coef, every); keys and values go to the pages as rows
    of head_dim.  Returns the queries: [T, nh * hd], or with ``expand`` [T, 2 nh * hd], each map a head of its own with zeros in
    the other's place.  ``k_pages`` None: ``qkv`` is [T, q] and nothing is written."""
    k = "diff_prep_kv_write"
    T = positions.numel()
    write = k_pages is not None
    _need(head_dim % 2 == 0 and 1 <= norm_dim <= head_dim // 2, k, "a head is two maps of half its width")
    _qkv_rows(k, qkv, T, (num_heads + (2 * num_kv_heads if write else 0)) * head_dim, head_dim)
    _check(positions, k, "positions", torch.int32, (T,))
    _check(seq_of_token, k, "seq_of_token", torch.int32, (T,))
    _check(block_table, k, "block_table", torch.int32)
    _need(block_table.dim() == 2, k, "block_table must be [B, pages]")
    _check(q_weight, k, "q_weight", tuple(_WTYPE), (head_dim // 2,))
    if write:
        _check(k_weight, k, "k_weight", q_weight.dtype, (head_dim // 2,))
    coef, every = temperature if temperature is not None else (0.0, 1.0)
    _need(every > 0, k, "the temperature's step must be positive")
    adt = ACT_DTYPES[dtype_name(act)]
    q = torch.empty((T, (2 if expand else 1) * num_heads * head_dim), dtype=adt, device=qkv.device)
    places, tiles = (None, None), (None, None, None, 0, 0)
    if write:
        places, tiles = _kv_places(k, k_pages, v_pages, layer_offset, page_size, page_stride, num_kv_heads, head_dim, block_table,
                                   runs, adt)
    _run(k, library(act).tq_diff_prep_kv_write(
        _ptr(qkv), qkv.stride(0), _ptr(positions), _ptr(seq_of_token), _ptr(block_table), block_table.shape[1], _ptr(q_weight),
        _ptr(k_weight) if write else None, _WTYPE[q_weight.dtype], float(eps), int(norm_dim), float(coef), float(every), _ptr(q),
        *places, page_size, page_stride, T, num_heads, num_kv_heads if write else 0, head_dim, int(write), int(expand), *tiles,
        _stream()))
    return q


def diff_attention_fused(act, head_dim: int, page_size: int, page_stride: int, scale: float) -> bool:
    """Whether ``diff_attention`` runs both maps of a head in one pass over keys and values (else two heads to a head's maps)."""
    return (dtype_name(act) == "bfloat16" and has_kernel(act, "tq_attention_mfma_diff") and head_dim % 32 == 0 and head_dim <= 256
            and page_size % 64 == 0 and page_stride % 8 == 0 and scale > 0)


def diff_attention(q: torch.Tensor, k_pages: torch.Tensor, v_pages: torch.Tensor, layer_offset: int, positions: torch.Tensor,
                   seq_of_token: torch.Tensor, block_table: torch.Tensor, page_size: int, page_stride: int, num_heads: int,
                   num_kv_heads: int, head_dim: int, scale: float, lam: float, eps: float, value_dim: int, post: float,
                   gate: torch.Tensor | None, act, runs: dict) -> torch.Tensor:
    """Differential attention behind ``diff_prep_kv_write``: both maps of every head over the cached rows, and ``diff_combine`` of
    what they leave; [T, nh * hd].  ``q`` as ``diff_prep_kv_write`` returns it: expanded, except where
    ``diff_attention_fused`` and the step is no decode step."""
    k = "diff_attention"
    T = positions.numel()
    if not diff_attention_fused(act, head_dim, page_size, page_stride, scale):
        o = attention(q, k_pages, v_pages, layer_offset, positions, seq_of_token, block_table, page_size, page_stride, 2 * num_heads,
                      num_kv_heads, head_dim, None, scale, act, runs=runs)
        return diff_combine(o, lam, eps, value_dim, post, gate, num_heads, head_dim, act)
    adt, lib = ACT_DTYPES[dtype_name(act)], library(act)
    decode = bool(runs["decode"])
    N = num_heads * head_dim
    _check(q, k, "q", adt, (T, (2 if decode else 1) * N))
    _check(k_pages, k, "k_pages", adt)
    _check(v_pages, k, "v_pages", adt)
    _check(block_table, k, "block_table", torch.int32)
    B = runs["slots"].numel()
    _check(runs["cu_seqlens"], k, "cu_seqlens", torch.int32, (B + 1,))
    _check(runs["slots"], k, "slots", torch.int32, (B,))
    _check(runs["start"], k, "start", torch.int32, (B,))
    _need(block_table.dim() == 2 and runs["max_end"] <= block_table.shape[1] * page_size, k, "positions reach beyond the page table")
    _need(num_heads % num_kv_heads == 0 and layer_offset + num_kv_heads * page_size * head_dim <= page_stride, k,
          "heads must be a multiple of kv heads, and the layer must fit in a page")
    _need(1 <= value_dim <= head_dim, k, "the values' width lies within the head")
    _need(gate is None or (gate.is_cuda and gate.dtype == torch.float32 and tuple(gate.shape) == (T, N) and gate.stride(1) == 1
                           and gate.stride(0) % 4 == 0 and gate.data_ptr() % 16 == 0), k,
          lambda: f"gate must be float32 [{T}, {N}] on the GPU, rows at multiples of 16 bytes")
    partial = None
    if decode:
        _need(T == B, k, "decoding brings one token per sequence")
        partial = torch.empty((lib.tq_attention_decode_scratch(B, 2 * num_heads, head_dim, int(runs["max_end"])),),
                              dtype=torch.float32, device=q.device)
    out = torch.empty((T, N), dtype=adt, device=q.device)
    esz = k_pages.element_size()
    _run("attention_mfma", lib.tq_attention_mfma_diff(
        _ptr(q), k_pages.data_ptr() + layer_offset * esz, v_pages.data_ptr() + layer_offset * esz, _ptr(block_table),
        block_table.shape[1], _ptr(runs["cu_seqlens"]), _ptr(runs["slots"]), _ptr(runs["start"]), page_size, page_stride, B, num_heads,
        num_kv_heads, head_dim, float(scale), float(lam), float(eps), int(value_dim), float(post), _ptr(gate),
        gate.stride(0) if gate is not None else 0, _ptr(out), _ptr(partial), int(decode), int(runs["max_new"]), int(runs["max_end"]),
        _stream()))
    return out


def diff_combine(o: torch.Tensor, lam: float, eps: float, value_dim: int, post: float, gate: torch.Tensor | None, num_heads: int,
                 head_dim: int, act) -> torch.Tensor:
    """The two maps' outputs of every head made one: r = o[t, 2 h] - lam o[t, 2 h + 1], divided by its root mean square over
    its first ``value_dim`` numbers, times ``post``, times sigmoid(gate).  ``o`` [T, 2 nh * hd] in the activation type, ``gate``
    float32 [T, nh * hd] (columns of a wider tensor allowed) or None; returns [T, nh * hd]."""
    k = "diff_combine"
    T = o.shape[0]
    _check(o, k, "o", ACT_DTYPES[dtype_name(act)], (T, 2 * num_heads * head_dim))
    N = num_heads * head_dim
    _need(gate is None or (gate.is_cuda and gate.dtype == torch.float32 and tuple(gate.shape) == (T, N) and gate.stride(1) == 1), k,
          lambda: f"gate must be float32 [{T}, {N}] on the GPU with unit stride along its rows")
    _need(1 <= value_dim <= head_dim, k, "the values' width lies within the head")
    out = torch.empty((T, N), dtype=o.dtype, device=o.device)
    _run(k, library(act).tq_diff_combine(_ptr(o), float(lam), float(eps), int(value_dim), float(post), _ptr(gate),
                                         gate.stride(0) if gate is not None else 0, _ptr(out), T, num_heads, head_dim, _stream()))
    return out


# ------------------------------------------------------------------ selective state spaces in their dual form
@dataclasses.dataclass(frozen=True)
class SsdDims:
    """Heads, value width, state width, groups and convolution taps of a Mamba-2 mixer."""
    heads: int
    vdim: int
    state: int
    groups: int
    taps: int

    @property
    def inner(self) -> int:
        return self.heads * self.vdim

    @property
    def channels(self) -> int:
        """Channels of the convolution: x, B and C."""
        return self.inner + 2 * self.groups * self.state

    @property
    def projections(self) -> int:
        """Numbers of a token's row of projections: z | x | B | C | dt."""
        return self.inner + self.channels + self.heads

    @property
    def state_floats(self) -> int:
        """Floats of a sequence's row of state: S [heads][state][vdim] and every channel's last taps - 1 inputs, filled up to a
        multiple of 4."""
        return -(-(self.heads * self.state * self.vdim + self.channels * (self.taps - 1)) // 4) * 4

    def sizes(self):
        return self.heads, self.vdim, self.state, self.groups, self.taps


def _ssd_proj(k: str, proj: torch.Tensor, d: SsdDims) -> None:
    _need(isinstance(proj, torch.Tensor) and proj.is_cuda and proj.dtype == torch.float32 and proj.dim() == 2
          and proj.stride(1) == 1 and proj.shape[1] >= d.projections, k,
          lambda: f"proj must be float32 [T, >= {d.projections}] on the GPU with unit stride along its rows")


def _ssd_state(k: str, state: torch.Tensor, d: SsdDims) -> int:
    _check(state, k, "state", torch.float32)
    _need(state.dim() == 2 and state.shape[1] == d.state_floats, k, lambda: f"state must be [slots, {d.state_floats}]")
    return state.stride(0)


def _ssd_runs(k: str, runs: dict) -> int:
    B = runs["slots"].numel()
    _check(runs["cu_seqlens"], k, "cu_seqlens", torch.int32, (B + 1,))
    _check(runs["slots"], k, "slots", torch.int32, (B,))
    return B


def ssd_prep(proj: torch.Tensor, slot_of_token: torch.Tensor, state: torch.Tensor, conv_w: torch.Tensor, conv_b: torch.Tensor,
             dt_bias: torch.Tensor, dims: SsdDims, act):
    """From the float32 projections [T, z | x | B | C | dt]: x, B and C behind the convolution and silu [T, channels], and
    softplus(dt + dt_bias) [T, heads].  Inputs before a token's run come from ``state``; nothing is written there."""
    k = "ssd_prep"
    T = slot_of_token.numel()
    _ssd_proj(k, proj, dims)
    _need(proj.shape[0] == T, k, "a row of projections per token")
    _check(slot_of_token, k, "slot_of_token", torch.int32, (T,))
    stride = _ssd_state(k, state, dims)
    _check(conv_w, k, "conv_w", torch.float32, (dims.channels, dims.taps))
    _check(conv_b, k, "conv_b", torch.float32, (dims.channels,))
    _check(dt_bias, k, "dt_bias", torch.float32, (dims.heads,))
    xbc = torch.empty((T, dims.channels), dtype=torch.float32, device=proj.device)
    dt = torch.empty((T, dims.heads), dtype=torch.float32, device=proj.device)
    _run(k, library(act).tq_ssd_prep(_ptr(proj), proj.stride(0), _ptr(slot_of_token), _ptr(state), stride, _ptr(conv_w), _ptr(conv_b),
                                     _ptr(dt_bias), *dims.sizes(), _ptr(xbc), _ptr(dt), T, _stream()))
    return xbc, dt


def _ssd_rows(k: str, xbc, dt, a_log, skip, d: SsdDims) -> int:
    T = xbc.shape[0]
    _check(xbc, k, "xbc", torch.float32, (T, d.channels))
    _check(dt, k, "dt", torch.float32, (T, d.heads))
    _check(a_log, k, "a_log", torch.float32, (d.heads,))
    _check(skip, k, "skip", torch.float32, (d.heads,))
    return T


def ssd_scan(xbc: torch.Tensor, dt: torch.Tensor, a_log: torch.Tensor, skip: torch.Tensor, runs: dict, state: torch.Tensor,
             dims: SsdDims, act) -> torch.Tensor:
    """S <- exp(-exp(a_log) dt) S + dt B x^T, y = S^T C + skip x over the step's runs of tokens, in order, from and into the
    sequences' rows of ``state``.  Returns y float32 [T, heads * vdim]."""
    k = "ssd_scan"
    T = _ssd_rows(k, xbc, dt, a_log, skip, dims)
    stride = _ssd_state(k, state, dims)
    _need(dims.state <= 1024, k, lambda: f"a state of {dims.state} channels is beyond the 1,024 this kernel takes")
    B = _ssd_runs(k, runs)
    y = torch.empty((T, dims.inner), dtype=torch.float32, device=xbc.device)
    _run(k, library(act).tq_ssd_scan(_ptr(xbc), _ptr(dt), _ptr(a_log), _ptr(skip), _ptr(runs["cu_seqlens"]), _ptr(runs["slots"]),
                                     _ptr(state), stride, *dims.sizes(), B, _ptr(y), _stream()))
    return y


def ssd_chunked(xbc: torch.Tensor, dt: torch.Tensor, a_log: torch.Tensor, skip: torch.Tensor, runs: dict, state: torch.Tensor,
                dims: SsdDims, act) -> torch.Tensor:
    """``ssd_scan`` for steps with long runs: the same sums over chunks of 64 tokens on the matrix cores, in float32 on both
    libraries (three launches), states of up to 256 channels.  ``runs`` also names ``max_new``, the longest run."""
    k = "ssd_chunked"
    T = _ssd_rows(k, xbc, dt, a_log, skip, dims)
    stride = _ssd_state(k, state, dims)
    _need(dims.state <= 256, k, lambda: f"a state of {dims.state} channels is beyond the 256 this kernel takes")
    B, max_new = _ssd_runs(k, runs), int(runs["max_new"])
    _need(1 <= max_new <= T, k, lambda: f"the longest run has {max_new} of {T} tokens")
    chunks = T // LIGHTNING_CHUNK + B
    scratch = torch.empty((chunks, dims.inner * dims.state), dtype=torch.float32, device=xbc.device)
    tot = torch.empty((chunks, dims.heads), dtype=torch.float32, device=xbc.device)
    y = torch.empty((T, dims.inner), dtype=torch.float32, device=xbc.device)
    _run(k, library(act).tq_ssd_chunked(_ptr(xbc), _ptr(dt), _ptr(a_log), _ptr(skip), _ptr(runs["cu_seqlens"]), _ptr(runs["slots"]),
                                        _ptr(state), stride, *dims.sizes(), B, max_new, _ptr(scratch), _ptr(tot), chunks, _ptr(y),
                                        _stream()))
    return y


def ssd_decode(proj: torch.Tensor, runs: dict, state: torch.Tensor, conv_w: torch.Tensor, conv_b: torch.Tensor,
               dt_bias: torch.Tensor, a_log: torch.Tensor, skip: torch.Tensor, dims: SsdDims, act) -> torch.Tensor:
    """``ssd_prep`` and ``ssd_scan`` of a step of one token per sequence, in one launch (``ssd_out`` moves the convolution's
    state on).  Returns y float32 [B, heads * vdim]."""
    k = "ssd_decode"
    _ssd_proj(k, proj, dims)
    stride = _ssd_state(k, state, dims)
    B = _ssd_runs(k, runs)
    _need(proj.shape[0] == B and runs["decode"], k, "decoding brings one token per sequence")
    _check(conv_w, k, "conv_w", torch.float32, (dims.channels, dims.taps))
    for name, t, n in (("conv_b", conv_b, dims.channels), ("dt_bias", dt_bias, dims.heads), ("a_log", a_log, dims.heads),
                       ("skip", skip, dims.heads)):
        _check(t, k, name, torch.float32, (n,))
    y = torch.empty((B, dims.inner), dtype=torch.float32, device=proj.device)
    _run(k, library(act).tq_ssd_decode(_ptr(proj), proj.stride(0), _ptr(runs["slots"]), _ptr(state), stride, _ptr(conv_w), _ptr(conv_b),
                                       _ptr(dt_bias), _ptr(a_log), _ptr(skip), *dims.sizes(), B, _ptr(y), _stream()))
    return y


def ssd_out(y: torch.Tensor, proj: torch.Tensor, weight: torch.Tensor, eps: float, parts: int, runs: dict, state: torch.Tensor,
            dims: SsdDims, act) -> torch.Tensor:
    """y silu(z) divided by its root mean square in ``parts`` equal parts, times ``weight`` [heads * vdim], in the activation
    type (z: the first columns of ``proj``); and the convolution's part of every sequence's state brought to its run's end."""
    k = "ssd_out"
    T = y.shape[0]
    _check(y, k, "y", torch.float32, (T, dims.inner))
    _ssd_proj(k, proj, dims)
    _need(proj.shape[0] == T and parts >= 1 and dims.inner % parts == 0, k, "a row of projections per token, and equal parts")
    _check(weight, k, "weight", tuple(_WTYPE), (dims.inner,))
    stride = _ssd_state(k, state, dims)
    B = _ssd_runs(k, runs)
    out = torch.empty((T, dims.inner), dtype=ACT_DTYPES[dtype_name(act)], device=y.device)
    _run(k, library(act).tq_ssd_out(_ptr(y), _ptr(proj), proj.stride(0), _ptr(weight), _WTYPE[weight.dtype], float(eps), int(parts),
                                    _ptr(runs["cu_seqlens"]), _ptr(runs["slots"]), _ptr(state), stride, *dims.sizes(), T, B,
                                    _ptr(out), _stream()))
    return out


# ------------------------------------------------------------------ sampling
def argmax(logits: torch.Tensor, act) -> torch.Tensor:
    k = "argmax"
    _check(logits, k, "logits", torch.float32)
    R, V = logits.shape
    out = torch.empty((R,), dtype=torch.int32, device=logits.device)
    _run(k, library(act).tq_argmax(_ptr(logits), R, V, _ptr(out), _stream()))
    return out


def nll(logits: torch.Tensor, targets: torch.Tensor, act) -> torch.Tensor:
    """-log softmax(logits[r])[targets[r]] per row, float32 [R] (NaN where the target is no token of the vocabulary)."""
    k = "nll"
    _check(logits, k, "logits", torch.float32)
    R, V = logits.shape
    _check(targets, k, "targets", torch.int32, (R,))
    out = torch.empty((R,), dtype=torch.float32, device=logits.device)
    _run(k, library(act).tq_nll(_ptr(logits), R, V, _ptr(targets), _ptr(out), _stream()))
    return out


def probs_half(logits: torch.Tensor, act, want_probs: bool = True,
               base: torch.Tensor | None = None) -> tuple[torch.Tensor | None, torch.Tensor | None]:
    """Each row's probabilities as the reference stores them with ``--save-logits`` (16-bit floats made by its own
    conversion: the mantissa cut, below 2^-14 zero; int16 [R, V], the bit patterns) and, with ``base`` (such rows of
    another run), the KL divergence of ``base`` against this row, float64 [R]
    (/root/reference/tools/quant.c:594-636)."""
    k = "probs_half"
    _check(logits, k, "logits", torch.float32)
    _need(logits.dim() == 2, k, "logits must be [R, V]")
    R, V = logits.shape
    _need(want_probs or base is not None, k, "nothing is asked for")
    probs = torch.empty((R, V), dtype=torch.int16, device=logits.device) if want_probs else None
    kl = None
    if base is not None:
        _check(base, k, "base", torch.int16, (R, V))
        kl = torch.empty((R,), dtype=torch.float64, device=logits.device)
    _run(k, library(act).tq_probs_half(_ptr(logits), R, V, _ptr(probs), _ptr(base), _ptr(kl), _stream()))
    return probs, kl


def rep_penalty(logits: torch.Tensor, recent: torch.Tensor, counts: torch.Tensor, penalty: float, act) -> None:
    k = "rep_penalty"
    _check(logits, k, "logits", torch.float32)
    R, V = logits.shape
    _check(recent, k, "recent", torch.int32)
    _need(recent.dim() == 2 and recent.shape[0] == R, k, lambda: f"recent must be [{R}, window]")
    _check(counts, k, "counts", torch.int32, (R,))
    _run(k, library(act).tq_rep_penalty(_ptr(logits), R, V, _ptr(recent), recent.shape[1], _ptr(counts),
                                        float(penalty), _stream()))


def sample_topp(logits: torch.Tensor, temperature: float, top_p: float, uniforms: torch.Tensor, act) -> torch.Tensor:
    k = "sample_topp"
    _check(logits, k, "logits", torch.float32)
    R, V = logits.shape
    _check(uniforms, k, "uniforms", torch.float32, (R,))
    _need(temperature > 0 and top_p > 0, k, "temperature and top_p must be positive (else use argmax)")
    probs = torch.empty((R, V), dtype=torch.float32, device=logits.device)
    out = torch.empty((R,), dtype=torch.int32, device=logits.device)
    lib = library(act)
    scratch = torch.empty((lib.tq_sample_topp_scratch(R),), dtype=torch.float32, device=logits.device)
    _run(k, lib.tq_sample_topp(_ptr(logits), R, V, float(temperature), float(top_p), _ptr(uniforms), _ptr(probs),
                               _ptr(scratch), _ptr(out), _stream()))
    return out


# ------------------------------------------------------------------------------------------------ probes
def probe_stream(buf: torch.Tensor, once: bool) -> None:
    """One read of all of ``buf`` (whole lines of 128 bytes per instruction; ``once``: with the read-once hint)."""
    k = "probe_stream"
    _need(buf.is_cuda and buf.is_contiguous(), k, "buf must be a contiguous tensor on the GPU")
    nbytes = buf.numel() * buf.element_size()
    out = torch.zeros((1,), dtype=torch.int32, device=buf.device)
    _run(k, library("bfloat16").tq_probe_stream(_ptr(buf), nbytes, int(once), 0x9e3779b9, _ptr(out), _stream()))


def probe_mfma(shape: int, workgroups: int, iters: int, seed: int, device) -> float:
    """A loop of bfloat16 matrix instructions alone (shape 32: 32x32x16, 16: 16x16x32); returns the number of
    floating-point operations that the launch does."""
    k = "probe_mfma"
    out = torch.empty((workgroups * 512,), dtype=torch.float32, device=device)
    _run(k, library("bfloat16").tq_probe_mfma(shape, workgroups, iters, seed, _ptr(out), _stream()))
    return float(workgroups) * 8 * iters * 196608.0
