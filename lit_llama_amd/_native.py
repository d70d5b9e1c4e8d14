"""ctypes binding of libmi355llama.so (include/mi355_llama.h).

The product path has no CPU fallback: if the shared library is missing or a GPU is absent, the
operators raise.  Only the structs / prototypes live here; all arithmetic is in csrc/*.hip.
"""
from __future__ import annotations

import ctypes as C
import os
from pathlib import Path
from typing import Optional

import torch

_PKG = Path(__file__).resolve().parent
LIB_PATH = _PKG / "libmi355llama.so"
CORE_LIB_PATH = _PKG / "libmi355core.so"  # the part a layered hybrid model needs (_build.build_core)

F32, BF16, F16 = 0, 1, 2
W_Q4, W_BF16, W_I8 = 0, 1, 2
EPI_STORE, EPI_ACCUM, EPI_SWIGLU, EPI_GEGLU, EPI_CLAMPGLU = 0, 1, 2, 3, 4
LF_RELU2, LF_NORM_ONE = 1, 2

_DTYPE_CODE = {torch.float32: F32, torch.bfloat16: BF16, torch.float16: F16}

c_void_p, c_int, c_int32, c_int64, c_float, c_size_t = C.c_void_p, C.c_int, C.c_int32, C.c_int64, C.c_float, C.c_size_t


class NativeError(RuntimeError):
    pass


class LinearArgs(C.Structure):
    _fields_ = [
        ("fmt", c_int32), ("R", c_int32), ("w", c_void_p), ("N", c_int32), ("K", c_int32),
        ("x", c_void_p), ("x_dtype", c_int32), ("M", c_int32), ("ldx", c_int64),
        ("norm_scale", c_void_p), ("norm_dtype", c_int32), ("eps", c_float),
        ("scales", c_void_p), ("zeros", c_void_p), ("scales2", c_void_p), ("zeros2", c_void_p),
        ("sz_dtype", c_int32), ("epi", c_int32), ("bias", c_void_p),
        ("y", c_void_p), ("y_dtype", c_int32), ("group_cols", c_int32), ("ldy", c_int64),
        ("waves", c_int32), ("grid", c_int32), ("prefetch", c_int32), ("flags", c_int32),
        ("attn_partials", c_void_p), ("attn_splits", c_int32), ("attn_heads", c_int32), ("attn_hs", c_int32),
        ("alpha", c_float), ("limit", c_float), ("slice_rows", c_int32), ("slice_stride", c_int64), ("debug_stamps", c_void_p),
    ]


class AttnArgs(C.Structure):
    _fields_ = [
        ("qkv", c_void_p), ("qkv_dtype", c_int32), ("B", c_int32), ("ld_qkv", c_int64),
        ("rope", c_void_p), ("pos", c_void_p), ("kcache", c_void_p), ("vcache", c_void_p),
        ("cache_dtype", c_int32), ("T", c_int32), ("n_head", c_int32), ("hs", c_int32),
        ("S", c_int32), ("y_dtype", c_int32), ("y", c_void_p), ("ldy", c_int64),
        ("kv_tmp", c_void_p), ("rope_gathered", c_int32), ("n_split", c_int32), ("partials", c_void_p),
        ("debug_stamps", c_void_p),
        ("adapter_k", c_void_p), ("adapter_v", c_void_p), ("adapter_gate", c_void_p),
        ("adapter_len", c_int32), ("reserved0", c_int32),
    ]


class AdapterArgs(C.Structure):
    _fields_ = [
        ("qkv", c_void_p), ("qkv_dtype", c_int32), ("B", c_int32), ("ld_qkv", c_int64),
        ("rope", c_void_p), ("pos", c_void_p), ("rope_gathered", c_int32), ("T", c_int32),
        ("n_head", c_int32), ("hs", c_int32), ("aT", c_int32), ("y_dtype", c_int32),
        ("ak", c_void_p), ("av", c_void_p), ("gate", c_void_p), ("y", c_void_p), ("ldy", c_int64),
    ]


class Int8Args(C.Structure):
    _fields_ = [
        ("w", c_void_p), ("scb", c_void_p), ("N", c_int32), ("K", c_int32),
        ("x", c_void_p), ("x_dtype", c_int32), ("M", c_int32), ("ldx", c_int64),
        ("norm_scale", c_void_p), ("norm_dtype", c_int32), ("eps", c_float),
        ("threshold", c_float), ("R", c_int32), ("bias", c_void_p), ("bias_dtype", c_int32),
        ("epi", c_int32), ("scb2", c_void_p), ("y", c_void_p), ("y_dtype", c_int32),
        ("waves", c_int32), ("ldy", c_int64), ("grid", c_int32), ("prefetch", c_int32),
        ("debug_stamps", c_void_p),
        ("attn_partials", c_void_p), ("attn_splits", c_int32), ("attn_heads", c_int32), ("attn_hs", c_int32),
        ("reserved0", c_int32),
    ]


class Weight(C.Structure):
    _fields_ = [
        ("fmt", c_int32), ("R", c_int32), ("w", c_void_p), ("N", c_int32), ("K", c_int32),
        ("scales", c_void_p), ("zeros", c_void_p), ("scales2", c_void_p), ("zeros2", c_void_p),
        ("scb", c_void_p), ("scb2", c_void_p),
        ("sz_dtype", c_int32), ("waves", c_int32), ("grid", c_int32), ("prefetch", c_int32),
        ("flags", c_int32), ("group_cols", c_int32),
    ]


class Layer(C.Structure):
    _fields_ = [
        ("rms1", c_void_p), ("rms2", c_void_p),
        ("attn", Weight), ("proj", Weight), ("fc", Weight), ("mproj", Weight),
        ("kcache", c_void_p), ("vcache", c_void_p),
        ("adapter_k", c_void_p), ("adapter_v", c_void_p), ("adapter_gate", c_void_p),
        ("adapter_len", c_int32), ("reserved0", c_int32),
    ]


class Model(C.Structure):
    _fields_ = [
        ("n_layer", c_int32), ("n_head", c_int32), ("n_embd", c_int32), ("hs", c_int32),
        ("n_hidden", c_int32), ("vocab", c_int32), ("S", c_int32), ("block_size", c_int32),
        ("param_dtype", c_int32), ("cache_dtype", c_int32), ("tp_world", c_int32), ("max_T", c_int32),
        ("eps", c_float), ("int8_threshold", c_float),
        ("wte", c_void_p), ("ln_f", c_void_p), ("lm_head", Weight), ("rope", c_void_p),
        ("layers", C.POINTER(Layer)),
        ("x", c_void_p), ("qkv", c_void_p), ("att", c_void_p), ("hbuf", c_void_p),
        ("partial", c_void_p), ("logits", c_void_p),
        ("tokens", c_void_p), ("pos", c_void_p), ("next_token", c_void_p), ("out_tokens", c_void_p),
        ("attn_part", c_void_p), ("attn_splits", c_int32), ("reserved0", c_int32),
        ("gemm_ws", c_void_p), ("gemm_ws_bytes", C.c_uint64),
    ]


class FusedStepArgs(C.Structure):
    _fields_ = [
        ("w", c_void_p), ("layer_stride", C.c_uint64),
        ("off_attn", C.c_uint32), ("off_proj", C.c_uint32), ("off_fc", C.c_uint32), ("off_mproj", C.c_uint32),
        ("layer_bytes", C.c_uint32), ("head_bytes", C.c_uint32),
        ("w_head", c_void_p), ("sz", c_void_p), ("sz_head", c_void_p), ("norms", c_void_p), ("wte", c_void_p),
        ("rope", c_void_p), ("kv", c_void_p),
        ("tokens", c_void_p), ("pos", c_void_p), ("next_token", c_void_p), ("out_tokens", c_void_p),
        ("logits", c_void_p), ("workspace", c_void_p), ("debug_stamps", c_void_p),
        ("n_layer", c_int32), ("n_head", c_int32), ("n_embd", c_int32), ("hs", c_int32),
        ("n_hidden", c_int32), ("vocab", c_int32), ("S", c_int32), ("mode", c_int32),
        ("eps", c_float), ("reserved0", c_int32),
        ("group_cols", c_int32), ("weight_fmt", c_int32), ("gt", c_void_p), ("gt_head", c_void_p),
        ("gt_layer_stride", C.c_uint64),
    ]


class TpComm(C.Structure):
    _fields_ = [
        ("world", c_int32), ("rank", c_int32), ("slot_floats", c_int32), ("reserved0", c_int32),
        ("peer_buf", c_void_p * 8), ("state", c_void_p),
    ]


class SeqBatch(C.Structure):
    _fields_ = [
        ("rows", c_int32), ("seqs", c_int32), ("max_count", c_int32), ("max_end", c_int32),
        ("row0", c_void_p), ("count", c_void_p), ("slot", c_void_p), ("pos", c_void_p),
    ]


class WindowAttnArgs(C.Structure):
    _fields_ = [
        ("proj", c_void_p), ("ld", c_int64), ("dtype", c_int32),
        ("heads", c_int32), ("kv_heads", c_int32), ("dim", c_int32), ("vdim", c_int32),
        ("off_q", c_int32), ("off_k", c_int32), ("off_v", c_int32), ("off_g", c_int32),
        ("scale", c_float), ("window", c_int32), ("ring", c_int32), ("rot_dims", c_int32), ("inv_freq", c_void_p),
        ("kring", c_void_p), ("vring", c_void_p), ("y", c_void_p), ("ldy", c_int64),
        ("partials", c_void_p), ("partials_bytes", C.c_uint64), ("path", c_int32),
        ("keep", c_int32), ("kept", c_int32), ("gate_values", c_int32), ("unit_qk", c_int32), ("unit_eps", c_float), ("sink", c_void_p),
        ("role", c_int32), ("chunked", c_int32), ("kv_rows", c_void_p),
        ("head_scale", c_void_p), ("slope", c_void_p), ("unit_v", c_int32), ("rot_at", c_int32), ("rows_per_seq", c_int64), ("ld_rows", c_int64),
        ("off_v_rows", c_int32), ("tail_dims", c_int32), ("key_tail", c_void_p), ("ld_tail", c_int64), ("tail_slot", c_int64),
        ("q_norm", c_void_p), ("k_norm", c_void_p), ("softcap", c_float), ("v_mix", c_float), ("v_first", c_void_p), ("ld_v_first", c_int64),
    ]


class RecurrentArgs(C.Structure):
    _fields_ = [
        ("kind", c_int32), ("dtype", c_int32), ("proj", c_void_p), ("ld", c_int64),
        ("heads", c_int32), ("kv_heads", c_int32), ("dim", c_int32), ("vdim", c_int32),
        ("off_q", c_int32), ("off_k", c_int32), ("off_v", c_int32), ("off_g", c_int32), ("off_a", c_int32), ("off_b", c_int32),
        ("q_scale", c_float), ("eps", c_float), ("taps", c_int32), ("rank", c_int32), ("inv_tau", c_float), ("unit_eps", c_float),
        ("conv_q", c_void_p), ("conv_k", c_void_p), ("conv_v", c_void_p), ("a_log", c_void_p), ("dt_bias", c_void_p),
        ("a2", c_void_p), ("a2_bias", c_void_p), ("head_norm", c_void_p), ("state", c_void_p), ("conv_ring", c_void_p),
        ("y", c_void_p), ("ldy", c_int64), ("scratch", c_void_p), ("scratch_bytes", C.c_uint64),
        ("path", c_int32), ("norm_ld", c_int32), ("bonus", c_void_p),
        ("conv_bq", c_void_p), ("conv_bk", c_void_p), ("conv_bv", c_void_p), ("skip", c_void_p),
    ]


class ExpertsArgs(C.Structure):
    _fields_ = [
        ("dtype", c_int32), ("rows", c_int32), ("width", c_int32), ("experts", c_int32), ("top", c_int32),
        ("ff", c_int32), ("ff_shared", c_int32), ("scale", c_float),
        ("norm", c_void_p), ("norm_dtype", c_int32), ("norm_add", c_float), ("eps", c_float), ("alpha", c_float),
        ("router", c_void_p), ("up", c_void_p), ("down", c_void_p), ("shared_up", c_void_p), ("shared_down", c_void_p),
        ("x", c_void_p), ("ldx", c_int64), ("scratch", c_void_p), ("scratch_bytes", C.c_uint64), ("path", c_int32),
        ("score", c_int32), ("act", c_int32), ("identity", c_int32), ("groups", c_int32), ("keep_groups", c_int32), ("reserved0", c_int32),
        ("correction", c_void_p), ("h", c_void_p), ("ldh", c_int64), ("logits", c_void_p), ("ld_logits", c_int64), ("out", c_void_p), ("ld_out", c_int64),
    ]


class Proj(C.Structure):
    _fields_ = [("w", c_void_p), ("N", c_int32), ("K", c_int32), ("bias", c_void_p)]


class JoinArgs(C.Structure):
    _fields_ = [
        ("dtype", c_int32), ("rows", c_int32), ("width", c_int32), ("eps", c_float), ("norm_add", c_float), ("n_stream", c_int32),
        ("tokens", c_void_p), ("embed", c_void_p), ("vocab", c_int32), ("gate_dtype", c_int32), ("t", c_void_p), ("ldt", c_int64),
        ("gate", c_void_p), ("ld_gate", c_int64), ("post", c_void_p), ("x", c_void_p), ("ldx", c_int64), ("stream", c_void_p),
        ("stream_stride", c_int64), ("stream_out", c_void_p), ("average", c_void_p), ("next", c_void_p), ("h", c_void_p), ("ldh", c_int64),
    ]


class LatentArgs(C.Structure):
    _fields_ = [
        ("proj", c_void_p), ("ld", c_int64), ("dtype", c_int32), ("heads", c_int32), ("dim", c_int32), ("rot_dim", c_int32), ("vdim", c_int32),
        ("q_rank", c_int32), ("kv_rank", c_int32), ("off_q", c_int32), ("off_c", c_int32), ("scale", c_float), ("eps", c_float),
        ("cache_rows", c_int32), ("q_norm", c_void_p), ("c_norm", c_void_p), ("inv_freq", c_void_p), ("sink", c_void_p),
        ("uq", Proj), ("expand", Proj), ("uk_t", c_void_p), ("uv", c_void_p), ("cache", c_void_p), ("y", c_void_p), ("ldy", c_int64),
        ("cq", c_void_p), ("q", c_void_p), ("qa", c_void_p), ("partials", c_void_p), ("partials_bytes", C.c_uint64),
        ("rows_c", c_void_p), ("kv_rows", c_void_p), ("expand_rows", c_int64), ("gemm_ws", c_void_p), ("gemm_ws_bytes", C.c_uint64),
        ("path", c_int32), ("reserved0", c_int32),
    ]


class NormArgs(C.Structure):
    _fields_ = [
        ("dtype", c_int32), ("rows", c_int32), ("width", c_int32), ("groups", c_int32), ("x", c_void_p), ("ldx", c_int64), ("want", c_void_p),
        ("eps", c_float), ("n_mix", c_int32), ("scale", c_void_p), ("h", c_void_p), ("ldh", c_int64), ("mu", c_void_p), ("shift", c_void_p),
        ("mix", c_void_p), ("mix_stride", c_int64),
    ]


class HybridLayer(C.Structure):
    _fields_ = [
        ("mixer", c_int32), ("mlp", c_int32), ("norm1", c_void_p), ("norm2", c_void_p),
        ("in", Proj), ("out", Proj), ("up", Proj), ("down", Proj),
        ("attn", WindowAttnArgs), ("rec", RecurrentArgs), ("moe", ExpertsArgs), ("kv_lender", c_int32), ("kv_last", c_int32),
        ("latent", LatentArgs), ("parallel", c_int32), ("hid_at", c_int32), ("cat", c_void_p), ("ld_cat", c_int64), ("limit", c_float),
        ("n_mix", c_int32), ("mu", c_void_p), ("shift", c_void_p), ("mix_w", Proj * 5), ("mix_at", c_int32 * 5), ("mix_stacked", c_int32),
        ("sandwich", c_int32), ("gate_at", c_int32), ("logits_at", c_int32), ("out_groups", c_int32), ("post1", c_void_p), ("post2", c_void_p),
        ("side", Proj), ("average", c_void_p), ("out_norm", c_void_p), ("proj_rows", c_void_p),
    ]


class HybridModel(C.Structure):
    _fields_ = [
        ("n_runs", c_int32), ("dtype", c_int32), ("norm_dtype", c_int32), ("width", c_int32),
        ("ldx", c_int32), ("vocab", c_int32), ("max_rows", c_int32), ("ld_logits", c_int32),
        ("eps", c_float), ("residual_mult", c_float), ("norm_add", c_float), ("logit_scale", c_float),
        ("norm_groups", c_int32), ("ld_n", c_int32),
        ("embed", c_void_p), ("final_norm", c_void_p), ("head", Proj), ("layers", C.POINTER(HybridLayer)),
        ("x", c_void_p), ("xw", c_void_p), ("xn", c_void_p), ("xb", c_void_p), ("mix", c_void_p), ("proj", c_void_p), ("att", c_void_p), ("hid", c_void_p),
        ("tmp", c_void_p), ("ld_att", c_int64), ("gemm_ws", c_void_p), ("gemm_ws_bytes", C.c_uint64),
        ("partials", c_void_p), ("partials_bytes", C.c_uint64), ("rec_scratch", c_void_p), ("rec_scratch_bytes", C.c_uint64),
        ("moe_scratch", c_void_p), ("moe_scratch_bytes", C.c_uint64),
        ("embed_norm", c_void_p), ("stream", c_void_p), ("side", c_void_p), ("ld_side", c_int64), ("mixed", c_void_p), ("ld_mixed", c_int64),
    ]


# name -> (restype, argtypes); must list every function declared in include/mi355_llama.h
PROTOTYPES = {
    "mi355_version": (c_int, []),
    "mi355_last_error": (C.c_char_p, []),
    "mi355_num_cus": (c_int, []),
    "mi355_packed_bytes": (c_size_t, [c_int, c_int, c_int, c_int, c_int]),
    "mi355_q4_repack": (c_int, [c_void_p, c_void_p, c_int64, c_int64, c_int, c_int, c_int, c_void_p, c_void_p]),
    "mi355_bf16_repack": (c_int, [c_void_p, c_void_p, c_int, c_int, c_int, c_int, c_void_p, c_void_p]),
    "mi355_i8_repack": (c_int, [c_void_p, c_void_p, c_int, c_int, c_int, c_void_p, c_void_p]),
    "mi355_u8_repack": (c_int, [c_void_p, c_void_p, c_int64, c_int64, c_int, c_int, c_int, c_void_p, c_void_p]),
    "mi355_linear_fast": (c_int, [C.POINTER(LinearArgs), c_void_p]),
    "mi355_linear_gemm_workspace_bytes": (c_size_t, [c_int, c_int]),
    "mi355_linear_gemm": (c_int, [C.POINTER(LinearArgs), c_void_p, c_size_t, c_void_p]),
    "mi355_linear_fast_batch": (c_int, [C.POINTER(LinearArgs), c_int, c_void_p]),
    "mi355_linear_dense": (c_int, [c_void_p, c_int64, c_void_p, c_void_p, c_void_p, c_int64, c_int, c_int, c_int,
                                   c_int, c_void_p]),
    "mi355_linear_colblock": (c_int, [c_void_p, c_int64, c_void_p, c_int64, c_int64, c_void_p, c_void_p, c_int, c_int,
                                      c_int, c_int, c_void_p, c_void_p, c_int64, c_int, c_int, c_int, c_int,
                                      c_void_p]),
    "mi355_colblock_dequant": (c_int, [c_void_p, c_int64, c_int64, c_void_p, c_void_p, c_int, c_int, c_int, c_int,
                                       c_void_p, c_int, c_int, c_int, c_void_p]),
    "mi355_rmsnorm": (c_int, [c_void_p, c_int64, c_void_p, c_int, c_float, c_void_p, c_int64, c_int, c_int, c_int,
                              c_int, c_void_p]),
    "mi355_apply_rope": (c_int, [c_void_p, c_void_p, c_void_p, c_int, c_int, c_int, c_int, c_int, c_void_p]),
    "mi355_swiglu": (c_int, [c_void_p, c_void_p, c_void_p, c_int64, c_int, c_void_p]),
    "mi355_add": (c_int, [c_void_p, c_void_p, c_void_p, c_int64, c_int, c_void_p]),
    "mi355_embedding": (c_int, [c_void_p, c_int, c_void_p, c_int, c_void_p, c_int, c_int, c_int, c_int, c_void_p]),
    "mi355_argmax": (c_int, [c_void_p, c_int, c_void_p, c_void_p, c_void_p, c_void_p]),
    "mi355_attention": (c_int, [C.POINTER(AttnArgs), c_void_p]),
    "mi355_adapter_prefix": (c_int, [C.POINTER(AdapterArgs), c_void_p]),
    "mi355_attn_combine": (c_int, [c_void_p, c_int, c_int, c_int, c_int, c_void_p, c_int, c_int64, c_void_p]),
    "mi355_kv_roll": (c_int, [c_void_p, c_void_p, c_int, c_int, c_int, c_int, c_int, c_void_p]),
    "mi355_int8_quant_rows": (c_int, [c_void_p, c_int, c_int, c_int, c_void_p, c_void_p, c_void_p]),
    "mi355_linear_int8": (c_int, [C.POINTER(Int8Args), c_void_p]),
    "mi355_linear_int8_gemm_workspace_bytes": (c_size_t, [c_int, c_int]),
    "mi355_linear_int8_gemm": (c_int, [C.POINTER(Int8Args), c_void_p, c_size_t, c_void_p]),
    "mi355_set_step": (c_int, [C.POINTER(Model), c_void_p, c_int, c_int, c_int, c_int, c_void_p]),
    "mi355_forward": (c_int, [C.POINTER(Model), c_int, c_int, c_int, c_void_p]),
    "mi355_forward_embed": (c_int, [C.POINTER(Model), c_int, c_void_p]),
    "mi355_forward_segment": (c_int, [C.POINTER(Model), c_int, c_int, c_int, c_int, c_void_p]),
    "mi355_residual_add": (c_int, [C.POINTER(Model), c_int, c_void_p]),
    "mi355_forward_head": (c_int, [C.POINTER(Model), c_int, c_int, c_int, c_void_p]),
    "mi355_graph_capture": (c_int, [C.POINTER(Model), c_int, c_void_p, C.POINTER(c_void_p)]),
    "mi355_graph_launch": (c_int, [c_void_p, c_void_p]),
    "mi355_graph_destroy": (c_int, [c_void_p]),
    "mi355_fused_step_workspace_bytes": (c_size_t, [c_int]),
    "mi355_fused_step_supported": (c_int, [c_int, c_int, c_int, c_int, c_int, c_int]),
    "mi355_fused_step": (c_int, [C.POINTER(FusedStepArgs), c_void_p]),
    "mi355_tp_comm_bytes": (c_size_t, [c_int, c_int]),
    "mi355_tp_buffer_alloc": (c_int, [c_size_t, C.POINTER(c_void_p)]),
    "mi355_tp_buffer_free": (c_int, [c_void_p]),
    "mi355_ipc_export": (c_int, [c_void_p, c_void_p]),
    "mi355_ipc_open": (c_int, [c_void_p, C.POINTER(c_void_p)]),
    "mi355_ipc_close": (c_int, [c_void_p]),
    "mi355_tp_step_begin": (c_int, [C.POINTER(TpComm), c_void_p]),
    "mi355_tp_allreduce": (c_int, [C.POINTER(TpComm), c_void_p, c_void_p, c_int, c_int, c_int, c_void_p]),
    "mi355_tp_argmax": (c_int, [C.POINTER(TpComm), c_void_p, c_int, c_int, c_void_p, c_void_p, c_void_p, c_void_p, c_int,
                                c_void_p]),
    "mi355_graph_begin": (c_int, [c_void_p]),
    "mi355_graph_end": (c_int, [c_void_p, C.POINTER(c_void_p)]),
    "mi355_sample": (c_int, [c_void_p, c_int, c_float, c_int, c_void_p, c_void_p, c_void_p, c_void_p, c_void_p, c_int,
                             c_void_p, c_void_p]),
    "mi355_sizeof": (c_int, [c_int]),
    "mi355_linear_max_rows": (c_int, [c_int, c_int, c_int, c_int]),
    "mi355_debug_time_next_launch": (c_int, [c_void_p, c_void_p]),
    "mi355_window_attention": (c_int, [C.POINTER(WindowAttnArgs), C.POINTER(SeqBatch), c_void_p]),
    "mi355_window_cache_write": (c_int, [C.POINTER(WindowAttnArgs), C.POINTER(SeqBatch), c_void_p]),
    "mi355_latent_attention": (c_int, [C.POINTER(LatentArgs), C.POINTER(SeqBatch), c_void_p]),
    "mi355_norm_groups": (c_int, [C.POINTER(NormArgs), C.POINTER(SeqBatch), c_void_p]),
    "mi355_join_rows": (c_int, [C.POINTER(JoinArgs), c_void_p]),
    "mi355_experts": (c_int, [C.POINTER(ExpertsArgs), c_void_p]),
    "mi355_experts_scratch_bytes": (c_size_t, [C.POINTER(ExpertsArgs)]),
    "mi355_recurrent": (c_int, [C.POINTER(RecurrentArgs), C.POINTER(SeqBatch), c_void_p]),
    "mi355_recurrent_scratch_bytes": (c_size_t, [c_int, c_int, c_int, c_int, c_int, c_int, c_int]),
    "mi355_hybrid_forward": (c_int, [C.POINTER(HybridModel), C.POINTER(SeqBatch), c_void_p, c_void_p, c_int, c_void_p, c_int, c_void_p]),
    "mi355_hybrid_reset_slots": (c_int, [C.POINTER(HybridModel), c_void_p, c_int, c_void_p]),
    "mi355_argmax_advance_rows": (c_int, [c_void_p, c_int64, c_int, c_int, c_void_p, c_void_p, c_void_p, c_void_p, c_int64, c_void_p]),
    "mi355_gptq_row_params": (c_int, [c_void_p, c_int64, c_int, c_int, c_int, c_int, c_void_p, c_void_p, c_void_p]),
    "mi355_gptq_block": (c_int, [c_void_p, c_int64, c_int, c_int, c_void_p, c_int64, c_void_p, c_void_p, c_int64,
                                 c_int64, c_int, c_void_p, c_void_p, c_void_p, c_int64, c_void_p]),
}

ABI_STRUCTS = [LinearArgs, AttnArgs, Int8Args, Weight, Layer, Model, FusedStepArgs, TpComm,
               SeqBatch, WindowAttnArgs, RecurrentArgs, Proj, HybridLayer, HybridModel, ExpertsArgs, LatentArgs, NormArgs, JoinArgs]

_lib: Optional[C.CDLL] = None


def _preload_hip_runtime() -> None:
    """Bind to the HIP runtime instance PyTorch ships (same soname libamdhip64.so.7 as /opt/rocm's)."""
    cand = Path(torch.__file__).resolve().parent / "lib" / "libamdhip64.so"
    if cand.exists():
        C.CDLL(str(cand), mode=C.RTLD_GLOBAL)


def lib() -> C.CDLL:
    """The loaded library; raises NativeError (never falls back) if it is not built."""
    global _lib
    if _lib is None:
        path = Path(os.environ.get("MI355_LLAMA_LIB", LIB_PATH))
        if not path.exists() and CORE_LIB_PATH.exists():
            path = CORE_LIB_PATH  # (a call outside the core then fails on its missing symbol)
        if not path.exists():
            raise NativeError(
                f"{path} not found: build it with `python -c 'import __graft_entry__ as g; g.build()'` "
                "(hipcc --offload-arch=gfx950).  There is no CPU fallback for the hot path."
            )
        _lib = _bind(path)
    return _lib


def _bind(path: Path) -> C.CDLL:
    _preload_hip_runtime()
    try:
        handle = C.CDLL(str(path))
    except OSError as e:  # pragma: no cover
        raise NativeError(f"cannot load {path}: {e}") from e
    core_only = path.name == CORE_LIB_PATH.name
    for name, (res, args) in PROTOTYPES.items():
        if core_only and not hasattr(handle, name):
            continue
        fn = getattr(handle, name)  # AttributeError if the .so is stale
        fn.restype = res
        fn.argtypes = args
    if handle.mi355_version() != 1:
        raise NativeError("libmi355llama ABI version mismatch; rebuild")
    for i, st in enumerate(ABI_STRUCTS):
        if handle.mi355_sizeof(i) != C.sizeof(st):
            raise NativeError(f"ABI struct {st.__name__}: C sizeof {handle.mi355_sizeof(i)} != ctypes {C.sizeof(st)}")
    return handle


E_ARG, E_SHAPE, E_DTYPE, E_STATE = -1, -2, -3, -4  # include/mi355_llama.h MI355_E_*


def last_error() -> str:
    return lib().mi355_last_error().decode(errors="replace")


def check(rc: int, what: str = "") -> None:
    if rc != 0:
        raise NativeError(f"{what or 'libmi355llama'} failed (rc={rc}): {last_error()}")


def require_gpu(t: torch.Tensor, what: str) -> None:
    if t.device.type != "cuda":
        raise NativeError(
            f"{what}: tensor is on {t.device}; the MI355X hot path runs on the GPU only "
            "(the CPU restatement of the reference lives in oracle/ and is test infrastructure)."
        )


def dtype_code(dt: torch.dtype) -> int:
    try:
        return _DTYPE_CODE[dt]
    except KeyError:
        raise NativeError(f"unsupported dtype {dt}") from None


def ptr(t: Optional[torch.Tensor]) -> Optional[int]:
    return None if t is None else t.data_ptr()


def stream_ptr(stream: Optional["torch.cuda.Stream"] = None) -> Optional[int]:
    s = stream if stream is not None else torch.cuda.current_stream()
    return s.cuda_stream or None


def num_cus() -> int:
    return int(lib().mi355_num_cus())
