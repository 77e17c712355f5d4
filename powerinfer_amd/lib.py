"""ctypes binding of libpowerinfer_hip.so (the C ABI declared in include/powerinfer_hip.h).

The library is loaded from this directory (built by `python -m powerinfer_amd.build`).  There is no CPU
fallback: without the shared object, or without a HIP device, everything here raises.
"""
import ctypes as C
import os

import numpy as np

HERE = os.path.dirname(os.path.abspath(__file__))
LIB_PATH = os.path.join(HERE, "libpowerinfer_hip.so")

F32, F16, Q4_0, I32, BF16 = 0, 1, 2, 18, 30
MIXER_LATENT, MIXER_GROUPED, MIXER_LINEAR, MIXER_KEYED = 0, 1, 2, 3
DECAY_CONST, DECAY_KEYED, DECAY_GATED = 0, 1, 2
FFN_NONE, FFN_MOE, FFN_GLU, FFN_GLU_MOE = 0, 1, 2, 3
ROT_PLAIN, ROT_WAVES, ROT_RAMP = 0, 1, 2
EPI_NONE, EPI_RELU, EPI_ADD, EPI_ADD2 = 0, 1, 2, 3
NORM_NONE, NORM_RMS, NORM_LAYER = 0, 1, 2

_vp, _i, _f, _sz, _u64 = C.c_void_p, C.c_int, C.c_float, C.c_size_t, C.c_uint64


class Norm(C.Structure):
    _fields_ = [("kind", C.c_int32), ("eps", C.c_float), ("w", C.c_void_p), ("b", C.c_void_p)]


class GroupGemm(C.Structure):
    _fields_ = [("W", _vp), ("w_gs", _sz), ("rows", C.c_int32), ("cols", C.c_int32), ("ldw", C.c_int32), ("n_group", C.c_int32),
                ("x", _vp), ("x_gs", _sz), ("ldx", C.c_int32), ("T", C.c_int32),
                ("y", _vp), ("y_gs", _sz), ("ldy", C.c_int32), ("y_f32", C.c_int32), ("relu2", C.c_int32),
                ("alpha", _f), ("off", _vp), ("gather", _vp), ("gather_div", C.c_int32),
                ("tiles", _vp), ("n_tiles", _vp), ("max_tiles", C.c_int32), ("glu", C.c_int32), ("glu_limit", _f), ("glu_gain", _f),
                ("pair_w", _vp), ("glu_plain_up", C.c_int32)]


class LatentPrep(C.Structure):
    _fields_ = [("z", _vp)] + [(n, C.c_int32) for n in ("ldz", "T", "n_head", "dim", "dim_ld", "rot_dim", "kv_rank", "rank_ld", "kd")] + [
        ("cs", _vp), ("norm_w", _vp), ("eps", _f), ("q_un", _vp), ("q_lat", _vp), ("cache", _vp), ("cell", _vp)]


class LatentAttn(C.Structure):
    _fields_ = [("q_lat", _vp), ("cache", _vp), ("lists", _vp), ("list_ld", _sz), ("work", _vp), ("n_vis", _vp)] + [
        (n, C.c_int32) for n in ("n_work", "T", "n_head", "kv_rank", "rank_ld", "kd", "n_parts")] + [
        ("scale", _f), ("sink", _vp), ("scratch", _vp), ("out_lat", _vp)]


class LatentExpanded(C.Structure):
    _fields_ = [(n, _vp) for n in ("q_un", "q_lat", "keys", "values", "cache", "list", "n_vis", "sink", "att")] + [
        (n, C.c_int32) for n in ("tok0", "T", "n_head", "dim", "dim_ld", "rot_dim", "vdim", "rank_ld", "kd", "ld_att")] + [("scale", _f)]


class FfnFront(C.Structure):
    _fields_ = [(n, C.c_int32) for n in ("off_glu", "ff", "ff_ld", "off_score")] + [("limit", _f), ("gain", _f), ("act", _vp)] + [
        (n, C.c_int32) for n in ("ld_act", "off_router", "n_expert", "n_top")] + [("ids", _vp), ("weights", _vp), ("plain_up", C.c_int32)]


class GqaPrep(C.Structure):
    _fields_ = [("z", _vp)] + [(n, C.c_int32) for n in ("ldz", "T", "n_head", "n_kv", "dim", "vdim", "rot_dim", "off_k", "off_v", "hd", "unit")] + [
        ("cs", _vp), ("eps", _f), ("q", _vp), ("cache", _vp), ("cell", _vp), ("rot_pairs", C.c_int32), ("unit_v", C.c_int32), ("q_norm", _vp), ("k_norm", _vp), ("temp", _vp),
        ("v_first", _vp), ("v_mix", _vp), ("v_keep", _vp), ("ld_first", C.c_int32)]


class GqaAttn(C.Structure):
    _fields_ = [("q", _vp), ("cache", _vp), ("lists", _vp), ("list_ld", _sz), ("work", _vp), ("n_vis", _vp)] + [
        (n, C.c_int32) for n in ("n_work", "T", "n_head", "n_kv", "dim", "vdim", "hd", "n_parts", "wide")] + [
        ("scale", _f), ("sink", _f), ("scratch", _vp), ("att", _vp), ("ld_att", C.c_int32), ("out_scale", _f), ("window", C.c_int32), ("first", _vp),
        ("softcap", _f), ("sinks", _vp), ("all_values", C.c_int32)]


class GqaMix(C.Structure):
    _fields_ = [("a", _vp), ("talk", _vp), ("z", _vp)] + [(n, C.c_int32) for n in ("ldz", "off_gate", "T", "n_head", "n_kv", "vdim")] + [("att", _vp), ("ld_att", C.c_int32), ("tokens", _vp), ("n_tokens", C.c_int32),
        ("parts", _vp), ("n_parts", C.c_int32)]


class Linear(C.Structure):
    _fields_ = [("z", _vp)] + [(n, C.c_int32) for n in ("ldz", "T", "n_head", "dim", "vdim", "off_k", "off_v")] + [
        ("decay", _vp), ("powers", _vp), ("state", _vp), ("runs", _vp), ("n_runs", C.c_int32), ("o", _vp), ("q", _vp), ("k", _vp), ("v", _vp), ("states", _vp)] + [
        (n, C.c_int32) for n in ("dim_ld", "vdim_ld", "n_chunks")] + [("chunks", _vp), ("first_chunk", _vp)] + [
        (n, C.c_int32) for n in ("decay_kind", "off_q", "plain")] + [("q_scale", _f), ("slot_ld", _sz), ("a2", _vp), ("a2_b", _vp)] + [
        (n, C.c_int32) for n in ("off_a", "rank", "rank_ld")] + [("tau", _f), ("i_b", _vp), ("f_b", _vp), ("off_i", C.c_int32), ("off_f", C.c_int32), ("cap", _f), ("den", _vp), ("gates", _vp)]


class GateNorm(C.Structure):
    _fields_ = [("o", _vp), ("z", _vp), ("w", _vp)] + [(n, C.c_int32) for n in ("ldz", "off_gate", "n", "T")] + [("eps", _f), ("att", _vp), ("ld_att", C.c_int32), ("scale", _f), ("heads", C.c_int32), ("silu", C.c_int32), ("den", _vp)]


class LayerOut(C.Structure):
    _fields_ = [("x", _vp), ("wo", _vp), ("att", _vp), ("rows", C.c_int32), ("ld_att", C.c_int32), ("T", C.c_int32),
                ("down", _vp), ("act", _vp), ("ids", _vp), ("ld_act", C.c_int32), ("top", C.c_int32), ("n_expert", C.c_int32),
                ("out", _vp), ("keep", _vp), ("scaled", C.c_int32), ("alpha", _f), ("gate_z", _vp), ("gate_b", _vp), ("ld_gate", C.c_int32), ("off_gate", C.c_int32)]


class ResNorm(C.Structure):
    _fields_ = [(n, _vp) for n in ("x", "mix", "gate_z", "gate_b", "w")] + [(n, C.c_int32) for n in ("ld_gate", "off_gate", "T", "cols")] + [
        ("alpha", _f), ("eps", _f), ("out", _vp), ("keep", _vp), ("h", _vp), ("ld", C.c_int32), ("ol", C.c_int32)]


class SumNorm(C.Structure):
    _fields_ = [("x", _vp), ("mix", _vp), ("y", _vp), ("inv", _vp), ("top", C.c_int32), ("y_w", _vp), ("w", _vp), ("mult", _f), ("w_next", _vp), ("rows", _vp)] + [
        (n, C.c_int32) for n in ("T", "cols", "groups")] + [("eps", _f), ("keep", _vp), ("h", _vp), ("ld", C.c_int32), ("ol", C.c_int32)]


class ConvNorm(C.Structure):
    _fields_ = [("x", _vp), ("w", _vp), ("taps_w", _vp)] + [(n, C.c_int32) for n in ("T", "cols", "groups", "taps")] + [
        ("eps", _f), ("state", _vp), ("slot_ld", _sz), ("items", _vp), ("n_items", C.c_int32), ("h", _vp), ("ld", C.c_int32), ("ol", C.c_int32)]


class PiError(RuntimeError):
    pass


_lib = None
_inited = False

_SIGS = {
    "pi_init": (_i, [_i]),
    "pi_last_error": (C.c_char_p, []),
    "pi_device_name": (_i, [C.c_char_p, _sz]),
    "pi_malloc": (_vp, [_sz]),
    "pi_free": (_i, [_vp]),
    "pi_malloc_host": (_vp, [_sz]),
    "pi_free_host": (_i, [_vp]),
    "pi_memset": (_i, [_vp, _i, _sz]),
    "pi_memcpy_h2d": (_i, [_vp, _vp, _sz]),
    "pi_memcpy_d2h": (_i, [_vp, _vp, _sz]),
    "pi_memcpy_d2d": (_i, [_vp, _vp, _sz]),
    "pi_sync": (_i, []),
    "pi_fill_normal_f16": (_i, [_vp, _sz, _u64, _f, _vp, _i, _vp]),
    "pi_fill_normal_bf16": (_i, [_vp, _sz, _u64, _f, _vp]),
    "pi_fill_normal_q4_0": (_i, [_vp, _sz, _u64, _f, _vp]),
    "pi_event_create": (_vp, []),
    "pi_event_record": (_i, [_vp, _vp]),
    "pi_event_elapsed_ms": (_i, [_vp, _vp, C.POINTER(_f)]),
    "pi_event_destroy": (_i, [_vp]),
    "pi_k_gemv": (_i, [_i, _vp, _i, _i, _vp, C.POINTER(Norm), _i, _vp, _vp, _vp, _vp]),
    "pi_k_gemv_multi_f16": (_i, [_vp, _vp, _i, _i, _vp, C.POINTER(Norm), _vp, _vp]),
    "pi_workspace_create": (_vp, [_i, _i]),
    "pi_workspace_destroy": (_i, [_vp]),
    "pi_k_predictor_fc2": (_i, [_vp, _i, _i, _vp, _f, _vp, _i, _vp, _vp, _vp, _vp, _vp, _vp]),
    "pi_k_compact_active": (_i, [_vp, _i, _f, _vp, _i, _vp, _vp, _vp, _vp]),
    "pi_k_sparse_upgate": (_i, [_i, _vp, _vp, _i, _i, _vp, C.POINTER(Norm), _i, _vp, _vp, _vp, _vp, _vp, _vp, _vp, _vp, _vp]),
    "pi_k_sparse_axpy": (_i, [_i, _vp, _i, _i, _vp, _vp, _vp, _vp, _vp, _i, _vp, _vp, _vp, _vp, _vp]),
    "pi_k_sparse_ffn_supported": (_i, [_i, _i, _i]),
    "pi_k_sparse_ffn_hot_supported": (_i, [_i, _i, _i]),
    "pi_k_sparse_ffn_workgroups": (_i, [_i, _i, _i]),
    "pi_k_sparse_ffn": (_i, [_vp, _i, _i, _vp, _f, _vp, _vp, _vp, _i, _vp, C.POINTER(Norm), _i, _vp, _vp, _vp, _vp, _vp, _vp, _vp, _vp]),
    "pi_k_sparse_ffn_noalloc_scratch_bytes": (_sz, []),
    "pi_k_sparse_ffn_noalloc_supported": (_i, [_i, _i, _i]),
    "pi_k_sparse_ffn_noalloc": (_i, [_vp, _i, _i, _vp, _f, _vp, _vp, _vp, _i, _vp, C.POINTER(Norm), _i, _vp, _vp, _vp, _vp, _vp, _vp, _vp]),
    "pi_k_pred_upgate_q4_supported": (_i, [_i, _i, _i]),
    "pi_k_pred_upgate_q4": (_i, [_vp, _i, _i, _vp, _f, _vp, _vp, _i, _vp, C.POINTER(Norm), _vp, _vp, _vp, _vp, _vp, _vp, _vp]),
    "pi_k_axpy_q4_partials": (_i, [_vp, _i, _i, _vp, _vp, _vp, _vp, _vp]),
    "pi_k_pred_upgate_q4_split": (_i, [_vp, _i, _i, _vp, _f, _vp, _vp, _vp, _vp, _i, _vp, C.POINTER(Norm), _vp, _vp, _vp, _vp, _vp, _vp, _vp]),
    "pi_k_axpy_q4_partials_split": (_i, [_vp, _vp, _i, _i, _vp, _vp, _vp, _vp, _vp]),
    "pi_k_axpy_q4_reduce": (_i, [_i, _i, _i, _vp, _vp, _vp, _vp, _vp, _vp]),
    "pi_k_k_shift": (_i, [_vp, _i, _i, _i, _i, _f, _f, _vp, _i, _vp]),
    "pi_k_k_shift_cells": (_i, [_vp, _i, _i, _i, _i, _i, _f, _f, _vp, _vp]),
    "pi_k_kv_compact": (_i, [_vp, _vp, _i, _i, _i, _vp, _i, _vp]),
    "pi_k_sparse_ffn_partials": (_i, [_vp, _i, _i, _vp, _f, _vp, _vp, _vp, _i, _vp, C.POINTER(Norm), _vp, _vp, _vp, _vp]),
    "pi_k_sparse_ffn_partials_hot": (_i, [_vp, _i, _i, _vp, _f, _vp, _vp, _vp, _i, _vp, C.POINTER(Norm), _vp, _vp, _vp, _vp, _vp, _vp, _vp]),
    "pi_k_sparse_ffn_reduce_hot": (_i, [_i, _i, _i, _vp, _vp, _vp, _vp, _vp, _vp]),
    "pi_k_sparse_ffn_reduce": (_i, [_i, _i, _i, _vp, _vp, _vp, _vp, _vp, _vp]),
    "pi_k_pred_upgate_supported": (_i, [_i, _i, _i]),
    "pi_k_pred_upgate": (_i, [_vp, _i, _i, _vp, _f, _vp, _vp, _i, _vp, C.POINTER(Norm), _vp, _vp, _vp, _vp]),
    "pi_k_sparse_axpy_dense": (_i, [_vp, _i, _i, _vp, _vp, _i, _vp, _vp, _vp, _vp, _vp]),
    "pi_k_norm_round_f16": (_i, [_vp, _i, _i, C.POINTER(Norm), _vp, _vp, _vp]),
    "pi_k_gemm_f16": (_i, [_vp, _i, _i, _vp, _i, _i, _vp, _vp, _vp, _vp, _vp]),
    "pi_k_gemm_bf16": (_i, [_vp, _i, _i, _vp, _i, _i, _vp, _vp, _vp, _vp, _vp]),
    "pi_k_batch_predictor_fc2": (_i, [_vp, _i, _i, _vp, _i, _f, _vp, _vp, _vp]),
    "pi_k_batch_sparse_ffn": (_i, [_vp, _i, _i, _f, _vp, _vp, _vp, _i, _vp, _i, _vp, _vp, _vp, _vp, _vp, _vp, _vp]),
    "pi_k_norm_round_f16_ol": (_i, [_vp, _i, _i, C.POINTER(Norm), _vp, _vp, _vp]),
    "pi_k_gemm_f16_ol": (_i, [_vp, _i, _i, _vp, _i, _i, _vp, _vp, _vp, _vp, _vp]),
    "pi_k_gemm_bf16_ol": (_i, [_vp, _i, _i, _vp, _i, _i, _vp, _vp, _vp, _vp, _vp]),
    "pi_k_batch_predictor_fc2_ol": (_i, [_vp, _i, _i, _vp, _i, _f, _vp, _vp, _vp]),
    "pi_k_batch_sparse_ffn_ol": (_i, [_vp, _i, _i, _f, _vp, _vp, _vp, _i, _vp, _i, _vp, _vp, _vp, _vp, _vp, _vp, _vp]),
    "pi_k_batch_union_count": (_i, [_i, _vp, _vp, _vp, _vp]),
    "pi_k_q4_split": (_i, [_vp, _i, _i, _vp, _vp, _vp]),
    "pi_k_norm_q8_blocks": (_i, [_vp, _i, _i, C.POINTER(Norm), _vp, _vp, _vp, _vp, _vp]),
    "pi_k_norm_q8_blocks_ol": (_i, [_vp, _i, _i, C.POINTER(Norm), _vp, _vp, _vp, _vp, _vp]),
    "pi_k_gemm_q4_t16": (_i, [_vp, _vp, _i, _i, _vp, _vp, _vp, _i, _i, _vp, _vp, _vp, _vp]),
    "pi_k_batch_sparse_ffn_q4": (_i, [_vp, _i, _i, _f, _vp, _vp, _vp, _vp, _vp, _vp, _i, _vp, _vp, _vp, _i, _vp, _vp, _vp, _vp, _vp, _vp, _vp, _vp, _vp]),
    "pi_k_gemm_tile_f16": (_i, [_vp, _i, _i, _vp, _i, _i, _vp, _vp, _vp, _vp, _i, _vp]),
    "pi_k_gemm_tile_bf16": (_i, [_vp, _i, _i, _vp, _i, _i, _vp, _vp, _vp, _vp, _i, _vp]),
    "pi_k_ffn_h_f16": (_i, [_vp, _vp, _vp, _f, _i, _i, _vp, _vp]),
    "pi_k_transpose_f16": (_i, [_vp, _i, _i, _vp, _vp]),
    "pi_k_norm_q8_round_f16": (_i, [_vp, _i, _i, C.POINTER(Norm), _vp, _vp, _vp]),
    "pi_k_ffn_h_q8_f16": (_i, [_vp, _vp, _vp, _f, _i, _i, _vp, _vp]),
    "pi_k_dequant_q4_f16": (_i, [_vp, _vp, _vp, _vp, _i, _i, _vp, _vp]),
    "pi_k_assemble_rows_f16": (_i, [_vp, _vp, _vp, _vp, _i, _i, _vp, _vp]),
    "pi_k_embed_batch_q4": (_i, [_vp, _i, _vp, _i, _vp, _vp]),
    "pi_k_host_signal": (_i, [_vp, _vp, _i, _i, _vp]),
    "pi_k_sparse_ffn_two_phase_supported": (_i, [_i, _i, _i]),
    "pi_k_sparse_ffn_logits_hot": (_i, [_vp, _i, _i, _vp, _f, _i, _vp, C.POINTER(Norm), _vp, _vp, _vp, _vp, _vp, _vp, _vp, _vp]),
    "pi_k_sparse_ffn_rows_hot": (_i, [_i, _f, _vp, _vp, _vp, _i, _vp, C.POINTER(Norm), _vp, _vp, _vp, _vp, _vp, _vp, _vp, _vp]),
    "pi_k_sparse_ffn_q4_partials": (_i, [_vp, _i, _i, _vp, _f, _vp, _vp, _vp, _vp, _vp, _vp, _i, _vp, C.POINTER(Norm), _vp, _vp, _vp, _vp, _vp, _vp]),
    "pi_k_sparse_ffn_q4_reduce": (_i, [_i, _i, _i, _vp, _vp, _vp, _vp, _vp, _vp]),
    "pi_k_pred_q4_logits": (_i, [_vp, _i, _i, _vp, _f, _i, _vp, C.POINTER(Norm), _vp, _vp, _vp, _vp, _vp, _vp]),
    "pi_k_upgate_q4_hot_rows": (_i, [_i, _f, _vp, _vp, _i, _vp, C.POINTER(Norm), _vp, _vp, _vp, _vp, _vp, _vp, _vp, _vp]),
    "pi_k_host_wait": (_i, [_vp, _vp, _i, _vp, C.c_double, _vp]),
    "pi_k_host_signal_wait": (_i, [_vp, _vp, _i, _i, _vp, C.c_double, _vp]),
    "pi_ggml_backend_get_stats": (None, [_vp]),
    "pi_ggml_backend_set_fusion": (None, [_i]),
    "pi_gemm_lib_create": (_vp, [C.c_size_t]),
    "pi_gemm_lib_destroy": (_i, [_vp]),
    "pi_gemm_lib_f16": (_i, [_vp, _vp, _i, _i, _vp, _i, _i, _vp, _vp, _vp, _vp, _vp]),
    "pi_gemm_lib_bf16": (_i, [_vp, _vp, _i, _i, _vp, _i, _i, _vp, _vp, _vp, _vp, _vp]),
    "pi_k_batch_sparse_mul_mat": (_i, [_vp, _i, _i, _vp, _i, _vp, _f, _vp, _vp, _vp, _vp, _vp]),
    "pi_k_batch_sparse_axpy": (_i, [_vp, _i, _i, _vp, _vp, _i, _f, _vp, _vp, _vp, _vp, _vp]),
    "pi_k_attn_split_supported": (_i, [_i, _i, _i]),
    "pi_k_attn_ggml_supported": (_i, [_i, _i, _i]),
    "pi_k_attn_ggml": (_i, [_vp, _vp, _vp, _vp, _i, _f, _f, _f, _vp, _vp, _i, _i, _i, _i, _i, _i, _vp, _vp, _vp, _vp]),
    "pi_k_attn_ggml_step": (_i, [_vp, _i, _vp, _i, _f, _f, _f, _vp, _vp, _i, _i, _i, _i, _i, _i, _i, _vp, _vp, _i, _vp, _i, _vp]),
    "pi_k_attn_split_scratch_floats": (_sz, [_i, _i, _i, _i]),
    "pi_k_attn_split": (_i, [_vp, _i, _vp, _vp, _vp, _sz, _i, _i, _i, _i, _i, _i, _i, _vp, _vp, _vp, _i, _vp, _vp]),
    "pi_k_attn_chunk_supported": (_i, [_i, _i, _i]),
    "pi_k_attn_chunk_long": (_i, [_vp, _i, _i, _i, _i, _i, _i, _f, _f, _vp, _i, _i, _vp, _vp, _vp, _vp, _vp, _vp, _vp]),
    "pi_k_attn_split_cached": (_i, [_vp, _vp, _vp, _i, _i, _i, _i, _i, _i, _vp, _vp, _vp, _vp]),
    "pi_k_attn_fused_batch": (_i, [_vp, _i, _vp, _vp, _vp, _sz, _i, _i, _i, _i, _i, _i, _vp, _vp, _i, _vp, _vp]),
    "pi_k_attn_fused_batch_ol": (_i, [_vp, _i, _vp, _vp, _vp, _sz, _i, _i, _i, _i, _i, _i, _vp, _vp, _i, _vp, _vp]),
    "pi_k_attn_fused_batch_q8": (_i, [_vp, _i, _vp, _vp, _vp, _sz, _i, _i, _i, _i, _i, _i, _vp, _vp, _i, _vp, _vp, _vp, _vp]),
    "pi_k_attn_chunk": (_i, [_vp, _i, _i, _i, _i, _i, _i, _f, _f, _vp, _i, _i, _vp, _vp, _vp, _vp, _i, _vp, _vp]),
    "pi_k_embed_batch": (_i, [_vp, _i, _vp, _i, _vp, _vp]),
    "pi_k_argmax_batch": (_i, [_vp, _i, _i, _vp, _vp, _vp, _vp, _i, _vp]),
    "pi_k_step_advance": (_i, [_vp, _vp]),
    "pi_k_rope_kv_store": (_i, [_vp, _i, _i, _i, _i, _f, _f, _vp, _i, _vp, _vp, _vp, _vp]),
    "pi_k_attn_decode": (_i, [_vp, _vp, _vp, _i, _i, _i, _i, _vp, _vp, _vp]),
    "pi_k_rope_table": (_i, [_vp, _i, _i, _i, _f, _f, _vp]),
    "pi_k_attn_fused_supported": (_i, [_i, _i]),
    "pi_k_attn_decode_supported": (_i, [_i, _i]),
    "pi_k_attn_fused": (_i, [_vp, _vp, _vp, _vp, _i, _i, _i, _i, _i, _vp, _vp, _vp]),
    "pi_k_embed": (_i, [_i, _vp, _i, _vp, _vp, _vp]),
    "pi_k_argmax": (_i, [_vp, _i, _vp, _vp]),
    "pi_k_embed_norm": (_i, [_vp, _i, _vp, _i, _vp, _f, _vp, _vp]),
    "pi_k_norm_pair": (_i, [_i, _vp, _vp, _i, _i, _f, _vp, _vp, _vp, _vp, _i, _i, _vp]),
    "pi_k_group_gemm": (_i, [_i, C.POINTER(GroupGemm), _vp]),
    "pi_k_group_gemm_tile": (_i, [C.POINTER(GroupGemm), _i, _vp]),
    "pi_k_rope_angles": (_i, [_vp, _i, _i, C.c_double, _vp, _vp]),
    "pi_k_latent_prep": (_i, [_i, C.POINTER(LatentPrep), _vp]),
    "pi_k_latent_attn_rows": (_i, [_i]),
    "pi_k_latent_attn_supported": (_i, [_i, _i, _i]),
    "pi_k_latent_attn_scratch_floats": (_sz, [_i, _i, _i]),
    "pi_k_latent_attn": (_i, [_i, C.POINTER(LatentAttn), _vp]),
    "pi_k_latent_expanded_supported": (_i, [_i, _i, _i]),
    "pi_k_latent_attn_expanded": (_i, [C.POINTER(LatentExpanded), _vp]),
    "pi_k_latent_shift": (_i, [_i, _vp, _i, _i, _i, _i, C.c_double, _vp, _vp]),
    "pi_k_route": (_i, [_vp, _i, _i, _i, _i, _i, _vp, _vp, _vp, _vp]),
    "pi_k_moe_sort": (_i, [_vp, _i, _i, _vp, _vp, _vp, _i, _vp, _vp, _vp]),
    "pi_k_moe_combine": (_i, [_i, _vp, _vp, _vp, _vp, _vp, _i, _i, _i, _vp, _vp, _vp]),
    "pi_k_gemm_bf16_ol_two": (_i, [_vp, _i, _vp, _vp, _vp, _i, _vp, _vp, _i, _i, _vp]),
    "pi_k_layer_step_supported": (_i, [_i, _i, _i]),
    "pi_k_latent_step": (_i, [C.POINTER(LatentPrep), _vp, _vp, _i, _i, _i, _i, _vp, _vp, _vp, _vp]),
    "pi_k_latent_attn_parts": (_i, [C.POINTER(LatentAttn), _vp]),
    "pi_k_value_up_step": (_i, [C.POINTER(LatentAttn), _vp, _i, _vp, _i, _vp, _i, _i, _i, _vp, _vp, _vp, _i, _vp, _i, _vp]),
    "pi_k_layer_out_step": (_i, [C.POINTER(LayerOut), _vp]),
    "pi_k_embed_bigram": (_i, [_vp, _i, _vp, _vp, _i, _f, _vp, C.c_int32, C.c_int64, C.c_int64, _i, _vp, _vp, _vp]),
    "pi_k_layer_norm": (_i, [_i, _vp, _vp, _i, _i, _f, _vp, _vp, _vp, _vp, _i, _i, _vp]),
    "pi_k_gqa_head_ld": (_i, [_i, _i, _i]),
    "pi_k_gqa_prep": (_i, [_i, C.POINTER(GqaPrep), C.POINTER(FfnFront), _vp]),
    "pi_k_gqa_rows": (_i, [_i]),
    "pi_k_gqa_scratch_floats": (_sz, [_i, _i, _i, _i, _i]),
    "pi_k_gqa_attn": (_i, [_i, C.POINTER(GqaAttn), _vp]),
    "pi_k_gqa_attn_parts": (_i, [C.POINTER(GqaAttn), _vp]),
    "pi_k_gqa_shift": (_i, [_i, _vp, _i, _i, _i, _i, C.c_double, _i, _vp, _vp]),
    "pi_k_gqa_shift_table": (_i, [_i, _vp, _i, _i, _i, _i, _vp, _i, _vp, _vp]),
    "pi_k_gqa_mix": (_i, [_i, C.POINTER(GqaMix), _vp]),
    "pi_k_gqa_talk_tokens": (_i, [_i, _i, _i, _i]),
    "pi_k_gqa_stats": (_i, [C.POINTER(GqaAttn), _vp, _vp]),
    "pi_k_gqa_talk": (_i, [C.POINTER(GqaAttn), C.POINTER(GqaMix), _vp, _vp, _i, _vp]),
    "pi_k_rope_angles_table": (_i, [_vp, _i, _i, _vp, C.c_double, _vp, _vp]),
    "pi_k_route_scores": (_i, [_vp, _i, _i, _i, _vp, _vp, _vp]),
    "pi_k_expert_up_step": (_i, [_vp, _i, _i, _i, _f, _f, _i, _i, _vp, _i, _vp, _vp, _i, _vp, _i, _vp]),
    "pi_k_sum_norm": (_i, [_i, C.POINTER(SumNorm), _vp]),
    "pi_k_conv_norm": (_i, [_i, C.POINTER(ConvNorm), _vp]),
    "pi_k_conv_tokens": (_i, [_i, _i]),
    "pi_k_linear_chunk": (_i, []),
    "pi_k_linear_supported": (_i, [_i, _i]),
    "pi_k_linear_states_bytes": (_sz, [_i, _i, _i, _i]),
    "pi_k_linear_copies": (_i, [_i]),
    "pi_k_linear_slot_floats": (_sz, [_i, _i, _i, _i]),
    "pi_k_linear_gate_floats": (_sz, [_i, _i, _i, _i, _i]),
    "pi_k_ffn_front": (_i, [_i, _vp, _i, _i, C.POINTER(FfnFront), _vp]),
    "pi_k_linear_step_beside": (_i, [_i, C.POINTER(Linear), C.POINTER(GqaPrep), _vp]),
    "pi_k_res_norm": (_i, [_i, C.POINTER(ResNorm), _vp]),
    "pi_k_gemm_bf16_ol_glu": (_i, [_vp, _i, _vp, _f, _f, _f, _vp, _i, _vp, _i, _vp, _i, _i, _vp]),
    "pi_k_linear_step": (_i, [_i, C.POINTER(Linear), C.POINTER(FfnFront), _vp]),
    "pi_k_linear_prep": (_i, [_i, C.POINTER(Linear), C.POINTER(FfnFront), _vp]),
    "pi_k_linear_chunks": (_i, [C.POINTER(Linear), _vp]),
    "pi_k_gate_norm": (_i, [_i, C.POINTER(GateNorm), _vp]),
    "pi_k_mix_up_step": (_i, [C.POINTER(GqaAttn), C.POINTER(GateNorm), _vp, _i, _i, _i, _f, _f, _vp, _i, _vp, _vp, _i, _vp, _i, _vp]),
    "pi_k_place_bf16": (_i, [_vp, C.c_int64, _i, _vp, _i, _i, _i, C.c_int64, _i, _vp]),
    "pi_k_pad_cols_bf16": (_i, [_vp, C.c_int64, _i, _vp, _i, _vp]),
    "pi_k_transpose_pad_bf16": (_i, [_vp, _i, _i, _i, _vp, _i, _vp]),
    "pi_k_cells_advance": (_i, [_i, _vp, _vp, _sz, _vp, _vp, _vp, _vp]),
}


def load():
    """dlopen the library and declare signatures (no device call)."""
    global _lib
    if _lib is None:
        if not os.path.exists(LIB_PATH):
            raise PiError(f"{LIB_PATH} is missing: run `python -m powerinfer_amd.build` (no CPU fallback exists)")
        L = C.CDLL(LIB_PATH)
        for name, (res, args) in _SIGS.items():
            fn = getattr(L, name)
            fn.restype, fn.argtypes = res, args
        _lib = L
    return _lib


def declared_symbols():
    from .model import ENGINE_SYMBOLS
    return sorted(list(_SIGS) + ENGINE_SYMBOLS)


def check(rc, what=""):
    if rc != 0:
        raise PiError(f"{what} failed ({rc}): {load().pi_last_error().decode()}")


def init(device=0):
    global _inited
    L = load()
    if not _inited:
        check(L.pi_init(device), "pi_init")
        _inited = True
    return L


def device_name():
    buf = C.create_string_buffer(256)
    check(init().pi_device_name(buf, 256), "pi_device_name")
    return buf.value.decode()


class DevBuf:
    """A device allocation with numpy upload/download helpers."""

    def __init__(self, nbytes=None, host=None):
        L = init()
        if host is not None:
            host = np.ascontiguousarray(host)
            nbytes = host.nbytes
        self.nbytes = int(nbytes)
        self.ptr = L.pi_malloc(max(self.nbytes, 1))
        if not self.ptr:
            raise PiError("pi_malloc: " + L.pi_last_error().decode())
        if host is not None and self.nbytes:
            check(L.pi_memcpy_h2d(self.ptr, host.ctypes.data_as(_vp), self.nbytes), "h2d")

    @classmethod
    def zeros(cls, nbytes):
        b = cls(nbytes)
        check(load().pi_memset(b.ptr, 0, b.nbytes), "memset")
        return b

    def upload(self, host, offset=0):
        host = np.ascontiguousarray(host)
        assert offset + host.nbytes <= self.nbytes
        check(load().pi_memcpy_h2d(self.ptr + offset, host.ctypes.data_as(_vp), host.nbytes), "h2d")

    def download(self, dtype, count=None, offset=0):
        dt = np.dtype(dtype)
        count = (self.nbytes - offset) // dt.itemsize if count is None else count
        out = np.empty(count, dt)
        if count:
            check(load().pi_memcpy_d2h(out.ctypes.data_as(_vp), self.ptr + offset, out.nbytes), "d2h")
        return out

    def free(self):
        if self.ptr:
            load().pi_free(self.ptr)
            self.ptr = None

    def __del__(self):
        try:
            self.free()
        except Exception:
            pass


def norm_arg(kind=NORM_NONE, eps=0.0, w=None, b=None):
    if kind == NORM_NONE:
        return None
    return C.byref(Norm(kind, eps, w.ptr if w is not None else None, b.ptr if b is not None else None))


def sync():
    check(init().pi_sync(), "pi_sync")
