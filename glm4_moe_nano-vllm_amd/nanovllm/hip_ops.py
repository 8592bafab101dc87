"""ctypes binding of libglm4moe_hip.so (include/glm4moe_hip.h) for torch tensors on ROCm.

This is the only place where Python touches the C-ABI: raw ``data_ptr()`` values plus the
current torch stream go in, nothing comes back but a status code.  There is NO CPU or eager
fallback: if the shared object is missing, or a tensor is not on the GPU, the call raises.
"""
from __future__ import annotations

import ctypes
import os
from dataclasses import dataclass
from ctypes import c_char_p, c_float, c_int, c_int64, c_size_t, c_void_p

import torch

_HERE = os.path.dirname(os.path.abspath(__file__))
LIB_PATH = os.environ.get(
    "GLM4MOE_HIP_LIB", os.path.join(_HERE, "..", "lib", "libglm4moe_hip.so"))

_lib = None

# name -> (restype, argtypes); mirrors include/glm4moe_hip.h one to one
_SIGNATURES = {
    "glm_abi_version": (c_int, []),
    "glm_last_error": (c_char_p, []),
    "glm_get_option": (c_int, [c_char_p, c_void_p]),
    "glm_set_option": (c_int, [c_char_p, c_int]),
    "glm_option_name": (c_char_p, [c_int]),
    "glm_rmsnorm": (c_int, [c_void_p, c_void_p, c_void_p, c_int64, c_int, c_float, c_void_p]),
    "glm_add_rmsnorm": (c_int, [c_void_p, c_void_p, c_void_p, c_void_p, c_void_p, c_int64, c_int,
                                c_float, c_void_p]),
    "glm_head_rmsnorm": (c_int, [c_void_p, c_int64, c_void_p, c_void_p, c_int64, c_int64, c_int,
                                 c_int, c_float, c_void_p]),
    "glm_rope_neox": (c_int, [c_void_p, c_int64, c_void_p, c_int64, c_void_p, c_int64, c_void_p,
                              c_int64, c_void_p, c_void_p, c_int64, c_int64, c_int, c_int, c_int,
                              c_int, c_void_p]),
    "glm_kv_store": (c_int, [c_void_p, c_int64, c_void_p, c_int64, c_void_p, c_void_p, c_void_p,
                             c_int64, c_int, c_int64, c_void_p]),
    "glm_qkv_split_norm_rope_store": (c_int, [c_void_p, c_int64, c_void_p, c_void_p, c_void_p,
                                              c_void_p, c_void_p, c_float, c_void_p, c_void_p,
                                              c_int64, c_int, c_void_p, c_void_p, c_void_p,
                                              c_int64, c_int64, c_int, c_int, c_int, c_void_p]),
    "glm_gemm_qkv_rope_store": (c_int, [c_void_p, c_int64, c_void_p, c_int64, c_void_p, c_int64, c_int, c_int, c_int, c_int,
                                        c_void_p, c_void_p, c_int, c_void_p, c_void_p, c_void_p, c_void_p, c_void_p, c_void_p,
                                        c_int64, c_void_p]),
    "glm_silu_and_mul": (c_int, [c_void_p, c_void_p, c_int64, c_int, c_void_p]),
    "glm_paged_attn_decode_workspace_bytes": (c_size_t, [c_int64, c_int, c_int, c_int]),
    "glm_paged_attn_decode_splits": (c_int, [c_int64, c_int, c_int, c_int64, c_int, c_int]),
    "glm_paged_attn_decode": (c_int, [c_void_p, c_void_p, c_void_p, c_void_p, c_void_p, c_int64,
                                      c_void_p, c_int64, c_int, c_int, c_int, c_int, c_int64,
                                      c_float, c_int, c_int, c_void_p, c_size_t, c_void_p]),
    "glm_paged_attn_decode_qkv": (c_int, [c_void_p, c_int64, c_void_p, c_void_p, c_int64, c_int, c_void_p, c_void_p, c_void_p,
                                          c_void_p, c_void_p, c_int64, c_void_p, c_int64, c_int, c_int, c_int, c_int,
                                          c_int64, c_float, c_int, c_int, c_void_p, c_size_t, c_void_p]),
    "glm_paged_attn_decode_qkv_partial": (c_int, [c_void_p, c_int, c_int64, c_void_p, c_void_p, c_void_p, c_int64, c_int,
                                                  c_void_p, c_void_p, c_void_p, c_void_p, c_void_p, c_int64, c_void_p,
                                                  c_int64, c_int, c_int, c_int, c_int, c_int64, c_float, c_int, c_int,
                                                  c_void_p, c_size_t, c_void_p]),
    "glm_varlen_attn_prefill": (c_int, [c_void_p, c_void_p, c_void_p, c_void_p, c_void_p,
                                        c_void_p, c_int64, c_void_p, c_int64, c_int, c_int, c_int,
                                        c_int, c_int, c_float, c_void_p]),
    "glm_router_topk": (c_int, [c_void_p, c_void_p, c_void_p, c_void_p, c_void_p, c_void_p,
                                c_int64, c_int, c_int, c_int, c_float, c_void_p]),
    "glm_moe_align_workspace_bytes": (c_size_t, [c_int64, c_int, c_int]),
    "glm_moe_align_parallel": (c_int, [c_void_p, c_void_p, c_void_p, c_void_p, c_void_p, c_void_p, c_int64, c_int, c_int,
                                       c_int, c_void_p, c_size_t, c_void_p]),
    "glm_router_select": (c_int, [c_void_p, c_int64, c_void_p, c_void_p, c_void_p, c_int64, c_int, c_int, c_float, c_void_p]),
    "glm_moe_align": (c_int, [c_void_p, c_void_p, c_void_p, c_void_p, c_void_p, c_void_p, c_int64,
                              c_int, c_int, c_int, c_void_p]),
    "glm_grouped_gemm_gateup_silu": (c_int, [c_void_p, c_int64, c_void_p, c_int64, c_int64, c_void_p,
                                             c_void_p, c_void_p, c_int64, c_int, c_int, c_int,
                                             c_void_p]),
    "glm_grouped_gemm_down": (c_int, [c_void_p, c_void_p, c_int64, c_int64, c_void_p, c_void_p, c_int,
                                      c_void_p, c_int64, c_int64, c_int, c_int, c_int, c_void_p]),
    "glm_fp8w_expand_scratch_bytes": (c_size_t, [c_int, c_int, c_int]),
    "glm_grouped_gemm_gateup_silu_fp8w": (c_int, [c_void_p, c_int64, c_void_p, c_int64, c_int64, c_void_p,
                                                  c_int64, c_void_p, c_void_p, c_void_p, c_int64, c_int,
                                                  c_int, c_int, c_void_p, c_size_t, c_void_p]),
    "glm_grouped_gemm_down_fp8w": (c_int, [c_void_p, c_void_p, c_int64, c_int64, c_void_p, c_int64, c_void_p,
                                           c_void_p, c_int, c_void_p, c_int64, c_int64, c_int, c_int, c_int,
                                           c_void_p, c_size_t, c_void_p]),
    "glm_moe_combine": (c_int, [c_void_p, c_int64, c_void_p, c_void_p, c_int64, c_int, c_int,
                                c_int64, c_void_p]),
    "glm_gemm_bf16": (c_int, [c_void_p, c_int64, c_void_p, c_int64, c_void_p, c_void_p, c_int64,
                              c_int64, c_int, c_int, c_void_p]),
    "glm_grouped_gemm_gateup_silu_fewtok": (c_int, [c_void_p, c_int64, c_int64, c_void_p, c_int64, c_int64, c_void_p,
                                                    c_void_p, c_void_p, c_int64, c_int, c_int, c_int, c_void_p]),
    "glm_grouped_gemm_down_fewtok": (c_int, [c_void_p, c_int64, c_void_p, c_int64, c_int64, c_void_p, c_void_p, c_int,
                                             c_void_p, c_int64, c_int64, c_int, c_int, c_int, c_void_p]),
    "glm_gemm_bf16_combine_norm": (c_int, [c_void_p, c_int64, c_void_p, c_int64, c_int, c_int64, c_void_p, c_void_p,
                                           c_float, c_void_p, c_void_p, c_void_p, c_int64, c_void_p, c_void_p, c_int64,
                                           c_int, c_int, c_void_p]),
    "glm_gemm_bf16_router_tail": (c_int, [c_void_p, c_void_p, c_int64, c_int, c_int, c_void_p, c_void_p, c_void_p, c_void_p,
                                          c_float, c_void_p, c_void_p, c_void_p, c_void_p, c_int, c_int, c_float, c_void_p,
                                          c_void_p, c_void_p, c_void_p, c_void_p, c_void_p, c_int, c_void_p]),
    "glm_quantize_fp8_rows": (c_int, [c_void_p, c_int64, c_void_p, c_int64, c_void_p, c_int64, c_int, c_void_p]),
    "glm_grouped_gemm_gateup_silu_fp8a8": (c_int, [c_void_p, c_int64, c_void_p, c_void_p, c_int64, c_int64, c_void_p, c_int64,
                                                   c_void_p, c_void_p, c_void_p, c_int64, c_void_p, c_int64, c_int, c_int,
                                                   c_int, c_void_p]),
    "glm_grouped_gemm_down_fp8a8": (c_int, [c_void_p, c_int64, c_void_p, c_void_p, c_int64, c_int64, c_void_p, c_int64,
                                            c_void_p, c_void_p, c_int, c_void_p, c_int64, c_int64, c_int, c_int, c_int,
                                            c_void_p]),
    "glm_decode_mlp_engine_workspace_bytes": (c_size_t, [c_int, c_int, c_int, c_int]),
    "glm_decode_mlp_engine": (c_int, [c_void_p, c_void_p, c_int64, c_int, c_int, c_void_p, c_void_p, c_float, c_void_p, c_void_p,
                                      c_void_p, c_void_p, c_int, c_int, c_float, c_void_p, c_void_p, c_void_p, c_void_p,
                                      c_void_p, c_void_p, c_void_p, c_int64, c_int64, c_void_p, c_int64, c_int64, c_int,
                                      c_void_p, c_void_p, c_int64, c_void_p, c_void_p]),
    "glm_gemm_bf16_partial_slices": (c_int, [c_int, c_int]),
    "glm_gemm_bf16_partial": (c_int, [c_void_p, c_int64, c_void_p, c_int64, c_void_p, c_int64, c_int, c_int,
                                      c_int, c_void_p]),
    "glm_add_rmsnorm_router_topk": (c_int, [c_void_p, c_void_p, c_int, c_int64, c_void_p, c_void_p, c_float, c_void_p,
                                            c_void_p, c_void_p, c_void_p, c_void_p, c_void_p, c_int64, c_int, c_int,
                                            c_int, c_float, c_void_p]),
    "glm_add_rmsnorm_router_topk_align": (c_int, [c_void_p, c_void_p, c_int, c_int64, c_void_p, c_void_p, c_float,
                                                  c_void_p, c_void_p, c_void_p, c_void_p, c_void_p, c_void_p, c_int64,
                                                  c_int, c_int, c_int, c_float, c_void_p, c_void_p, c_void_p, c_void_p,
                                                  c_int, c_void_p, c_size_t, c_void_p]),
    "glm_router_workspace_bytes": (c_size_t, [c_int64, c_int]),
    "glm_allreduce_oneshot_buffer_elems": (c_size_t, [c_int, c_int64]),
    "glm_comm_alloc": (c_int, [c_void_p, c_size_t, c_int]),
    "glm_comm_free": (c_int, [c_void_p]),
    "glm_comm_ipc_export": (c_int, [c_void_p, c_void_p]),
    "glm_comm_ipc_open": (c_int, [c_void_p, c_void_p]),
    "glm_comm_ipc_close": (c_int, [c_void_p]),
    "glm_allreduce_oneshot": (c_int, [c_void_p, c_void_p, c_void_p, c_void_p, c_int, c_int, c_int64, c_int64, c_void_p,
                                      c_void_p]),
    "glm_ep_plan": (c_int, [c_void_p, c_void_p, c_int64, c_int, c_int, c_int, c_int, c_int, c_void_p, c_void_p, c_void_p,
                            c_void_p, c_void_p, c_void_p, c_void_p]),
    "glm_grouped_gemm_gateup_silu_cap": (c_int, [c_void_p, c_int64, c_void_p, c_int64, c_int64, c_void_p, c_void_p,
                                                 c_void_p, c_int64, c_int64, c_int, c_int, c_int, c_void_p]),
    "glm_grouped_gemm_down_cap": (c_int, [c_void_p, c_void_p, c_int64, c_int64, c_void_p, c_void_p, c_int, c_void_p,
                                          c_int64, c_int64, c_int64, c_int, c_int, c_int, c_void_p]),
    "glm_gather_rows": (c_int, [c_void_p, c_int64, c_void_p, c_int64, c_void_p, c_int64, c_int, c_void_p]),
    "glm_scatter_rows": (c_int, [c_void_p, c_int64, c_void_p, c_int64, c_void_p, c_int64, c_int, c_void_p]),
    "glm_moe_combine_scaled": (c_int, [c_void_p, c_int64, c_void_p, c_void_p, c_void_p, c_int64, c_void_p, c_int64, c_int,
                                       c_int, c_void_p]),
    "glm_moe_combine_add_rmsnorm": (c_int, [c_void_p, c_int64, c_void_p, c_int64, c_int, c_int, c_int64, c_void_p,
                                            c_void_p, c_void_p, c_void_p, c_float, c_void_p]),
    "glm_add_rmsnorm_partial": (c_int, [c_void_p, c_int, c_int64, c_void_p, c_void_p, c_void_p, c_void_p,
                                        c_int64, c_int, c_float, c_void_p]),
    "glm_gemm_bf16_act": (c_int, [c_void_p, c_int64, c_void_p, c_int64, c_void_p, c_void_p, c_int64, c_int64, c_int,
        c_int, c_int, c_int, c_float, c_float, c_void_p]),
    "glm_gemm_f32": (c_int, [c_void_p, c_int64, c_int64, c_void_p, c_int64, c_int64, c_void_p, c_void_p, c_int64,
        c_int64, c_int64, c_int, c_int, c_int, c_int, c_float, c_float, c_void_p]),
    "glm_seq_norm_taps": (c_int, [c_int]),
    "glm_seq_norm": (c_int, [c_void_p, c_void_p, c_int64, c_void_p, c_void_p, c_int64, c_void_p, c_int64, c_int, c_int,
        c_int64, c_void_p, c_void_p, c_void_p, c_int, c_void_p, c_int64, c_void_p, c_void_p, c_void_p, c_void_p,
        c_void_p, c_void_p, c_int64, c_int, c_int64, c_int, c_int, c_float, c_void_p]),
    "glm_embed_rows": (c_int, [c_void_p, c_void_p, c_int64, c_int64, c_void_p, c_void_p, c_void_p, c_int64, c_void_p, c_int64, c_int,
        c_int64, c_int, c_int, c_float, c_void_p]),
    "glm_latent_prepare": (c_int, [c_void_p, c_int64, c_int, c_int64, c_int64, c_int, c_int, c_int, c_int, c_void_p,
        c_float, c_void_p, c_void_p, c_int64, c_void_p, c_void_p, c_int64, c_void_p, c_void_p, c_int, c_void_p]),
    "glm_latent_gather": (c_int, [c_void_p, c_int64, c_void_p, c_void_p, c_int64, c_void_p, c_int64, c_int, c_void_p]),
    "glm_latent_attn_max_rows": (c_int, [c_int]),
    "glm_latent_attn": (c_int, [c_void_p, c_void_p, c_int64, c_int, c_void_p, c_void_p, c_int, c_int, c_void_p, c_void_p, c_void_p,
        c_int64, c_int64, c_int, c_int, c_int, c_int, c_float, c_void_p, c_int, c_void_p, c_void_p, c_void_p, c_int, c_void_p]),
    "glm_attn_merge": (c_int, [c_void_p, c_void_p, c_void_p, c_int, c_void_p, c_int64, c_int64, c_int, c_int, c_void_p, c_void_p]),
    "glm_latent_up": (c_int, [c_void_p, c_void_p, c_void_p, c_void_p, c_int64, c_int64, c_int64, c_int, c_int, c_int, c_void_p]),
    "glm_window_attn_prefill": (c_int, [c_void_p, c_int64, c_void_p, c_void_p, c_int64, c_void_p, c_int64, c_int, c_void_p, c_void_p,
        c_int64, c_void_p, c_int64, c_void_p, c_void_p, c_void_p, c_void_p, c_int, c_int, c_int64, c_int64, c_int, c_int, c_int, c_int,
        c_float, c_void_p, c_void_p]),
    "glm_gemm_bf16_glu": (c_int, [c_void_p, c_int64, c_void_p, c_int64, c_void_p, c_int64, c_int64, c_int, c_int, c_float, c_float,
        c_void_p]),
    "glm_glu_f32": (c_int, [c_void_p, c_int64, c_void_p, c_int64, c_int64, c_int, c_float, c_float, c_void_p]),
    "glm_stream_norm": (c_int, [c_void_p, c_int64, c_int64, c_void_p, c_void_p, c_void_p, c_int64, c_int, c_void_p, c_void_p,
        c_void_p, c_float, c_void_p, c_void_p, c_int64, c_void_p, c_void_p, c_void_p, c_void_p, c_void_p,
        c_void_p, c_int64, c_int, c_int64, c_int, c_int, c_int, c_float, c_void_p]),
    "glm_group_kv_store": (c_int, [c_void_p, c_int64, c_int64, c_int64, c_int, c_void_p, c_int64, c_void_p, c_void_p, c_int64, c_int,
        c_int, c_int, c_int, c_void_p]),
    "glm_group_attn_prefill": (c_int, [c_void_p, c_int64, c_void_p, c_void_p, c_int64, c_int, c_void_p, c_int64, c_int, c_void_p, c_void_p,
        c_void_p, c_void_p, c_int, c_int, c_int, c_int, c_int, c_int, c_void_p, c_void_p, c_int64, c_void_p]),
    "glm_group_attn_decode": (c_int, [c_void_p, c_int64, c_void_p, c_void_p, c_int64, c_int, c_void_p, c_int64, c_void_p, c_void_p,
        c_void_p, c_void_p, c_int, c_int, c_int, c_int, c_int, c_int, c_void_p, c_void_p, c_void_p, c_int64, c_void_p, c_void_p, c_void_p,
        c_int64, c_int, c_void_p, c_void_p, c_void_p]),
    "glm_group_attn_plain": (c_int, [c_void_p, c_int64, c_void_p, c_void_p, c_int64, c_int, c_void_p, c_int64, c_void_p, c_void_p, c_int64,
        c_int, c_int, c_int, c_int, c_void_p, c_void_p, c_int64, c_int, c_void_p]),
    "glm_group_rotate_store": (c_int, [c_void_p, c_int64, c_int, c_int, c_int, c_int, c_int, c_int, c_int, c_int, c_int, c_int, c_void_p, c_int,
        c_void_p, c_int64, c_void_p, c_void_p, c_int64, c_int, c_void_p]),
    "glm_group_norm_store": (c_int, [c_void_p, c_int64, c_int, c_int, c_int, c_int, c_int, c_int, c_int, c_void_p, c_int, c_int, c_int, c_float,
        c_float, c_int, c_void_p, c_void_p, c_int64, c_void_p, c_void_p, c_int64, c_int, c_void_p]),
    "glm_gemm_bf16_slices": (c_int, [c_int64, c_int, c_int]),
    "glm_residual_norm": (c_int, [c_void_p, c_void_p, c_void_p, c_int64, c_int, c_int, c_int64, c_void_p, c_int64, c_int64, c_void_p, c_void_p,
        c_void_p, c_void_p, c_int64, c_int, c_int64, c_int, c_int, c_float, c_void_p]),
    "glm_memory_recurrent": (c_int, [c_void_p, c_int64, c_int64, c_int64, c_int64, c_void_p, c_int64, c_void_p, c_int64, c_int, c_void_p,
        c_void_p, c_void_p, c_int64, c_void_p, c_void_p, c_void_p, c_int64, c_void_p, c_void_p, c_void_p,
        c_void_p, c_int, c_int, c_int, c_int, c_int, c_int, c_float, c_float, c_int, c_void_p]),
    "glm_memory_gates": (c_int, [c_void_p, c_int64, c_void_p, c_int64, c_int, c_void_p, c_void_p, c_int64, c_void_p, c_void_p,
        c_void_p, c_int, c_int, c_float, c_void_p]),
    "glm_memory_chunkwise": (c_int, [c_void_p, c_int64, c_int64, c_int64, c_void_p, c_int64, c_void_p, c_int64, c_void_p, c_void_p,
        c_void_p, c_int64, c_void_p, c_void_p, c_void_p, c_void_p, c_int, c_int, c_int, c_int, c_int,
        c_void_p]),
    "glm_memory_output": (c_int, [c_void_p, c_int64, c_void_p, c_int64, c_void_p, c_void_p, c_int64, c_int64, c_int, c_int, c_int,
        c_float, c_void_p]),
    "glm_linear_recurrent": (c_int, [c_void_p, c_int64, c_int64, c_int64, c_void_p, c_void_p, c_int64, c_void_p, c_int64, c_void_p,
        c_void_p, c_void_p, c_void_p, c_int, c_int, c_int, c_int, c_int, c_void_p]),
    "glm_linear_chunkwise": (c_int, [c_void_p, c_int64, c_int64, c_int64, c_void_p, c_int64, c_void_p, c_int64, c_void_p, c_int64, c_void_p,
        c_void_p, c_void_p, c_void_p, c_int, c_int, c_int, c_int, c_void_p]),
    "glm_row_norm_gate": (c_int, [c_void_p, c_int64, c_int, c_void_p, c_int64, c_void_p, c_void_p, c_int64, c_int64, c_int, c_int,
        c_float, c_int, c_void_p]),
    "glm_depth_norm_taps": (c_int, [c_int]),
    "glm_depth_norm": (c_int, [c_void_p, c_void_p, c_int64, c_void_p, c_int64, c_void_p, c_void_p, c_int, c_int64, c_void_p, c_void_p,
        c_void_p, c_int64, c_void_p, c_int64, c_int, c_void_p, c_void_p, c_void_p, c_void_p, c_int, c_void_p, c_int64, c_void_p,
        c_void_p, c_void_p, c_void_p, c_void_p, c_void_p, c_int64, c_int, c_int64, c_int, c_int, c_int, c_float, c_void_p]),
    "glm_router_softmax": (c_int, [c_void_p, c_int64, c_void_p, c_void_p, c_int64, c_int, c_int, c_void_p]),
    "glm_router_softmax_align": (c_int, [c_void_p, c_int64, c_void_p, c_void_p, c_void_p, c_void_p, c_void_p, c_int64, c_int, c_int,
        c_void_p]),
    "glm_moe_combine_weighted": (c_int, [c_void_p, c_int64, c_int64, c_void_p, c_void_p, c_void_p, c_int64, c_int64, c_int, c_int, c_int,
        c_void_p]),
    "glm_grouped_gemm_f32": (c_int, [c_void_p, c_int64, c_void_p, c_int64, c_int64, c_void_p, c_void_p, c_void_p, c_int64, c_int64,
        c_int, c_int, c_int, c_void_p]),
    "glm_swiglu_f32": (c_int, [c_void_p, c_int64, c_void_p, c_int64, c_int64, c_int, c_void_p]),
    "glm_mul_f32": (c_int, [c_void_p, c_int64, c_void_p, c_int64, c_int64, c_int, c_void_p]),
    "glm_rope_pairs": (c_int, [c_void_p, c_void_p, c_int, c_float, c_void_p, c_int64, c_int, c_void_p]),
    "glm_latent_rows": (c_int, [c_void_p, c_int64, c_int, c_int, c_int, c_int, c_void_p, c_void_p, c_float, c_void_p, c_void_p, c_int64,
        c_void_p, c_void_p, c_int64, c_int, c_int, c_int, c_void_p, c_void_p, c_int64, c_int64, c_int, c_void_p]),
    "glm_latent_absorb": (c_int, [c_void_p, c_int64, c_int64, c_int, c_int, c_int, c_int, c_void_p, c_void_p, c_void_p, c_int, c_void_p]),
}

EXPORTED_SYMBOLS = tuple(_SIGNATURES)


def load_library(path: str | None = None) -> ctypes.CDLL:
    """dlopen the HIP library and attach prototypes; raises if it is missing."""
    global _lib
    if _lib is not None and path is None:
        return _lib
    p = os.path.abspath(path or LIB_PATH)
    if not os.path.exists(p):
        raise RuntimeError(
            f"libglm4moe_hip.so not found at {p}: build it with "
            "`python glm4_moe_nano-vllm_amd/build.py` (there is no CPU fallback)")
    lib = ctypes.CDLL(p)
    for name, (res, args) in _SIGNATURES.items():
        # (a library of one model's kernels, build.py --kernel-set, lacks the other models' entry points)
        if os.path.basename(p) != "libglm4moe_hip.so" and not hasattr(lib, name):
            continue
        fn = getattr(lib, name)
        fn.restype = res
        fn.argtypes = args
    if path is None:
        _lib = lib
        _read_host_options()
    return lib


# ---- options -----------------------------------------------------------------------------------------------------------
# Host-side switches of the launch paths (which fused launch a layer takes, which collective form): read from the
# environment ONCE, when the library is loaded, like the library's own table (glm_get_option / glm_set_option).  A path never
# consults os.environ afterwards; tests and A/B tools call set_option().  options() is the effective set of both sides
# (bench.py prints it in its line's config).
_HOST_OPTION_ENV = {  # name -> (environment variable, default)
    "fuse_combine_qkv": ("GLM4MOE_FUSE_COMBINE_QKV", 1),    # one token: combine + input norm + QKV in one launch
    "fuse_oproj_router": ("GLM4MOE_FUSE_OPROJ_ROUTER", 1),  # one token: o_proj + norm + router + bucketing in one launch
    "defer_qkv_reduce": ("GLM4MOE_DEFER_QKV_REDUCE", 1),    # QKV as K-slice partial sums reduced by the attention's loads
    "fuse_qkv_rope": ("GLM4MOE_FUSE_QKV_ROPE", 1),          # prefill: split + rotary + K/V store in the QKV GEMM's epilogue
    "t1_engine": ("GLM4MOE_T1_ENGINE", 0),                  # one token: o_proj .. down projection as ONE persistent launch (r05; opt-in:
                                                            # bit-identical, 5-6 us per layer slower — profiles/r05/decode_engine_stamps.txt)
    "ep_fixed": ("GLM_EP_FIXED", 1),                        # expert parallelism: fixed-capacity dispatch at decode sizes
    "oneshot_allreduce": ("GLM_ONESHOT_ALLREDUCE", 0),      # opt-in one-hop all-reduce over mapped peer buffers
}
_host_opts: dict = {}


def _read_host_options() -> None:
    for name, (env, dflt) in _HOST_OPTION_ENV.items():
        v = os.environ.get(env)
        _host_opts[name] = int(v) if v not in (None, "") else dflt


def opt(name: str) -> int:
    """Effective value of a launch-path option (host-side table or the library's)."""
    if not _host_opts:
        load_library()
    if name in _host_opts:
        return _host_opts[name]
    v = c_int(0)
    _check(load_library().glm_get_option(name.encode(), ctypes.byref(v)), "glm_get_option")
    return v.value


def set_option(name: str, value: int) -> int:
    """Change an option for the launches that follow (NOT for HIP graphs captured earlier); returns the old value."""
    old = opt(name)
    if name in _host_opts:
        _host_opts[name] = int(value)
    else:
        _check(load_library().glm_set_option(name.encode(), int(value)), "glm_set_option")
    return old


class option:
    """`with hip_ops.option("tinym", 0): ...`"""

    def __init__(self, name: str, value: int):
        self.name, self.value = name, value

    def __enter__(self):
        self.old = set_option(self.name, self.value)

    def __exit__(self, *exc):
        set_option(self.name, self.old)
        return False


def options() -> dict:
    lib = load_library()
    out, i = {}, 0
    while True:
        n = lib.glm_option_name(i)
        if not n:
            break
        out[n.decode()] = opt(n.decode())
        i += 1
    out.update(_host_opts)
    return out


GLM_ERR_UNSUPPORTED = -2  # include/glm4moe_hip.h


def _check(rc: int, name: str) -> None:
    if rc != 0:
        msg = load_library().glm_last_error()
        raise RuntimeError(f"{name} failed ({rc}): {msg.decode() if msg else '?'}")


def _stream() -> int:
    return torch.cuda.current_stream().cuda_stream


def _p(t: torch.Tensor | None) -> int | None:
    if t is None:
        return None
    if not t.is_cuda:
        raise RuntimeError("glm4moe HIP ops need GPU tensors (no CPU fallback)")
    return t.data_ptr()


def _bf16(t: torch.Tensor, name: str) -> None:
    if t.dtype != torch.bfloat16:
        raise TypeError(f"{name}: expected bfloat16, got {t.dtype}")
    if t.stride(-1) != 1:
        raise ValueError(f"{name}: innermost stride must be 1")


# ------------------------------------------------------------------------------------------
# norms
def rmsnorm(x: torch.Tensor, weight: torch.Tensor, eps: float) -> torch.Tensor:
    _bf16(x, "x"); _bf16(weight, "weight")
    H = x.shape[-1]
    x2 = x.reshape(-1, H)
    if not x2.is_contiguous():
        x2 = x2.contiguous()
    y = torch.empty_like(x2)
    _check(load_library().glm_rmsnorm(_p(x2), _p(weight), _p(y), x2.shape[0], H, eps, _stream()),
           "glm_rmsnorm")
    return y.view(x.shape)


def add_rmsnorm(x: torch.Tensor, residual: torch.Tensor, weight: torch.Tensor,
                eps: float) -> tuple[torch.Tensor, torch.Tensor]:
    _bf16(x, "x"); _bf16(residual, "residual"); _bf16(weight, "weight")
    H = x.shape[-1]
    x2 = x.reshape(-1, H).contiguous()
    r2 = residual.reshape(-1, H).contiguous()
    y = torch.empty_like(x2)
    ro = torch.empty_like(x2)
    _check(load_library().glm_add_rmsnorm(_p(x2), _p(r2), _p(weight), _p(y), _p(ro), x2.shape[0],
                                          H, eps, _stream()), "glm_add_rmsnorm")
    return y.view(x.shape), ro.view(x.shape)


def head_rmsnorm(x: torch.Tensor, weight: torch.Tensor, eps: float) -> torch.Tensor:
    """x: [T, n_heads, hd] (head stride hd, arbitrary token stride) -> contiguous result."""
    _bf16(x, "x"); _bf16(weight, "weight")
    T, nh, hd = x.shape
    if x.stride(1) != hd:
        x = x.contiguous()
    y = torch.empty((T, nh, hd), dtype=x.dtype, device=x.device)
    _check(load_library().glm_head_rmsnorm(_p(x), x.stride(0), _p(weight), _p(y), nh * hd, T, nh,
                                           hd, eps, _stream()), "glm_head_rmsnorm")
    return y


# ------------------------------------------------------------------------------------------
# rotary / kv cache
def rope_neox(positions: torch.Tensor, q: torch.Tensor, k: torch.Tensor,
              cos_sin_cache: torch.Tensor, rotary_dim: int) -> tuple[torch.Tensor, torch.Tensor]:
    """q: [T,nh,hd], k: [T,nkv,hd] (head stride hd) -> new contiguous (q, k)."""
    _bf16(q, "q"); _bf16(k, "k")
    T, nh, hd = q.shape
    nkv = k.shape[1]
    if q.stride(1) != hd:
        q = q.contiguous()
    if k.stride(1) != hd:
        k = k.contiguous()
    assert positions.dtype == torch.int64 and cos_sin_cache.dtype == torch.float32
    cs = cos_sin_cache.reshape(cos_sin_cache.shape[0], -1)
    assert cs.is_contiguous() and cs.shape[1] == rotary_dim
    qo = torch.empty((T, nh, hd), dtype=q.dtype, device=q.device)
    ko = torch.empty((T, nkv, hd), dtype=k.dtype, device=k.device)
    _check(load_library().glm_rope_neox(_p(q), q.stride(0), _p(k), k.stride(0), _p(qo), nh * hd,
                                        _p(ko), nkv * hd, _p(positions.contiguous()), _p(cs),
                                        cs.shape[0], T, nh, nkv, hd, rotary_dim, _stream()),
           "glm_rope_neox")
    return qo, ko


def kv_store(key: torch.Tensor, value: torch.Tensor, k_cache: torch.Tensor, v_cache: torch.Tensor,
             slot_mapping: torch.Tensor) -> None:
    _bf16(key, "key"); _bf16(value, "value")
    N, nh, hd = key.shape
    D = nh * hd
    assert key.stride(1) == hd and value.stride(1) == hd
    assert k_cache.stride(1) == D and v_cache.stride(1) == D
    assert slot_mapping.numel() == N and slot_mapping.dtype == torch.int32
    n_slots = k_cache.numel() // D
    _check(load_library().glm_kv_store(_p(key), key.stride(0), _p(value), value.stride(0),
                                       _p(k_cache), _p(v_cache), _p(slot_mapping), N, D, n_slots,
                                       _stream()), "glm_kv_store")


def qkv_split_norm_rope_store(qkv: torch.Tensor, nh: int, nkv: int, hd: int,
                              positions: torch.Tensor, cos_sin_cache: torch.Tensor,
                              rotary_dim: int, q_norm_w: torch.Tensor | None,
                              k_norm_w: torch.Tensor | None, eps: float,
                              k_cache: torch.Tensor | None, v_cache: torch.Tensor | None,
                              slot_mapping: torch.Tensor | None, need_kv_out: bool):
    """Fused split + (qk-norm) + rotary + cache scatter; returns (q, k|None, v|None)."""
    _bf16(qkv, "qkv")
    T = qkv.shape[0]
    assert qkv.shape[1] == (nh + 2 * nkv) * hd
    cs = cos_sin_cache.reshape(cos_sin_cache.shape[0], -1)
    q = torch.empty((T, nh, hd), dtype=qkv.dtype, device=qkv.device)
    k = torch.empty((T, nkv, hd), dtype=qkv.dtype, device=qkv.device) if need_kv_out else None
    v = torch.empty((T, nkv, hd), dtype=qkv.dtype, device=qkv.device) if need_kv_out else None
    store = k_cache is not None and k_cache.numel() > 0 and slot_mapping is not None
    n_slots = (k_cache.numel() // (nkv * hd)) if store else 0
    _check(load_library().glm_qkv_split_norm_rope_store(
        _p(qkv), qkv.stride(0), _p(q), _p(k), _p(v), _p(q_norm_w), _p(k_norm_w), eps,
        _p(positions), _p(cs), cs.shape[0], rotary_dim,
        _p(k_cache) if store else None, _p(v_cache) if store else None,
        _p(slot_mapping) if store else None, n_slots, T, nh, nkv, hd, _stream()),
        "glm_qkv_split_norm_rope_store")
    return q, k, v


def gemm_qkv_rope_store(x: torch.Tensor, w: torch.Tensor, bias: torch.Tensor | None, nh: int, nkv: int, hd: int,
                        positions: torch.Tensor, cos_sin_cache: torch.Tensor, rotary_dim: int,
                        k_cache: torch.Tensor | None, v_cache: torch.Tensor | None, slot_mapping: torch.Tensor | None,
                        need_kv: bool):
    """Prefill: QKV projection + split + rotary + K/V cache store in ONE launch (glm_gemm_qkv_rope_store).  Returns
    (q [T,nh,hd], k, v [T,nkv,hd] or None) — or None when the launcher does not cover the shape (nothing was enqueued:
    the caller takes gemm_bf16 + qkv_split_norm_rope_store)."""
    if x.dim() != 2 or x.shape[0] < 96 or hd != 128 or rotary_dim != 64 or opt("fuse_qkv_rope") == 0:
        return None
    _bf16(x, "x"); _bf16(w, "w")
    T, K = x.shape
    assert w.shape == ((nh + 2 * nkv) * hd, K) and w.stride(1) == 1 and positions.dtype == torch.int64
    assert cos_sin_cache.dtype == torch.float32 and cos_sin_cache.is_contiguous() and cos_sin_cache.shape[-1] == rotary_dim
    q = torch.empty((T, nh, hd), dtype=x.dtype, device=x.device)
    k = torch.empty((T, nkv, hd), dtype=x.dtype, device=x.device) if need_kv else None
    v = torch.empty_like(k) if need_kv else None
    has_cache = k_cache is not None and slot_mapping is not None
    if has_cache and slot_mapping.numel() != T:
        # never skip the K/V store silently: later decode steps would read unwritten cache rows (kv_store asserts too)
        raise ValueError(f"gemm_qkv_rope_store: slot_mapping has {slot_mapping.numel()} entries for {T} token rows")
    if positions.numel() != T or positions.device != x.device or (bias is not None and bias.data_ptr() % 8):
        return None   # the two-launch path checks / handles these
    if has_cache:
        assert k_cache.is_contiguous() and v_cache.is_contiguous() and slot_mapping.dtype == torch.int32
    n_slots = k_cache.shape[0] * k_cache.shape[1] if has_cache else 0
    rc = load_library().glm_gemm_qkv_rope_store(
        _p(x), x.stride(0), _p(w), w.stride(0), _p(bias), T, nh, nkv, hd, K, _p(positions), _p(cos_sin_cache), rotary_dim,
        _p(q), _p(k), _p(v), _p(k_cache) if has_cache else None, _p(v_cache) if has_cache else None,
        _p(slot_mapping) if has_cache else None, n_slots, _stream())
    if rc == GLM_ERR_UNSUPPORTED:
        return None
    _check(rc, "glm_gemm_qkv_rope_store")
    return q, k, v


def padded_weight(rows: int, cols: int, *lead: int, dtype=None, device=None) -> torch.Tensor:
    """Allocate [*lead, rows, cols] whose row pitch avoids HBM channel aliasing.

    A wave of the streaming GEMM reads 16-32 weight rows at once; when the row pitch is a multiple
    of 4 KiB those rows land on the same channels (measured 4.7 vs 5.8 TB/s at K=4096).  64 extra
    elements per row (never read) fix that; the returned tensor is the [.., rows, cols] view."""
    pad = 64 if (cols * 2) % 4096 == 0 else 0
    t = torch.empty((*lead, rows, cols + pad), dtype=dtype, device=device)
    return t[..., :cols] if pad else t


def silu_and_mul(x: torch.Tensor) -> torch.Tensor:
    _bf16(x, "x")
    I = x.shape[-1] // 2
    x2 = x.reshape(-1, 2 * I).contiguous()
    y = torch.empty((x2.shape[0], I), dtype=x.dtype, device=x.device)
    _check(load_library().glm_silu_and_mul(_p(x2), _p(y), x2.shape[0], I, _stream()),
           "glm_silu_and_mul")
    return y.view(*x.shape[:-1], I)


# ------------------------------------------------------------------------------------------
# attention
# Split-KV scratch of the decode attention: ONE grow-only buffer per device, sized for the split count the launch
# really uses (none at all once B * nkv >= 256).  Keyed by device only: launches of one engine on one device are stream
# ordered (eager step, then capture on torch's side stream, then replays), and a per-stream key would make every graph
# capture miss the buffer reserve_attn_workspace() laid down on the default stream.  A replaced buffer stays referenced:
# HIP graphs captured earlier hold its address.  reserve_attn_workspace() lets the runner size it for max_num_seqs
# BEFORE the KV cache takes the rest of the memory; growing inside a stream capture is an error (the allocation and
# its memset would land in that graph's private pool).
_attn_ws: dict = {}
_attn_ws_retired: list = []


def _grow_only(table: dict, retired: list, device, need: int, what: str) -> torch.Tensor:
    device = torch.device(device)
    key = (device.type, device.index if device.index is not None else torch.cuda.current_device())
    ws = table.get(key)
    if ws is None or ws.numel() < need:
        if torch.cuda.is_current_stream_capturing():
            raise RuntimeError(f"{what}: {need} bytes needed while a HIP graph is being captured, {0 if ws is None else ws.numel()} "
                               "reserved — run one eager step (or the reserve_* call) at this size before capturing")
        if ws is not None:
            retired.append(ws)
        ws = torch.zeros(need, dtype=torch.uint8, device=device)  # zeros: the head of it holds arrival counters
        table[key] = ws
    return ws


def _attn_workspace(device, need: int) -> torch.Tensor | None:
    if need <= 0:
        return None
    return _grow_only(_attn_ws, _attn_ws_retired, device, need, "decode attention split-KV scratch")


def attn_workspace_bytes(B: int, nh: int, nkv: int, hd: int, block_size: int, bt_stride: int, num_splits: int = 0,
                         max_context_len: int = 0) -> int:
    lib = load_library()
    s = lib.glm_paged_attn_decode_splits(B, nkv, block_size, bt_stride, num_splits, max_context_len)
    return lib.glm_paged_attn_decode_workspace_bytes(B, nh, hd, s) if s > 1 else 0


def reserve_attn_workspace(device, max_batch: int, nh: int, nkv: int, hd: int, block_size: int, bt_stride: int) -> int:
    """Size the split-KV scratch for every decode batch size up to max_batch (worst case over B); returns the bytes."""
    need = max((attn_workspace_bytes(b, nh, nkv, hd, block_size, bt_stride) for b in range(1, max_batch + 1)), default=0)
    _attn_workspace(device, need)
    return need


def paged_attn_decode(q: torch.Tensor, k_cache: torch.Tensor, v_cache: torch.Tensor,
                      context_lens: torch.Tensor, block_tables: torch.Tensor, scale: float,
                      num_splits: int = 0, max_context_len: int = 0) -> torch.Tensor:
    """q: [B,nh,hd]; caches [n_blocks, block_size, nkv, hd] -> [B,nh,hd]."""
    _bf16(q, "q"); _bf16(k_cache, "k_cache"); _bf16(v_cache, "v_cache")
    B, nh, hd = q.shape
    n_blocks, block_size, nkv, _ = k_cache.shape
    assert q.is_contiguous() and k_cache.is_contiguous() and v_cache.is_contiguous()
    assert context_lens.dtype == torch.int32 and block_tables.dtype == torch.int32
    assert block_tables.stride(1) == 1
    lib = load_library()
    need = attn_workspace_bytes(B, nh, nkv, hd, block_size, block_tables.stride(0), num_splits, max_context_len)
    ws = _attn_workspace(q.device, need)
    out = torch.empty_like(q)
    _check(lib.glm_paged_attn_decode(_p(q), _p(k_cache), _p(v_cache), _p(context_lens),
                                     _p(block_tables), block_tables.stride(0), _p(out), B, nh, nkv,
                                     hd, block_size, n_blocks, scale, num_splits, max_context_len,
                                     _p(ws), ws.numel() if ws is not None else 0, _stream()), "glm_paged_attn_decode")
    return out


def paged_attn_decode_qkv(qkv, nh: int, nkv: int, hd: int, positions: torch.Tensor,
                          cos_sin_cache: torch.Tensor, rotary_dim: int, slot_mapping: torch.Tensor,
                          k_cache: torch.Tensor, v_cache: torch.Tensor, context_lens: torch.Tensor,
                          block_tables: torch.Tensor, scale: float, num_splits: int = 0,
                          max_context_len: int = 0, qkv_bias: torch.Tensor | None = None) -> torch.Tensor:
    """Decode attention straight from the packed QKV rows [B, (nh+2nkv)*hd]: rotary on Q/K, K/V cache store and the
    paged attention in one launch (no head RMSNorm, rotary_dim 64).  qkv may be a PartialSum (K-slice partial sums of
    the QKV projection, gemm_bf16_partial) together with the projection's bias: the kernel reduces them on load."""
    _bf16(k_cache, "k_cache"); _bf16(v_cache, "v_cache")
    partial = isinstance(qkv, PartialSum)
    if partial:
        part = qkv.part
        assert part.is_contiguous() and part.dtype == torch.float32 and part.shape[2] == (nh + 2 * nkv) * hd
        if qkv_bias is not None:
            _bf16(qkv_bias, "qkv_bias")
            assert qkv_bias.is_contiguous() and qkv_bias.numel() == part.shape[2]
        B = part.shape[1]
        dev_, dt_ = part.device, k_cache.dtype
    else:
        _bf16(qkv, "qkv")
        assert qkv_bias is None, "a bias belongs to partial sums only (bf16 rows already include it)"
        B = qkv.shape[0]
        dev_, dt_ = qkv.device, qkv.dtype
    n_blocks, block_size, nkv_c, _ = k_cache.shape
    assert nkv_c == nkv and (partial or (qkv.dim() == 2 and qkv.stride(1) == 1))
    assert k_cache.is_contiguous() and v_cache.is_contiguous() and cos_sin_cache.dtype == torch.float32
    assert cos_sin_cache.is_contiguous() and cos_sin_cache.shape[-1] == rotary_dim
    assert positions.dtype == torch.int64 and slot_mapping.dtype == torch.int32
    assert context_lens.dtype == torch.int32 and block_tables.dtype == torch.int32 and block_tables.stride(1) == 1
    lib = load_library()
    need = attn_workspace_bytes(B, nh, nkv, hd, block_size, block_tables.stride(0), num_splits, max_context_len)
    ws = _attn_workspace(dev_, need)
    out = torch.empty((B, nh, hd), dtype=dt_, device=dev_)
    if partial:
        _check(lib.glm_paged_attn_decode_qkv_partial(
            _p(part), part.shape[0], part.shape[1] * part.shape[2], _p(qkv_bias), _p(positions), _p(cos_sin_cache),
            cos_sin_cache.numel() // rotary_dim, rotary_dim, _p(slot_mapping), _p(k_cache), _p(v_cache), _p(context_lens),
            _p(block_tables), block_tables.stride(0), _p(out), B, nh, nkv, hd, block_size, n_blocks, scale, num_splits,
            max_context_len, _p(ws), ws.numel() if ws is not None else 0, _stream()), "glm_paged_attn_decode_qkv_partial")
        return out
    _check(lib.glm_paged_attn_decode_qkv(_p(qkv), qkv.stride(0), _p(positions), _p(cos_sin_cache),
                                         cos_sin_cache.numel() // rotary_dim, rotary_dim,
                                         _p(slot_mapping), _p(k_cache), _p(v_cache), _p(context_lens),
                                         _p(block_tables), block_tables.stride(0), _p(out), B, nh, nkv, hd,
                                         block_size, n_blocks, scale, num_splits, max_context_len, _p(ws),
                                         ws.numel() if ws is not None else 0, _stream()), "glm_paged_attn_decode_qkv")
    return out


def varlen_attn_prefill(q, k, v, cu_seqlens_q, cu_seqlens_k, max_seqlen_q, scale,
                        block_tables=None, block_size=256) -> torch.Tensor:
    _bf16(q, "q"); _bf16(k, "k"); _bf16(v, "v")
    Tq, nh, hd = q.shape
    nkv = k.shape[-2]
    B = cu_seqlens_q.numel() - 1
    out = torch.empty((Tq, nh, hd), dtype=q.dtype, device=q.device)
    q = q.contiguous(); k = k.contiguous(); v = v.contiguous()
    bts = block_tables.stride(0) if block_tables is not None else 0
    _check(load_library().glm_varlen_attn_prefill(_p(q), _p(k), _p(v), _p(cu_seqlens_q),
                                                  _p(cu_seqlens_k), _p(block_tables), bts, _p(out),
                                                  B, max_seqlen_q, nh, nkv, hd, block_size, scale,
                                                  _stream()), "glm_varlen_attn_prefill")
    return out


# ------------------------------------------------------------------------------------------
# MoE
# From this many rows on the router's logits (R1, moe.py:33: bf16(x . Wg^T)) are computed as what they are at that size,
# a [T, H] x [H, E] GEMM, and glm_router_select does R2..R7 from them; below, the token-per-workgroup kernel
# (glm_router_topk / the fused add-RMSNorm + router + bucketing launch), which is built for decode latency: at T = 16384
# it takes 1.2 ms per layer against 0.34 ms for norm + GEMM + select + bucketing (tools/prefill_router_probe.py).
ROUTER_GEMM_MIN_ROWS = 1024


def router_by_gemm(T: int, E: int) -> bool:
    return T >= ROUTER_GEMM_MIN_ROWS and E % 8 == 0  # the GEMM kernels want 16-byte output rows


def router_select(logits: torch.Tensor, bias: torch.Tensor, k: int, routed_scaling_factor: float):
    """R2..R7 from bf16 logits [T, E] (glm_router_select): (topk_idx int64 ascending per row, topk_w bf16)."""
    _bf16(logits, "logits")
    assert bias.dtype == torch.float32 and logits.dim() == 2 and logits.stride(1) == 1
    T, E = logits.shape
    idx = torch.empty((T, k), dtype=torch.int64, device=logits.device)
    w = torch.empty((T, k), dtype=torch.bfloat16, device=logits.device)
    _check(load_library().glm_router_select(_p(logits), logits.stride(0), _p(bias), _p(idx), _p(w), T, E, k,
                                            routed_scaling_factor, _stream()), "glm_router_select")
    return idx, w


def router_topk(x: torch.Tensor, gate_w: torch.Tensor, bias: torch.Tensor, k: int,
                routed_scaling_factor: float, return_logits: bool = False):
    _bf16(x, "x"); _bf16(gate_w, "gate_w")
    assert bias.dtype == torch.float32
    T, H = x.shape
    E = gate_w.shape[0]
    x = x.contiguous()
    if router_by_gemm(T, E):
        logits = gemm_bf16(x, gate_w, None)
        idx, w = router_select(logits, bias, k, routed_scaling_factor)
        return (idx, w, logits) if return_logits else (idx, w)
    idx = torch.empty((T, k), dtype=torch.int64, device=x.device)
    w = torch.empty((T, k), dtype=torch.bfloat16, device=x.device)
    logits = torch.empty((T, E), dtype=torch.bfloat16, device=x.device) if return_logits else None
    _check(load_library().glm_router_topk(_p(x), _p(gate_w), _p(bias), _p(idx), _p(w), _p(logits),
                                          T, H, E, k, routed_scaling_factor, _stream()),
           "glm_router_topk")
    return (idx, w, logits) if return_logits else (idx, w)


_router_ws: dict = {}
_router_ws_retired: list = []


def _router_workspace(device, T: int, E: int) -> torch.Tensor:
    """Workspace of the fused router + align launch (arrival counters, zero-initialised and restored by the kernel, then
    the T x E logits scratch): one grow-only buffer per device (see _grow_only); a replaced buffer stays referenced
    because HIP graphs captured earlier hold its address."""
    return _grow_only(_router_ws, _router_ws_retired, device, load_library().glm_router_workspace_bytes(T, E),
                      "router workspace")


def reserve_router_workspace(device, max_tokens: int, E: int) -> int:
    """Size the router workspace for every batch size up to max_tokens (the runner calls this before graph capture)."""
    need = load_library().glm_router_workspace_bytes(max_tokens, E)
    _grow_only(_router_ws, _router_ws_retired, device, need, "router workspace")
    return need


def add_rmsnorm_router_topk(x, residual: torch.Tensor, norm_weight: torch.Tensor, eps: float,
                            gate_w: torch.Tensor, bias: torch.Tensor, k: int, routed_scaling_factor: float,
                            align_with_shared: bool | None = None):
    """Post-attention add-RMSNorm + router in one launch.  x: bf16 [T,H] tensor or PartialSum (o_proj partial sums).
    Returns (normalised hidden, residual_out, topk_idx, topk_w); with align_with_shared = True/False the same launch
    also builds moe_align's (expert_offsets, sorted_token, sorted_scale, pair_pos), returned as a fifth element."""
    _bf16(residual, "residual"); _bf16(norm_weight, "norm_weight"); _bf16(gate_w, "gate_w")
    assert bias.dtype == torch.float32
    H = residual.shape[-1]
    r2 = residual.reshape(-1, H).contiguous()
    T = r2.shape[0]
    E = gate_w.shape[0]
    if router_by_gemm(T, E) and not isinstance(x, PartialSum):
        # prefill sizes: norm, logits GEMM + selection, bucketing as separate launches (see ROUTER_GEMM_MIN_ROWS)
        yn, rn = add_rmsnorm(x.reshape(-1, H), r2, norm_weight, eps)
        idx, w = router_topk(yn, gate_w, bias, k, routed_scaling_factor)
        if align_with_shared is None:
            return yn.view(residual.shape), rn.view(residual.shape), idx, w
        return (yn.view(residual.shape), rn.view(residual.shape), idx, w,
                moe_align(idx, w, E, bool(align_with_shared)))
    y = torch.empty_like(r2)
    ro = torch.empty_like(r2)
    idx = torch.empty((T, k), dtype=torch.int64, device=r2.device)
    w = torch.empty((T, k), dtype=torch.bfloat16, device=r2.device)
    if isinstance(x, PartialSum):
        part = x.part
        assert part.is_contiguous() and part.shape[1:] == (T, H)
        xp, pp, ns, stride = None, _p(part), part.shape[0], T * H
    else:
        _bf16(x, "x")
        x2 = x.reshape(-1, H).contiguous()
        assert x2.shape[0] == T
        xp, pp, ns, stride = _p(x2), None, 0, 0
    if align_with_shared is not None and 8 * (E + 1) <= 2 * H:
        ws = bool(align_with_shared)
        G, R, dev = E + (1 if ws else 0), T * k + (T if ws else 0), r2.device
        offs = torch.empty(G + 1, dtype=torch.int32, device=dev)
        tok = torch.empty(R, dtype=torch.int32, device=dev)
        scale = torch.empty(R, dtype=torch.bfloat16, device=dev)
        pos = torch.empty(T * k, dtype=torch.int32, device=dev)
        rws = _router_workspace(dev, T, E)
        _check(load_library().glm_add_rmsnorm_router_topk_align(
            xp, pp, ns, stride, _p(r2), _p(norm_weight), eps, _p(y), _p(ro), _p(gate_w), _p(bias), _p(idx), _p(w), T, H,
            E, k, routed_scaling_factor, _p(offs), _p(tok), _p(scale), _p(pos), 1 if ws else 0, _p(rws), rws.numel(),
            _stream()), "glm_add_rmsnorm_router_topk_align")
        return y.view(residual.shape), ro.view(residual.shape), idx, w, (offs, tok, scale, pos)
    _check(load_library().glm_add_rmsnorm_router_topk(xp, pp, ns, stride, _p(r2), _p(norm_weight), eps, _p(y), _p(ro),
                                                      _p(gate_w), _p(bias), _p(idx), _p(w), T, H, E, k,
                                                      routed_scaling_factor, _stream()),
           "glm_add_rmsnorm_router_topk")
    if align_with_shared is not None:
        return y.view(residual.shape), ro.view(residual.shape), idx, w, moe_align(idx, w, E, bool(align_with_shared))
    return y.view(residual.shape), ro.view(residual.shape), idx, w


ALIGN_PARALLEL_MIN_PAIRS = 16384  # from here on the one-workgroup bucketing kernel is the slower one (200 us at 131072 pairs)


def moe_align(topk_idx: torch.Tensor, topk_w: torch.Tensor | None, E: int, with_shared: bool):
    """topk_w None: no scales (the rows are weighed where they are summed up)."""
    T, k = topk_idx.shape
    G = E + (1 if with_shared else 0)
    R = T * k + (T if with_shared else 0)
    dev = topk_idx.device
    offs = torch.empty(G + 1, dtype=torch.int32, device=dev)
    tok = torch.empty(R, dtype=torch.int32, device=dev)
    scale = torch.empty(R, dtype=torch.bfloat16, device=dev) if topk_w is not None else None
    pos = torch.empty(T * k, dtype=torch.int32, device=dev)
    if T * k >= ALIGN_PARALLEL_MIN_PAIRS:  # prefill sizes: count / offsets / scatter over many workgroups
        lib = load_library()
        ws = torch.zeros(lib.glm_moe_align_workspace_bytes(T, k, E) // 4, dtype=torch.int32, device=dev)
        _check(lib.glm_moe_align_parallel(_p(topk_idx), _p(topk_w), _p(offs), _p(tok), _p(scale), _p(pos), T, k, E,
                                          1 if with_shared else 0, _p(ws), ws.numel() * 4, _stream()),
               "glm_moe_align_parallel")
        return offs, tok, scale, pos
    _check(load_library().glm_moe_align(_p(topk_idx), _p(topk_w), _p(offs), _p(tok), _p(scale),
                                        _p(pos), T, k, E, 1 if with_shared else 0, _stream()),
           "glm_moe_align")
    return offs, tok, scale, pos


TINYM_MAX_ROWS = 1  # token rows the single-sequence GEMV body takes (csrc/gemm_tinym.hip)


def grouped_gemm_gateup_silu(x, w13, expert_offsets, sorted_token, R: int, max_rows_per_group: int | None = None) -> torch.Tensor:
    """x [T,H]; w13 [G, 2I, H] -> act [R, I].  max_rows_per_group: an upper bound the caller knows (T for a top-k routing
    with the shared group); with ONE token row it selects the single-sequence GEMV body."""
    _bf16(x, "x"); _bf16(w13, "w13")
    G, I2, H = w13.shape
    I = I2 // 2
    assert w13.stride(2) == 1  # rows may be padded (stride(1) >= H), groups strided
    act = torch.empty((R, I), dtype=x.dtype, device=x.device)
    if x.shape[0] <= TINYM_MAX_ROWS and max_rows_per_group is not None and max_rows_per_group <= x.shape[0]:
        # single-sequence decode: the GEMV body (the caller vouches that no group holds more rows than there are tokens;
        # the body computes ONE row per group and would silently drop further ones — at least the row count must allow it)
        if R > G:
            raise ValueError(f"grouped_gemm_gateup_silu: {R} rows over {G} groups cannot be one row per group")
        _check(load_library().glm_grouped_gemm_gateup_silu_fewtok(
            _p(x), x.stride(0), x.shape[0], _p(w13), w13.stride(0), w13.stride(1), _p(expert_offsets), _p(sorted_token),
            _p(act), R, H, I, G, _stream()), "glm_grouped_gemm_gateup_silu_fewtok")
        return act
    _check(load_library().glm_grouped_gemm_gateup_silu(_p(x), x.stride(0), _p(w13), w13.stride(0),
                                                       w13.stride(1),
                                                       _p(expert_offsets), _p(sorted_token),
                                                       _p(act), R, H, I, G, _stream()),
           "glm_grouped_gemm_gateup_silu")
    return act


def grouped_gemm_down(act, w2, expert_offsets, sorted_scale, n_scaled_groups: int,
                      max_rows_per_group: int | None = None) -> torch.Tensor:
    """act [R,I]; w2 [G, H, I] -> y [R, H]."""
    _bf16(act, "act"); _bf16(w2, "w2")
    G, H, I = w2.shape
    R = act.shape[0]
    assert w2.stride(2) == 1 and act.is_contiguous()
    y = torch.empty((R, H), dtype=act.dtype, device=act.device)
    if max_rows_per_group is not None and max_rows_per_group <= TINYM_MAX_ROWS:
        if act.shape[0] > w2.shape[0] * max(1, max_rows_per_group):
            raise ValueError(f"grouped_gemm_down: {act.shape[0]} rows over {w2.shape[0]} groups exceed {max_rows_per_group} per group")
        _check(load_library().glm_grouped_gemm_down_fewtok(_p(act), max_rows_per_group, _p(w2), w2.stride(0), w2.stride(1),
                                                           _p(expert_offsets), _p(sorted_scale), n_scaled_groups, _p(y), H,
                                                           R, H, I, G, _stream()), "glm_grouped_gemm_down_fewtok")
        return y
    _check(load_library().glm_grouped_gemm_down(_p(act), _p(w2), w2.stride(0), w2.stride(1),
                                                _p(expert_offsets),
                                                _p(sorted_scale), n_scaled_groups, _p(y), H, R, H,
                                                I, G, _stream()), "glm_grouped_gemm_down")
    return y


FP8_MAX = 448.0  # largest finite OCP e4m3fn value


def quantize_fp8_rowwise(w: torch.Tensor):
    """Weight-only quantisation used for the experts: per-row scale s = max|row| / 448,
    q = e4m3fn(row / s).  Returns (q as uint8 with a padded row pitch, s as fp32)."""
    rows, cols = w.shape[-2], w.shape[-1]
    s = (w.abs().amax(dim=-1).to(torch.float32) / FP8_MAX).clamp_min(1e-12)
    q = (w.to(torch.float32) / s.unsqueeze(-1)).clamp(-FP8_MAX, FP8_MAX).to(torch.float8_e4m3fn)
    pad = 128 if cols % 4096 == 0 else 0  # same channel-aliasing rule as padded_weight (bytes)
    store = torch.empty((*w.shape[:-1], cols + pad), dtype=torch.uint8, device=w.device)
    view = store[..., :cols]
    view.copy_(q.view(torch.uint8))
    return view, s.contiguous()


def quantize_fp8_rows(x: torch.Tensor):
    """Dynamic per-row e4m3 quantisation of activation rows (glm_quantize_fp8_rows): x [T, H] bf16 ->
    (q [T, H] uint8, scale [T] fp32) with x ~ q * scale[:, None]."""
    _bf16(x, "x")
    assert x.dim() == 2 and x.stride(1) == 1
    T, H = x.shape
    q = torch.empty((T, H), dtype=torch.uint8, device=x.device)
    s = torch.empty(T, dtype=torch.float32, device=x.device)
    _check(load_library().glm_quantize_fp8_rows(_p(x), x.stride(0), _p(q), q.stride(0), _p(s), T, H, _stream()),
           "glm_quantize_fp8_rows")
    return q, s


def grouped_gemm_gateup_silu_fp8a8(x_q, x_scale, w13_q, w13_s, expert_offsets, sorted_token, R: int):
    """fp8 x fp8 gate|up on the block-scaled MFMA (glm_grouped_gemm_gateup_silu_fp8a8).  x_q [T, H] uint8 + x_scale [T];
    w13_q [G, 2I, H] uint8 + w13_s [G, 2I].  Returns (act_q [R, I] uint8, act_bscale [R, 64] uint8: E8M0 per 32 columns) — or
    None when the launcher does not cover the shape (nothing enqueued: take the weight-only path)."""
    G, I2, H = w13_q.shape
    I = I2 // 2
    assert x_q.dtype == torch.uint8 and w13_q.dtype == torch.uint8 and x_q.stride(1) == 1 and w13_q.stride(2) == 1
    assert x_scale.dtype == torch.float32 and w13_s.dtype == torch.float32 and w13_s.stride(1) == 1
    act = torch.empty((R, I), dtype=torch.uint8, device=x_q.device)
    bs = torch.zeros((R, 64), dtype=torch.uint8, device=x_q.device)
    rc = load_library().glm_grouped_gemm_gateup_silu_fp8a8(
        _p(x_q), x_q.stride(0), _p(x_scale), _p(w13_q), w13_q.stride(0), w13_q.stride(1), _p(w13_s), w13_s.stride(0),
        _p(expert_offsets), _p(sorted_token), _p(act), act.stride(0), _p(bs), R, H, I, G, _stream())
    if rc == GLM_ERR_UNSUPPORTED:
        return None
    _check(rc, "glm_grouped_gemm_gateup_silu_fp8a8")
    return act, bs


def grouped_gemm_down_fp8a8(act_q, act_bscale, w2_q, w2_s, expert_offsets, sorted_scale, n_scaled_groups: int):
    """fp8 x fp8 down projection with the act rows' E8M0 block scales inside the MFMA; y [R, H] bf16, or None (shape not
    covered)."""
    G, H, I = w2_q.shape
    R = act_q.shape[0]
    assert act_q.dtype == torch.uint8 and w2_q.dtype == torch.uint8 and act_bscale.dtype == torch.uint8
    assert act_bscale.shape == (R, 64) and act_bscale.is_contiguous() and w2_q.stride(2) == 1 and w2_s.stride(1) == 1
    y = torch.empty((R, H), dtype=torch.bfloat16, device=act_q.device)
    rc = load_library().glm_grouped_gemm_down_fp8a8(
        _p(act_q), act_q.stride(0), _p(act_bscale), _p(w2_q), w2_q.stride(0), w2_q.stride(1), _p(w2_s), w2_s.stride(0),
        _p(expert_offsets), _p(sorted_scale), n_scaled_groups, _p(y), y.stride(0), R, H, I, G, _stream())
    if rc == GLM_ERR_UNSUPPORTED:
        return None
    _check(rc, "glm_grouped_gemm_down_fp8a8")
    return y


_FP8_LARGE_MIN_AVG_ROWS = 96  # api.hip LARGEM_MIN_AVG_ROWS
_fp8_scratch: dict = {}


def _fp8_expand_scratch(device, G: int, rows: int, cols: int, R: int):
    """Scratch for the prefill-regime fp8 expert GEMM where the tiled kernel cannot take the fp8 bytes directly (K not a
    multiple of 64): bf16 copy of ONE weight stack, reused by every layer and both projections.  None at decode row counts
    (streaming fp8 kernel) and for the shapes the fp8-operand kernel covers."""
    if R // max(G, 1) < _FP8_LARGE_MIN_AVG_ROWS:
        return None, 0
    need = load_library().glm_fp8w_expand_scratch_bytes(G, rows, cols)
    if need == 0:  # the tiled kernel takes the fp8 bytes themselves
        return None, 0
    buf = _fp8_scratch.get(device)
    if buf is None or buf.numel() < need:
        buf = torch.empty(need, dtype=torch.uint8, device=device)
        _fp8_scratch[device] = buf
    return buf, buf.numel()


def grouped_gemm_gateup_silu_fp8w(x, w13_q, w13_s, expert_offsets, sorted_token, R: int) -> torch.Tensor:
    """x [T,H] bf16; w13_q [G,2I,H] uint8 (fp8 e4m3); w13_s [G,2I] fp32 -> act [R,I]."""
    _bf16(x, "x")
    G, I2, H = w13_q.shape
    I = I2 // 2
    assert w13_q.dtype == torch.uint8 and w13_q.stride(2) == 1 and w13_s.dtype == torch.float32
    assert w13_s.stride(1) == 1
    act = torch.empty((R, I), dtype=x.dtype, device=x.device)
    scr, scr_n = _fp8_expand_scratch(x.device, G, I2, H, R)
    _check(load_library().glm_grouped_gemm_gateup_silu_fp8w(
        _p(x), x.stride(0), _p(w13_q), w13_q.stride(0), w13_q.stride(1), _p(w13_s), w13_s.stride(0),
        _p(expert_offsets), _p(sorted_token), _p(act), R, H, I, G, _p(scr), scr_n, _stream()),
        "glm_grouped_gemm_gateup_silu_fp8w")
    return act


def grouped_gemm_down_fp8w(act, w2_q, w2_s, expert_offsets, sorted_scale, n_scaled_groups: int) -> torch.Tensor:
    _bf16(act, "act")
    G, H, I = w2_q.shape
    R = act.shape[0]
    assert w2_q.dtype == torch.uint8 and w2_q.stride(2) == 1 and w2_s.dtype == torch.float32 and act.is_contiguous()
    y = torch.empty((R, H), dtype=act.dtype, device=act.device)
    scr, scr_n = _fp8_expand_scratch(act.device, G, H, I, R)
    _check(load_library().glm_grouped_gemm_down_fp8w(
        _p(act), _p(w2_q), w2_q.stride(0), w2_q.stride(1), _p(w2_s), w2_s.stride(0), _p(expert_offsets),
        _p(sorted_scale), n_scaled_groups, _p(y), H, R, H, I, G, _p(scr), scr_n, _stream()),
        "glm_grouped_gemm_down_fp8w")
    return y


def ep_plan(topk_idx: torch.Tensor, topk_w: torch.Tensor, E: int, ep: int, rank: int, cap: int):
    """Fixed-capacity expert-parallel dispatch plan (glm_ep_plan) from the replicated routing [T, k]: device tensors
    (send_gather, slot_scale, pair_slot, recv_offs, recv_gidx, overflow); no host synchronisation."""
    T, k = topk_idx.shape
    _bf16(topk_w, "topk_w")
    assert topk_idx.dtype == torch.int64 and topk_idx.is_contiguous() and topk_w.is_contiguous() and E % ep == 0
    dev = topk_idx.device
    per = (T + ep - 1) // ep
    Tl = max(0, min(T, (rank + 1) * per) - min(T, rank * per))
    send_gather = torch.empty(ep * cap, dtype=torch.int32, device=dev)
    slot_scale = torch.zeros(ep * cap, dtype=torch.bfloat16, device=dev)
    pair_slot = torch.empty(max(Tl * k, 1), dtype=torch.int32, device=dev)
    recv_offs = torch.empty(E // ep + 1, dtype=torch.int32, device=dev)
    recv_gidx = torch.empty(ep * cap, dtype=torch.int32, device=dev)
    overflow = torch.empty(1, dtype=torch.int32, device=dev)
    _check(load_library().glm_ep_plan(_p(topk_idx), _p(topk_w), T, k, E, ep, rank, cap, _p(send_gather), _p(slot_scale),
                                      _p(pair_slot), _p(recv_offs), _p(recv_gidx), _p(overflow), _stream()), "glm_ep_plan")
    return send_gather, slot_scale, pair_slot, recv_offs, recv_gidx, overflow


def grouped_gemm_gateup_silu_cap(x, w13, expert_offsets, sorted_token, R_cap: int, R_expected: int) -> torch.Tensor:
    """grouped_gemm_gateup_silu over a capacity-sized row array: expert_offsets say which of the R_cap rows are real."""
    _bf16(x, "x"); _bf16(w13, "w13")
    G, I2, H = w13.shape
    I = I2 // 2
    assert w13.stride(2) == 1
    act = torch.empty((R_cap, I), dtype=x.dtype, device=x.device)
    _check(load_library().glm_grouped_gemm_gateup_silu_cap(_p(x), x.stride(0), _p(w13), w13.stride(0), w13.stride(1),
                                                           _p(expert_offsets), _p(sorted_token), _p(act), R_cap, R_expected,
                                                           H, I, G, _stream()), "glm_grouped_gemm_gateup_silu_cap")
    return act


def grouped_gemm_down_cap(act, w2, expert_offsets, R_expected: int) -> torch.Tensor:
    """Unscaled grouped down projection over a capacity-sized row array (the routing weight is applied at home)."""
    _bf16(act, "act"); _bf16(w2, "w2")
    G, H, I = w2.shape
    R_cap = act.shape[0]
    assert w2.stride(2) == 1 and act.is_contiguous()
    y = torch.empty((R_cap, H), dtype=act.dtype, device=act.device)
    _check(load_library().glm_grouped_gemm_down_cap(_p(act), _p(w2), w2.stride(0), w2.stride(1), _p(expert_offsets), None, 0,
                                                    _p(y), H, R_cap, R_expected, H, I, G, _stream()),
           "glm_grouped_gemm_down_cap")
    return y


def moe_combine(y, pair_pos, T: int, k: int, shared_base: int) -> torch.Tensor:
    H = y.shape[1]
    out = torch.empty((T, H), dtype=y.dtype, device=y.device)
    _check(load_library().glm_moe_combine(_p(y), y.stride(0), _p(pair_pos), _p(out), T, k, H,
                                          shared_base, _stream()), "glm_moe_combine")
    return out


def gather_rows(src: torch.Tensor, idx: torch.Tensor) -> torch.Tensor:
    """dst[i] = src[idx[i]] (rows of bf16; idx int32; idx < 0: the row is left uninitialised)."""
    _bf16(src, "src")
    assert src.dim() == 2 and idx.dtype == torch.int32 and idx.is_contiguous()
    dst = torch.empty((idx.numel(), src.shape[1]), dtype=src.dtype, device=src.device)
    _check(load_library().glm_gather_rows(_p(src), src.stride(0), _p(dst), dst.stride(0), _p(idx), idx.numel(),
                                          src.shape[1], _stream()), "glm_gather_rows")
    return dst


def scatter_rows(src: torch.Tensor, idx: torch.Tensor, n_rows: int | None = None, no_init: bool = False) -> torch.Tensor:
    """dst[idx[i]] = src[i] (idx < 0: skipped); rows of dst no index points at stay zero (no_init: uninitialised)."""
    _bf16(src, "src")
    assert src.dim() == 2 and idx.dtype == torch.int32 and idx.is_contiguous() and idx.numel() == src.shape[0]
    alloc = torch.empty if no_init else torch.zeros
    dst = alloc((n_rows if n_rows is not None else src.shape[0], src.shape[1]), dtype=src.dtype, device=src.device)
    _check(load_library().glm_scatter_rows(_p(src), src.stride(0), _p(dst), dst.stride(0), _p(idx), idx.numel(),
                                           src.shape[1], _stream()), "glm_scatter_rows")
    return dst


def moe_combine_scaled(y, pair_pos, row_scale, shared_rows, T: int, k: int) -> torch.Tensor:
    """Expert-parallel combine: routing weight applied here to the unscaled rows, ascending-expert bf16 adds, + shared."""
    _bf16(y, "y"); _bf16(row_scale, "row_scale")
    H = y.shape[1]
    out = torch.empty((T, H), dtype=y.dtype, device=y.device)
    if shared_rows is not None:
        _bf16(shared_rows, "shared_rows")
    _check(load_library().glm_moe_combine_scaled(_p(y), y.stride(0), _p(pair_pos), _p(row_scale), _p(shared_rows),
                                                 shared_rows.stride(0) if shared_rows is not None else 0, _p(out), T, k,
                                                 H, _stream()), "glm_moe_combine_scaled")
    return out


class DeferredCombine:
    """Rows of the grouped down projection plus the per-token row list: the MoE combine (moe_combine) that has not
    been run yet because the consumer — the next layer's add-RMSNorm — performs it in the same launch."""
    __slots__ = ("y", "pair_pos", "T", "k", "shared_base", "out_shape")

    def __init__(self, y, pair_pos, T, k, shared_base, out_shape):
        self.y, self.pair_pos, self.T, self.k, self.shared_base, self.out_shape = y, pair_pos, T, k, shared_base, out_shape

    @property
    def shape(self):
        return self.out_shape

    def materialize(self) -> torch.Tensor:
        return moe_combine(self.y, self.pair_pos, self.T, self.k, self.shared_base).view(self.out_shape)


def moe_combine_add_rmsnorm(dc: DeferredCombine, residual: torch.Tensor, weight: torch.Tensor,
                            eps: float) -> tuple[torch.Tensor, torch.Tensor]:
    """moe_combine + add_rmsnorm(combined, residual) in one launch."""
    _bf16(residual, "residual"); _bf16(weight, "weight")
    H = dc.y.shape[1]
    r2 = residual.reshape(-1, H).contiguous()
    assert r2.shape[0] == dc.T
    out = torch.empty_like(r2)
    ro = torch.empty_like(r2)
    _check(load_library().glm_moe_combine_add_rmsnorm(_p(dc.y), dc.y.stride(0), _p(dc.pair_pos), dc.T, dc.k, H,
                                                      dc.shared_base, _p(r2), _p(weight), _p(out), _p(ro), eps,
                                                      _stream()), "glm_moe_combine_add_rmsnorm")
    return out.view(residual.shape), ro.view(residual.shape)


def combine_add_rmsnorm_gemm(dc: DeferredCombine, residual: torch.Tensor, norm_weight: torch.Tensor, eps: float,
                             w: torch.Tensor, bias: torch.Tensor | None):
    """ONE token: moe_combine + add_rmsnorm(combined, residual) + (x @ w.T + bias) in ONE launch (glm_gemm_bf16_combine_norm).
    Returns (y [T, N], residual_out [T, H]); the normalised hidden state itself is never written."""
    _bf16(residual, "residual"); _bf16(norm_weight, "norm_weight"); _bf16(w, "w")
    H = dc.y.shape[1]
    N = w.shape[0]
    r2 = residual.reshape(-1, H).contiguous()
    assert r2.shape[0] == dc.T and w.shape[1] == H and w.stride(1) == 1
    y = torch.empty((dc.T, N), dtype=r2.dtype, device=r2.device)
    ro = torch.empty_like(r2)
    _check(load_library().glm_gemm_bf16_combine_norm(_p(dc.y), dc.y.stride(0), _p(dc.pair_pos), dc.T, dc.k, dc.shared_base,
                                                     _p(r2), _p(norm_weight), eps, _p(ro), None, _p(w), w.stride(0),
                                                     _p(bias), _p(y), N, N, H, _stream()), "glm_gemm_bf16_combine_norm")
    return y, ro.view(residual.shape)


def can_combine_norm_gemm(dc, H: int) -> bool:
    return (isinstance(dc, DeferredCombine) and dc.T <= TINYM_MAX_ROWS and H % 8 == 0 and H <= 4096
            and opt("tinym") != 0 and opt("fuse_combine_qkv") != 0)


_tail_ws: dict = {}
_tail_ws_retired: list = []


def check_router_tail(device=None) -> None:
    """Raise if a one-token o_proj + router-tail launch gave up its bounded wait since the last call (its outputs were
    poisoned; word 2 of the tail workspace is the sticky status).  One 4-byte read: call it where the step is synchronised
    anyway (ModelRunner.run).  The workspace is re-zeroed so that the next launch starts from clean counters."""
    for key, ws in list(_tail_ws.items()):
        if device is not None and torch.device(device).index not in (None, key[1]):
            continue
        st = int(ws[8:12].view(torch.int32).item())
        if st:
            torch.cuda.synchronize(torch.device(key[0], key[1]))
            ws.zero_()
            raise RuntimeError(f"one-token router tail: designated workgroup {st - 1} gave up waiting for the projection; "
                               "the outputs of that step are NaN")


def can_gemm_router_tail(x: torch.Tensor, H: int, E: int) -> bool:
    return (x.dim() == 2 and x.shape[0] == 1 and 2048 <= H <= 4096 and H % 8 == 0 and E <= 256 and x.is_contiguous()
            and opt("tinym") != 0 and opt("fuse_oproj_router") != 0)


def gemm_add_rmsnorm_router_topk_align(x: torch.Tensor, w: torch.Tensor, residual: torch.Tensor, norm_weight: torch.Tensor,
                                       eps: float, gate_w: torch.Tensor, bias: torch.Tensor, k: int,
                                       routed_scaling_factor: float, with_shared: bool):
    """ONE token: o_proj + post-attention add-RMSNorm + router + bucketing in one launch (glm_gemm_bf16_router_tail).
    x [1, K], w [H, K].  Returns what add_rmsnorm_router_topk(..., align_with_shared=...) returns — or None when the
    launcher does not cover the shape (nothing was enqueued: take the two-launch path)."""
    _bf16(x, "x"); _bf16(w, "w"); _bf16(residual, "residual"); _bf16(norm_weight, "norm_weight"); _bf16(gate_w, "gate_w")
    assert bias.dtype == torch.float32 and x.shape[0] == 1 and w.stride(1) == 1
    K, H, E = x.shape[1], w.shape[0], gate_w.shape[0]
    dev = x.device
    r2 = residual.reshape(1, H).contiguous()
    o_row = torch.empty((1, H), dtype=x.dtype, device=dev)
    y, ro = torch.empty_like(r2), torch.empty_like(r2)
    idx = torch.empty((1, k), dtype=torch.int64, device=dev)
    tw = torch.empty((1, k), dtype=torch.bfloat16, device=dev)
    G, R = E + (1 if with_shared else 0), k + (1 if with_shared else 0)
    offs = torch.empty(G + 1, dtype=torch.int32, device=dev)
    tok = torch.empty(R, dtype=torch.int32, device=dev)
    scale = torch.empty(R, dtype=torch.bfloat16, device=dev)
    pos = torch.empty(k, dtype=torch.int32, device=dev)
    # two self-restoring counters + E floats of logits scratch, one grow-only zeroed buffer per device
    ticket = _grow_only(_tail_ws, _tail_ws_retired, dev, 16 + 4 * 256, "router-tail workspace").data_ptr()
    rc = load_library().glm_gemm_bf16_router_tail(
        _p(x), _p(w), w.stride(0), K, H, _p(o_row), ticket, _p(r2), _p(norm_weight), eps, _p(y), _p(ro), _p(gate_w),
        _p(bias), E, k, routed_scaling_factor, _p(idx), _p(tw), _p(offs), _p(tok), _p(scale), _p(pos), 1 if with_shared else 0,
        _stream())
    if rc == GLM_ERR_UNSUPPORTED:
        # the launcher's own limits (K window of the tail's LDS scratch, rows per wave vs experts) are checked before anything
        # is enqueued: nothing ran, the caller falls back to o_proj + add_rmsnorm_router_topk (two launches)
        return None
    _check(rc, "glm_gemm_bf16_router_tail")
    return y.view(residual.shape), ro.view(residual.shape), idx, tw, (offs, tok, scale, pos)


_engine_ws: dict = {}
_engine_ws_retired: list = []


def can_decode_mlp_engine(x: torch.Tensor, H: int, E: int, k: int, I: int) -> bool:
    return (opt("t1_engine") != 0 and x.dim() == 2 and x.shape[0] == 1 and H in (2048, 4096) and x.shape[1] % 2048 == 0
            and E <= 256 and k <= 64 and 1024 <= I <= 1536 and I % 8 == 0 and x.is_contiguous())


def decode_mlp_engine(x: torch.Tensor, w_o: torch.Tensor, residual: torch.Tensor, norm_weight: torch.Tensor, eps: float,
                      gate_w: torch.Tensor, bias: torch.Tensor, k: int, routed_scaling_factor: float, w13: torch.Tensor,
                      w2: torch.Tensor, want_act: bool = False):
    """ONE token: o_proj + post-attention add-RMSNorm + router + bucketing + grouped gate|up + SiLU*mul + grouped down x
    routing weight in ONE persistent launch (glm_decode_mlp_engine, csrc/decode_engine.hip).  x [1, K]; w_o [H, K];
    w13 [E+1, 2I, H], w2 [E+1, H, I] (group E = the shared expert).  Returns (y_norm, residual_out, topk_idx, topk_w,
    (offs, tok, scale, pos), y [k+1, H], act or None) — exactly what gemm_add_rmsnorm_router_topk_align +
    grouped_gemm_gateup_silu + grouped_gemm_down return, bit for bit — or None when the launcher does not cover the shape
    (nothing was enqueued)."""
    _bf16(x, "x"); _bf16(w_o, "w_o"); _bf16(residual, "residual"); _bf16(norm_weight, "norm_weight"); _bf16(gate_w, "gate_w")
    _bf16(w13, "w13"); _bf16(w2, "w2")
    assert bias.dtype == torch.float32 and x.shape[0] == 1 and w_o.stride(1) == 1 and w13.stride(2) == 1 and w2.stride(2) == 1
    K, H, E = x.shape[1], w_o.shape[0], gate_w.shape[0]
    I = w2.shape[2]
    assert w13.shape[0] == E + 1 and w13.shape[1] == 2 * I and w13.shape[2] == H and w2.shape[0] == E + 1 and w2.shape[1] == H
    dev = x.device
    r2 = residual.reshape(1, H).contiguous()
    y_norm, ro = torch.empty_like(r2), torch.empty_like(r2)
    idx = torch.empty((1, k), dtype=torch.int64, device=dev)
    tw = torch.empty((1, k), dtype=torch.bfloat16, device=dev)
    offs = torch.empty(E + 2, dtype=torch.int32, device=dev)
    tok = torch.empty(k + 1, dtype=torch.int32, device=dev)
    scale = torch.empty(k + 1, dtype=torch.bfloat16, device=dev)
    pos = torch.empty(k, dtype=torch.int32, device=dev)
    y = torch.empty((k + 1, H), dtype=x.dtype, device=dev)
    act = torch.empty((k + 1, I), dtype=x.dtype, device=dev) if want_act else None
    lib = load_library()
    ws = _grow_only(_engine_ws, _engine_ws_retired, dev, lib.glm_decode_mlp_engine_workspace_bytes(H, E, k, I),
                    "decode engine workspace")
    rc = lib.glm_decode_mlp_engine(
        _p(x), _p(w_o), w_o.stride(0), K, H, _p(r2), _p(norm_weight), eps, _p(y_norm), _p(ro), _p(gate_w), _p(bias), E, k,
        routed_scaling_factor, _p(idx), _p(tw), _p(offs), _p(tok), _p(scale), _p(pos), _p(w13), w13.stride(0), w13.stride(1),
        _p(w2), w2.stride(0), w2.stride(1), I, _p(act), _p(y), y.stride(0), ws.data_ptr(), _stream())
    if rc == GLM_ERR_UNSUPPORTED:
        return None
    _check(rc, "glm_decode_mlp_engine")
    return y_norm.view(residual.shape), ro.view(residual.shape), idx, tw, (offs, tok, scale, pos), y, act


def check_decode_engine(device=None) -> None:
    """Raise if a bounded wait inside a glm_decode_mlp_engine launch expired since the last call (word 1 of its workspace is
    the sticky status; y was NaN-filled).  One 4-byte read; the workspace is re-zeroed."""
    for key, ws in list(_engine_ws.items()):
        if device is not None and torch.device(device).index not in (None, key[1]):
            continue
        st = int(ws[4:8].view(torch.int32).item())
        if st:
            torch.cuda.synchronize(torch.device(key[0], key[1]))
            ws.zero_()
            raise RuntimeError(f"one-token decode engine: a bounded wait expired (code 0x{st & 0xf00:x}, workgroup {st & 0xff}); "
                               "the outputs of that step are NaN")


class PartialSum:
    """fp32 K-slice partial sums [nslices, M, N] of a bias-free linear layer whose reduction (and bf16 rounding) is
    deferred to the consumer kernel (add_rmsnorm_partial)."""
    __slots__ = ("part",)

    def __init__(self, part: torch.Tensor):
        self.part = part

    @property
    def shape(self):
        return self.part.shape[1:]


def gemm_bf16_partial(x: torch.Tensor, w: torch.Tensor, want_slices: int = 8) -> PartialSum:
    """K-slice partial sums of x @ w.T for decode batches: M <= 32, or gemm_slices of them; see glm_gemm_bf16_partial."""
    _bf16(x, "x"); _bf16(w, "w")
    K = x.shape[-1]
    N = w.shape[0]
    assert x.dim() == 2 and w.shape[1] == K and w.stride(1) == 1 and x.stride(1) == 1
    M = x.shape[0]
    lib = load_library()
    ns = lib.glm_gemm_bf16_partial_slices(K, want_slices) if M <= 32 else want_slices
    part = torch.empty((ns, M, N), dtype=torch.float32, device=x.device)
    _check(lib.glm_gemm_bf16_partial(_p(x), x.stride(0), _p(w), w.stride(0), _p(part), M, N, K, ns, _stream()),
           "glm_gemm_bf16_partial")
    return PartialSum(part)


def gemm_slices(M: int, N: int, K: int) -> int:
    """K slices that spread a projection of some hundred rows over the chip (1: its output tiles do)."""
    return load_library().glm_gemm_bf16_slices(M, N, K)


def add_rmsnorm_partial(ps: PartialSum, residual: torch.Tensor, weight: torch.Tensor,
                        eps: float) -> tuple[torch.Tensor, torch.Tensor]:
    """add_rmsnorm whose x is bf16(sum of the K-slice partial sums)."""
    _bf16(residual, "residual"); _bf16(weight, "weight")
    part = ps.part
    ns, T, H = part.shape
    r2 = residual.reshape(-1, H).contiguous()
    assert r2.shape[0] == T and part.is_contiguous()
    y = torch.empty_like(r2)
    ro = torch.empty_like(r2)
    _check(load_library().glm_add_rmsnorm_partial(_p(part), ns, T * H, _p(r2), _p(weight), _p(y), _p(ro), T, H, eps,
                                                  _stream()), "glm_add_rmsnorm_partial")
    return y.view(residual.shape), ro.view(residual.shape)


def gemm_bf16(x: torch.Tensor, w: torch.Tensor, bias: torch.Tensor | None = None) -> torch.Tensor:
    """y = bf16(x @ w.T + bias); x [..., K], w [N, K]."""
    _bf16(x, "x"); _bf16(w, "w")
    K = x.shape[-1]
    N = w.shape[0]
    assert w.shape[1] == K and w.stride(1) == 1  # row pitch w.stride(0) may be padded
    x2 = x.reshape(-1, K)
    if x2.stride(-1) != 1:
        x2 = x2.contiguous()
    M = x2.shape[0]
    y = torch.empty((M, N), dtype=x.dtype, device=x.device)
    _check(load_library().glm_gemm_bf16(_p(x2), x2.stride(0), _p(w), w.stride(0), _p(bias), _p(y), N,
                                        M, N, K, _stream()), "glm_gemm_bf16")
    return y.view(*x.shape[:-1], N)


# ------------------------------------------------------------------------------------------
# decoders with a 32-bit residual stream, latent attention and short convolutions over time (no counterpart in the
# reference).  Activations are bf16 or fp32 (`act dtype`): every op below takes either and picks the kernel by dtype.
ACT_NONE, ACT_XIELU, ACT_SOFTCAP = 0, 1, 2
ACT_GATE, ACT_SILU_GATE = 4, 5     # columns below the constant pass / go through SiLU, the others through the sigmoid
ACT_RELU2_GATE = 6                 # columns below the first constant: relu squared; below the second: pass; the others: sigmoid
NO_ACT = (ACT_NONE, 0.0, 0.0)


def round8(n: int) -> int:
    return (n + 7) // 8 * 8


def _is_f32(dtype) -> int:
    if dtype == torch.float32:
        return 1
    if dtype == torch.bfloat16:
        return 0
    raise TypeError(f"activations are bfloat16 or float32, not {dtype}")


def linear_act(x: torch.Tensor, w: torch.Tensor, bias: torch.Tensor | None = None, act=NO_ACT, out_f32: bool = False, out: torch.Tensor | None = None) -> torch.Tensor:
    """act(x @ w.T + bias), x [M, K], w [N, K] (row pitches free), in x's dtype or — out_f32 — unrounded fp32; out: where to (a view with
    its own row pitch)."""
    M, K = x.shape
    N = w.shape[0]
    assert w.shape[1] == K and w.dtype == x.dtype and x.stride(1) == 1 and w.stride(1) == 1
    f32 = _is_f32(x.dtype)
    assert bias is None or (bias.dtype == x.dtype and bias.numel() == N and bias.is_contiguous())
    dt = torch.float32 if (f32 or out_f32) else x.dtype
    y = torch.empty((M, N), dtype=dt, device=x.device) if out is None else out
    assert y.shape == (M, N) and y.dtype == dt and y.stride(1) == 1
    if f32:
        _check(load_library().glm_gemm_f32(_p(x), x.stride(0), 0, _p(w), w.stride(0), 0, _p(bias), _p(y), y.stride(0), 0, M, N, K, 1, *act,
                                           _stream()), "glm_gemm_f32")
    elif act[0] == ACT_NONE and not out_f32:
        _check(load_library().glm_gemm_bf16(_p(x), x.stride(0), _p(w), w.stride(0), _p(bias), _p(y), y.stride(0), M, N, K, _stream()),
               "glm_gemm_bf16")
    else:
        _check(load_library().glm_gemm_bf16_act(_p(x), x.stride(0), _p(w), w.stride(0), _p(bias), _p(y), y.stride(0), M, N, K,
                                                int(out_f32), *act, _stream()), "glm_gemm_bf16_act")
    return y


def batched_gemm_f32(x: torch.Tensor, w: torch.Tensor, y: torch.Tensor) -> None:
    """y[b] = x[b] @ w[b].T for strided fp32 views x [B, M, K], w [B, N, K], y [B, M, N]."""
    B, M, K = x.shape
    N = w.shape[1]
    assert w.shape == (B, N, K) and y.shape == (B, M, N) and x.stride(2) == w.stride(2) == y.stride(2) == 1
    assert x.dtype == w.dtype == y.dtype == torch.float32
    _check(load_library().glm_gemm_f32(_p(x), x.stride(1), x.stride(0), _p(w), w.stride(1), w.stride(0), None, _p(y), y.stride(1),
                                       y.stride(0), M, N, K, B, *NO_ACT, _stream()), "glm_gemm_f32")


def embed_rows(ids: torch.Tensor, table: torch.Tensor, wp: int, cast: torch.Tensor | None = None, pos: torch.Tensor | None = None,
               freq: torch.Tensor | None = None, scale: float = 1.0, out: torch.Tensor | None = None) -> torch.Tensor:
    """fp32 residual rows [T, wp] (`out` or new) of the token ids, times scale; `cast` ([T, >= wp], the table's dtype) receives a copy.  freq (fp64, one per
    pair of columns): the sinusoidal vector of the positions `pos` is added."""
    T = ids.numel()
    assert ids.dtype == torch.int64 and table.stride(1) == 1
    x = torch.empty((T, wp), dtype=torch.float32, device=table.device) if out is None else out
    assert x.shape == (T, wp) and x.dtype == torch.float32 and x.is_contiguous()
    assert cast is None or (cast.shape[0] == T and cast.stride(1) == 1 and cast.dtype == table.dtype)
    assert freq is None or (freq.dtype == torch.float64 and freq.numel() >= (table.shape[1] + 1) // 2 and pos.dtype == torch.int32 and pos.numel() == T)
    _check(load_library().glm_embed_rows(_p(ids), _p(table), table.stride(0), table.shape[0], _p(pos) if freq is not None else None, _p(freq), _p(x), wp, _p(cast),
                                         cast.stride(0) if cast is not None else wp, _is_f32(table.dtype), T, table.shape[1], wp,
                                         scale, _stream()), "glm_embed_rows")
    return x


def seq_norm_taps(taps: int) -> int:
    t = load_library().glm_seq_norm_taps(taps)
    if t < 0:
        raise NotImplementedError(f"a convolution over {taps} tokens is not built")
    return t


def seq_norm(x: torch.Tensor, width: int, eps: float, y=None, g_post: torch.Tensor | None = None,
             g_pre: torch.Tensor | None = None, conv=None, meta=None, rows: torch.Tensor | None = None, act_dtype=torch.bfloat16,
             x_cast: torch.Tensor | None = None, keep_x: bool = True):
    """Between two sublayers (glm_seq_norm): returns (x_out, h).  y: the finished sublayer's output [T, wp] (bf16, fp32 or a
    PartialSum), g_post its norm's gain; g_pre the gain of the norm in front of the next sublayer (None: no h); conv =
    (bf16 weights [taps, wp], fp32 state [n, taps-1, wp]) with the step's `meta` (pos, seq_of, q_start, state_in, state_out); rows:
    gather of rows (no convolution); x_cast receives x_out in the activation dtype."""
    wp = x.shape[1]
    assert x.dtype == torch.float32 and x.is_contiguous() and wp % 8 == 0 and width <= wp
    T = rows.numel() if rows is not None else x.shape[0]
    yp, ldy, y_f32, ns, sstride = None, wp, 0, 1, 0
    if y is not None:
        t = y.part if isinstance(y, PartialSum) else y
        assert t.is_contiguous() and t.shape[-2:] == x.shape and g_post is not None and g_post.numel() == wp
        yp, ldy, y_f32 = _p(t), t.shape[-1], _is_f32(t.dtype)
        if t.dim() == 3:
            ns, sstride = t.shape[0], t.shape[1] * t.shape[2]
    x_out = torch.empty((T, wp), dtype=torch.float32, device=x.device) if (y is not None and keep_x) else None
    h = torch.empty((T, wp), dtype=act_dtype, device=x.device) if g_pre is not None else None
    w = st = pos = seq_of = q_start = s_in = s_out = None
    taps, n_state = 1, 0
    if conv is not None:
        w, st = conv
        taps, n_state = w.shape[0], st.shape[0]
        assert w.dtype == torch.bfloat16 and st.dtype == torch.float32 and w.is_contiguous() and st.is_contiguous() and w.shape[1] == wp
        assert taps == 1 or (st.shape[1:] == (taps - 1, wp) and meta is not None and rows is None)
    if taps > 1:
        pos, seq_of, q_start, s_in, s_out = meta.pos, meta.seq_of, meta.q_start, meta.state_in, meta.state_out
        assert pos.numel() == seq_of.numel() == T and q_start.numel() == s_in.numel() + 1 == s_out.numel() + 1
        if y is None:
            assert x_out is None
    for g in (g_post, g_pre):
        assert g is None or (g.dtype == torch.float32 and g.is_contiguous() and g.numel() == wp)
    assert x_cast is None or (x_cast.dtype == act_dtype and x_cast.stride(1) == 1 and x_cast.shape[0] == T)
    _check(load_library().glm_seq_norm(
        _p(x), _p(rows), wp, _p(x_out), _p(x_cast), x_cast.stride(0) if x_cast is not None else wp, yp, ldy, y_f32, ns, sstride,
        _p(g_post) if y is not None else None, _p(g_pre), _p(w) if taps > 1 else None, taps, _p(st) if taps > 1 else None, n_state,
        _p(pos), _p(seq_of), _p(q_start), _p(s_in), _p(s_out), _p(h), wp, _is_f32(act_dtype), T, width, wp, eps, _stream()),
        "glm_seq_norm")
    return (x if x_out is None else x_out), h


def latent_prepare(qc: torch.Tensor, c_off: int, heads: int, dimp: int, rank: int, norm_w: torch.Tensor, eps: float,
                   slots: torch.Tensor, cache: torch.Tensor, Ta: int, wukt: torch.Tensor, crow: torch.Tensor | None = None,
                   n_crows: int = 0):
    """Latent norm + cache store of every row of qc, q' = W_uk^T q of the first Ta rows.  Returns (q' [Ta, H, rp], c_out
    [n_crows, rp] or None)."""
    T, rp, f32 = qc.shape[0], cache.shape[-1], _is_f32(qc.dtype)
    assert qc.stride(1) == 1 and cache.is_contiguous() and cache.dtype == qc.dtype and slots.numel() == T
    assert slots.dtype == torch.int32 and norm_w.dtype == torch.float32 and norm_w.numel() == rp and wukt.shape == (heads, rp, dimp)
    assert wukt.is_contiguous() and (crow is None or (crow.dtype == torch.int32 and crow.numel() == T))
    qa = torch.empty((Ta, heads, rp), dtype=qc.dtype, device=qc.device)
    c_out = torch.empty((n_crows, rp), dtype=qc.dtype, device=qc.device) if crow is not None else None
    _check(load_library().glm_latent_prepare(
        _p(qc), qc.stride(0), c_off, T, Ta, heads, dimp, rank, rp, _p(norm_w), eps, _p(slots), _p(cache), cache.numel() // rp,
        _p(crow), _p(c_out), n_crows, _p(wukt), _p(qa) if Ta else None, f32, _stream()), "glm_latent_prepare")
    if f32 and Ta:
        q = qc[:Ta, : heads * dimp].view(Ta, heads, dimp)
        batched_gemm_f32(q.transpose(0, 1), wukt, qa.transpose(0, 1))
    return qa, c_out


def mul_f32(y: torch.Tensor, g: torch.Tensor) -> None:
    """y *= g, fp32 rows."""
    assert y.shape == g.shape and y.dtype == g.dtype == torch.float32 and y.stride(1) == g.stride(1) == 1
    _check(load_library().glm_mul_f32(_p(y), y.stride(0), _p(g), g.stride(0), y.shape[0], y.shape[1], _stream()), "glm_mul_f32")


def rope_pairs(pos: torch.Tensor, freq: torch.Tensor, mscale: float, pairs: int) -> torch.Tensor:
    """cos and sin [T, pairs, 2] of pos x freq (fp64) times mscale; pairs behind the last frequency do not turn."""
    assert pos.dtype == torch.int32 and freq.dtype == torch.float64 and freq.numel() <= pairs
    cs = torch.empty((pos.numel(), pairs, 2), dtype=torch.float32, device=pos.device)
    _check(load_library().glm_rope_pairs(_p(pos), _p(freq), freq.numel(), mscale, _p(cs), pos.numel(), pairs, _stream()), "glm_rope_pairs")
    return cs


def latent_rows(x: torch.Tensor, c_off: int, rank: int, norm_w: torch.Tensor, cs: torch.Tensor | None, eps: float, slots: torch.Tensor, cache: torch.Tensor,
                query: tuple | None = None, crow: torch.Tensor | None = None, n_crows: int = 0):
    """In front of the query projection: rows x hold the raw latent (and the rotated key part behind it) at c_off; norm, rotation and cache
    store; query = (column, rank, gain) of the queries' latent.  Returns (query latent [T, round8(rank)], c_out [n_crows, cache columns])."""
    T, rc, rp = x.shape[0], cache.shape[-1], round8(rank)
    assert x.stride(1) == 1 and cache.is_contiguous() and cache.dtype == x.dtype and slots.numel() == T and slots.dtype == torch.int32
    assert norm_w.dtype == torch.float32 and norm_w.numel() == rp and (crow is None or (crow.dtype == torch.int32 and crow.numel() == T))
    assert rc == rp or (cs.dtype == torch.float32 and cs.is_contiguous() and cs.numel() == T * (rc - rp))
    c_out = torch.empty((n_crows, rc), dtype=x.dtype, device=x.device) if crow is not None else None
    q_off, q_rank, q_gain = query or (0, 0, None)
    assert q_gain is None or (q_gain.dtype == torch.float32 and q_gain.numel() == round8(q_rank))
    cq = torch.empty((T, round8(q_rank)), dtype=x.dtype, device=x.device) if query else None
    _check(load_library().glm_latent_rows(
        _p(x), x.stride(0), c_off, rank, rp, rc - rp, _p(norm_w), _p(cs), eps, _p(slots), _p(cache), cache.numel() // rc, _p(crow), _p(c_out), n_crows, q_off, q_rank,
        round8(q_rank), _p(q_gain), _p(cq), round8(q_rank), T, _is_f32(x.dtype), _stream()), "glm_latent_rows")
    return cq, c_out


def latent_absorb(q: torch.Tensor, heads: int, dimp: int, cs: torch.Tensor | None, wukt: torch.Tensor, rotp: int) -> torch.Tensor:
    """W_uk^T q | rotated rest for every row and head of q ([Ta, heads * (dimp + rotp)])."""
    Ta, rp = q.shape[0], wukt.shape[1]
    assert q.shape[1] == heads * (dimp + rotp) and q.stride(1) == 1 and wukt.shape == (heads, rp, dimp) and wukt.is_contiguous()
    assert rotp == 0 or (cs.dtype == torch.float32 and cs.is_contiguous() and cs.numel() >= Ta * rotp)
    qa = torch.empty((Ta, heads, rp + rotp), dtype=q.dtype, device=q.device)
    f32 = _is_f32(q.dtype)
    _check(load_library().glm_latent_absorb(_p(q), q.stride(0), Ta, heads, dimp, rp, rotp, _p(cs), _p(wukt), _p(qa), f32, _stream()), "glm_latent_absorb")
    if f32 and Ta:
        qh = q.as_strided((Ta, heads, dimp), (q.stride(0), dimp + rotp, 1), q.storage_offset())
        batched_gemm_f32(qh.transpose(0, 1), wukt, qa[..., :rp].transpose(0, 1))
    return qa


def latent_gather(cache: torch.Tensor, slots: torch.Tensor, rows: torch.Tensor, out: torch.Tensor) -> None:
    """out[rows[i]] = cache row slots[i]."""
    rp = cache.shape[-1]
    assert out.shape[1] == rp and out.dtype == cache.dtype and out.is_contiguous() and cache.is_contiguous()
    assert slots.dtype == rows.dtype == torch.int32 and slots.numel() == rows.numel()
    _check(load_library().glm_latent_gather(_p(cache), cache.numel() // rp, _p(slots), _p(rows), slots.numel(), _p(out), out.shape[0],
                                            rp * cache.element_size(), _stream()), "glm_latent_gather")


def latent_attn_max_rows(rp: int) -> int:
    n = load_library().glm_latent_attn_max_rows(rp)
    if n <= 0:
        raise NotImplementedError(f"a latent of {rp} columns is not built")
    return n


def latent_tokens_per_tile(rp: int, heads: int) -> int:
    """Query tokens of one sequence that share a workgroup's pass over the cache."""
    rows = latent_attn_max_rows(rp)
    groups = -(-heads // rows)
    return max(1, rows // -(-heads // groups))


def latent_attn(qa: torch.Tensor, cache: torch.Tensor, tile_tok: torch.Tensor, tile_n: torch.Tensor, tokens_per_tile: int,
                pos: torch.Tensor, seq_of: torch.Tensor, block_tables: torch.Tensor, window: int, scale: float,
                sink: torch.Tensor, wuv: torch.Tensor, out: torch.Tensor, num_splits: int = 0, gate: torch.Tensor | None = None) -> None:
    """Absorbed attention of the rows qa [Ta, H, rp] over the paged rows (all rp columns make the scores, the first wuv.shape[2] of
    them are the latent), then W_uv and the gate rows ([T, H * vdimp], factors): writes out[:Ta] ([T, H * vdimp])."""
    Ta, H, rp = qa.shape
    n_blocks, bs, _ = cache.shape
    vdimp, vp = wuv.shape[1:]
    if Ta == 0:
        return
    assert qa.is_contiguous() and cache.is_contiguous() and cache.dtype == qa.dtype and wuv.is_contiguous()
    assert wuv.shape[0] == H and vp <= rp == cache.shape[2] and sink.dtype == torch.float32 and sink.numel() == H and block_tables.stride(1) == 1
    for t in (tile_tok, tile_n, pos, seq_of, block_tables):
        assert t.dtype == torch.int32
    assert pos.numel() >= Ta and seq_of.numel() >= Ta and out.stride(1) == 1 and out.shape[0] >= Ta and out.shape[1] == H * vdimp
    assert gate is None or (gate.dtype == out.dtype and gate.stride(1) == 1 and gate.shape[0] >= Ta and gate.shape[1] == H * vdimp)
    lib, f32 = load_library(), _is_f32(qa.dtype)
    part_o = part_ml = None
    ns = 1
    if not f32:
        # as many (tile, head group, KV split) workgroups as the chip has CUs, at least two 64-key tiles per split
        rows = latent_attn_max_rows(rp)
        wgs = tile_tok.numel() * -(-H // rows)
        keys = min(window + tokens_per_tile, block_tables.shape[1] * bs)
        # (and no more keys per split than a workgroup's slice of the block table covers)
        ns = num_splits or max(1, min(64, 256 // max(1, wgs), -(-keys // 128)), -(-keys // (900 * bs)))
    ctx = torch.empty((Ta, H, vp), dtype=qa.dtype, device=qa.device)
    if ns > 1:
        part_o = torch.empty((Ta * H, ns, vp), dtype=torch.float32, device=qa.device)
        part_ml = torch.empty((Ta * H, ns, 2), dtype=torch.float32, device=qa.device)
    _check(lib.glm_latent_attn(_p(qa), _p(cache), n_blocks, bs, _p(tile_tok), _p(tile_n), tile_tok.numel(), tokens_per_tile, _p(pos),
                               _p(seq_of), _p(block_tables), block_tables.stride(0), Ta, H, rp, vp, window, scale, _p(sink), ns,
                               _p(ctx), _p(part_o), _p(part_ml), f32, _stream()), "glm_latent_attn")
    if f32:
        batched_gemm_f32(ctx.transpose(0, 1), wuv, out[:Ta].view(Ta, H, vdimp).transpose(0, 1))
        if gate is not None:
            mul_f32(out[:Ta], gate[:Ta])
        return
    if ns > 1:
        _check(lib.glm_attn_merge(_p(part_o), _p(part_ml), _p(sink), ns, _p(ctx), H * vp, Ta, H, vp, None, _stream()), "glm_attn_merge")
    _check(lib.glm_latent_up(_p(ctx), _p(wuv), _p(out), _p(gate), gate.stride(0) if gate is not None else 0, out.stride(0), Ta, H, vdimp, vp, _stream()),
           "glm_latent_up")


WINDOW_ATTN_MAX_DIM = 256  # head sizes of glm_window_attn_prefill


def window_attn_prefill(q: torch.Tensor, k: torch.Tensor, v: torch.Tensor, out: torch.Tensor, q_start: torch.Tensor,
                        k_start: torch.Tensor, tile_seq: torch.Tensor, tile_off: torch.Tensor, heads: int, dk: int, dv: int,
                        window: int, scale: float, sink: torch.Tensor, kr: torch.Tensor | None = None, cs: torch.Tensor | None = None,
                        gate: torch.Tensor | None = None) -> None:
    """q, out: rows of the step's long portions (views with free row pitch); k, v: expanded rows, see the header.  kr [Tk, rotp]: the
    rotated key part that all heads share, the last of dk columns (k holds the others), cs the rotation of these query columns."""
    _bf16(q, "q"); _bf16(k, "k"); _bf16(v, "v"); _bf16(out, "out")
    rotp = kr.shape[1] if kr is not None else 0
    assert q.shape[1] == heads * dk and k.shape[1] == heads * (dk - rotp) and v.shape[1] == out.shape[1] == heads * dv and k.stride(0) == v.stride(0)
    assert k.shape[0] == v.shape[0] and out.shape[0] == q.shape[0] and sink.dtype == torch.float32 and sink.numel() == heads
    for t in (q_start, k_start, tile_seq, tile_off):
        assert t.dtype == torch.int32
    S = q_start.numel() - 1
    assert k_start.numel() == S + 1 and tile_seq.numel() == tile_off.numel()
    if rotp:
        _bf16(kr, "kr")
        assert kr.shape[0] == k.shape[0] and kr.stride(1) == 1 and cs.dtype == torch.float32 and cs.is_contiguous() and cs.numel() == q.shape[0] * rotp
    if gate is not None:
        _bf16(gate, "gate")
        assert gate.shape == out.shape and gate.stride(1) == 1
    _check(load_library().glm_window_attn_prefill(
        _p(q), q.stride(0), _p(k), _p(v), k.stride(0), _p(kr), kr.stride(0) if rotp else 0, rotp, _p(cs), _p(gate), gate.stride(0) if gate is not None else 0,
        _p(out), out.stride(0), _p(q_start), _p(k_start), _p(tile_seq), _p(tile_off),
        tile_seq.numel(), S, q.shape[0], k.shape[0], heads, dk, dv, window, scale, _p(sink), _stream()), "glm_window_attn_prefill")


# ------------------------------------------------------------------------------------------
# decoders whose residual is several streams, with grouped-head attention over chunks and a gated matrix memory
GLU_SLOPE = 1.702


def gated_glu(x: torch.Tensor, w: torch.Tensor, limit: float, slope: float = GLU_SLOPE) -> torch.Tensor:
    """Clamped gated unit of x @ w.T, w [2 N, K] rows gate | up -> [M, N]."""
    M, K = x.shape
    N = w.shape[0] // 2
    assert w.shape == (2 * N, K) and w.dtype == x.dtype and x.stride(1) == 1 and w.stride(1) == 1
    y = torch.empty((M, N), dtype=x.dtype, device=x.device)
    if _is_f32(x.dtype):
        z = linear_act(x, w)
        _check(load_library().glm_glu_f32(_p(z), z.stride(0), _p(y), N, M, N, limit, slope, _stream()), "glm_glu_f32")
    else:
        _check(load_library().glm_gemm_bf16_glu(_p(x), x.stride(0), _p(w), w.stride(0), _p(y), N, M, N, K, limit, slope, _stream()),
               "glm_gemm_bf16_glu")
    return y


def stream_norm(x: torch.Tensor, streams: int, width: int, eps: float, y: torch.Tensor | None = None, y_scale: torch.Tensor | None = None,
                mix_out: torch.Tensor | None = None, w_in: torch.Tensor | None = None, gain: float = 1.0, shift: torch.Tensor | None = None,
                state: torch.Tensor | None = None, meta=None, rows: torch.Tensor | None = None, act_dtype=torch.bfloat16, keep_x: bool = True):
    """Between two sublayers (glm_stream_norm): returns (streams, h).  x: [T, wp] (all streams are that row) or [T, streams, wp], fp32;
    y: the finished sublayer's output [T, wp]; w_in: weights of the next sublayer's input (None: no h); shift + state: token shift with
    the step's `meta`; rows: gather of rows (streams are not kept)."""
    wp = x.shape[-1]
    assert x.dtype == torch.float32 and x.is_contiguous() and wp % 8 == 0 and width <= wp and (x.dim() == 2 or x.shape[1] == streams)
    T = rows.numel() if rows is not None else x.shape[0]
    for t, n in ((y_scale, wp), (mix_out, streams * (streams + 1)), (w_in, streams), (shift, wp)):
        assert t is None or (t.dtype == torch.float32 and t.is_contiguous() and t.numel() == n)
    assert y is None or (y.stride(1) == 1 and y.shape == (x.shape[0], wp) and y_scale is not None and mix_out is not None)
    x_out = torch.empty((T, streams, wp), dtype=torch.float32, device=x.device) if (y is not None and keep_x and rows is None) else None
    h = torch.empty((T, wp), dtype=act_dtype, device=x.device) if w_in is not None else None
    pos = seq_of = q_start = s_in = s_out = None
    if shift is not None:
        pos, seq_of, q_start, s_in, s_out = meta.pos, meta.seq_of, meta.q_start, meta.state_in, meta.state_out
        assert pos.numel() == seq_of.numel() == T and q_start.numel() == s_in.numel() + 1 == s_out.numel() + 1
        assert state.dtype == torch.float32 and state.is_contiguous() and state.shape[1] == wp
    if x_out is not None or h is not None:
        _check(load_library().glm_stream_norm(
            _p(x), x.stride(0), x.stride(1) if x.dim() == 3 else 0, _p(rows), _p(x_out), _p(y), y.stride(0) if y is not None else wp,
            _is_f32(y.dtype) if y is not None else 0, _p(y_scale), _p(mix_out), _p(w_in), gain, _p(shift), _p(state) if shift is not None else None,
            state.shape[0] if shift is not None else 0, _p(pos), _p(seq_of), _p(q_start), _p(s_in), _p(s_out), _p(h), wp, _is_f32(act_dtype), T,
            streams, width, wp, eps, _stream()), "glm_stream_norm")
    return (x if x_out is None else x_out), h


GROUP_ATTN_MAX_DIM = 256   # head sizes of glm_group_attn_prefill / _decode
GROUP_ATTN_ROWS = 16       # (token, head) rows a decode workgroup takes


def group_kv_store(src: torch.Tensor, k_off: int, v_off: int, slots: torch.Tensor, k_cache: torch.Tensor, v_cache: torch.Tensor) -> None:
    """Key and value columns of projection rows -> their cache rows.  Caches [blocks, G, block size, head size]."""
    n, G, bs, dk = k_cache.shape
    assert v_cache.shape[:3] == (n, G, bs) and k_cache.dtype == v_cache.dtype == src.dtype and k_cache.is_contiguous() and v_cache.is_contiguous()
    assert slots.dtype == torch.int32 and slots.numel() == src.shape[0] and src.stride(1) == 1
    _check(load_library().glm_group_kv_store(_p(src), src.stride(0), k_off, v_off, _is_f32(src.dtype), _p(slots), src.shape[0], _p(k_cache), _p(v_cache),
                                             n * bs, bs, G, dk, v_cache.shape[3], _stream()), "glm_group_kv_store")


class _GroupForm(ctypes.Structure):
    _fields_ = [("window", c_int), ("chunk", c_int), ("scale", c_float), ("slope", c_void_p), ("sink", c_void_p), ("cap", c_float), ("maps", c_int),
                ("lam", c_float), ("post", c_float), ("eps", c_float), ("vn", c_int), ("sigmoid", c_int), ("bias", c_void_p), ("kscale", c_void_p),
                ("gate", c_void_p), ("ldg", c_int64), ("gate_cols", c_int)]


@dataclass
class GroupParts:
    """What an attention with grouped heads may have beside window, chunk, slope and sink (include/glm4moe_hip.h, glm_group_form)."""
    cap: float = 0.0                       # soft cap on the scores
    maps: int = 1                          # 2: two queries / keys per head side by side, output post d / rms(d), d = o_1 - lam o_2, over vn columns
    lam: float = 0.0
    post: float = 1.0
    eps: float = 0.0
    vn: int = 0
    sigmoid: bool = False                  # weights sigmoid(score + bias), not normalised
    bias: torch.Tensor | None = None       # fp32 [heads]
    kscale: torch.Tensor | None = None     # fp32 [blocks, block size]: the keys are the values, their products times this
    gate: torch.Tensor | None = None       # factors of the output, a row per row of q; [T, heads] or, gate_cols, [T, heads * value columns]
    gate_cols: bool = False


NO_PARTS = GroupParts()


def _group_form(window, chunk, scale, slope, sink, p: GroupParts, q, k_cache, v_cache, heads: int) -> _GroupForm:
    assert p.bias is None or (p.bias.dtype == torch.float32 and p.bias.numel() == heads)
    assert p.kscale is None or (p.kscale.dtype == torch.float32 and p.kscale.is_contiguous() and p.kscale.numel() == k_cache.shape[0] * k_cache.shape[2])
    assert p.gate is None or (p.gate.dtype == q.dtype and p.gate.stride(1) == 1 and p.gate.shape[0] >= q.shape[0]
                              and p.gate.shape[1] >= (heads * v_cache.shape[3] if p.gate_cols else heads))
    return _GroupForm(window, chunk, scale, _p(slope), _p(sink), p.cap, p.maps, p.lam, p.post, p.eps, p.vn, int(p.sigmoid), _p(p.bias), _p(p.kscale), _p(p.gate),
                      p.gate.stride(0) if p.gate is not None else 0, int(p.gate_cols))


def _group_shape(q, k_cache, v_cache, out, heads, slope, sink):
    n, G, bs, dk = k_cache.shape
    dv = v_cache.shape[3]
    assert v_cache.shape[:3] == (n, G, bs) and k_cache.dtype == v_cache.dtype == q.dtype == out.dtype and k_cache.is_contiguous() and v_cache.is_contiguous()
    assert q.shape[1] == heads * dk and out.shape[1] == heads * dv and q.stride(1) == out.stride(1) == 1 and out.shape[0] >= q.shape[0]
    for t in (slope, sink):
        assert t is None or (t.dtype == torch.float32 and t.numel() == heads)
    return n, G, bs, dk, dv


def group_attn_tile_rows(heads: int, kv_heads: int, maps: int = 1) -> int:
    """Query rows per workgroup of glm_group_attn_prefill: two heads of a group share a tile where they pair up, and so do two maps."""
    return 64 if maps == 2 or (heads // kv_heads) % 2 == 0 else 128


def group_attn_rows(maps: int = 1) -> int:
    """(token, head) rows a workgroup of glm_group_attn_decode takes."""
    return GROUP_ATTN_ROWS // maps


def group_attn_prefill(q: torch.Tensor, k_cache: torch.Tensor, v_cache: torch.Tensor, block_tables: torch.Tensor, seq0: int, q_start: torch.Tensor,
                       pos: torch.Tensor, tile_seq: torch.Tensor, tile_off: torch.Tensor, heads: int, window: int, chunk: int, scale: float, slope, sink,
                       out: torch.Tensor, parts: GroupParts = NO_PARTS) -> None:
    """Long portions (rows of q, q_start relative to them) over the paged caches; block table of portion s in row seq0 + s; tiles of
    group_attn_tile_rows rows."""
    n, G, bs, dk, dv = _group_shape(q, k_cache, v_cache, out, heads, slope, sink)
    for t in (block_tables, q_start, pos, tile_seq, tile_off):
        assert t.dtype == torch.int32
    assert pos.numel() == q.shape[0] and tile_seq.numel() == tile_off.numel() and block_tables.shape[0] >= seq0 + q_start.numel() - 1
    form = _group_form(window, chunk, scale, slope, sink, parts, q, k_cache, v_cache, heads)
    _check(load_library().glm_group_attn_prefill(
        _p(q), q.stride(0), _p(k_cache), _p(v_cache), n, bs, _p(block_tables), block_tables.stride(0), seq0, _p(q_start), _p(pos), _p(tile_seq), _p(tile_off),
        tile_seq.numel(), group_attn_tile_rows(heads, G, parts.maps), heads, G, dk, dv, ctypes.byref(form), _p(out), out.stride(0), _stream()),
        "glm_group_attn_prefill")


def group_attn_splits(tiles: int, tokens_per_tile: int, heads: int, kv_heads: int, keys: int, maps: int = 1) -> int:
    """KV splits of a decode launch: about one workgroup per CU, at least 128 keys each."""
    wgs = tiles * kv_heads * -(-tokens_per_tile * (heads // kv_heads) // group_attn_rows(maps))
    return max(1, min(64, 256 // max(1, wgs), -(-keys // 128)))


def group_attn_decode(q: torch.Tensor, k_cache: torch.Tensor, v_cache: torch.Tensor, block_tables: torch.Tensor, pos: torch.Tensor, seq_of: torch.Tensor,
                      tile_tok: torch.Tensor, tile_n: torch.Tensor, tokens_per_tile: int, heads: int, window: int, chunk: int, scale: float, slope, sink,
                      out: torch.Tensor, num_splits: int = 0, new=None, parts: GroupParts = NO_PARTS) -> None:
    """Decoded tokens and short portions (the rows of q) over the paged caches; out is written row by row from its first.  new =
    (keys, values, q_start, slots): the rows' own keys and values are taken from there and stored to their cache rows."""
    n, G, bs, dk, dv = _group_shape(q, k_cache, v_cache, out, heads, slope, sink)
    T = q.shape[0]
    if T == 0:
        return
    for t in (block_tables, pos, seq_of, tile_tok, tile_n):
        assert t.dtype == torch.int32
    assert pos.numel() >= T and seq_of.numel() >= T and tile_tok.numel() == tile_n.numel()
    keys = block_tables.shape[1] * bs
    for w in (window, chunk):
        keys = min(keys, w + tokens_per_tile) if w else keys
    ns = num_splits or group_attn_splits(tile_tok.numel(), tokens_per_tile, heads, G, keys, parts.maps)
    part_o = part_ml = None
    if ns > 1 or parts.maps > 1:
        part_o = torch.empty((T * heads * parts.maps, ns, dv), dtype=torch.float32, device=q.device)
        part_ml = torch.empty((T * heads * parts.maps, ns, 2), dtype=torch.float32, device=q.device)
    kn = vn = q_start = slots = None
    if new is not None:
        kn, vn, q_start, slots = new
        assert kn.shape == (T, G * dk) and vn.shape == (T, G * dv) and kn.stride() == vn.stride() and kn.stride(1) == 1 and kn.dtype == vn.dtype == q.dtype
        assert q_start.dtype == slots.dtype == torch.int32 and slots.numel() >= T
    lib, form = load_library(), _group_form(window, chunk, scale, slope, sink, parts, q, k_cache, v_cache, heads)
    _check(lib.glm_group_attn_decode(
        _p(q), q.stride(0), _p(k_cache), _p(v_cache), n, bs, _p(block_tables), block_tables.stride(0), _p(pos), _p(seq_of), _p(tile_tok), _p(tile_n),
        tile_tok.numel(), tokens_per_tile, heads, G, dk, dv, ctypes.byref(form), _p(kn), _p(vn),
        kn.stride(0) if kn is not None else 0, _p(q_start), _p(slots), _p(out), out.stride(0), ns, _p(part_o), _p(part_ml),
        _stream()), "glm_group_attn_decode")
    if part_o is not None:
        _check(lib.glm_attn_merge(_p(part_o), _p(part_ml), _p(sink), ns, _p(out), out.stride(0), T, heads, dv, ctypes.byref(form), _stream()), "glm_attn_merge")


def group_attn_plain(q: torch.Tensor, k_cache: torch.Tensor, v_cache: torch.Tensor, block_tables: torch.Tensor, pos: torch.Tensor, seq_of: torch.Tensor,
                     heads: int, window: int, chunk: int, scale: float, slope, sink, out: torch.Tensor, parts: GroupParts = NO_PARTS) -> None:
    """The same for any head size, in fp32 arithmetic whatever the dtype of the rows and caches."""
    n, G, bs, dk, dv = _group_shape(q, k_cache, v_cache, out, heads, slope, sink)
    for t in (block_tables, pos, seq_of):
        assert t.dtype == torch.int32
    assert pos.numel() >= q.shape[0] and seq_of.numel() >= q.shape[0]
    form = _group_form(window, chunk, scale, slope, sink, parts, q, k_cache, v_cache, heads)
    _check(load_library().glm_group_attn_plain(
        _p(q), q.stride(0), _p(k_cache), _p(v_cache), n, bs, _p(block_tables), block_tables.stride(0), _p(pos), _p(seq_of), q.shape[0], heads, G, dk, dv,
        ctypes.byref(form), _p(out), out.stride(0), _is_f32(q.dtype), _stream()), "glm_group_attn_plain")


def group_rotate_store(x: torch.Tensor, q_off: int, k_off: int, v_off: int, heads: int, maps: int, dims: int, cs: torch.Tensor, slots: torch.Tensor,
                       k_cache: torch.Tensor, v_cache: torch.Tensor) -> None:
    """Rows of a projection: queries at q_off are rotated in place (column i < dims / 2 of a head's map with column i + dims / 2, table cs of
    rope_pairs), rotated keys at k_off and the values at v_off go to their cache rows [blocks, G, block size, maps * columns | value columns]."""
    n, G, bs, dk = k_cache.shape
    dv, T = v_cache.shape[3], x.shape[0]
    assert v_cache.shape[:3] == (n, G, bs) and k_cache.dtype == v_cache.dtype == x.dtype and k_cache.is_contiguous() and v_cache.is_contiguous() and x.stride(1) == 1
    assert slots.dtype == torch.int32 and slots.numel() == T and cs.dtype == torch.float32 and cs.shape[0] == T and cs.is_contiguous() and dk % maps == 0
    assert max(q_off + heads * dk, k_off + G * dk, v_off + G * dv) <= x.shape[1]
    _check(load_library().glm_group_rotate_store(_p(x), x.stride(0), q_off, k_off, v_off, _is_f32(x.dtype), heads, G, maps, dk // maps, dv, dims, _p(cs), cs.shape[1],
                                                 _p(slots), T, _p(k_cache), _p(v_cache), n * bs, bs, _stream()), "glm_group_rotate_store")


def group_norm_store(x: torch.Tensor, q_off: int, k_off: int, gain: torch.Tensor, q_true: int, k_cols: int, k_true: int, first: int, eps: float, pos: torch.Tensor,
                     slots: torch.Tensor, cache: torch.Tensor, kscale: torch.Tensor, temperature: tuple = (0.0, 0)) -> None:
    """Rows of a projection whose keys are the values: queries at q_off (as many columns as gain, q_true of them true) <- q / rms(q) gain, times
    1 + coef ln(floor((p + 1) / every) + 1) with temperature = (coef, every); key heads `first`.. of the k_cols columns at k_off go to the
    cache as they are, 1 / rms of all of them (k_true true ones) to kscale."""
    n, G, bs, dm = cache.shape
    T = x.shape[0]
    assert cache.dtype == x.dtype and cache.is_contiguous() and x.stride(1) == 1 and gain.dtype == torch.float32 and gain.is_contiguous()
    assert kscale.dtype == torch.float32 and kscale.is_contiguous() and kscale.numel() == n * bs
    assert pos.dtype == slots.dtype == torch.int32 and pos.numel() == slots.numel() == T and max(q_off + gain.numel(), k_off + k_cols) <= x.shape[1]
    _check(load_library().glm_group_norm_store(_p(x), x.stride(0), q_off, gain.numel(), q_true, k_off, k_cols, k_true, _is_f32(x.dtype), _p(gain), dm, first, G, eps,
                                               *temperature, _p(pos), _p(slots), T, _p(cache), _p(kscale), n * bs, bs, _stream()), "glm_group_norm_store")


def residual_norm(x: torch.Tensor | None, width: int, wp: int, eps: float, y=None, embed: tuple | None = None, g: torch.Tensor | None = None, rows: torch.Tensor | None = None,
                  act_dtype=torch.bfloat16, keep_x: bool = True):
    """Between two layers (glm_residual_norm): returns (x_out, h) with x_out = x + y + rows of an embedding table and h its norm with gain g (None: no
    h).  y: [T, wp] in bf16, fp32 or a PartialSum; embed: (ids, table); rows: gather of rows."""
    T = rows.numel() if rows is not None else (x.shape[0] if x is not None else embed[0].numel())
    dev = embed[1].device if x is None else x.device
    assert x is None or (x.dtype == torch.float32 and x.is_contiguous() and x.shape[1] == wp)
    yp, ldy, y_f32, ns, sstride = None, wp, 0, 1, 0
    if y is not None:
        t = y.part if isinstance(y, PartialSum) else y
        assert t.shape[-1] == wp and t.is_contiguous() and (x is None or t.shape[-2] == x.shape[0])
        yp, y_f32 = _p(t), _is_f32(t.dtype)
        if isinstance(y, PartialSum):
            ns, sstride = t.shape[0], t.shape[1] * t.shape[2]
    ids, table = embed or (None, None)
    if embed is not None:
        assert ids.dtype == torch.int64 and ids.is_contiguous() and table.stride(1) == 1 and table.shape[1] >= wp and table.dtype == act_dtype
        assert x is None or ids.numel() == x.shape[0]
    assert rows is None or rows.dtype == torch.int32
    assert g is None or (g.dtype == torch.float32 and g.numel() == wp)
    x_out = torch.empty((T, wp), dtype=torch.float32, device=dev) if keep_x else None
    h = torch.empty((T, wp), dtype=act_dtype, device=dev) if g is not None else None
    _check(load_library().glm_residual_norm(_p(x), _p(rows), yp, ldy, y_f32, ns, sstride, _p(table), table.stride(0) if table is not None else wp,
                                            table.shape[0] if table is not None else 0, _p(ids), _p(x_out), _p(g), _p(h), wp, _is_f32(act_dtype), T, width, wp, eps, _stream()),
           "glm_residual_norm")
    return x_out, h


MEMORY_CHUNK_MAX_DIM = 256   # key size of glm_memory_chunkwise


def _memory_state(state, heads, dimp, vdimp):
    S, n, m = state
    assert S.shape[1:] == (heads, dimp, vdimp) and n.shape == (S.shape[0], heads, dimp) and m.shape == (S.shape[0], heads)
    for t in state:
        assert t.dtype == torch.float32 and t.is_contiguous()
    return S, n, m


def memory_recurrent(x: torch.Tensor, hrow: torch.Tensor, wif: torch.Tensor, bif: torch.Tensor, norm: torch.Tensor, y: torch.Tensor, state, pos, q_start, state_in,
                     state_out, heads: int, dim: int, vdim: int, cap: float, eps: float) -> None:
    """Gated matrix memory token by token, gates and output norm included: rows x = q | k | v | g (heads padded to multiples of 8) -> y."""
    dimp, vdimp = round8(dim), round8(vdim)
    S, n, m = _memory_state(state, heads, dimp, vdimp)
    kd, vd = heads * dimp, heads * vdimp
    assert x.shape[1] >= 2 * kd + 2 * vd and x.stride(1) == hrow.stride(1) == wif.stride(1) == y.stride(1) == 1 and x.dtype == hrow.dtype == wif.dtype == y.dtype
    assert wif.shape == (2 * heads, hrow.shape[1]) and bif.numel() == 2 * heads and norm.numel() == vd and bif.dtype == norm.dtype == torch.float32
    for t in (pos, q_start, state_in, state_out):
        assert t.dtype == torch.int32
    seqs = q_start.numel() - 1
    assert state_in.numel() >= seqs and state_out.numel() >= seqs
    _check(load_library().glm_memory_recurrent(
        _p(x), x.stride(0), kd, 2 * kd, 2 * kd + vd, _p(hrow), hrow.stride(0), _p(wif), wif.stride(0), hrow.shape[1], _p(bif), _p(norm), _p(y), y.stride(0), _p(S), _p(n),
        _p(m), S.shape[0], _p(pos), _p(q_start), _p(state_in), _p(state_out), seqs, heads, dim, dimp, vdim, vdimp, cap, eps, _is_f32(x.dtype), _stream()),
        "glm_memory_recurrent")


def memory_chunkwise(x: torch.Tensor, hrow: torch.Tensor, wif: torch.Tensor, bif: torch.Tensor, norm: torch.Tensor, y: torch.Tensor, state, pos, q_start, state_in,
                     state_out, tile_seq, tile_off, heads: int, dim: int, vdim: int, cap: float, eps: float) -> None:
    """The same for long portions (bf16), 64 tokens at a time; q_start, pos and the 128-row tiles relative to the rows of x."""
    _bf16(x, "x"); _bf16(y, "y"); _bf16(hrow, "hrow"); _bf16(wif, "wif")
    dimp, vdimp = round8(dim), round8(vdim)
    S, n, m = _memory_state(state, heads, dimp, vdimp)
    kd, vd, T = heads * dimp, heads * vdimp, x.shape[0]
    assert x.shape[1] >= 2 * kd + 2 * vd and hrow.shape[0] == T and x.stride(1) == y.stride(1) == hrow.stride(1) == wif.stride(1) == 1
    assert wif.shape == (2 * heads, hrow.shape[1]) and bif.numel() == 2 * heads and norm.numel() == vd and bif.dtype == norm.dtype == torch.float32
    for t in (pos, q_start, state_in, state_out, tile_seq, tile_off):
        assert t.dtype == torch.int32
    seqs = q_start.numel() - 1
    assert state_in.numel() >= seqs and state_out.numel() >= seqs and pos.numel() == T and tile_seq.numel() == tile_off.numel()
    o = torch.empty((T, vd), dtype=x.dtype, device=x.device)
    gates = torch.empty((3, heads, T), dtype=torch.float32, device=x.device)
    lib = load_library()
    _check(lib.glm_memory_gates(_p(hrow), hrow.stride(0), _p(wif), wif.stride(0), hrow.shape[1], _p(bif), _p(gates), T, _p(q_start), _p(tile_seq), _p(tile_off),
                                tile_seq.numel(), heads, cap, _stream()), "glm_memory_gates")
    _check(lib.glm_memory_chunkwise(_p(x), x.stride(0), kd, 2 * kd, _p(gates), T, _p(o), vd, _p(S), _p(n), _p(m), S.shape[0], _p(pos), _p(q_start),
                                    _p(state_in), _p(state_out), seqs, heads, dim, dimp, vdimp, _stream()), "glm_memory_chunkwise")
    _check(lib.glm_memory_output(_p(o), vd, _p(x[:, 2 * kd + vd:]), x.stride(0), _p(norm), _p(y), y.stride(0), T, heads, vdim, vdimp, eps, _stream()),
           "glm_memory_output")


def linear_recurrent(x: torch.Tensor, decay: torch.Tensor, S: torch.Tensor, pos, q_start, state_in, state_out, heads: int, dimp: int, vdimp: int) -> torch.Tensor:
    """Linear memory (constant decay) token by token: rows x = q | k | v | ... -> fp32 rows o [T, heads * vdimp] in front of their norm."""
    kd, T = heads * dimp, x.shape[0]
    assert S.shape[1:] == (heads, dimp, vdimp) and S.dtype == torch.float32 and S.is_contiguous() and decay.dtype == torch.float32 and decay.numel() == heads
    assert x.shape[1] >= 2 * kd + heads * vdimp and x.stride(1) == 1
    for t in (pos, q_start, state_in, state_out):
        assert t.dtype == torch.int32
    seqs = q_start.numel() - 1
    assert state_in.numel() >= seqs and state_out.numel() >= seqs
    o = torch.empty((T, heads * vdimp), dtype=torch.float32, device=x.device)
    _check(load_library().glm_linear_recurrent(
        _p(x), x.stride(0), kd, 2 * kd, _p(decay), _p(o), heads * vdimp, _p(S), S.shape[0], _p(pos), _p(q_start), _p(state_in), _p(state_out), seqs, heads, dimp, vdimp,
        _is_f32(x.dtype), _stream()), "glm_linear_recurrent")
    return o


def linear_chunkwise(x: torch.Tensor, powers: torch.Tensor, S: torch.Tensor, pos, q_start, state_in, state_out, heads: int, dimp: int, vdimp: int) -> torch.Tensor:
    """The same for long portions (bf16), 64 tokens at a time; powers [heads, 65] = decay^j; q_start and pos relative to the rows of x."""
    _bf16(x, "x")
    kd, T = heads * dimp, x.shape[0]
    assert S.shape[1:] == (heads, dimp, vdimp) and S.dtype == torch.float32 and S.is_contiguous() and powers.dtype == torch.float32 and powers.shape == (heads, 65) and powers.is_contiguous()
    assert x.shape[1] >= 2 * kd + heads * vdimp and x.stride(1) == 1 and pos.numel() == T
    for t in (pos, q_start, state_in, state_out):
        assert t.dtype == torch.int32
    seqs = q_start.numel() - 1
    assert state_in.numel() >= seqs and state_out.numel() >= seqs
    o = torch.empty((T, heads * vdimp), dtype=x.dtype, device=x.device)
    _check(load_library().glm_linear_chunkwise(
        _p(x), x.stride(0), kd, 2 * kd, _p(powers), T, _p(o), heads * vdimp, _p(S), S.shape[0], _p(pos), _p(q_start), _p(state_in), _p(state_out), seqs, heads, dimp, vdimp,
        _stream()), "glm_linear_chunkwise")
    return o


def row_norm_gate(o: torch.Tensor, gate: torch.Tensor, norm: torch.Tensor, n: int, eps: float, y: torch.Tensor) -> None:
    """y = o / rms(o) . norm . gate per row; n of the columns are true, the others zeros."""
    T, np_ = o.shape
    assert gate.shape == y.shape == o.shape and gate.dtype == y.dtype and o.stride(1) == gate.stride(1) == y.stride(1) == 1 and norm.dtype == torch.float32 and norm.numel() == np_
    _check(load_library().glm_row_norm_gate(_p(o), o.stride(0), _is_f32(o.dtype), _p(gate), gate.stride(0), _p(norm), _p(y), y.stride(0), T, n, np_, eps, _is_f32(y.dtype), _stream()),
           "glm_row_norm_gate")


# ------------------------------------------------------------------------------------------
# decoders whose sublayers read the residual as it is, with norms in groups, an average over depth and softmax-routed experts
def depth_norm_taps(taps: int) -> int:
    t = load_library().glm_depth_norm_taps(taps)
    if t < 0:
        raise NotImplementedError(f"a convolution over {taps} tokens is not built")
    return t


class ExpertRows:
    """Unscaled rows of the experts [R, N] with the row and the fp32 weight of each of a token's k experts: what a feed-forward of experts
    hands to the launch that closes it."""

    def __init__(self, rows: torch.Tensor, pair_pos: torch.Tensor, weights: torch.Tensor):
        self.rows, self.pair_pos, self.weights = rows, pair_pos, weights


def depth_norm(x: torch.Tensor, width: int, groups: int, eps: float, y=None, g_post: torch.Tensor | None = None, x_out: torch.Tensor | None = None,
               cast: bool = False, depth: tuple | None = None, x_next: torch.Tensor | None = None, g_pre: torch.Tensor | None = None, conv: tuple | None = None,
               meta=None, rows: torch.Tensor | None = None, act_dtype=torch.bfloat16):
    """Between two sublayers (glm_depth_norm).  y: sublayer output [T, wp] or ExpertRows, g_post the gain of its norm; x_out receives the
    residual behind it, cast: also in the activation dtype (returned); depth = (planes [n, T, wp], coefficients [n + 1]), their average
    goes to x_next; h is the result of `conv` (bf16 weights, state) or of the norm with gain g_pre.  Returns (cast, h)."""
    wp = x.shape[1]
    T = rows.numel() if rows is not None else x.shape[0]
    dev, f32 = x.device, _is_f32(act_dtype)
    for t in (x, x_out, x_next):
        assert t is None or (t.dtype == torch.float32 and t.is_contiguous() and t.shape[1] == wp)
    assert x_out is None or x_out.shape[0] == T
    assert x_next is None or x_next.shape[0] == T
    yp = pos_p = w_p = None
    ldy, k, n_rows = wp, 0, 0
    if y is not None:
        t = y.rows if isinstance(y, ExpertRows) else y
        assert t.dtype == act_dtype and t.stride(1) == 1 and t.shape[1] == wp and g_post is not None
        yp, ldy = _p(t), t.stride(0)
        if isinstance(y, ExpertRows):
            k, n_rows = y.weights.shape[1], t.shape[0]
            assert y.weights.shape[0] == x.shape[0] and y.weights.dtype == torch.float32 and y.pair_pos.dtype == torch.int32 and y.pair_pos.numel() == y.weights.numel()
            pos_p, w_p = _p(y.pair_pos), _p(y.weights)
        else:
            assert t.shape[0] == x.shape[0]
    for g in (g_post, g_pre):
        assert g is None or (g.dtype == torch.float32 and g.is_contiguous() and g.numel() == wp)
    dp = cp = None
    n_depth = stride = 0
    if depth is not None:
        planes, coef = depth
        n_depth, stride = planes.shape[0], planes.stride(0)
        assert planes.shape[1:] == x.shape and planes.dtype == torch.float32 and planes.stride(1) == wp and planes.stride(2) == 1
        assert coef.dtype == torch.float32 and coef.numel() == n_depth + 1
        dp, cp = _p(planes), _p(coef)
    x_cast = torch.empty((T, wp), dtype=act_dtype, device=dev) if cast else None
    h = torch.empty((T, wp), dtype=act_dtype, device=dev) if (conv is not None or g_pre is not None) else None
    taps, n_state, cw, st = 1, 0, None, None
    args = (None,) * 5
    if conv is not None:
        cw, st = conv
        taps, n_state = cw.shape[0], st.shape[0]
        assert cw.dtype == torch.bfloat16 and st.dtype == torch.float32 and cw.is_contiguous() and st.is_contiguous() and cw.shape[1] == wp
        if taps == 1:
            raise ValueError("a convolution of one tap keeps two (depth_norm_taps)")
        assert st.shape[1:] == (taps - 1, wp) and rows is None
        args = (meta.pos, meta.seq_of, meta.q_start, meta.state_in, meta.state_out)
        assert meta.pos.numel() == meta.seq_of.numel() == T
    _check(load_library().glm_depth_norm(
        _p(x), _p(rows), wp, yp, ldy, pos_p, w_p, k, n_rows, _p(g_post) if y is not None else None, _p(x_out), _p(x_cast), wp, dp, stride, n_depth, cp, _p(x_next), _p(g_pre),
        _p(cw), taps, _p(st), n_state, *(_p(a) for a in args), _p(h), wp, f32, T, width, wp, groups, eps, _stream()), "glm_depth_norm")
    return x_cast, h


def softmax_router(logits: torch.Tensor, E: int, k: int):
    """The k largest scores of softmax(logits[:, :E]) per row: (experts int64 [T, k], weights fp32 [T, k]), not renormalised."""
    T = logits.shape[0]
    assert logits.dtype == torch.float32 and logits.stride(1) == 1 and logits.shape[1] >= E
    idx = torch.empty((T, k), dtype=torch.int64, device=logits.device)
    w = torch.empty((T, k), dtype=torch.float32, device=logits.device)
    _check(load_library().glm_router_softmax(_p(logits), logits.stride(0), _p(idx), _p(w), T, E, k, _stream()), "glm_router_softmax")
    return idx, w


ROUTER_ALIGN_MAX_ROWS = 64    # rows up to which one workgroup routes and buckets them (1024 pairs at most)


def softmax_router_align(logits: torch.Tensor, E: int, k: int):
    """softmax_router and the bucketing of its pairs: (weights [T, k], offsets [E + 1], source rows [T k], pair positions [T k])."""
    T, dev = logits.shape[0], logits.device
    if T > ROUTER_ALIGN_MAX_ROWS or E > 256 or T * k > 1024:
        idx, w = softmax_router(logits, E, k)
        offs, tok, _, pos = moe_align(idx, None, E, False)
        return w, offs, tok, pos
    assert logits.dtype == torch.float32 and logits.stride(1) == 1 and logits.shape[1] >= E
    idx = torch.empty((T, k), dtype=torch.int64, device=dev)
    w = torch.empty((T, k), dtype=torch.float32, device=dev)
    offs, tok, pos = (torch.empty(n, dtype=torch.int32, device=dev) for n in (E + 1, T * k, T * k))
    _check(load_library().glm_router_softmax_align(_p(logits), logits.stride(0), _p(idx), _p(w), _p(offs), _p(tok), _p(pos), T, E, k, _stream()), "glm_router_softmax_align")
    return w, offs, tok, pos


def combine_weighted(y: ExpertRows) -> torch.Tensor:
    """Sum of the experts' rows with their weights, one row per token."""
    r, (T, k) = y.rows, y.weights.shape
    out = torch.empty((T, r.shape[1]), dtype=r.dtype, device=r.device)
    _check(load_library().glm_moe_combine_weighted(_p(r), r.stride(0), r.shape[0], _p(y.pair_pos), _p(y.weights), _p(out), out.stride(0), T, k, r.shape[1], _is_f32(r.dtype), _stream()),
           "glm_moe_combine_weighted")
    return out


def grouped_swiglu(x: torch.Tensor, w13: torch.Tensor, offs: torch.Tensor, tok: torch.Tensor) -> torch.Tensor:
    """silu(gate) up of the gathered rows, w13 [G, 2 I, K] rows gate | up, bf16 or fp32 -> [rows, I]."""
    if x.dtype == torch.bfloat16:
        return grouped_gemm_gateup_silu(x, w13, offs, tok, tok.numel(), max_rows_per_group=x.shape[0])
    G, I2, K = w13.shape
    R = tok.numel()
    t = torch.empty((R, I2), dtype=x.dtype, device=x.device)
    act = torch.empty((R, I2 // 2), dtype=x.dtype, device=x.device)
    lib = load_library()
    _check(lib.glm_grouped_gemm_f32(_p(x), x.stride(0), _p(w13), w13.stride(0), w13.stride(1), _p(offs), _p(tok), _p(t), I2, R, I2, K, G, _stream()), "glm_grouped_gemm_f32")
    _check(lib.glm_swiglu_f32(_p(t), I2, _p(act), I2 // 2, R, I2 // 2, _stream()), "glm_swiglu_f32")
    return act


def grouped_down(act: torch.Tensor, w2: torch.Tensor, offs: torch.Tensor, max_rows_per_group: int) -> torch.Tensor:
    """Unscaled down projection of the experts' rows, w2 [G, N, I]."""
    if act.dtype == torch.bfloat16:
        return grouped_gemm_down(act, w2, offs, None, 0, max_rows_per_group=max_rows_per_group)
    G, N, I = w2.shape
    y = torch.empty((act.shape[0], N), dtype=act.dtype, device=act.device)
    _check(load_library().glm_grouped_gemm_f32(_p(act), I, _p(w2), w2.stride(0), w2.stride(1), _p(offs), None, _p(y), N, act.shape[0], N, I, G, _stream()), "glm_grouped_gemm_f32")
    return y
