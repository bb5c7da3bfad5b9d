"""Flat re-export of the operator surface (reference: src/pygpukit/ops/basic.py)."""

from pygpukit_amd.ops.elementwise import add, add_inplace, clamp, copy_to, div, mul, mul_inplace, sub, where
from pygpukit_amd.ops.embedding import (embedding_lookup, embedding_lookup_batch, embedding_lookup_ptr,
                                       kv_cache_prefill, kv_cache_prefill_gqa, kv_cache_update, kv_cache_update_gqa, kv_cache_update_gqa_ptr)
from pygpukit_amd.ops.matmul import (batched_matmul, gemm_w8a16_init_lut, gemv_bf16, gemv_bf16_opt_available, gemv_fp8_bf16,
                                    gemv_fp8_bf16_batched, linear_bias_gelu, matmul, matmul_nt, transpose, w8a16_gemm,
                                    w8a16_gemm_nk, w8a16_gemm_sm120)
from pygpukit_amd.ops.matmul.fp8 import *  # noqa: F401,F403
from pygpukit_amd.ops.nn import (bias_add_inplace, conv_silu, delta_rule, gated_recurrence, geglu, gelu, glu_packed, latent_rows, layernorm, layernorm_f32, mixture_of_experts, relu2, rmsnorm, rmsnorm_residual, rope_inplace,
                                rope_inplace_f32table, sdpa_causal, sdpa_causal_fixed_cache, sdpa_causal_fixed_cache_ptr,
                                sdpa_causal_strided, rotate_pairs, state_space, window_attention, head_gate, rmsnorm_f32, rmsnorm_add_f32, short_conv, sigmoid, sigmoid_mul, silu, slice_rows_range_ptr, split_qkv_batch, swiglu, tanh, xielu,
                                gelu_erf, group_norm_f32, head_norm_rope, hyper_read, hyper_write, poly_norm, soft_cap, table_experts, talk_attention)
from pygpukit_amd.ops.reduction import argmax, argmax_int, argmax_rows, max, mean, min, softmax, sum, sum_axis
from pygpukit_amd.ops.unary import abs, cos, exp, log, neg, relu, rsqrt, sin, sqrt
from pygpukit_amd.ops.sampling import (sample_greedy, sample_multinomial, sample_token_gpu, sample_topk, sample_topk_to_buf_ptr,
                                       sample_topp, set_sampling_seed)
from pygpukit_amd.ops.tensor import (cast_bf16_to_f32, cast_f16_to_f32, cast_f32_to_bf16, cast_f32_to_f16, concat_axis0, pad_2d,
                                    repeat_interleave_axis1, reshape_copy, transpose_3d_012, transpose_3d_021, transpose_4d_0132,
                                    transpose_4d_0213)

__all__ = [n for n in dir() if not n.startswith("_")]
