from pygpukit_amd.ops.nn.activation import gelu, gelu_erf, poly_norm, relu2, sigmoid, silu, soft_cap, tanh, xielu
from pygpukit_amd.ops.nn.attention import (sdpa_causal, sdpa_causal_fixed_cache, sdpa_causal_fixed_cache_ptr,
                                          sdpa_causal_strided, window_attention, head_gate, head_norm_rope, sigmoid_mul, talk_attention)
from pygpukit_amd.ops.nn.fused import geglu, glu_packed, rmsnorm_residual, swiglu
from pygpukit_amd.ops.nn.hyper import hyper_read, hyper_write
from pygpukit_amd.ops.nn.latent import latent_rows, rotate_pairs
from pygpukit_amd.ops.nn.linear import bias_add_inplace, slice_rows_range_ptr, split_qkv_batch
from pygpukit_amd.ops.nn.norm import group_norm_f32, layernorm, layernorm_f32, rmsnorm, rmsnorm_add_f32, rmsnorm_f32
from pygpukit_amd.ops.nn.moe import mixture_of_experts, table_experts
from pygpukit_amd.ops.nn.recurrence import conv_silu, delta_rule, gated_recurrence, short_conv, state_space
from pygpukit_amd.ops.nn.rope import rope_inplace, rope_inplace_f32table

__all__ = ["gelu", "silu", "sigmoid", "tanh", "relu2", "sdpa_causal", "sdpa_causal_fixed_cache",
           "sdpa_causal_fixed_cache_ptr", "sdpa_causal_strided", "rmsnorm_residual", "swiglu", "geglu", "glu_packed",
           "bias_add_inplace", "split_qkv_batch", "slice_rows_range_ptr", "layernorm", "rmsnorm", "rope_inplace",
           "rope_inplace_f32table", "window_attention", "head_gate", "sigmoid_mul", "xielu", "short_conv", "gated_recurrence", "rmsnorm_f32", "rmsnorm_add_f32",
           "conv_silu", "delta_rule", "state_space", "mixture_of_experts", "layernorm_f32", "latent_rows", "rotate_pairs", "gelu_erf", "poly_norm", "soft_cap",
           "head_norm_rope", "talk_attention", "hyper_read", "hyper_write", "group_norm_f32", "table_experts"]
