"""LLM layer of pygpukit_amd: config, layers, CausalTransformerModel, decode strategies, native engine."""

from pygpukit_amd.llm.buffers import DecodeBuffers, PrefillBuffers
from pygpukit_amd.llm.config import (FETEZEN_SPEC, GPT2_SPEC, LLAMA_SPEC, MODEL_SPECS, QWEN2_SPEC, QWEN3_SPEC, TOTOLORN_SPEC, MALASUN_SPEC, RATASUN_SPEC, ExpertsConfig, GPT2Config, LayerConfig, LlamaConfig, LoopConfig, ModelSpec,
                                    Qwen3Config, TransformerConfig, detect_model_spec, layer_list_config)
from pygpukit_amd.llm.decode import DecodeBatch, DecodeM1, DecodeM1Graph, DecodeStrategy
from pygpukit_amd.llm.engine import Engine, StackEngine
from pygpukit_amd.llm.layers import (MLP, Attention, ChannelDelta, GatedRecurrence, GatedWindowAttention, HyperBlock, HyperConnection, LatentAttention, Linear, LinearBF16, LinearFP8, MixtureOfExperts, Norm, ParallelBlock,
                                    StateSpace, TableExperts, TalkingAttention, TransformerBlock, apply_rotary_pos_emb_numpy, precompute_freqs_cis)
from pygpukit_amd.llm.models import CausalTransformerModel, FetezenModel, GPT2Model, LlamaModel, MalasunModel, QwenModel, RatasunModel, TotolornModel
from pygpukit_amd.llm.loader import (FP8QuantConfig, load_gpt2_from_safetensors, load_llama_from_safetensors,  # noqa: E402
                                     load_model_from_safetensors, load_qwen3_from_safetensors, load_totolorn_from_safetensors, load_malasun_from_safetensors, load_ratasun_from_safetensors,
                                     load_fetezen_from_safetensors)
from pygpukit_amd.llm.scheduler import BatchScheduler  # noqa: E402
from pygpukit_amd.llm.safetensors import Dtype, SafeTensorsFile, ShardedSafeTensorsFile, TensorInfo, load_safetensors  # noqa: E402
from pygpukit_amd.llm.sampling import sample_token

# legacy component names (models/causal.py:1496-1501)
RMSNorm = LayerNorm = Norm
LlamaAttention = CausalSelfAttention = Attention
LlamaMLP = MLP
LlamaBlock = TransformerBlock

__all__ = ["load_model_from_safetensors", "load_qwen3_from_safetensors", "load_llama_from_safetensors", "load_gpt2_from_safetensors",
           "FP8QuantConfig", "SafeTensorsFile", "ShardedSafeTensorsFile", "TensorInfo", "Dtype", "load_safetensors",
           "DecodeBuffers", "PrefillBuffers", "ModelSpec", "TransformerConfig", "GPT2_SPEC", "LLAMA_SPEC", "QWEN2_SPEC",
           "QWEN3_SPEC", "MODEL_SPECS", "detect_model_spec", "DecodeStrategy", "DecodeM1", "DecodeM1Graph", "DecodeBatch",
           "Engine", "MLP", "Attention", "Linear", "LinearBF16", "LinearFP8", "Norm", "TransformerBlock",
           "precompute_freqs_cis", "CausalTransformerModel", "GPT2Model", "LlamaModel", "QwenModel", "sample_token",
           "GPT2Config", "LlamaConfig", "Qwen3Config", "apply_rotary_pos_emb_numpy", "RMSNorm", "LayerNorm", "LlamaAttention",
           "CausalSelfAttention", "LlamaMLP", "LlamaBlock", "TOTOLORN_SPEC", "LayerConfig", "layer_list_config", "StackEngine", "LatentAttention", "TotolornModel",
           "load_totolorn_from_safetensors", "BatchScheduler", "MALASUN_SPEC", "MalasunModel", "GatedWindowAttention", "GatedRecurrence",
           "load_malasun_from_safetensors", "RATASUN_SPEC", "RatasunModel", "ExpertsConfig", "LoopConfig", "ChannelDelta", "StateSpace", "MixtureOfExperts",
           "ParallelBlock", "load_ratasun_from_safetensors", "FETEZEN_SPEC", "FetezenModel", "HyperBlock", "HyperConnection", "TableExperts", "TalkingAttention",
           "load_fetezen_from_safetensors"]
