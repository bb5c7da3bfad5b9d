from .attention import Attention
from .block import LoopInput, ParallelBlock, TransformerBlock
from .delta import ChannelDelta
from .experts import MixtureOfExperts
from .latent_attention import LatentAttention
from .linear import Linear, LinearBF16, LinearFP8, quantize_linear_fp8
from .mlp import MLP
from .norm import Norm
from .recurrence import GatedRecurrence
from .rope import apply_rotary_pos_emb_numpy, precompute_freqs_cis
from .state_space import StateSpace
from .window_attention import GatedWindowAttention

__all__ = ["Attention", "LatentAttention", "GatedWindowAttention", "GatedRecurrence", "ChannelDelta", "StateSpace", "MixtureOfExperts", "TransformerBlock", "ParallelBlock", "LoopInput", "Linear", "LinearBF16", "LinearFP8", "MLP", "Norm", "precompute_freqs_cis", "apply_rotary_pos_emb_numpy",
           "quantize_linear_fp8"]
