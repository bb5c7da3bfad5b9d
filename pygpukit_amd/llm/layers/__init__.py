from .attention import Attention
from .block import HyperBlock, HyperConnection, LoopInput, ParallelBlock, TransformerBlock
from .delta import ChannelDelta
from .experts import MixtureOfExperts, TableExperts
from .latent_attention import LatentAttention
from .linear import Linear, LinearBF16, LinearFP8, quantize_linear_fp8
from .mlp import MLP
from .norm import Norm
from .recurrence import GatedRecurrence
from .rope import apply_rotary_pos_emb_numpy, precompute_freqs_cis
from .state_space import StateSpace
from .talking_attention import TalkingAttention
from .window_attention import GatedWindowAttention

__all__ = ["Attention", "LatentAttention", "GatedWindowAttention", "GatedRecurrence", "ChannelDelta", "StateSpace", "MixtureOfExperts", "TransformerBlock", "ParallelBlock", "LoopInput", "HyperBlock", "HyperConnection", "TableExperts", "TalkingAttention", "Linear", "LinearBF16", "LinearFP8", "MLP", "Norm", "precompute_freqs_cis", "apply_rotary_pos_emb_numpy",
           "quantize_linear_fp8"]
