from .causal import CausalTransformerModel, GPT2Model, LlamaModel, QwenModel, TotolornModel, MalasunModel, RatasunModel, FetezenModel

__all__ = ["CausalTransformerModel", "GPT2Model", "LlamaModel", "QwenModel", "TotolornModel", "MalasunModel", "RatasunModel", "FetezenModel"]
