from .causal import CausalTransformerModel, GPT2Model, LlamaModel, QwenModel, TotolornModel, MalasunModel, RatasunModel

__all__ = ["CausalTransformerModel", "GPT2Model", "LlamaModel", "QwenModel", "TotolornModel", "MalasunModel", "RatasunModel"]
