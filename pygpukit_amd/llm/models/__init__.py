from .causal import CausalTransformerModel, GPT2Model, LlamaModel, QwenModel, TotolornModel, MalasunModel

__all__ = ["CausalTransformerModel", "GPT2Model", "LlamaModel", "QwenModel", "TotolornModel", "MalasunModel"]
