from .causal import CausalTransformerModel, GPT2Model, LlamaModel, QwenModel, TotolornModel

__all__ = ["CausalTransformerModel", "GPT2Model", "LlamaModel", "QwenModel", "TotolornModel"]
