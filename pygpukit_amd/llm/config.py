"""Model configuration (reference: src/pygpukit/llm/config.py:20-507).

TransformerConfig carries the dimensions; ModelSpec is the data-only description of one
architecture family (HF tensor-name patterns + architecture flags + default hyper-parameters).
Described are the dense families GPT-2, Llama, Qwen2, Qwen3 and the layer-list families Totolorn, Malasun, Ratasun (whose
feed-forwards are mixtures of experts) and Fetezen (dense layers beside experts that a table of tokens chooses).  A layer-list model's config.json spells out every layer: LayerConfig."""

from __future__ import annotations

from dataclasses import dataclass
from typing import Literal


@dataclass(frozen=True)
class ModelSpec:
    name: str
    embed_tokens: str
    position_embed: str | None
    lm_head: str | None
    final_norm: str
    final_norm_bias: str | None
    attn_norm: str | None
    attn_norm_bias: str | None
    q_proj: str
    k_proj: str | None
    v_proj: str | None
    o_proj: str
    q_bias: str | None
    k_bias: str | None
    v_bias: str | None
    o_bias: str | None
    q_norm: str | None
    k_norm: str | None
    mlp_norm: str | None
    mlp_norm_bias: str | None
    fc1: str | None
    fc1_bias: str | None
    fc2: str | None
    fc2_bias: str | None
    gate_proj: str | None
    up_proj: str | None
    down_proj: str | None
    moe_gate: str | None = None
    expert_gate_proj: str | None = None
    expert_up_proj: str | None = None
    expert_down_proj: str | None = None
    norm_type: Literal["rmsnorm", "layernorm"] = "rmsnorm"
    activation: Literal["gelu", "silu", "xielu", "poly_norm"] = "silu"
    use_rope: bool = True
    use_qk_norm: bool = False
    use_position_embed: bool = False
    qkv_combined: bool = False
    weight_transpose: bool = False
    is_moe: bool = False
    default_norm_eps: float = 1e-5
    default_rope_theta: float = 10000.0
    hf_model_type: str = ""
    # layer-list families: config.json's "architecture", and what their layers add to the fields above
    architecture: str = ""
    post_attn_norm: str | None = None      # norm of the sublayer's output, before the residual add
    post_mlp_norm: str | None = None
    kv_down_proj: str | None = None        # latent attention: hidden -> latent, its norm, latent -> keys / values
    kv_down_norm: str | None = None
    k_up_proj: str | None = None
    v_up_proj: str | None = None
    head_gate: str | None = None           # one sigmoid gate per head
    q_conv: str | None = None              # taps over time on the channels of q, k, v
    k_conv: str | None = None
    v_conv: str | None = None
    out_gate: str | None = None            # one sigmoid gate per element of the mixer's output
    forget_proj: str | None = None         # gated recurrence: forget gate, its bias and lower bound, norm of a head's output
    forget_bias: str | None = None
    forget_lower: str | None = None
    head_norm: str | None = None
    act_params: str | None = None          # numbers of the activation
    norm_scalar: bool = False              # a norm's weight is one number
    norm_weight_offset: float = 0.0        # norms multiply by offset + weight (1: weights stored around zero)
    residual_f32: bool = False             # the residual stream stays fp32 whatever the element type
    parallel: bool = False                 # mixer and feed-forward read one norm, both results are added
    strength: str | None = None            # delta rule: write strength, the two maps of the decay and of the output gate
    decay_down: str | None = None
    decay_up: str | None = None
    gate_down: str | None = None
    gate_up: str | None = None
    decay_log: str | None = None           # recurrences: logarithm of the decay rate, bias of its step
    step_bias: str | None = None
    in_proj: str | None = None             # state space: all projections in one matrix, taps and their bias, skip, norm of the output
    conv: str | None = None
    conv_bias: str | None = None
    skip: str | None = None
    out_norm: str | None = None
    router: str | None = None              # experts: router, correction of the choice
    router_correction: str | None = None
    loop_in: str | None = None             # passes over a stretch of layers: map of [stream; embedding], one vector per pass
    loop_step: str | None = None
    talk: str | None = None                # attention: mix of the heads' scores, sinks
    sink: str | None = None
    chunked: bool = False                  # an attention mask's size is a chunk, not a sliding window
    hyper: str | None = None               # hyper-connections of sublayer {sublayer}: prefix of its in, out and mix
    expert_table: str | None = None        # experts: table of tokens instead of a router; the shared expert and its gate
    shared_up_proj: str | None = None
    shared_down_proj: str | None = None
    shared_gate: str | None = None


def _hf_decoder_spec(name: str, *, qk_norm: bool, qkv_bias: bool, eps: float, theta: float) -> ModelSpec:
    """Llama-style HF checkpoint naming: model.layers.{layer}.{self_attn|mlp}.*"""
    L = "model.layers.{layer}."
    A = L + "self_attn."
    return ModelSpec(
        name=name, embed_tokens="model.embed_tokens.weight", position_embed=None, lm_head="lm_head.weight",
        final_norm="model.norm.weight", final_norm_bias=None,
        attn_norm=L + "input_layernorm.weight", attn_norm_bias=None,
        q_proj=A + "q_proj.weight", k_proj=A + "k_proj.weight", v_proj=A + "v_proj.weight", o_proj=A + "o_proj.weight",
        q_bias=A + "q_proj.bias" if qkv_bias else None, k_bias=A + "k_proj.bias" if qkv_bias else None,
        v_bias=A + "v_proj.bias" if qkv_bias else None, o_bias=None,
        q_norm=A + "q_norm.weight" if qk_norm else None, k_norm=A + "k_norm.weight" if qk_norm else None,
        mlp_norm=L + "post_attention_layernorm.weight", mlp_norm_bias=None,
        fc1=None, fc1_bias=None, fc2=None, fc2_bias=None,
        gate_proj=L + "mlp.gate_proj.weight", up_proj=L + "mlp.up_proj.weight", down_proj=L + "mlp.down_proj.weight",
        norm_type="rmsnorm", activation="silu", use_rope=True, use_qk_norm=qk_norm,
        default_norm_eps=eps, default_rope_theta=theta, hf_model_type=name)


LLAMA_SPEC = _hf_decoder_spec("llama", qk_norm=False, qkv_bias=False, eps=1e-5, theta=10000.0)
QWEN2_SPEC = _hf_decoder_spec("qwen2", qk_norm=False, qkv_bias=True, eps=1e-6, theta=1000000.0)
QWEN3_SPEC = _hf_decoder_spec("qwen3", qk_norm=True, qkv_bias=False, eps=1e-6, theta=1000000.0)

_G = "h.{layer}."
GPT2_SPEC = ModelSpec(
    name="gpt2", embed_tokens="wte.weight", position_embed="wpe.weight", lm_head=None,
    final_norm="ln_f.weight", final_norm_bias="ln_f.bias",
    attn_norm=_G + "ln_1.weight", attn_norm_bias=_G + "ln_1.bias",
    q_proj=_G + "attn.c_attn.weight", k_proj=_G + "attn.c_attn.weight", v_proj=_G + "attn.c_attn.weight",
    o_proj=_G + "attn.c_proj.weight",
    q_bias=_G + "attn.c_attn.bias", k_bias=_G + "attn.c_attn.bias", v_bias=_G + "attn.c_attn.bias",
    o_bias=_G + "attn.c_proj.bias", q_norm=None, k_norm=None,
    mlp_norm=_G + "ln_2.weight", mlp_norm_bias=_G + "ln_2.bias",
    fc1=_G + "mlp.c_fc.weight", fc1_bias=_G + "mlp.c_fc.bias", fc2=_G + "mlp.c_proj.weight", fc2_bias=_G + "mlp.c_proj.bias",
    gate_proj=None, up_proj=None, down_proj=None,
    norm_type="layernorm", activation="gelu", use_rope=False, use_qk_norm=False, use_position_embed=True,
    qkv_combined=True, weight_transpose=True, default_norm_eps=1e-5, default_rope_theta=10000.0, hf_model_type="gpt2")

_T = "l{layer}."
TOTOLORN_SPEC = ModelSpec(
    name="totolorn", embed_tokens="embed", position_embed="pos", lm_head="head", final_norm="final.norm", final_norm_bias=None,
    attn_norm=_T + "norm1", attn_norm_bias=None, q_proj=_T + "mix.q", k_proj=None, v_proj=None, o_proj=_T + "mix.o",
    q_bias=None, k_bias=None, v_bias=None, o_bias=None, q_norm=None, k_norm=None, mlp_norm=_T + "norm2", mlp_norm_bias=None,
    fc1=None, fc1_bias=None, fc2=None, fc2_bias=None, gate_proj=_T + "mlp.gate", up_proj=_T + "mlp.up", down_proj=_T + "mlp.down",
    norm_type="rmsnorm", activation="silu", use_rope=False, use_position_embed=True, architecture="Totolorn",
    post_attn_norm=_T + "norm1b", post_mlp_norm=_T + "norm2b", kv_down_proj=_T + "mix.dkv", kv_down_norm=_T + "mix.dkv.norm",
    k_up_proj=_T + "mix.uk", v_up_proj=_T + "mix.uv", head_gate=_T + "mix.g", norm_weight_offset=1.0, residual_f32=True)

MALASUN_SPEC = ModelSpec(
    name="malasun", embed_tokens="embed", position_embed=None, lm_head="head", final_norm="final.norm", final_norm_bias=None,
    attn_norm=None, attn_norm_bias=None, q_proj=_T + "mix.q", k_proj=_T + "mix.k", v_proj=_T + "mix.v", o_proj=_T + "mix.o",
    q_bias=_T + "mix.q.b", k_bias=_T + "mix.k.b", v_bias=_T + "mix.v.b", o_bias=None, q_norm=_T + "mix.q.norm", k_norm=_T + "mix.k.norm",
    mlp_norm=None, mlp_norm_bias=None, fc1=_T + "mlp.up", fc1_bias=None, fc2=_T + "mlp.down", fc2_bias=None,
    gate_proj=None, up_proj=None, down_proj=None, norm_type="rmsnorm", activation="xielu", use_rope=False, use_qk_norm=True,
    architecture="Malasun", post_attn_norm=_T + "norm1", post_mlp_norm=_T + "norm2", q_conv=_T + "mix.q.conv", k_conv=_T + "mix.k.conv",
    v_conv=_T + "mix.v.conv", out_gate=_T + "mix.g", forget_proj=_T + "mix.f", forget_bias=_T + "mix.f.b", forget_lower=_T + "mix.lower",
    head_norm=_T + "mix.norm", act_params=_T + "mlp.act", norm_scalar=True, residual_f32=True)

RATASUN_SPEC = ModelSpec(
    name="ratasun", embed_tokens="embed", position_embed=None, lm_head="head", final_norm="final.norm", final_norm_bias=None,
    attn_norm=_T + "norm1", attn_norm_bias=None, q_proj=_T + "mix.q", k_proj=_T + "mix.k", v_proj=_T + "mix.v", o_proj=_T + "mix.o",
    q_bias=None, k_bias=None, v_bias=None, o_bias=None, q_norm=None, k_norm=None, mlp_norm=None, mlp_norm_bias=None,
    fc1=None, fc1_bias=None, fc2=None, fc2_bias=None, gate_proj=None, up_proj=None, down_proj=None,
    expert_gate_proj=_T + "mlp.e{expert}.gate", expert_up_proj=_T + "mlp.e{expert}.up", expert_down_proj=_T + "mlp.e{expert}.down",
    norm_type="layernorm", activation="silu", use_rope=True, is_moe=True, architecture="Ratasun", parallel=True, residual_f32=True,
    kv_down_proj=_T + "mix.dkv", kv_down_norm=_T + "mix.dkv.norm", k_up_proj=_T + "mix.uk", v_up_proj=_T + "mix.uv",
    q_conv=_T + "mix.q.conv", k_conv=_T + "mix.k.conv", v_conv=_T + "mix.v.conv", head_norm=_T + "mix.norm", strength=_T + "mix.b",
    decay_down=_T + "mix.a1", decay_up=_T + "mix.a2", gate_down=_T + "mix.g1", gate_up=_T + "mix.g2", decay_log=_T + "mix.A_log",
    step_bias=_T + "mix.dt_bias", in_proj=_T + "mix.in", conv=_T + "mix.conv", conv_bias=_T + "mix.conv.b", skip=_T + "mix.D", out_norm=_T + "mix.norm",
    router=_T + "mlp.router", router_correction=_T + "mlp.correction", loop_in="loop.in", loop_step="loop.step")

FETEZEN_SPEC = ModelSpec(
    name="fetezen", embed_tokens="embed", position_embed=None, lm_head="head", final_norm="final.norm", final_norm_bias=None,
    attn_norm=_T + "norm1", attn_norm_bias=None, q_proj=_T + "mix.q", k_proj=_T + "mix.k", v_proj=_T + "mix.v", o_proj=_T + "mix.o",
    q_bias=_T + "mix.q.b", k_bias=_T + "mix.k.b", v_bias=_T + "mix.v.b", o_bias=_T + "mix.o.b", q_norm=_T + "mix.q.norm", k_norm=_T + "mix.k.norm",
    mlp_norm=_T + "norm2", mlp_norm_bias=None, fc1=_T + "mlp.up", fc1_bias=None, fc2=_T + "mlp.down", fc2_bias=None, gate_proj=None, up_proj=None, down_proj=None,
    expert_up_proj=_T + "mlp.e{expert}.up", expert_down_proj=_T + "mlp.e{expert}.down", norm_type="rmsnorm", activation="poly_norm", use_rope=True, use_qk_norm=True,
    is_moe=True, architecture="Fetezen", act_params=_T + "mlp.act", residual_f32=True, talk=_T + "mix.talk", sink=_T + "mix.sink", chunked=True, hyper=_T + "hc{sublayer}.",
    expert_table=_T + "mlp.table", shared_up_proj=_T + "mlp.shared.up", shared_down_proj=_T + "mlp.shared.down", shared_gate=_T + "mlp.shared.sg")

MODEL_SPECS: dict[str, ModelSpec] = {"gpt2": GPT2_SPEC, "llama": LLAMA_SPEC, "qwen3": QWEN3_SPEC, "qwen2": QWEN2_SPEC,
                                     "totolorn": TOTOLORN_SPEC, "malasun": MALASUN_SPEC, "ratasun": RATASUN_SPEC, "fetezen": FETEZEN_SPEC}


def detect_model_spec(tensor_names: list[str], config: dict | None = None) -> ModelSpec:
    """Pick the family: config.json's "architecture" if it names one of ours, else the checkpoint's tensor names
    (config.py:380-431): QK-norm -> Qwen3, QKV biases -> Qwen2, model.embed_tokens -> Llama, wte -> GPT-2.  MoE checkpoints are
    rejected."""
    arch = (config or {}).get("architecture")
    if arch:
        for spec in MODEL_SPECS.values():
            if spec.architecture == arch:
                return spec
        raise ValueError(f"unknown architecture {arch!r} (known: {[s.architecture for s in MODEL_SPECS.values() if s.architecture]})")
    names = set(tensor_names)
    if any("block_sparse_moe" in n or "mlp.experts" in n for n in names):
        raise ValueError("MoE checkpoints of the Hugging Face families are not supported by pygpukit_amd")
    if any("q_norm" in n for n in names):
        return QWEN3_SPEC
    if "model.embed_tokens.weight" in names:
        return QWEN2_SPEC if "model.layers.0.self_attn.q_proj.bias" in names else LLAMA_SPEC
    if "wte.weight" in names:
        return GPT2_SPEC
    raise ValueError(f"Cannot detect model type from tensor names. First 10 names: {list(tensor_names)[:10]}")


@dataclass(frozen=True)
class ExpertsConfig:
    """A layer's mixture of experts; with groups > 0 only experts of the `keep` best groups of neighbours can be chosen.  With `table` a
    table of token ids chooses; shared_size: width of one more expert that every token runs (None: none)."""

    count: int
    top: int
    groups: int
    keep: int
    scale: float                      # of the chosen experts' weights, which sum to it
    table: bool = False
    shared_size: int | None = None


@dataclass(frozen=True)
class LoopConfig:
    """Layers start .. stop - 1 run `times` times with the same weights, every pass with caches of its own."""

    start: int
    stop: int
    times: int

    def runs(self, num_layers: int) -> list[tuple[int, int | None]]:
        """(layer, number of the pass that starts with it or None) in the order they run."""
        head = [(i, None) for i in range(self.start)]
        body = [(i, t if i == self.start else None) for t in range(self.times) for i in range(self.start, self.stop)]
        return head + body + [(i, None) for i in range(self.stop, num_layers)]


@dataclass(frozen=True)
class LayerConfig:
    """One layer of a layer-list model."""

    mixer: Literal["latent_attention", "attention", "hgrn2", "channel_delta", "mamba2"]
    num_heads: int
    head_dim: int                     # query / key width of a head
    v_head_dim: int                   # value width of a head
    kv_rank: int                      # latent attention: latent size, what the cache holds per token
    window: int | None                # keys a query sees, itself included (None: all before it)
    scale: float                      # multiplies q . k
    intermediate_size: int | None     # feed-forward width; None: the layer has no feed-forward
    num_kv_heads: int = 0             # attention: key / value heads
    conv_taps: int | None = None      # attention: taps over time on q, k, v (None: no convolution)
    kv_from: int | None = None        # attention: the layer whose keys and values this one uses (None: its own)
    # rotated query / key columns (0: none), pair i turns by position * base^(-2i / rot_dim): latent attention: beside head_dim's, neighbours
    # are a pair; attention: the first of head_dim's, i and i + rot_dim / 2 are a pair
    rot_dim: int = 0
    rot_base: float = 10000.0
    norm_groups: int = 1              # state space: equal parts of the output that are normed on their own
    experts: ExpertsConfig | None = None
    chunked: bool = False             # attention: `window` is the size of the chunks of positions that see only themselves


def parse_experts(i: int, mlp: dict, table: bool = False) -> tuple[ExpertsConfig, int]:
    r, shared = mlp["router"], mlp.get("shared")
    g = r.get("groups")
    e = ExpertsConfig(int(r["experts"]), int(r["top"]), int(g["count"]) if g else 0, int(g["keep"]) if g else 0, float(r.get("scale", 1.0)), table,
                      int(shared["ff"]) if shared else None)
    if not 1 <= e.top <= e.count or (e.groups and (e.count % e.groups or not 1 <= e.keep <= e.groups or e.keep * (e.count // e.groups) < e.top)):
        raise ValueError(f"layer {i}: cannot choose {e.top} of {e.count} experts in {e.keep} of {e.groups} groups")
    return e, int(mlp["expert"]["ff"])


def parse_layer(i: int, entry: dict, spec: ModelSpec | None = None) -> LayerConfig:
    kind, mlp = entry.get("type"), entry.get("mlp")
    if kind not in ("latent_attention", "attention", "hgrn2", "channel_delta", "mamba2"):
        raise ValueError(f"layer {i}: unknown mixer {kind!r}")
    m = entry["mixer"]
    if mlp is not None and mlp.get("kind") not in ("dense", "moe"):
        raise ValueError(f"layer {i}: unknown feed-forward {mlp.get('kind')!r}")
    experts, ff = (None, None) if mlp is None else parse_experts(i, mlp, spec is not None and spec.expert_table is not None) if mlp["kind"] == "moe" else (None, int(mlp["ff"]))
    heads, vdim = int(m["heads"]), int(m["vdim"])
    dim = int(m["state"] if kind == "mamba2" else m["dim"])
    if kind == "hgrn2":
        return LayerConfig(kind, heads, dim, vdim, 0, None, 1.0, ff, experts=experts)
    if kind in ("channel_delta", "mamba2"):
        lc = LayerConfig(kind, heads, dim, vdim, 0, None, 1.0, ff, int(m["kv_heads" if kind == "channel_delta" else "groups"]), int(m["conv"]),
                         norm_groups=int(m.get("norm_groups", 1)), experts=experts)
        if lc.num_kv_heads < 1 or heads % lc.num_kv_heads or heads * vdim % lc.norm_groups or lc.conv_taps < 1:
            raise ValueError(f"layer {i}: {heads} heads of {vdim} over {lc.num_kv_heads} key heads, {lc.conv_taps} taps, {lc.norm_groups} norm groups")
        return lc
    mask = m.get("mask")
    window = int(mask["size"]) if mask else None
    if kind == "latent_attention":
        rot, rd = m.get("rot"), int(m.get("rot_dim", 0))
        if rd % 2 or (rot is not None and int(rot["dims"]) != rd):
            raise ValueError(f"layer {i}: {rd} rotated columns, rotation of {rot}")
        return LayerConfig(kind, heads, dim, vdim, int(m["kv_rank"]), window, float(m["scale"]), ff, rot_dim=rd, rot_base=float(rot["base"]) if rot else 10000.0,
                           experts=experts)
    taps, src, rot = m.get("conv"), m.get("kv_from"), m.get("rot") if spec is not None and spec.use_rope else None
    rd = int(rot["dims"]) if rot else 0
    if rd % 2 or not 0 <= rd <= dim or (window is not None and window < 1):
        raise ValueError(f"layer {i}: {rd} rotated columns of {dim}, mask of {window}")
    return LayerConfig(kind, heads, dim, vdim, 0, window, float(m["scale"]), ff, int(m["kv_heads"]), int(taps) if taps is not None else None,
                       int(src) if src is not None else None, rot_dim=rd, rot_base=float(rot["base"]) if rot else 10000.0, experts=experts,
                       chunked=window is not None and spec is not None and spec.chunked)


def distance_slopes(heads: int) -> list[float]:
    """Slopes of the distance bias: 2^(-8 (h + 1) / heads) for head h."""
    return [2.0 ** (-8.0 * (h + 1) / heads) for h in range(heads)]


NO_POSITION_LIMIT = 2**30       # models without learned positions


def layer_list_config(config: dict) -> "TransformerConfig":
    """config.json of a layer-list model -> TransformerConfig.  The per-model head fields take the first layer's values."""
    found = next((s for s in MODEL_SPECS.values() if s.architecture and s.architecture == config.get("architecture")), None)
    layers = tuple(parse_layer(i, e, found) for i, e in enumerate(config["layers"]))
    if not layers:
        raise ValueError("config.json lists no layers")
    for i, l in enumerate(layers):
        if l.mixer == "attention" and (l.num_kv_heads < 1 or l.num_heads % l.num_kv_heads):
            raise ValueError(f"layer {i}: {l.num_heads} query heads over {l.num_kv_heads} key heads")
        if l.kv_from is not None:
            s = layers[l.kv_from] if 0 <= l.kv_from < i else None
            if s is None or s.mixer != "attention" or s.kv_from is not None or (s.num_kv_heads, s.head_dim, s.v_head_dim) != (l.num_kv_heads, l.head_dim, l.v_head_dim):
                raise ValueError(f"layer {i}: cannot take the keys and values of layer {l.kv_from}")
    first = layers[0]
    loop = config.get("loop")
    if loop is not None:
        loop = LoopConfig(int(loop["start"]), int(loop["stop"]), int(loop["times"]))
        if not 0 <= loop.start < loop.stop <= len(layers) or loop.times < 1 or any(l.kv_from is not None for l in layers):
            raise ValueError(f"cannot run layers {loop.start} .. {loop.stop - 1} of {len(layers)} {loop.times} times")
    spec = found or TOTOLORN_SPEC
    width, streams, groups, cap = int(config["width"]), int(config.get("streams", 1)), int(config["norm"].get("groups", 1)), config.get("logit_softcap")
    if groups < 1 or width % groups or streams < 1 or (cap is not None and not float(cap) > 0) or (spec.hyper is None and (streams, groups, cap) != (1, 1, None)):
        raise ValueError(f"{spec.name}: width {width} in {groups} norm groups, {streams} streams, logits capped at {cap}")
    return TransformerConfig(vocab_size=int(config["vocab"]), hidden_size=width, num_layers=len(layers), num_heads=first.num_heads,
                             num_kv_heads=first.num_kv_heads or first.num_heads, intermediate_size=max([l.intermediate_size or 0 for l in layers]),
                             _head_dim=first.head_dim, norm_type=spec.norm_type, activation=spec.activation, use_rope=spec.use_rope, loop=loop,
                             logit_scale=float(config.get("logit_scale", 1.0)),
                             max_position_embeddings=int(config["max_positions"]) if spec.use_position_embed else NO_POSITION_LIMIT,
                             norm_eps=float(config["norm"]["eps"]), tie_word_embeddings=False, layers=layers, residual_mult=float(config.get("residual_mult", 1.0)),
                             streams=streams, norm_groups=groups, logit_softcap=None if cap is None else float(cap))


@dataclass
class TransformerConfig:
    """config.py:440-507.  head_dim defaults to hidden_size // num_heads unless _head_dim is given
    (Qwen3-0.6B: hidden 1024, 16 heads, head_dim 128)."""

    vocab_size: int = 32000
    hidden_size: int = 2048
    num_layers: int = 22
    num_heads: int = 32
    num_kv_heads: int | None = None
    intermediate_size: int | None = None
    _head_dim: int | None = None
    num_experts: int | None = None
    num_experts_per_tok: int = 2
    moe_intermediate_size: int | None = None
    norm_type: Literal["rmsnorm", "layernorm"] = "rmsnorm"
    activation: Literal["gelu", "silu", "xielu", "poly_norm"] = "silu"
    use_rope: bool = True
    causal: bool = True
    max_position_embeddings: int = 2048
    norm_eps: float = 1e-5
    rope_theta: float = 10000.0
    tie_word_embeddings: bool = True
    layers: tuple[LayerConfig, ...] | None = None    # layer-list models: every layer's own sizes
    residual_mult: float = 1.0                       # factor of every sublayer's contribution to the residual stream
    loop: LoopConfig | None = None                   # layer-list models: a stretch of layers that runs several times
    logit_scale: float = 1.0                         # factor of the logits (the loader multiplies the output norm's weight by it)
    streams: int = 1                                 # hyper-connected models: residual streams
    norm_groups: int = 1                             # equal parts of the width that the norms treat on their own
    logit_softcap: float | None = None               # logits become cap * tanh(logits / cap)

    def __post_init__(self):
        if self.num_kv_heads is None:
            self.num_kv_heads = self.num_heads
        if self.intermediate_size is None:
            self.intermediate_size = 4 * self.hidden_size
        if self.moe_intermediate_size is None:
            self.moe_intermediate_size = self.intermediate_size

    @property
    def is_moe(self) -> bool:
        return self.num_experts is not None and self.num_experts > 1

    @property
    def head_dim(self) -> int:
        return self._head_dim if self._head_dim is not None else self.hidden_size // self.num_heads

    @property
    def num_kv_groups(self) -> int:
        return self.num_heads // self.num_kv_heads


# ---- legacy per-family configs (config.py:515-620): HF-style field names, converted to TransformerConfig ----------
@dataclass
class GPT2Config:
    vocab_size: int = 50257
    n_embd: int = 768
    n_layer: int = 12
    n_head: int = 12
    n_positions: int = 1024
    layer_norm_eps: float = 1e-5

    @property
    def n_inner(self) -> int:
        return 4 * self.n_embd

    def to_transformer_config(self) -> TransformerConfig:
        return TransformerConfig(vocab_size=self.vocab_size, hidden_size=self.n_embd, num_layers=self.n_layer, num_heads=self.n_head,
                                 num_kv_heads=self.n_head, intermediate_size=self.n_inner, norm_type="layernorm", activation="gelu",
                                 use_rope=False, causal=True, max_position_embeddings=self.n_positions, norm_eps=self.layer_norm_eps)


@dataclass
class LlamaConfig:
    vocab_size: int = 32000
    hidden_size: int = 2048
    intermediate_size: int = 5632
    num_hidden_layers: int = 22
    num_attention_heads: int = 32
    num_key_value_heads: int = 4
    max_position_embeddings: int = 2048
    rms_norm_eps: float = 1e-5
    rope_theta: float = 10000.0

    @property
    def head_dim(self) -> int:
        return self.hidden_size // self.num_attention_heads

    def to_transformer_config(self) -> TransformerConfig:
        return TransformerConfig(vocab_size=self.vocab_size, hidden_size=self.hidden_size, num_layers=self.num_hidden_layers,
                                 num_heads=self.num_attention_heads, num_kv_heads=self.num_key_value_heads,
                                 intermediate_size=self.intermediate_size, norm_type="rmsnorm", activation="silu", use_rope=True,
                                 causal=True, max_position_embeddings=self.max_position_embeddings, norm_eps=self.rms_norm_eps,
                                 rope_theta=self.rope_theta)


@dataclass
class Qwen3Config:
    vocab_size: int = 151936
    hidden_size: int = 4096
    intermediate_size: int = 12288
    num_hidden_layers: int = 36
    num_attention_heads: int = 32
    num_key_value_heads: int = 8
    head_dim: int = 128            # not hidden_size // heads: Qwen3-0.6B is 1024 / 16 heads with 128
    max_position_embeddings: int = 40960
    rms_norm_eps: float = 1e-6
    rope_theta: float = 1000000.0

    def to_transformer_config(self) -> TransformerConfig:
        """The reference's conversion drops head_dim (config.py:600-616) and so gets 64 for Qwen3-0.6B; it is carried
        through here."""
        return TransformerConfig(vocab_size=self.vocab_size, hidden_size=self.hidden_size, num_layers=self.num_hidden_layers,
                                 num_heads=self.num_attention_heads, num_kv_heads=self.num_key_value_heads,
                                 intermediate_size=self.intermediate_size, _head_dim=self.head_dim, norm_type="rmsnorm",
                                 activation="silu", use_rope=True, causal=True, max_position_embeddings=self.max_position_embeddings,
                                 norm_eps=self.rms_norm_eps, rope_theta=self.rope_theta)
