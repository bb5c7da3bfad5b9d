"""Checkpoint loading (reference: src/pygpukit/llm/loader.py:63-612): a .safetensors file (or a sharded index) ->
CausalTransformerModel, architecture and dimensions inferred from tensor names and shapes exactly as the reference does
(detect_model_spec; head_dim from the QK-norm weight or the 128/64/256 probe; rope_theta / rms_norm_eps and the FP8
`quantization_config` from a sibling config.json).  Tensors whose stored dtype equals the target dtype go from the file
mapping straight to device memory; others are converted on the host first.  Experts are served in the layer-list families only."""

from __future__ import annotations

import ctypes as C
import json
import os
from dataclasses import dataclass

import numpy as np

from pygpukit_amd import _hip
from pygpukit_amd.core.array import GPUArray
from pygpukit_amd.core.dtypes import bfloat16, float16, float32, uint8
from pygpukit_amd.core.factory import from_numpy
from pygpukit_amd.llm.config import (FETEZEN_SPEC, GPT2_SPEC, LLAMA_SPEC, MALASUN_SPEC, QWEN3_SPEC, RATASUN_SPEC, TOTOLORN_SPEC, LayerConfig, ModelSpec, TransformerConfig,
                                     detect_model_spec, distance_slopes, layer_list_config)
from pygpukit_amd.llm.layers import (MLP, Attention, ChannelDelta, GatedRecurrence, GatedWindowAttention, HyperBlock, HyperConnection, LatentAttention, LoopInput,
                                     MixtureOfExperts, Norm, ParallelBlock, StateSpace, TableExperts, TalkingAttention, TransformerBlock)
from pygpukit_amd.llm.layers.linear import LinearBF16, LinearFP8
from pygpukit_amd.llm.models.causal import CausalTransformerModel
from pygpukit_amd.llm.safetensors import Dtype, load_safetensors


@dataclass
class FP8QuantConfig:
    """`quantization_config` of an FP8 checkpoint's config.json (loader.py:29-60)."""
    quant_method: str
    fmt: str
    weight_block_size: tuple[int, int]
    modules_to_not_convert: list[str]

    @classmethod
    def from_config(cls, config: dict) -> "FP8QuantConfig | None":
        qc = config.get("quantization_config")
        if not qc or qc.get("quant_method") != "fp8":
            return None
        bs = qc.get("weight_block_size", [128, 128])
        return cls("fp8", qc.get("fmt", "e4m3"), (int(bs[0]), int(bs[1])), list(qc.get("modules_to_not_convert", [])))


def _read_config(model_path: str) -> dict:
    p = os.path.join(os.path.dirname(os.path.abspath(model_path)), "config.json")
    if not os.path.exists(p):
        return {}
    try:
        with open(p, encoding="utf-8") as f:
            return json.load(f)
    except (OSError, ValueError):
        return {}


def load_model_from_safetensors(model_path: str, dtype: str = "bfloat16", spec: ModelSpec | None = None,
                                repack_weights: bool = True) -> CausalTransformerModel:
    """loader.py:132-612.  dtype: "float32" | "float16" | "bfloat16" (the reference defaults to float32; bf16 is the
    native format of the checkpoints this path serves).  `repack_weights` is accepted for signature compatibility: arrays
    come from the device pool already.  `model_path` may be the checkpoint's folder (model.safetensors or its index)."""
    if os.path.isdir(model_path):
        one = os.path.join(model_path, "model.safetensors")
        model_path = one if os.path.exists(one) else os.path.join(model_path, "model.safetensors.index.json")
    st = load_safetensors(model_path)
    names = set(st.tensor_names)
    target = {"float32": (float32, Dtype.Float32, np.float32), "float16": (float16, Dtype.Float16, np.float16),
              "bfloat16": (bfloat16, Dtype.BFloat16, np.uint16)}.get(dtype)
    if target is None:
        raise ValueError(f"load_model_from_safetensors: unsupported dtype {dtype}")
    target_dt, target_id, target_np = target
    hf_config = _read_config(model_path)
    if spec is None:
        spec = detect_model_spec(st.tensor_names, hf_config)
    fp8 = FP8QuantConfig.from_config(hf_config)

    def load_tensor(name: str, do_transpose: bool = False) -> GPUArray:
        info = st.tensor_info(name)
        if info.dtype == target_id and not do_transpose:
            out = GPUArray(tuple(info.shape), target_dt)
            st.upload(name, out)                       # file mapping -> device, no host copy
            return out
        if info.dtype in (Dtype.Float8E4M3, Dtype.Float8E5M2):
            raise ValueError(f"{name}: FP8 tensor without quantization_config / _scale_inv companion")
        arr = st.tensor_as_f32(name)
        if do_transpose and arr.ndim == 2:
            arr = arr.T
        arr = np.ascontiguousarray(arr)
        if target_id == Dtype.BFloat16:
            u = arr.view(np.uint32)
            arr = ((u + 0x7FFF + ((u >> 16) & 1)) >> 16).astype(np.uint16)
        else:
            arr = arr.astype(target_np)
        return from_numpy(arr) if target_id != Dtype.BFloat16 else _bf16_array(arr)

    def try_load(name: str | None, do_transpose: bool = False) -> GPUArray | None:
        return load_tensor(name, do_transpose) if name is not None and name in names else None

    def is_fp8_weight(name: str) -> bool:
        return fp8 is not None and name + "_scale_inv" in names

    def load_linear(weight_name: str, bias_name: str | None = None, do_transpose: bool = False):
        bias = try_load(bias_name)
        if is_fp8_weight(weight_name):
            info = st.tensor_info(weight_name)
            codes = GPUArray(tuple(info.shape), uint8)
            st.upload(weight_name, codes)
            sname = weight_name + "_scale_inv"
            sinfo = st.tensor_info(sname)
            if sinfo.dtype == Dtype.BFloat16:
                scale = GPUArray(tuple(sinfo.shape), bfloat16)
                st.upload(sname, scale)
            else:
                s32 = np.ascontiguousarray(st.tensor_as_f32(sname))
                u = s32.view(np.uint32)
                scale = _bf16_array(((u + 0x7FFF + ((u >> 16) & 1)) >> 16).astype(np.uint16))
            return LinearFP8(codes, scale, bias, fp8.weight_block_size)
        return LinearBF16(load_tensor(weight_name, do_transpose), bias)

    def nm(pattern: str | None, layer: int) -> str | None:
        return None if pattern is None else pattern.format(layer=layer)

    if spec.architecture:
        return _load_layer_list(st, spec, hf_config, target_dt, load_tensor, try_load)

    embed_info = st.tensor_info(spec.embed_tokens)
    vocab_size, hidden_size = embed_info.shape
    num_layers = 0
    while nm(spec.attn_norm, num_layers) in names:
        num_layers += 1
    if num_layers == 0:
        raise ValueError(f"no layers found for spec '{spec.name}' (looked for {nm(spec.attn_norm, 0)})")

    q_info = st.tensor_info(nm(spec.q_proj, 0))
    if spec.qkv_combined:                       # GPT-2: c_attn is [hidden, 3 hidden] (Conv1D layout)
        q_dim = hidden_size
        head_dim = 64 if hidden_size % 64 == 0 else hidden_size
    else:
        q_dim = q_info.shape[0]
        head_dim = 0
        if spec.use_qk_norm and nm(spec.q_norm, 0) in names:
            head_dim = st.tensor_info(nm(spec.q_norm, 0)).shape[0]
        if not head_dim:
            for hd in (128, 64, 256):
                if q_dim % hd == 0 and hidden_size % hd == 0 and 4 <= q_dim // hd <= 128:
                    head_dim = hd
                    break
        if not head_dim:
            head_dim = hf_config.get("head_dim") or hidden_size // int(hf_config.get("num_attention_heads", 1))
    if spec.qkv_combined and "n_head" in hf_config:
        head_dim = hidden_size // int(hf_config["n_head"])
    num_heads = q_dim // head_dim
    num_kv_heads = num_heads if spec.qkv_combined else st.tensor_info(nm(spec.k_proj, 0)).shape[0] // head_dim
    if spec.activation == "silu":
        intermediate = st.tensor_info(nm(spec.gate_proj, 0)).shape[0]
    else:
        fc1 = st.tensor_info(nm(spec.fc1, 0)).shape
        intermediate = fc1[1] if spec.weight_transpose else fc1[0]
    cfg = TransformerConfig(vocab_size=vocab_size, hidden_size=hidden_size, num_layers=num_layers, num_heads=num_heads,
                            num_kv_heads=num_kv_heads, intermediate_size=intermediate,
                            _head_dim=head_dim if head_dim != hidden_size // num_heads else None, norm_type=spec.norm_type,
                            activation=spec.activation, use_rope=spec.use_rope,
                            max_position_embeddings=int(hf_config.get("max_position_embeddings", hf_config.get("n_positions", 2048))),
                            norm_eps=float(hf_config.get("rms_norm_eps", hf_config.get("layer_norm_epsilon", spec.default_norm_eps))),
                            rope_theta=float(hf_config.get("rope_theta", spec.default_rope_theta)))
    eps = cfg.norm_eps

    blocks = []
    for layer in range(num_layers):
        attn_norm = Norm(load_tensor(nm(spec.attn_norm, layer)), try_load(nm(spec.attn_norm_bias, layer)), spec.norm_type, eps)
        mlp_norm = Norm(load_tensor(nm(spec.mlp_norm, layer)), try_load(nm(spec.mlp_norm_bias, layer)), spec.norm_type, eps)
        qn = kn = None
        if spec.use_qk_norm:
            qw, kw = try_load(nm(spec.q_norm, layer)), try_load(nm(spec.k_norm, layer))
            qn = Norm(qw, None, spec.norm_type, eps) if qw is not None else None
            kn = Norm(kw, None, spec.norm_type, eps) if kw is not None else None
        if spec.qkv_combined:
            w = st.tensor_as_f32(nm(spec.q_proj, layer))
            w = w.T if spec.weight_transpose else w                       # -> [3 hidden, hidden]
            b = st.tensor_as_f32(nm(spec.q_bias, layer)) if nm(spec.q_bias, layer) in names else None
            parts = [_to_device(np.ascontiguousarray(w[i * hidden_size:(i + 1) * hidden_size]), target_id, target_np) for i in range(3)]
            biases = [None] * 3 if b is None else [_to_device(np.ascontiguousarray(b[i * hidden_size:(i + 1) * hidden_size]), target_id, target_np)
                                                   for i in range(3)]
            o = load_linear(nm(spec.o_proj, layer), nm(spec.o_bias, layer), spec.weight_transpose)
            attn = Attention(parts[0], parts[1], parts[2], o, cfg, q_bias=biases[0], k_bias=biases[1], v_bias=biases[2])
        else:
            attn = Attention(load_linear(nm(spec.q_proj, layer), nm(spec.q_bias, layer)), load_linear(nm(spec.k_proj, layer), nm(spec.k_bias, layer)),
                             load_linear(nm(spec.v_proj, layer), nm(spec.v_bias, layer)), load_linear(nm(spec.o_proj, layer), nm(spec.o_bias, layer)),
                             cfg, q_norm=qn, k_norm=kn)
        if spec.activation == "silu":
            g, u_, d = (load_linear(nm(spec.gate_proj, layer)), load_linear(nm(spec.up_proj, layer)), load_linear(nm(spec.down_proj, layer)))
            if isinstance(g, LinearBF16) and isinstance(u_, LinearBF16) and g.bias is None and u_.bias is None:
                g, u_ = g.weight, u_.weight                               # lets MLP fuse gate|up into one matrix
            mlp = MLP(cfg, gate_proj=g, up_proj=u_, down_proj=d)
        else:
            mlp = MLP(cfg, fc1_weight=load_tensor(nm(spec.fc1, layer), spec.weight_transpose), fc1_bias=try_load(nm(spec.fc1_bias, layer)),
                      fc2_weight=load_tensor(nm(spec.fc2, layer), spec.weight_transpose), fc2_bias=try_load(nm(spec.fc2_bias, layer)))
        blocks.append(TransformerBlock(attn_norm, attn, mlp_norm, mlp))

    final_norm = Norm(load_tensor(spec.final_norm), try_load(spec.final_norm_bias), spec.norm_type, eps)
    lm_head = try_load(spec.lm_head) if spec.lm_head else None            # tied embeddings when absent
    position_embed = try_load(spec.position_embed) if spec.use_position_embed else None
    return CausalTransformerModel(cfg, load_tensor(spec.embed_tokens), blocks, final_norm, lm_head, position_embed, spec)


def _load_layer_list(st, spec: ModelSpec, config: dict, dtype, load_tensor, try_load) -> CausalTransformerModel:
    """A layer-list checkpoint: config.json gives every layer's kind and sizes, the tensors are checked against it."""
    if not config:
        raise ValueError(f"a {spec.name} checkpoint needs its config.json beside it")
    cfg = layer_list_config(config)

    def tensor(name: str, shape: tuple[int, ...]) -> GPUArray:
        if name not in st:
            raise ValueError(f"checkpoint has no tensor {name!r}")
        got = tuple(st.tensor_info(name).shape)
        if got != shape:
            raise ValueError(f"{name}: shape {got}, config.json says {shape}")
        return load_tensor(name)

    def fp32(name: str, size: int) -> np.ndarray:
        if name not in st or int(np.prod(st.tensor_info(name).shape)) != size:
            raise ValueError(f"{name}: missing or not of {size} elements")
        return np.ascontiguousarray(st.tensor_as_f32(name), dtype=np.float32).reshape(size)

    def norm(name: str, width: int, offset: float, scalar: bool = False, kind: str = "rmsnorm", mult: float = 1.0) -> Norm:
        w = np.repeat(fp32(name, 1), width) if scalar else fp32(name, width)
        return Norm(from_numpy((w + np.float32(offset)) * np.float32(mult)), None, kind, cfg.norm_eps, stream_dtype=dtype, groups=cfg.norm_groups if width == cfg.hidden_size and spec.hyper else 1)

    H, off, one = cfg.hidden_size, spec.norm_weight_offset, spec.norm_scalar
    blocks: list[TransformerBlock] = []

    def latent_mixer(lc: LayerConfig, nm) -> LatentAttention:
        rot = lc.rot_dim
        freq = from_numpy((lc.rot_base ** (-2.0 * np.arange(rot // 2) / rot)).astype(np.float32)) if rot else None
        gate = tensor(nm(spec.head_gate), (lc.num_heads, H)) if spec.head_gate else None
        return LatentAttention(tensor(nm(spec.q_proj), (lc.num_heads * (lc.head_dim + rot), H)), tensor(nm(spec.kv_down_proj), (lc.kv_rank + rot, H)),
                               norm(nm(spec.kv_down_norm), lc.kv_rank, 0.0), tensor(nm(spec.k_up_proj), (lc.num_heads * lc.head_dim, lc.kv_rank)),
                               tensor(nm(spec.v_up_proj), (lc.num_heads * lc.v_head_dim, lc.kv_rank)),
                               tensor(nm(spec.o_proj), (H, lc.num_heads * lc.v_head_dim)), num_heads=lc.num_heads, head_dim=lc.head_dim,
                               v_head_dim=lc.v_head_dim, scale=lc.scale, window=lc.window, head_gate=gate, rot_dim=rot, rot_freq=freq)

    def attention_mixer(lc: LayerConfig, nm) -> GatedWindowAttention:
        q, k, v = lc.num_heads * lc.head_dim, lc.num_kv_heads * lc.head_dim, lc.num_kv_heads * lc.v_head_dim
        own = lc.kv_from is None

        def proj(weight: str, bias: str, rows: int) -> LinearBF16:
            return LinearBF16(tensor(nm(weight), (rows, H)), tensor(nm(bias), (rows,)))

        def conv(name: str, rows: int) -> GPUArray | None:
            return None if lc.conv_taps is None else tensor(nm(name), (rows, lc.conv_taps))

        return GatedWindowAttention(
            proj(spec.q_proj, spec.q_bias, q), proj(spec.k_proj, spec.k_bias, k) if own else None, proj(spec.v_proj, spec.v_bias, v) if own else None,
            tensor(nm(spec.o_proj), (H, lc.num_heads * lc.v_head_dim)), tensor(nm(spec.out_gate), (lc.num_heads * lc.v_head_dim, H)), num_heads=lc.num_heads,
            num_kv_heads=lc.num_kv_heads, head_dim=lc.head_dim, v_head_dim=lc.v_head_dim, scale=lc.scale, window=lc.window, q_norm=norm(nm(spec.q_norm), q, 0.0),
            k_norm=norm(nm(spec.k_norm), k, 0.0) if own else None, q_conv=conv(spec.q_conv, q), k_conv=conv(spec.k_conv, k) if own else None,
            v_conv=conv(spec.v_conv, v) if own else None, slopes=from_numpy(np.asarray(distance_slopes(lc.num_heads), np.float32)),
            source=None if own else blocks[lc.kv_from].attn, kv_from=lc.kv_from)

    def talking_mixer(lc: LayerConfig, nm) -> TalkingAttention:
        q, k, v = lc.num_heads * lc.head_dim, lc.num_kv_heads * lc.head_dim, lc.num_kv_heads * lc.v_head_dim
        own, rot = lc.kv_from is None, lc.rot_dim
        freq = from_numpy((lc.rot_base ** (-2.0 * np.arange(rot // 2) / rot)).astype(np.float32)) if rot else None

        def proj(weight: str, bias: str, rows: int, cols: int = H) -> LinearBF16:
            return LinearBF16(tensor(nm(weight), (rows, cols)), tensor(nm(bias), (rows,)))

        def head_norm(name: str) -> Norm:
            return Norm(from_numpy(fp32(nm(name), lc.head_dim)), None, "rmsnorm", cfg.norm_eps, stream_dtype=dtype)

        return TalkingAttention(
            proj(spec.q_proj, spec.q_bias, q), proj(spec.k_proj, spec.k_bias, k) if own else None, proj(spec.v_proj, spec.v_bias, v) if own else None,
            proj(spec.o_proj, spec.o_bias, H, lc.num_heads * lc.v_head_dim), num_heads=lc.num_heads, num_kv_heads=lc.num_kv_heads, head_dim=lc.head_dim,
            v_head_dim=lc.v_head_dim, scale=lc.scale, window=lc.window, chunked=lc.chunked, q_norm=head_norm(spec.q_norm), k_norm=head_norm(spec.k_norm) if own else None,
            rot_freq=freq, talk=from_numpy(fp32(nm(spec.talk), lc.num_heads ** 2).reshape(lc.num_heads, lc.num_heads)), sink=from_numpy(fp32(nm(spec.sink), lc.num_heads)),
            source=None if own else blocks[lc.kv_from].attn, kv_from=lc.kv_from)

    def recurrent_mixer(lc: LayerConfig, nm) -> GatedRecurrence:
        qk, v = lc.num_heads * lc.head_dim, lc.num_heads * lc.v_head_dim
        return GatedRecurrence(tensor(nm(spec.q_proj), (qk, H)), tensor(nm(spec.forget_proj), (qk, H)), tensor(nm(spec.v_proj), (v, H)), tensor(nm(spec.o_proj), (H, v)),
                               from_numpy(fp32(nm(spec.forget_bias), qk)), from_numpy(fp32(nm(spec.forget_lower), qk)), from_numpy(fp32(nm(spec.head_norm), lc.v_head_dim)),
                               num_heads=lc.num_heads, head_dim=lc.head_dim, v_head_dim=lc.v_head_dim, eps=cfg.norm_eps)

    def decay_rates(name: str, heads: int) -> GPUArray:
        return from_numpy(np.exp(fp32(name, heads).astype(np.float64)).astype(np.float32))

    def rows_of(name: str) -> int:
        if name not in st or len(st.tensor_info(name).shape) != 2:
            raise ValueError(f"checkpoint has no matrix {name!r}")
        return int(st.tensor_info(name).shape[0])

    def taps(name: str, channels: int, n: int) -> GPUArray:
        return _transposed(tensor(name, (channels, n)))

    def delta_mixer(lc: LayerConfig, nm) -> ChannelDelta:
        k, q, v, n = lc.num_kv_heads * lc.head_dim, lc.num_heads * lc.head_dim, lc.num_heads * lc.v_head_dim, lc.conv_taps

        def maps(down: str, up: str, rows: int) -> tuple[GPUArray, GPUArray]:
            rank = rows_of(nm(down))
            return tensor(nm(down), (rank, H)), tensor(nm(up), (rows, rank))

        return ChannelDelta(tensor(nm(spec.q_proj), (k, H)), tensor(nm(spec.k_proj), (k, H)), tensor(nm(spec.v_proj), (v, H)), tensor(nm(spec.o_proj), (H, v)),
                            tensor(nm(spec.strength), (lc.num_heads, H)), maps(spec.decay_down, spec.decay_up, q), maps(spec.gate_down, spec.gate_up, v),
                            (taps(nm(spec.q_conv), k, n), taps(nm(spec.k_conv), k, n), taps(nm(spec.v_conv), v, n)), decay_rates(nm(spec.decay_log), lc.num_heads),
                            from_numpy(fp32(nm(spec.step_bias), q)), from_numpy(fp32(nm(spec.head_norm), lc.v_head_dim)), num_heads=lc.num_heads,
                            num_kv_heads=lc.num_kv_heads, head_dim=lc.head_dim, v_head_dim=lc.v_head_dim, eps=cfg.norm_eps)

    def state_space_mixer(lc: LayerConfig, nm) -> StateSpace:
        v, ch, heads = lc.num_heads * lc.v_head_dim, lc.num_heads * lc.v_head_dim + 2 * lc.num_kv_heads * lc.head_dim, lc.num_heads
        w = tensor(nm(spec.in_proj), (v + ch + heads, H))
        parts = (w._view(0, (v, H)), w._view(v * H, (ch, H)), w._view((v + ch) * H, (heads, H)))
        return StateSpace(parts, tensor(nm(spec.o_proj), (H, v)), taps(nm(spec.conv), ch, lc.conv_taps), from_numpy(fp32(nm(spec.conv_bias), ch)),
                          decay_rates(nm(spec.decay_log), heads), from_numpy(fp32(nm(spec.step_bias), heads)), from_numpy(fp32(nm(spec.skip), heads)),
                          from_numpy(fp32(nm(spec.out_norm), v)), num_heads=heads, num_groups=lc.num_kv_heads, state_dim=lc.head_dim, v_head_dim=lc.v_head_dim,
                          norm_groups=lc.norm_groups, eps=cfg.norm_eps)

    def expert_mlp(lc: LayerConfig, nm) -> MixtureOfExperts:
        e, I = lc.experts, lc.intermediate_size
        gate_up, down = GPUArray((e.count, 2 * I, H), dtype), GPUArray((e.count, H, I), dtype)
        for k in range(e.count):
            for out, at, pattern, shape in ((gate_up, 2 * k, spec.expert_gate_proj, (I, H)), (gate_up, 2 * k + 1, spec.expert_up_proj, (I, H)), (down, k, spec.expert_down_proj, (H, I))):
                w = tensor(nm(pattern, expert=k), shape)
                _hip.call("pgk_memcpy_d2d", C.c_void_p(out.data_ptr() + at * w.nbytes), w._p, w.nbytes, None)
        return MixtureOfExperts(tensor(nm(spec.router), (e.count, H)), from_numpy(fp32(nm(spec.router_correction), e.count)), gate_up, down, top=e.top, groups=e.groups,
                                keep=e.keep, scale=e.scale)

    def table_mlp(i: int, lc: LayerConfig, nm) -> TableExperts:
        e, I = lc.experts, lc.intermediate_size
        name = nm(spec.expert_table)
        if name not in st or tuple(st.tensor_info(name).shape) != (cfg.vocab_size, e.top) or st.tensor_info(name).dtype not in (Dtype.Int32, Dtype.Int64):
            raise ValueError(f"{name}: missing, or not integers [{cfg.vocab_size}, {e.top}]")
        table = np.ascontiguousarray(st.tensor_numpy(name))
        if table.min() < 0 or table.max() >= e.count:
            raise ValueError(f"{name}: names experts outside [0, {e.count})")
        up, down = GPUArray((e.count, I, H), dtype), GPUArray((e.count, H, I), dtype)
        for k in range(e.count):
            for out, pattern, shape in ((up, spec.expert_up_proj, (I, H)), (down, spec.expert_down_proj, (H, I))):
                w = tensor(nm(pattern, expert=k), shape)
                _hip.call("pgk_memcpy_d2d", C.c_void_p(out.data_ptr() + k * w.nbytes), w._p, w.nbytes, None)
        shared = {}
        if e.shared_size is not None:
            shared = dict(shared_up=tensor(nm(spec.shared_up_proj), (e.shared_size, H)), shared_down=tensor(nm(spec.shared_down_proj), (H, e.shared_size)),
                          shared_gate=tensor(nm(spec.shared_gate), (1, H)))
        return TableExperts(from_numpy(table.astype(np.int32)), up, down, **shared)

    def hyper(nm, sublayer: int) -> HyperConnection:
        p, n = nm(spec.hyper, sublayer=sublayer), cfg.streams
        return HyperConnection(from_numpy(fp32(p + "in", n)), from_numpy(fp32(p + "out", n)), from_numpy(fp32(p + "mix", n * n).reshape(n, n)))

    def hyper_block(i: int, lc: LayerConfig, nm, attn) -> HyperBlock:
        mlp = None
        if lc.experts is not None:
            mlp = table_mlp(i, lc, nm)
        elif lc.intermediate_size is not None:
            I = lc.intermediate_size
            mlp = MLP(cfg, fc1_weight=tensor(nm(spec.fc1), (I, H)), fc2_weight=tensor(nm(spec.fc2), (H, I)), act_params=from_numpy(fp32(nm(spec.act_params), 4)), act_eps=cfg.norm_eps)
        return HyperBlock(norm(nm(spec.attn_norm), H, off), attn, hyper(nm, 1), None if mlp is None else norm(nm(spec.mlp_norm), H, off), mlp, None if mlp is None else hyper(nm, 2))

    mixers = {"latent_attention": (latent_mixer, spec.kv_down_proj), "attention": (talking_mixer, spec.talk) if spec.talk else (attention_mixer, spec.out_gate), "hgrn2": (recurrent_mixer, spec.forget_proj),
              "channel_delta": (delta_mixer, spec.decay_down), "mamba2": (state_space_mixer, spec.in_proj)}
    for i, lc in enumerate(cfg.layers):
        nm = lambda pattern, **kw: pattern.format(layer=i, **kw)  # noqa: E731, B023
        make, known = mixers[lc.mixer]
        if known is None:
            raise ValueError(f"layer {i}: {spec.name} models have no {lc.mixer} layers")
        mlp = mlp_norm = post_mlp = None
        attn = make(lc, nm)
        if spec.hyper:
            blocks.append(hyper_block(i, lc, nm, attn))
            continue
        if (lc.experts is not None) != (spec.is_moe and lc.intermediate_size is not None):
            raise ValueError(f"layer {i}: {spec.name} models have {'no dense feed-forwards' if spec.is_moe else 'no experts'}")
        if spec.parallel:
            blocks.append(ParallelBlock(norm(nm(spec.attn_norm), H, off, one, spec.norm_type), attn, None if lc.experts is None else expert_mlp(lc, nm)))
            continue
        if lc.intermediate_size is not None:
            I = lc.intermediate_size
            if spec.activation == "xielu":
                p, q = (float(x) for x in np.logaddexp(0.0, fp32(nm(spec.act_params), 2).astype(np.float64)))
                mlp = MLP(cfg, fc1_weight=tensor(nm(spec.fc1), (I, H)), fc2_weight=tensor(nm(spec.fc2), (H, I)), act_params=(p, 0.5 + q))
            else:
                mlp = MLP(cfg, gate_proj=tensor(nm(spec.gate_proj), (I, H)), up_proj=tensor(nm(spec.up_proj), (I, H)), down_proj=tensor(nm(spec.down_proj), (H, I)))
            mlp_norm = norm(nm(spec.mlp_norm), H, off, one) if spec.mlp_norm else None
            post_mlp = norm(nm(spec.post_mlp_norm), H, off, one)
        blocks.append(TransformerBlock(norm(nm(spec.attn_norm), H, off, one) if spec.attn_norm else None, attn, mlp_norm, mlp,
                                       norm(nm(spec.post_attn_norm), H, off, one), post_mlp, cfg.residual_mult))
    lm_head = tensor(spec.lm_head, (cfg.vocab_size, H)) if spec.lm_head in st else None
    pos = tensor(spec.position_embed, (cfg.max_position_embeddings, H)) if spec.use_position_embed else None
    loop = None
    if cfg.loop is not None:
        if spec.loop_in is None:
            raise ValueError(f"{spec.name} models have no loop")
        loop = LoopInput(tensor(spec.loop_in, (H, 2 * H)), from_numpy(fp32(spec.loop_step, cfg.loop.times * H).reshape(cfg.loop.times, H)))
    return CausalTransformerModel(cfg, tensor(spec.embed_tokens, (cfg.vocab_size, H)), blocks, norm(spec.final_norm, H, off, one, spec.norm_type, cfg.logit_scale), lm_head, pos, spec, loop)


def _transposed(w: GPUArray) -> GPUArray:
    return from_numpy(np.ascontiguousarray(w.to_numpy().T))


def _bf16_array(bits: np.ndarray) -> GPUArray:
    out = GPUArray(tuple(bits.shape), bfloat16)
    out.copy_from_numpy(np.ascontiguousarray(bits, dtype=np.uint16))
    return out


def _to_device(arr_f32: np.ndarray, target_id: int, target_np) -> GPUArray:
    if target_id == Dtype.BFloat16:
        u = np.ascontiguousarray(arr_f32, dtype=np.float32).view(np.uint32)
        return _bf16_array(((u + 0x7FFF + ((u >> 16) & 1)) >> 16).astype(np.uint16))
    return from_numpy(np.ascontiguousarray(arr_f32).astype(target_np))


def load_gpt2_from_safetensors(model_path: str, dtype: str = "float32") -> CausalTransformerModel:
    return load_model_from_safetensors(model_path, dtype=dtype, spec=GPT2_SPEC)


def load_llama_from_safetensors(model_path: str, dtype: str = "bfloat16") -> CausalTransformerModel:
    return load_model_from_safetensors(model_path, dtype=dtype, spec=LLAMA_SPEC)


def load_qwen3_from_safetensors(model_path: str, dtype: str = "bfloat16") -> CausalTransformerModel:
    return load_model_from_safetensors(model_path, dtype=dtype, spec=QWEN3_SPEC)


def load_totolorn_from_safetensors(model_path: str, dtype: str = "bfloat16") -> CausalTransformerModel:
    return load_model_from_safetensors(model_path, dtype=dtype, spec=TOTOLORN_SPEC)


def load_malasun_from_safetensors(model_path: str, dtype: str = "bfloat16") -> CausalTransformerModel:
    return load_model_from_safetensors(model_path, dtype=dtype, spec=MALASUN_SPEC)


def load_fetezen_from_safetensors(model_path: str, dtype: str = "bfloat16") -> CausalTransformerModel:
    return load_model_from_safetensors(model_path, dtype=dtype, spec=FETEZEN_SPEC)


def load_ratasun_from_safetensors(model_path: str, dtype: str = "bfloat16") -> CausalTransformerModel:
    return load_model_from_safetensors(model_path, dtype=dtype, spec=RATASUN_SPEC)


__all__ = ["load_fetezen_from_safetensors", "load_ratasun_from_safetensors", "load_malasun_from_safetensors", "load_totolorn_from_safetensors", "load_model_from_safetensors", "load_gpt2_from_safetensors", "load_llama_from_safetensors", "load_qwen3_from_safetensors",
           "FP8QuantConfig"]
