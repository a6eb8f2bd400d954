"""Named model-architecture presets for bench/tests (random-init weights;
there is no network for checkpoints).  Shapes follow the published HF
configs of the models BASELINE.json names."""

from __future__ import annotations

from ..config import ModelConfig


def _tuvutar(width: int, heads: int, ff: int, vocab: int, period: str,
             repeats: int, dim: int = 128, rot: int = 64, rank: int = 512,
             delta_heads: int = 0, delta_kv: int = 0) -> dict:
    """A Tuvutar config: ``period`` repeated, "d" a gated-delta layer, "a" a
    latent-attention layer with rows of its own, "s" one that reads the rows of
    the latest "a"."""
    layers, last = [], None
    for kind in period * repeats:
        if kind == "d":
            mixer = {"heads": delta_heads or 2 * heads,
                     "kv_heads": delta_kv or heads, "dim": 128, "vdim": 128,
                     "conv": 4}
        else:
            mixer = {"heads": heads, "dim": dim, "rot_dim": rot, "vdim": dim,
                     "kv_rank": rank, "scale": (dim + rot) ** -0.5,
                     "rot": {"base": 10000.0, "dims": rot,
                             "scaling": {"factor": 8.0, "original": 4096,
                                         "fast": 32.0, "slow": 1.0}}}
            if kind == "s":
                mixer["kv_from"] = last
            else:
                last = len(layers)
        layers.append({"type": "delta" if kind == "d" else "latent_attention",
                       "mixer": mixer, "mlp": {"kind": "dense", "ff": ff}})
    return {"architecture": "Tuvutar", "width": width, "vocab": vocab,
            "norm": {"eps": 1e-6}, "layers": layers}


def _lepizen(width: int, heads: int, kv_heads: int, ff: int, vocab: int,
             n_layers: int, dim: int = 128) -> dict:
    mixer = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": dim,
             "scale": dim ** -0.5, "v_mix": True}
    return {"architecture": "Lepizen", "width": width, "vocab": vocab,
            "norm": {"eps": 1e-6}, "residual_mult": 0.7, "logit_scale": 0.25,
            "logit_softcap": 50.0,
            "layers": [{"type": "attention", "mixer": dict(mixer),
                        "mlp": {"kind": "dense", "ff": ff}}
                       for _ in range(n_layers)]}


def _sadosun(width: int, heads: int, kv_heads: int, ff: int, vocab: int,
             period: str, repeats: int = 1, dim: int = 128, window: int = 1024,
             experts: int = 64, identity: int = 8, top: int = 6,
             inner: int = 0, state: int = 16, side: int = 256) -> dict:
    """A Sadosun config: ``period`` repeated, "a" a windowed-attention layer,
    "m" a selective-scan layer; ff: units of one expert."""
    layers = []
    for kind in period * repeats:
        if kind == "m":
            mixer = {"inner": inner or 2 * width, "state": state,
                     "dt_rank": width // 16, "conv": 4}
        else:
            mixer = {"heads": heads, "kv_heads": kv_heads, "dim": dim,
                     "vdim": dim, "scale": dim ** -0.5,
                     "rot": {"base": 10000.0, "dims": dim},
                     "mask": {"size": window}}
        layers.append({
            "type": "mamba1" if kind == "m" else "attention", "mixer": mixer,
            "mlp": {"kind": "moe", "expert": {"ff": ff},
                    "router": {"experts": experts, "identity": identity,
                               "top": top}}})
    return {"architecture": "Sadosun", "width": width, "vocab": vocab,
            "norm": {"eps": 1e-6}, "embedding": {"scale": 12.0},
            "canon": {"taps": 4}, "token_side": {"dim": side},
            "layers": layers}


def _dufinex(width: int, heads: int, kv_heads: int, ff: int, vocab: int,
             period: str, repeats: int = 1, dim: int = 128, expert_ff: int = 0,
             experts: int = 64, top: int = 6, delta_heads: int = 0,
             delta_kv: int = 0, rank: int = 128, scale: float = 50.0) -> dict:
    """A Dufinex config: ``period`` repeated, "d" a delta layer, "a" an attention
    layer, "s" one that reads the keys and values of the latest "a"; capitals
    have routed experts in place of a dense feed-forward."""
    layers, last = [], None
    for kind in period * repeats:
        low = kind.lower()
        if low == "d":
            mixer = {"heads": delta_heads or heads, "kv_heads": delta_kv or heads,
                     "dim": 128, "vdim": 128, "conv": 4, "decay_rank": rank,
                     "gate_rank": rank}
        else:
            mixer = {"heads": heads, "kv_heads": kv_heads, "dim": dim,
                     "vdim": dim, "scale": dim ** -0.5}
            if low == "s":
                mixer["kv_from"] = last
            else:
                last = len(layers)
        mlp = {"kind": "dense", "ff": ff, "limit": 7.0}
        if kind != low:
            mlp = {"kind": "moe", "expert": {"ff": expert_ff, "limit": 7.0},
                   "router": {"experts": experts, "top": top}}
        layers.append({"type": "channel_delta" if low == "d" else "attention",
                       "mixer": mixer, "mlp": mlp})
    return {"architecture": "Dufinex", "width": width, "vocab": vocab,
            "norm": {"eps": 1e-6}, "embedding": {"scale": scale},
            "layers": layers}


def _llama(width: int, heads: int, kv_heads: int, ff: int, vocab: int,
           n_layers: int) -> dict:
    return {"model_type": "llama", "hidden_size": width,
            "num_hidden_layers": n_layers, "intermediate_size": ff,
            "num_attention_heads": heads, "num_key_value_heads": kv_heads,
            "vocab_size": vocab, "rms_norm_eps": 1e-6, "rope_theta": 10000.0}


def _dense_mla(width: int, heads: int, ff: int, vocab: int, n_layers: int,
               dim: int = 128, rot: int = 64, rank: int = 512) -> dict:
    """A DeepSeek-V2 config without experts (latent attention + dense MLP)."""
    return {"model_type": "deepseek_v2", "hidden_size": width,
            "num_hidden_layers": n_layers, "intermediate_size": ff,
            "num_attention_heads": heads, "vocab_size": vocab,
            "rms_norm_eps": 1e-6, "rope_theta": 10000.0, "q_lora_rank": None,
            "kv_lora_rank": rank, "qk_nope_head_dim": dim,
            "qk_rope_head_dim": rot, "v_head_dim": dim}


def _moe_mla(width: int, heads: int, ff: int, vocab: int, n_layers: int,
             experts: int = 64, top: int = 6) -> dict:
    """A DeepSeek-V2 config with routed experts of ``ff`` units everywhere."""
    return {**_dense_mla(width, heads, ff, vocab, n_layers),
            "moe_intermediate_size": ff, "n_routed_experts": experts,
            "num_experts_per_tok": top, "n_shared_experts": 0,
            "first_k_dense_replace": 0, "moe_layer_freq": 1}


PRESETS = {
    # headline model: DeepSeek-Coder-V2-Lite-Instruct (15.7B total, 2.4B active)
    "deepseek-v2-lite": {
        "model_type": "deepseek_v2",
        "hidden_size": 2048,
        "num_hidden_layers": 27,
        "intermediate_size": 10944,
        "moe_intermediate_size": 1408,
        "num_attention_heads": 16,
        "vocab_size": 102400,
        "rms_norm_eps": 1e-6,
        "rope_theta": 10000.0,
        "q_lora_rank": None,
        "kv_lora_rank": 512,
        "qk_nope_head_dim": 128,
        "qk_rope_head_dim": 64,
        "v_head_dim": 128,
        "n_routed_experts": 64,
        "n_shared_experts": 2,
        "num_experts_per_tok": 6,
        "n_group": 1,
        "topk_group": 1,
        "topk_method": "greedy",
        "norm_topk_prob": False,
        "routed_scaling_factor": 1.0,
        "first_k_dense_replace": 1,
        "moe_layer_freq": 1,
        "max_position_embeddings": 163840,
        "rope_scaling": {"type": "yarn", "factor": 40.0, "beta_fast": 32,
                         "beta_slow": 1, "mscale": 0.707, "mscale_all_dim": 0.707,
                         "original_max_position_embeddings": 4096},
    },
    "llama-3-8b": {
        "model_type": "llama",
        "hidden_size": 4096,
        "num_hidden_layers": 32,
        "intermediate_size": 14336,
        "num_attention_heads": 32,
        "num_key_value_heads": 8,
        "vocab_size": 128256,
        "rms_norm_eps": 1e-5,
        "rope_theta": 500000.0,
        "max_position_embeddings": 8192,
    },
    "llama-3-70b": {
        "model_type": "llama",
        "hidden_size": 8192,
        "num_hidden_layers": 80,
        "intermediate_size": 28672,
        "num_attention_heads": 64,
        "num_key_value_heads": 8,
        "vocab_size": 128256,
        "rms_norm_eps": 1e-5,
        "rope_theta": 500000.0,
        "max_position_embeddings": 8192,
    },
    "gemma-2-9b": {
        "model_type": "gemma2",
        "hidden_size": 3584,
        "num_hidden_layers": 42,
        "intermediate_size": 14336,
        "num_attention_heads": 16,
        "num_key_value_heads": 8,
        "head_dim": 256,
        "vocab_size": 256000,
        "rms_norm_eps": 1e-6,
        "rope_theta": 10000.0,
        "query_pre_attn_scalar": 256,
        "attn_logit_softcapping": 50.0,
        "final_logit_softcapping": 30.0,
        "sliding_window": 4096,
        "max_position_embeddings": 8192,
    },
    "tinyllama-1.1b": {
        "model_type": "llama",
        "hidden_size": 2048,
        "num_hidden_layers": 22,
        "intermediate_size": 5632,
        "num_attention_heads": 32,
        "num_key_value_heads": 4,
        "vocab_size": 32000,
        "rms_norm_eps": 1e-5,
        "rope_theta": 10000.0,
    },
    # Qwen2-7B-Instruct shapes (config.json of Qwen/Qwen2-7B-Instruct);
    # llama-family remap with QKV-only attention biases
    "qwen2-7b": {
        "model_type": "qwen2",
        "hidden_size": 3584,
        "num_hidden_layers": 28,
        "intermediate_size": 18944,
        "num_attention_heads": 28,
        "num_key_value_heads": 4,
        "vocab_size": 152064,
        "rms_norm_eps": 1e-6,
        "rope_theta": 1000000.0,
        "tie_word_embeddings": False,
        "max_position_embeddings": 32768,
    },

    # small debug model (CPU-runnable; 8 layers so a CPU smoke of the
    # 8-stage pipeline gives every rank at least one layer)
    "debug-llama": {
        "model_type": "llama",
        "hidden_size": 256,
        "num_hidden_layers": 8,
        "intermediate_size": 512,
        "num_attention_heads": 8,
        "num_key_value_heads": 4,
        "vocab_size": 1024,
        "rms_norm_eps": 1e-5,
        "rope_theta": 10000.0,
    },
    "tuvutar-2b": _tuvutar(2048, 16, 8192, 32000, "dddadds", 4),
    "tuvutar-8b": _tuvutar(4096, 32, 14336, 32000, "dddadds", 4,
                           delta_heads=32, delta_kv=16),
    "lepizen-2b": _lepizen(2048, 16, 4, 8192, 32000, 28),
    "lepizen-8b": _lepizen(4096, 32, 8, 16384, 32000, 36),
    "sadosun-7b": _sadosun(2048, 16, 4, 1024, 32000, "maamaa", 4),
    "dufinex-7b": _dufinex(2048, 16, 4, 8192, 32000, "dDaDdDsD", 3,
                           expert_ff=1024),
    "debug-dufinex": {
        "architecture": "Dufinex", "width": 80, "vocab": 320,
        "norm": {"eps": 1e-5}, "embedding": {"scale": 0.8},
        "layers": [
            {"type": "attention",
             "mixer": {"heads": 4, "kv_heads": 2, "dim": 24, "vdim": 16,
                       "scale": 0.2},
             "mlp": {"kind": "moe", "expert": {"ff": 40, "limit": 2.0},
                     "router": {"experts": 5, "top": 2}}},
            {"type": "channel_delta",
             "mixer": {"heads": 4, "kv_heads": 2, "dim": 16, "vdim": 24,
                       "conv": 3, "decay_rank": 12, "gate_rank": 8},
             "mlp": {"kind": "dense", "ff": 112, "limit": 3.0}},
            {"type": "attention",
             "mixer": {"heads": 4, "kv_heads": 2, "dim": 24, "vdim": 16,
                       "scale": 0.2, "kv_from": 0},
             "mlp": None},
        ],
    },
    "debug-sadosun": {
        "architecture": "Sadosun", "width": 80, "vocab": 320,
        "norm": {"eps": 1e-6}, "embedding": {"scale": 4.0},
        "canon": {"taps": 3}, "token_side": {"dim": 20},
        "layers": [
            {"type": "attention",
             "mixer": {"heads": 6, "kv_heads": 2, "dim": 24, "vdim": 16,
                       "scale": 0.2, "rot": {"base": 1000.0, "dims": 16},
                       "mask": {"size": 50}},
             "mlp": {"kind": "moe", "expert": {"ff": 48},
                     "router": {"experts": 6, "identity": 1, "top": 2}}},
            {"type": "mamba1",
             "mixer": {"inner": 120, "state": 10, "dt_rank": 6, "conv": 4},
             "mlp": None},
        ],
    },
    "debug-lepizen": {
        "architecture": "Lepizen", "width": 96, "vocab": 320,
        "norm": {"eps": 1e-6}, "residual_mult": 0.6, "logit_scale": 0.4,
        "logit_softcap": 20.0,
        "layers": [
            {"type": "attention", "mlp": None,
             "mixer": {"heads": 6, "kv_heads": 3, "dim": 24, "vdim": 40,
                       "scale": 0.2, "v_mix": False}},
            {"type": "attention", "mlp": {"kind": "dense", "ff": 160},
             "mixer": {"heads": 8, "kv_heads": 2, "dim": 16, "vdim": 24,
                       "scale": 0.25, "v_mix": True}},
            {"type": "attention", "mlp": {"kind": "dense", "ff": 112},
             "mixer": {"heads": 4, "kv_heads": 4, "dim": 32, "vdim": 12,
                       "scale": 0.18, "v_mix": True}},
        ],
    },
    "debug-tuvutar": {
        "architecture": "Tuvutar", "width": 96, "vocab": 320,
        "norm": {"eps": 1e-6},
        "layers": [
            {"type": "delta", "mlp": None,
             "mixer": {"heads": 4, "kv_heads": 2, "dim": 24, "vdim": 40,
                       "conv": 4}},
            {"type": "latent_attention", "mlp": {"kind": "dense", "ff": 160},
             "mixer": {"heads": 3, "dim": 32, "rot_dim": 16, "vdim": 24,
                       "kv_rank": 48, "scale": 0.14,
                       "rot": {"base": 10000.0, "dims": 16,
                               "scaling": {"factor": 4.0, "original": 512,
                                           "fast": 32.0, "slow": 1.0}}}},
            {"type": "delta", "mlp": {"kind": "dense", "ff": 128},
             "mixer": {"heads": 2, "kv_heads": 2, "dim": 16, "vdim": 16,
                       "conv": 3}},
            {"type": "latent_attention", "mlp": {"kind": "dense", "ff": 96},
             "mixer": {"heads": 5, "dim": 16, "rot_dim": 16, "vdim": 32,
                       "kv_rank": 48, "scale": 0.2, "kv_from": 1,
                       "rot": {"base": 10000.0, "dims": 16,
                               "scaling": {"factor": 4.0, "original": 512,
                                           "fast": 32.0, "slow": 1.0}}}},
        ],
    },
    "debug-deepseek": {
        "model_type": "deepseek_v2",
        "hidden_size": 128,
        "num_hidden_layers": 8,
        "intermediate_size": 256,
        "moe_intermediate_size": 64,
        "num_attention_heads": 4,
        "vocab_size": 512,
        "rms_norm_eps": 1e-6,
        "rope_theta": 10000.0,
        "q_lora_rank": None,
        "kv_lora_rank": 64,
        "qk_nope_head_dim": 32,
        "qk_rope_head_dim": 16,
        "v_head_dim": 32,
        "n_routed_experts": 8,
        "n_shared_experts": 1,
        "num_experts_per_tok": 2,
        "first_k_dense_replace": 1,
        "moe_layer_freq": 1,
        "rope_scaling": {"type": "yarn", "factor": 4.0, "beta_fast": 32,
                         "beta_slow": 1, "mscale": 0.707, "mscale_all_dim": 0.707,
                         "original_max_position_embeddings": 4096},
    },
}


def get_preset(name: str, quant: bool = False,
               group_size: int = 64, bits: int = 4) -> ModelConfig:
    raw = dict(PRESETS[name])
    if quant:
        raw["quantization"] = {"group_size": group_size, "bits": bits}
    return ModelConfig.from_dict(raw)
