"""Model registry: a checkpoint directory's config.json -> a Decoder with its weights.

The architecture is chosen by config.json: Hugging Face style files of the Phi, Qwen2, Gemma and Phi-3 families (the
serde Config structs rai-models/src/llm/phi2.rs:9-24, qwen2.rs:8-24, gemma.rs:12-27, phi3.rs read the same keys) by
"model_type" or the first entry of "architectures", and Lelitar files by "architecture".
"""
from __future__ import annotations

import json
from pathlib import Path

from .models import Decoder, safetensors_index_files


class ConfigError(ValueError):
    pass


def read_config(model_dir):
    return json.loads((Path(model_dir) / "config.json").read_text())


def architecture(cfg):
    """The registry name of a parsed config.json."""
    name = cfg.get("model_type") or cfg.get("architecture") or (cfg.get("architectures") or [""])[0]
    key = name.lower()
    for suffix in ("forcausallm", "model"):
        key = key.removesuffix(suffix)
    key = {"phi": "phi2", "phi-msft": "phi2"}.get(key, key)
    if key not in REGISTRY:
        raise ConfigError(f"config.json: architecture {name!r} is not one of {sorted(REGISTRY)}")
    return key


def _hf_kwargs(arch, c):
    heads = c["num_attention_heads"]
    head_dim = c.get("head_dim") or c["hidden_size"] // heads
    rotary = int(c.get("partial_rotary_factor", 0.5 if arch == "phi2" else 1.0) * head_dim)
    return dict(vocab_size=c["vocab_size"], hidden_size=c["hidden_size"], intermediate_size=c["intermediate_size"],
                num_hidden_layers=c["num_hidden_layers"], num_attention_heads=heads,
                num_key_value_heads=c.get("num_key_value_heads") or heads, head_dim=head_dim, rotary_dim=rotary,
                max_position_embeddings=c["max_position_embeddings"],
                hidden_act=c.get("hidden_act") or c.get("hidden_activation") or "gelu_new",
                tie_word_embeddings=bool(c.get("tie_word_embeddings", arch == "gemma")),
                rope_theta=c.get("rope_theta", 10000.0), norm_eps=c.get("rms_norm_eps", c.get("layer_norm_eps", 1e-5)),
                qk_layernorm=bool(c.get("qk_layernorm", False)))


def _hf(arch):
    def build(c, dtype, max_batch, max_context, dev):
        kw = _hf_kwargs(arch, c)
        max_context = min(max_context or kw["max_position_embeddings"], kw["max_position_embeddings"])
        return Decoder(arch, dtype, max_batch=max_batch, max_context=max_context, dev=dev, **kw)
    return build


def lelitar_layers(c):
    """The layer list of a Lelitar config.json as Decoder.latent takes it.  Activations and the router's form are fixed
    by the design: relu in a dense MLP, silu in an expert, sigmoid scores on the expert's input."""
    out = []
    for i, spec in enumerate(c["layers"]):
        if spec["type"] != "latent_attention":
            raise ConfigError(f"config.json: layer {i} has mixer {spec['type']!r}; Lelitar layers are 'latent_attention'")
        m, mlp = spec["mixer"], spec.get("mlp")
        y = dict(heads=m["heads"], qk_dim=m["dim"], v_dim=m["vdim"], q_rank=m["q_rank"], kv_rank=m["kv_rank"],
                 window=(m.get("mask") or {}).get("size") or 0, attn_scale=m["scale"])
        if mlp is None:
            y.update(mlp_kind="none")
        elif mlp["kind"] == "dense":
            y.update(mlp_kind="dense", mlp_act="relu", intermediate=mlp["ff"])
        elif mlp["kind"] == "moe":
            y.update(mlp_kind="moe", mlp_act="silu", intermediate=mlp["expert"]["ff"], experts=mlp["router"]["experts"],
                     top=mlp["router"]["top"])
        else:
            raise ConfigError(f"config.json: layer {i} has mlp kind {mlp['kind']!r}")
        out.append(y)
    return out


def _lelitar(c, dtype, max_batch, max_context, dev):
    return Decoder.latent(dtype, vocab_size=c["vocab"], width=c["width"], layers=lelitar_layers(c),
                          norm_eps=c["norm"]["eps"], norm_groups=c["norm"].get("groups", 1),
                          residual_mult=c["residual_mult"], max_batch=max_batch, max_context=max_context or 2048, dev=dev)


REGISTRY = {"phi2": _hf("phi2"), "qwen2": _hf("qwen2"), "gemma": _hf("gemma"), "phi3": _hf("phi3"), "lelitar": _lelitar}


def decoder_from_config(cfg, dtype="bf16", *, max_batch=1, max_context=None, dev=0):
    """A decoder without weights for a parsed config.json."""
    return REGISTRY[architecture(cfg)](cfg, dtype, max_batch, max_context, dev)


def load_model(model_dir, dtype="bf16", *, max_batch=1, max_context=None, dev=0):
    """config.json and the safetensors file(s) of a directory -> a Decoder ready to run."""
    model_dir = Path(model_dir)
    dec = decoder_from_config(read_config(model_dir), dtype, max_batch=max_batch, max_context=max_context, dev=dev)
    index = model_dir / "model.safetensors.index.json"
    dec.load_safetensors(safetensors_index_files(index) if index.exists() else model_dir / "model.safetensors")
    return dec
