"""Model registry: a checkpoint directory's config.json -> a Decoder with its weights.

The architecture is chosen by config.json: Hugging Face style files of the Phi, Qwen2, Gemma and Phi-3 families (the
serde Config structs rai-models/src/llm/phi2.rs:9-24, qwen2.rs:8-24, gemma.rs:12-27, phi3.rs read the same keys) by
"model_type" or the first entry of "architectures", Lelitar and Bezadra files by "architecture".
"""
from __future__ import annotations

import json
import struct
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
    def build(c, dtype, max_batch, max_context, dev, shapes):
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


def _lelitar(c, dtype, max_batch, max_context, dev, shapes):
    return Decoder.latent(dtype, vocab_size=c["vocab"], width=c["width"], layers=lelitar_layers(c),
                          norm_eps=c["norm"]["eps"], norm_groups=c["norm"].get("groups", 1),
                          residual_mult=c["residual_mult"], max_batch=max_batch, max_context=max_context or 2048, dev=dev)


def bezadra_layers(c, shapes):
    """The layer list of a Bezadra config.json as Decoder.hybrid takes it.  The ranks of a delta rule's two low-rank factors
    are not in the file: they are the row counts of the tensors in `shapes` (name -> shape)."""
    out = []
    for i, spec in enumerate(c["layers"]):
        m, mlp = spec["mixer"], spec.get("mlp")
        y = dict(mixer=spec["type"], heads=m["heads"], kv_heads=m["kv_heads"], qk_dim=m["dim"], v_dim=m["vdim"])
        if spec["type"] == "attention":
            rot, scaling = m["rot"], m["rot"].get("scaling")
            y.update(attn_scale=m["scale"], softcap=m.get("softcap") or 0.0, rot_dims=rot["dims"], rot_base=rot["base"])
            if scaling:
                y.update(rot_factor=scaling["factor"], rot_low=scaling["low"], rot_high=scaling["high"], rot_original=scaling["original"])
        elif spec["type"] == "channel_delta":
            names = f"l{i}.mix.a1", f"l{i}.mix.g1"
            missing = [n for n in names if n not in (shapes or {})]
            if missing:
                raise ConfigError(f"layer {i}: the ranks of its low-rank factors come from the shapes of {missing}, which are not given")
            y.update(conv_taps=m["conv"], decay_rank=shapes[names[0]][0], gate_rank=shapes[names[1]][0])
        else:
            raise ConfigError(f"config.json: layer {i} has mixer {spec['type']!r}; Bezadra layers are 'attention' or 'channel_delta'")
        if mlp is None:
            y.update(mlp_kind="none")
        elif mlp["kind"] == "dense":
            y.update(mlp_kind="dense", intermediate=mlp["ff"], mlp_limit=mlp["limit"], mlp_alpha=1.702)
        else:
            raise ConfigError(f"config.json: layer {i} has mlp kind {mlp['kind']!r}")
        out.append(y)
    return out


def _bezadra(c, dtype, max_batch, max_context, dev, shapes):
    loop = c.get("loop")
    return Decoder.hybrid(dtype, vocab_size=c["vocab"], width=c["width"], layers=bezadra_layers(c, shapes), norm_eps=c["norm"]["eps"],
                          embed_scale=c["embedding"]["scale"], logit_scale=c["logit_scale"],
                          loop=(loop["start"], loop["stop"], loop["times"]) if loop else None,
                          max_batch=max_batch, max_context=max_context or 2048, dev=dev)


REGISTRY = {"phi2": _hf("phi2"), "qwen2": _hf("qwen2"), "gemma": _hf("gemma"), "phi3": _hf("phi3"), "lelitar": _lelitar, "bezadra": _bezadra}


def tensor_shapes(paths):
    """name -> shape of every tensor of some safetensors files, from their headers alone."""
    out = {}
    for path in paths:
        with open(path, "rb") as f:
            n = struct.unpack("<Q", f.read(8))[0]
            out.update((k, v["shape"]) for k, v in json.loads(f.read(n)).items() if k != "__metadata__")
    return out


def decoder_from_config(cfg, dtype="bf16", *, max_batch=1, max_context=None, dev=0, shapes=None):
    """A decoder without weights for a parsed config.json; `shapes` (see tensor_shapes) for designs whose config.json leaves
    sizes to the tensors."""
    return REGISTRY[architecture(cfg)](cfg, dtype, max_batch, max_context, dev, shapes)


def load_model(model_dir, dtype="bf16", *, max_batch=1, max_context=None, dev=0):
    """config.json and the safetensors file(s) of a directory -> a Decoder ready to run."""
    model_dir = Path(model_dir)
    index = model_dir / "model.safetensors.index.json"
    files = safetensors_index_files(index) if index.exists() else [model_dir / "model.safetensors"]
    cfg = read_config(model_dir)
    shapes = tensor_shapes(files) if architecture(cfg) == "bezadra" else None
    dec = decoder_from_config(cfg, dtype, max_batch=max_batch, max_context=max_context, dev=dev, shapes=shapes)
    dec.load_safetensors(files)
    return dec
