"""Small Bezadra configurations and weights for the tests, and the device model built from them."""
import copy

import numpy as np

from oracle import bezadra
from oracle.dtypes import rnd, to_storage

SCALING = {"factor": 3.0, "low": 1.5, "high": 5.0, "original": 60}


def mlp_of(ff, limit):
    return None if ff is None else {"kind": "dense", "ff": ff, "limit": limit}


def attention(heads=6, kv_heads=3, dim=24, vdim=40, dims=16, base=900.0, scaling=SCALING, scale=0.6, softcap=2.5, ff=88, limit=1.1):
    rot = {"dims": dims, "base": base}
    if scaling:
        rot["scaling"] = dict(scaling)
    return {"type": "attention", "mlp": mlp_of(ff, limit),
            "mixer": dict(heads=heads, kv_heads=kv_heads, dim=dim, vdim=vdim, rot=rot, scale=scale, softcap=softcap)}


def delta(heads=4, kv_heads=2, dim=20, vdim=36, conv=3, ff=72, limit=1.3):
    return {"type": "channel_delta", "mlp": mlp_of(ff, limit), "mixer": dict(heads=heads, kv_heads=kv_heads, dim=dim, vdim=vdim, conv=conv)}


def config(layers, loop=None, vocab=301, width=120, eps=1e-5, embed_scale=3.0, logit_scale=0.7):
    c = {"architecture": "Bezadra", "vocab": vocab, "width": width, "norm": {"eps": eps}, "embedding": {"scale": embed_scale},
         "logit_scale": logit_scale, "layers": layers}
    if loop:
        c["loop"] = dict(zip(("start", "stop", "times"), loop))
    return c


def mixed_config(**kw):
    """Every kind of layer, each with sizes of its own, two of them looped three times."""
    kw.setdefault("loop", (1, 3, 3))
    return config([delta(), attention(), delta(heads=3, kv_heads=3, dim=40, vdim=24, conv=5, ff=None),
                   attention(heads=4, kv_heads=1, dim=32, vdim=16, dims=32, scaling=None, ff=None),
                   delta(heads=5, kv_heads=1, dim=8, vdim=72, conv=2, ff=40)], **kw)


def build(cfg, params, dt, max_batch=1, max_context=256):
    from rai_amd.config import decoder_from_config

    shapes = {k: list(v.shape) for k, v in params.items()}
    dec = decoder_from_config(cfg, dt, max_batch=max_batch, max_context=max_context, shapes=shapes)
    names = dec.param_names()
    assert {k: int(np.prod(s)) for k, s in shapes.items()} == names
    for n in names:
        dec.load_param(n, to_storage(np.asarray(params[n], np.float32), dt))
    return dec


def marked(params, marker):
    """Embedding rows that share feature 0, with feature 1 the marker's alone."""
    params["embed"][:, 0] = 3.0
    params["embed"][:, 1] = 0.0
    params["embed"][marker, 1] = 4.0
    return params


def standout_key_params(cfg, dt, seed, marker, strength=4.0):
    """Random weights under which the key of token `marker` wins every query of every attention head by a wide margin,
    however far back it is: queries are nearly constant along one feature that does not turn (or turns slowest), and
    only the marker's key has a large share along it; every other share of a score is small."""
    p = marked(bezadra.random_params(cfg, "f32", seed), marker)
    for i, spec in enumerate(cfg["layers"]):
        m, q = spec["mixer"], f"l{i}.mix."
        if spec["type"] != "attention":
            continue
        f = m["dim"] - 1 if m["rot"]["dims"] < m["dim"] else m["rot"]["dims"] // 2 - 1
        for name, heads, feature in (("q", m["heads"], 0), ("k", m["kv_heads"], 1)):
            p[q + name] *= 0.2
            for h in range(heads):
                p[q + name][h * m["dim"] + f] = 0.0
                p[q + name][h * m["dim"] + f, feature] = strength
        p[q + "sink"][:] = 1.0
    return {k: rnd(v, dt) for k, v in p.items()}


def long_memory_params(cfg, dt, seed, marker):
    """Random weights under which the recurrence keeps what token `marker` wrote: slow decays, a key of the marker's own
    that every query reads along, and a large value behind it."""
    p = marked(bezadra.random_params(cfg, "f32", seed), marker)
    for i, spec in enumerate(cfg["layers"]):
        m, q = spec["mixer"], f"l{i}.mix."
        if spec["type"] != "channel_delta":
            continue
        p[q + "dt_bias"][:] = -9.0
        for name in "qkv":
            p[q + name + ".conv"][:, -1] = 1.0
        for h in range(m["kv_heads"]):
            row = h * m["dim"]
            for name, feature in (("q", 0), ("k", 1)):
                p[q + name][row] = 0.0
                p[q + name][row, feature] = 3.0
        p[q + "v"][:, 1] *= 4.0
    return {k: rnd(v, dt) for k, v in p.items()}


def without(cfg, what):
    """The configuration with one thing changed: what a model that leaves a mechanism out would compute."""
    c = copy.deepcopy(cfg)
    for spec in c["layers"]:
        m = spec["mixer"]
        if what == "softcap" and spec["type"] == "attention":
            m["softcap"] = 1e6
        if what == "scaling" and spec["type"] == "attention":
            m["rot"].pop("scaling", None)
        if what == "limit" and spec["mlp"]:
            spec["mlp"]["limit"] = 1e6
    return c


def run_portions(dec, ids, sizes):
    """Logits of every token of `ids` [B, n], fed in portions of the given sizes (the last size repeats)."""
    ids = np.atleast_2d(ids)
    b, n = ids.shape
    dec.clear_kv_cache()
    out, at, k = [], 0, 0
    while at < n:
        s = min(sizes[min(k, len(sizes) - 1)], n - at)
        out.append(dec.forward_rows(ids[:, at:at + s], range(b * s)).reshape(b, s, -1))
        at, k = at + s, k + 1
    return np.concatenate(out, axis=1)
