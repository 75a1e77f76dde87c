"""Small Lelitar configurations and weights for the tests, and the device model built from them."""
import copy

import numpy as np

from oracle import lelitar
from oracle.dtypes import rnd, to_storage


def layer(heads=3, dim=24, vdim=40, q_rank=48, kv_rank=72, window=19, scale=0.2, mlp="dense", ff=88, experts=6, top=2):
    mixer = dict(heads=heads, dim=dim, vdim=vdim, q_rank=q_rank, kv_rank=kv_rank, scale=scale,
                 mask=None if window is None else {"size": window})
    if mlp == "dense":
        mlp = {"kind": "dense", "ff": ff}
    elif mlp == "moe":
        mlp = {"kind": "moe", "expert": {"ff": ff}, "router": {"experts": experts, "top": top}}
    return {"type": "latent_attention", "mixer": mixer, "mlp": mlp}


def config(layers, vocab=301, width=120, groups=3, eps=1e-5, mult=0.45):
    return {"architecture": "Lelitar", "vocab": vocab, "width": width, "norm": {"eps": eps, "groups": groups},
            "residual_mult": mult, "layers": layers}


def mixed_config(**kw):
    """Every kind of layer, each with sizes of its own."""
    return config([layer(), layer(heads=5, dim=32, vdim=16, q_rank=40, kv_rank=64, window=33, mlp="moe", ff=48),
                   layer(heads=2, dim=72, vdim=24, q_rank=24, kv_rank=136, window=None, mlp=None),
                   layer(heads=1, dim=8, vdim=8, q_rank=72, kv_rank=24, window=7, mlp="moe", ff=24, experts=70, top=3)], **kw)


def clear_routing(cfg, params, seed):
    """Gives every token one of a few classes, in features that no layer writes and only the routers read, and every
    class its own ranking of the experts with even distances between their logits.  No choice is then a close call that
    a rounding could turn, which would change a token's whole mixture."""
    rng = np.random.Generator(np.random.PCG64(seed + 1000))
    n = max(2, min(16, cfg["width"] // 5))
    block = slice(cfg["width"] - n, cfg["width"])
    params["embed"][:, block] = 0.0
    params["embed"][np.arange(cfg["vocab"]), cfg["width"] - n + np.arange(cfg["vocab"]) % n] = 5.0
    for name, a in params.items():
        if name.endswith(("mix.o", ".down")):
            a[block] = 0.0
        elif name.endswith(".router"):
            a[:] = 0.0
            for c in range(n):
                a[:, cfg["width"] - n + c] = 0.2 - 0.1 * rng.permutation(len(a))
    return params


def random_params(cfg, dt, seed=0):
    p = lelitar.random_params(cfg, "f32", seed)
    if any((spec["mlp"] or {}).get("kind") == "moe" for spec in cfg["layers"]):
        clear_routing(cfg, p, seed)
    return {k: rnd(v, dt) for k, v in p.items()}


def build(cfg, params, dt, max_batch=1, max_context=256):
    from rai_amd.config import decoder_from_config

    dec = decoder_from_config(cfg, dt, max_batch=max_batch, max_context=max_context)
    names = dec.param_names()
    assert {k: int(np.prod(s)) for k, s in lelitar.param_shapes(cfg).items()} == names
    for n in names:
        dec.load_param(n, to_storage(np.asarray(params[n], np.float32), dt))
    return dec


def standout_params(cfg, dt, seed, marker, strength=0.5):
    """Random weights under which the key of token `marker` wins every query of every head by a wide margin, so that
    seeing or missing it decides the attention's output.  All tokens share feature 0, from which the queries are made
    nearly constant; feature 1 is the marker's alone and its key direction is the query's."""
    p = random_params(cfg, "f32", seed)
    p["embed"][:, 0] = 3.0
    p["embed"][:, 1] = 0.0
    p["embed"][marker, 1] = 8.0
    for i, spec in enumerate(cfg["layers"]):
        m, q = spec["mixer"], f"l{i}.mix."
        p[q + "dq"][0] = 0.0
        p[q + "dq"][0, 0] = 4.0                      # first query latent: feature 0
        p[q + "dkv"][0] = 0.0
        p[q + "dkv"][0, 1] = 4.0                     # first key latent: feature 1
        for h in range(m["heads"]):
            uq = p[q + "uq"][h * m["dim"]:(h + 1) * m["dim"], 0]
            p[q + "uk"][h * m["dim"]:(h + 1) * m["dim"], 0] = strength * uq / max(np.linalg.norm(uq), 1e-3)
            uq *= strength / max(np.linalg.norm(uq), 1e-3)
    return {k: rnd(v, dt) for k, v in p.items()}


def with_window(cfg, delta):
    """The configuration with every window shifted by delta: what an off-by-one mask would compute."""
    c = copy.deepcopy(cfg)
    for spec in c["layers"]:
        if spec["mixer"]["mask"]:
            spec["mixer"]["mask"]["size"] += delta
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
