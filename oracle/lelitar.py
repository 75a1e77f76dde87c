"""Plain NumPy restatement of the Lelitar decoder (test infrastructure only, see oracle/__init__.py).

One function per mechanism, everything in float64 over the stored weights, no cache: a sequence is always evaluated
whole.  Notation: x[t, :] is the residual stream of token t, W x is a Linear with W stored [out, in].

    x_0        = E[token]
    x_{l+1}    = x_l + m * (attention_l(n1_l(x_l)) + mlp_l(n2_l(x_l)))
    logits     = head . n(x_L)

`cfg` is a dict with the keys of the model's config.json (see rai_amd/config.py for the reader of the product).
"""
import numpy as np

F = np.float64


def rms(x, eps):
    """x / sqrt(mean(x^2) + eps) over the last axis."""
    return x / np.sqrt(np.mean(x * x, axis=-1, keepdims=True) + eps)


def grouped_rms_norm(x, w, groups, eps):
    """The last axis in `groups` equal runs, each divided by its own root mean square; one weight per element."""
    parts = x.reshape(x.shape[:-1] + (groups, x.shape[-1] // groups))
    return rms(parts, eps).reshape(x.shape) * w


def sigmoid(z):
    return np.where(z >= 0, 1.0 / (1.0 + np.exp(-np.abs(z))), np.exp(-np.abs(z)) / (1.0 + np.exp(-np.abs(z))))


def softmax(z):
    e = np.exp(z - z.max(axis=-1, keepdims=True))
    return e / e.sum(axis=-1, keepdims=True)


def window_mask(n, size):
    """mask[i, j]: position i sees j, the last `size` positions up to and including itself (None: every earlier one)."""
    i, j = np.arange(n)[:, None], np.arange(n)[None, :]
    return (j <= i) & ((i - j < size) if size is not None else True)


def latent_attention(h, p, heads, dim, vdim, scale, window, eps):
    """Attention over a latent: q from one low-rank factor, every head's k and v from another (h [n, width]).

    p: dq, dq.norm, uq, dkv, dkv.norm, uk, uv, g, o."""
    n = h.shape[0]
    cq = rms(h @ p["dq"].T, eps) * p["dq.norm"]
    c = rms(h @ p["dkv"].T, eps) * p["dkv.norm"]
    q = (cq @ p["uq"].T).reshape(n, heads, dim)
    k = (c @ p["uk"].T).reshape(n, heads, dim)
    v = (c @ p["uv"].T).reshape(n, heads, vdim)
    see = window_mask(n, window)
    out = np.empty((n, heads, vdim), F)
    for hd in range(heads):
        s = np.where(see, (q[:, hd] @ k[:, hd].T) * scale, -np.inf)
        out[:, hd] = softmax(s) @ v[:, hd]
    return (out.reshape(n, heads * vdim) * sigmoid(h @ p["g"].T)) @ p["o"].T


def gated_mlp(h, p, act):
    """down(act(gate h) * (up h))."""
    return (act(h @ p["gate"].T) * (h @ p["up"].T)) @ p["down"].T


def relu(z):
    return np.maximum(z, 0.0)


def silu(z):
    return z * sigmoid(z)


def route(h, router, top):
    """(chosen [n, top], weights [n, top]): the largest sigmoid scores, not renormalised."""
    s = sigmoid(h @ router.T)
    chosen = np.argsort(-s, axis=-1, kind="stable")[:, :top]
    return chosen, np.take_along_axis(s, chosen, -1)


def mixture(h, p, top):
    """Sum over the chosen experts of expert(score * h): the score scales what goes into the expert."""
    chosen, w = route(h, p["router"], top)
    out = np.zeros_like(h)
    for t in range(h.shape[0]):
        for e, s in zip(chosen[t], w[t]):
            out[t] += gated_mlp(s * h[t], {k: p[f"e{e}.{k}"] for k in ("gate", "up", "down")}, silu)
    return out


def sub(params, prefix):
    """The parameters under a dotted prefix, without it."""
    return {k[len(prefix) + 1:]: v for k, v in params.items() if k.startswith(prefix + ".")}


def layer(x, cfg, i, params):
    """One block: both branches read the same x, each behind its own norm."""
    spec, norm = cfg["layers"][i], cfg["norm"]
    mx = spec["mixer"]
    n1 = grouped_rms_norm(x, params[f"l{i}.norm1"], norm["groups"], norm["eps"])
    window = (mx.get("mask") or {}).get("size")
    y = latent_attention(n1, sub(params, f"l{i}.mix"), mx["heads"], mx["dim"], mx["vdim"], mx["scale"], window, norm["eps"])
    if spec["mlp"] is not None:
        n2 = grouped_rms_norm(x, params[f"l{i}.norm2"], norm["groups"], norm["eps"])
        p = sub(params, f"l{i}.mlp")
        y = y + (gated_mlp(n2, p, relu) if spec["mlp"]["kind"] == "dense" else mixture(n2, p, spec["mlp"]["router"]["top"]))
    return x + cfg["residual_mult"] * y


class Model:
    def __init__(self, cfg, params):
        self.cfg, self.p = cfg, {k: np.asarray(v, F) for k, v in params.items()}

    def hidden(self, ids):
        """Residual stream after every layer, [layers, n, width], of one sequence of token ids."""
        x, out = self.p["embed"][np.asarray(ids, np.int64)], []
        for i in range(len(self.cfg["layers"])):
            x = layer(x, self.cfg, i, self.p)
            out.append(x)
        return np.stack(out)

    def logits(self, ids, hidden=None):
        """[n, vocab] of one sequence."""
        x = self.hidden(ids)[-1] if hidden is None else hidden
        norm = self.cfg["norm"]
        return grouped_rms_norm(x, self.p["final.norm"], norm["groups"], norm["eps"]) @ self.p["head"].T

    def greedy(self, prompt, n_new):
        """Tokens (and the logits they were chosen from), each step over the whole sequence so far."""
        ids, rows = list(prompt), []
        for _ in range(n_new):
            rows.append(self.logits(ids)[-1])
            ids.append(int(np.argmax(rows[-1])))
        return np.array(ids[len(prompt):], np.uint32), np.stack(rows)


def param_shapes(cfg):
    """Tensor names and shapes of a model with this configuration."""
    h, v = cfg["width"], cfg["vocab"]
    out = {"embed": (v, h)}
    for i, spec in enumerate(cfg["layers"]):
        mx, ml, p = spec["mixer"], spec["mlp"], f"l{i}."
        qd, vd = mx["heads"] * mx["dim"], mx["heads"] * mx["vdim"]
        out[p + "norm1"] = (h,)
        if ml is not None:
            out[p + "norm2"] = (h,)
        out.update({p + "mix.dq": (mx["q_rank"], h), p + "mix.dq.norm": (mx["q_rank"],), p + "mix.uq": (qd, mx["q_rank"]),
                    p + "mix.dkv": (mx["kv_rank"], h), p + "mix.dkv.norm": (mx["kv_rank"],),
                    p + "mix.uk": (qd, mx["kv_rank"]), p + "mix.uv": (vd, mx["kv_rank"]), p + "mix.g": (vd, h),
                    p + "mix.o": (h, vd)})
        if ml is None:
            continue
        if ml["kind"] == "dense":
            out.update({p + "mlp.gate": (ml["ff"], h), p + "mlp.up": (ml["ff"], h), p + "mlp.down": (h, ml["ff"])})
        else:
            ff = ml["expert"]["ff"]
            for e in range(ml["router"]["experts"]):
                q = f"{p}mlp.e{e}."
                out.update({q + "gate": (ff, h), q + "up": (ff, h), q + "down": (h, ff)})
            out[p + "mlp.router"] = (ml["router"]["experts"], h)
    out.update({"final.norm": (h,), "head": (v, h)})
    return out


def random_params(cfg, dt, seed=0):
    """Random weights whose values `dt` can hold: matrices scaled by their fan-in, norm weights around 1."""
    from .dtypes import rnd

    rng = np.random.Generator(np.random.PCG64(seed))
    out = {}
    for name, shape in param_shapes(cfg).items():
        a = rng.standard_normal(shape, dtype=np.float32)
        if len(shape) == 1:
            a = np.float32(1) + np.float32(0.1) * a
        elif name not in ("embed",):
            a *= np.float32(1.0 / np.sqrt(shape[1]))
        out[name] = rnd(a, dt)
    return out
