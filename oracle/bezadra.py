"""Plain NumPy restatement of the Bezadra decoder (test infrastructure only, see oracle/__init__.py).

One function per mechanism, everything in float64 over the stored weights, no cache: a sequence is always evaluated
whole, the recurrence one token after the other.  Notation: x[t, :] is the residual stream of token t, W x is a Linear
with W stored [out, in].

    x0         = s E[token]
    x         <- x + mixer(n(x)) + mlp(n(x))            one norm for both, layer after layer
    x         <- Win [x; x0] + step[t]                  ahead of pass t of the looped run of layers
    logits     = c E n(x)

`cfg` is a dict with the keys of the model's config.json (see rai_amd/config.py for the reader of the product).
"""
import numpy as np

F = np.float64


def layer_norm(x, w, eps):
    d = x - x.mean(axis=-1, keepdims=True)
    return d / np.sqrt((d * d).mean(axis=-1, keepdims=True) + eps) * w


def rms(x, eps):
    return x / np.sqrt((x * x).mean(axis=-1, keepdims=True) + eps)


def unit(x):
    return x / np.sqrt((x * x).sum(axis=-1, keepdims=True) + 1e-6)


def sigmoid(z):
    e = np.exp(-np.abs(z))
    return np.where(z >= 0, 1.0 / (1.0 + e), e / (1.0 + e))


def silu(z):
    return z * sigmoid(z)


def softplus(z):
    return np.maximum(z, 0.0) + np.log1p(np.exp(-np.abs(z)))


def rotation_frequencies(dims, base, scaling=None):
    """f_i of the pairs of `dims` rotated features.  With `scaling`, waves longer than original / low positions are
    stretched by `factor`, those shorter than original / high kept, and the ones between blended by where original /
    wavelength falls between low and high."""
    f = float(base) ** (-2.0 * np.arange(dims // 2) / dims)
    if not scaling:
        return f
    turns = scaling["original"] * f / (2 * np.pi)       # original / wavelength
    s = np.clip((turns - scaling["low"]) / (scaling["high"] - scaling["low"]), 0.0, 1.0)
    return (1 - s) * f / scaling["factor"] + s * f


def rotate(x, positions, freq):
    """x [n, heads, dim]: feature i turns with feature i + len(freq); the rest stay."""
    k = len(freq)
    a = positions[:, None, None] * freq
    u, v = x[..., :k], x[..., k:2 * k]
    return np.concatenate([u * np.cos(a) - v * np.sin(a), v * np.cos(a) + u * np.sin(a), x[..., 2 * k:]], axis=-1)


def sink_softmax(s, sink):
    """Softmax over the last axis whose denominator has one more term, exp(sink)."""
    m = np.maximum(s.max(axis=-1, keepdims=True), sink)
    e = np.exp(s - m)
    return e / (e.sum(axis=-1, keepdims=True) + np.exp(sink - m))


def attention(h, p, heads, kv_heads, dim, vdim, scale, softcap, rot):
    """Grouped-query attention with rotation, capped scores, a sink in the softmax and an output gate (h [n, width]).

    p: q, k, v, sink, g, o."""
    n = h.shape[0]
    pos = np.arange(n)
    freq = rotation_frequencies(rot["dims"], rot["base"], rot.get("scaling"))
    q = rotate((h @ p["q"].T).reshape(n, heads, dim), pos, freq)
    k = rotate((h @ p["k"].T).reshape(n, kv_heads, dim), pos, freq)
    v = (h @ p["v"].T).reshape(n, kv_heads, vdim)
    see = pos[None, :] <= pos[:, None]
    out = np.empty((n, heads, vdim), F)
    for hd in range(heads):
        kv = hd // (heads // kv_heads)
        s = (q[:, hd] @ k[:, kv].T) * scale
        if softcap:
            s = softcap * np.tanh(s / softcap)
        out[:, hd] = sink_softmax(np.where(see, s, -np.inf), p["sink"][hd]) @ v[:, kv]
    return (out.reshape(n, heads * vdim) * sigmoid(h @ p["g"].T)) @ p["o"].T


def causal_conv(x, w):
    """x [n, channels], w [channels, taps]: the last tap meets the token itself, zeros lie before the first one."""
    n, taps = x.shape[0], w.shape[1]
    past = np.concatenate([np.zeros((taps - 1, x.shape[1]), F), x])
    return sum(past[j:j + n] * w[:, j] for j in range(taps))


def decays(h, p, heads, dim):
    """g [n, heads, dim] in (0, 1): the rate per head, its time step per key channel from a low-rank factor."""
    dt = softplus((h @ p["a1"].T) @ p["a2"].T + p["dt_bias"]).reshape(h.shape[0], heads, dim)
    return np.exp(-np.exp(p["A_log"])[:, None] * dt)


def delta_recurrence(q, k, v, g, beta):
    """One head, token by token from an empty state S [dim, vdim]: decay the rows, write the part of v that the
    decayed state does not already return for k, read with q.  q, k, g [n, dim]; v [n, vdim]; beta [n]."""
    S = np.zeros((k.shape[1], v.shape[1]), F)
    out = np.empty_like(v)
    for t in range(len(k)):
        S = g[t][:, None] * S
        S = S + np.outer(k[t], beta[t] * (v[t] - S.T @ k[t]))
        out[t] = S.T @ q[t]
    return out


def channel_delta(h, p, heads, kv_heads, dim, vdim, eps):
    """Gated delta rule with a decay per key channel (h [n, width]).

    p: q, k, v and their .conv, b, a1, a2, A_log, dt_bias, norm, g1, g2, o."""
    n = h.shape[0]
    q, k, v = (silu(causal_conv(h @ p[c].T, p[c + ".conv"])) for c in "qkv")
    q = unit(q.reshape(n, kv_heads, dim)) * dim ** -0.5
    k = unit(k.reshape(n, kv_heads, dim))
    v = v.reshape(n, heads, vdim)
    beta = sigmoid(h @ p["b"].T)
    g = decays(h, p, heads, dim)
    out = np.empty((n, heads, vdim), F)
    for hd in range(heads):
        kv = hd // (heads // kv_heads)
        out[:, hd] = delta_recurrence(q[:, kv], k[:, kv], v[:, hd], g[:, hd], beta[:, hd])
    gate = sigmoid((h @ p["g1"].T) @ p["g2"].T).reshape(n, heads, vdim)
    return (rms(out, eps) * p["norm"] * gate).reshape(n, heads * vdim) @ p["o"].T


def clamped_mlp(h, p, limit):
    """down(a sigmoid(1.702 a) (u + 1)) with a = gate h cut off above `limit` and u = up h on both sides."""
    a = np.minimum(h @ p["gate"].T, limit)
    u = np.clip(h @ p["up"].T, -limit, limit)
    return (a * sigmoid(1.702 * a) * (u + 1.0)) @ p["down"].T


def loop_entry(x, x0, w_in, step):
    return np.concatenate([x, x0], axis=-1) @ w_in.T + step


def sub(params, prefix):
    """The parameters under a dotted prefix, without it."""
    return {k[len(prefix) + 1:]: v for k, v in params.items() if k.startswith(prefix + ".")}


def layer(x, cfg, i, params):
    spec, eps = cfg["layers"][i], cfg["norm"]["eps"]
    mx, p = spec["mixer"], sub(params, f"l{i}.mix")
    h = layer_norm(x, params[f"l{i}.norm1"], eps)
    if spec["type"] == "attention":
        y = attention(h, p, mx["heads"], mx["kv_heads"], mx["dim"], mx["vdim"], mx["scale"], mx["softcap"], mx["rot"])
    else:
        y = channel_delta(h, p, mx["heads"], mx["kv_heads"], mx["dim"], mx["vdim"], eps)
    if spec["mlp"] is not None:
        y = y + clamped_mlp(h, sub(params, f"l{i}.mlp"), spec["mlp"]["limit"])
    return x + y


def schedule(cfg):
    """(layer, pass or None) in the order they run; pass t is given on the first layer of each pass."""
    n, loop = len(cfg["layers"]), cfg.get("loop")
    if not loop:
        return [(i, None) for i in range(n)]
    run = list(range(loop["start"], loop["stop"]))
    out = [(i, None) for i in range(loop["start"])]
    for t in range(loop["times"]):
        out += [(i, t if i == run[0] else None) for i in run]
    return out + [(i, None) for i in range(loop["stop"], n)]


class Model:
    def __init__(self, cfg, params):
        self.cfg, self.p = cfg, {k: np.asarray(v, F) for k, v in params.items()}

    def hidden(self, ids):
        """Residual stream after every layer run, [layer runs, n, width], of one sequence of token ids."""
        x0 = self.p["embed"][np.asarray(ids, np.int64)] * self.cfg["embedding"]["scale"]
        x, out = x0, []
        for i, t in schedule(self.cfg):
            if t is not None:
                x = loop_entry(x, x0, self.p["loop.in"], self.p["loop.step"][t])
            x = layer(x, self.cfg, i, self.p)
            out.append(x)
        return np.stack(out)

    def logits(self, ids, hidden=None):
        """[n, vocab] of one sequence."""
        x = self.hidden(ids)[-1] if hidden is None else hidden
        return layer_norm(x, self.p["final.norm"], self.cfg["norm"]["eps"]) @ self.p["embed"].T * self.cfg["logit_scale"]

    def greedy(self, prompt, n_new):
        """Tokens (and the logits they were chosen from), each step over the whole sequence so far."""
        ids, rows = list(prompt), []
        for _ in range(n_new):
            rows.append(self.logits(ids)[-1])
            ids.append(int(np.argmax(rows[-1])))
        return np.array(ids[len(prompt):], np.uint32), np.stack(rows)


def param_shapes(cfg, a_rank=12, g_rank=20):
    """Tensor names and shapes of a model with this configuration; the ranks of the two low-rank factors of a
    channel_delta mixer are not in the configuration."""
    h, v = cfg["width"], cfg["vocab"]
    out = {"embed": (v, h)}
    if cfg.get("loop"):
        out.update({"loop.in": (h, 2 * h), "loop.step": (cfg["loop"]["times"], h)})
    for i, spec in enumerate(cfg["layers"]):
        mx, ml, p = spec["mixer"], spec["mlp"], f"l{i}."
        qd, kd = mx["heads"] * mx["dim"], mx["kv_heads"] * mx["dim"]
        vd = mx["heads"] * mx["vdim"]
        out[p + "norm1"] = (h,)
        if spec["type"] == "attention":
            out.update({p + "mix.q": (qd, h), p + "mix.k": (kd, h), p + "mix.v": (mx["kv_heads"] * mx["vdim"], h),
                        p + "mix.sink": (mx["heads"],), p + "mix.g": (vd, h), p + "mix.o": (h, vd)})
        else:
            taps = mx["conv"]
            out.update({p + "mix.q": (kd, h), p + "mix.q.conv": (kd, taps), p + "mix.k": (kd, h), p + "mix.k.conv": (kd, taps),
                        p + "mix.v": (vd, h), p + "mix.v.conv": (vd, taps), p + "mix.b": (mx["heads"], h),
                        p + "mix.A_log": (mx["heads"],), p + "mix.norm": (mx["vdim"],), p + "mix.a1": (a_rank, h),
                        p + "mix.a2": (qd, a_rank), p + "mix.dt_bias": (qd,), p + "mix.g1": (g_rank, h), p + "mix.g2": (vd, g_rank),
                        p + "mix.o": (h, vd)})
        if ml is not None:
            out.update({p + "mlp.gate": (ml["ff"], h), p + "mlp.up": (ml["ff"], h), p + "mlp.down": (h, ml["ff"])})
    out["final.norm"] = (h,)
    return out


def random_params(cfg, dt, seed=0, **ranks):
    """Random weights whose values `dt` can hold: matrices scaled by their fan-in, norm weights around 1, decays between
    a few tokens' memory and a few hundred's."""
    from .dtypes import rnd

    rng = np.random.Generator(np.random.PCG64(seed))
    out = {}
    for name, shape in param_shapes(cfg, **ranks).items():
        a = rng.standard_normal(shape, dtype=np.float32)
        if name.endswith(("norm1", ".norm")):
            a = np.float32(1) + np.float32(0.1) * a
        elif name.endswith("A_log"):
            a = np.float32(0.5) * a
        elif name.endswith("dt_bias"):
            a = np.float32(-3) + np.float32(1.5) * a
        elif name.endswith(".conv"):
            a *= np.float32(1.0 / np.sqrt(shape[1]))
        elif name == "embed":
            a *= np.float32(0.3)
        elif name not in ("loop.step",) and not name.endswith("sink"):
            a *= np.float32(1.0 / np.sqrt(shape[1]))
        out[name] = rnd(a, dt)
    return out
