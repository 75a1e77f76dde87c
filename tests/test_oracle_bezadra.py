"""The Bezadra restatement against sums written out term by term, and the config.json reader (CPU)."""
import json
import math
import struct

import numpy as np
import pytest

from oracle import bezadra
from tests import bezadra_models as bm


def rng(seed):
    return np.random.Generator(np.random.PCG64(seed))


def sig(z):
    return 1 / (1 + math.exp(-z))


def test_layer_norm_term_by_term():
    x, w = rng(0).standard_normal((2, 12)) + 3, rng(1).standard_normal(12)
    got = bezadra.layer_norm(x, w, 0.25)
    for t in range(2):
        mean = sum(map(float, x[t])) / 12
        var = sum((float(v) - mean) ** 2 for v in x[t]) / 12
        for i in range(12):
            assert math.isclose(got[t, i], (x[t, i] - mean) / math.sqrt(var + 0.25) * w[i], rel_tol=1e-10)


def test_frequencies_in_three_ranges():
    s = dict(factor=4.0, low=1.0, high=4.0, original=1000)
    plain, got = (bezadra.rotation_frequencies(32, 30000.0, x) for x in (None, s))
    kinds = set()
    for i in range(16):
        f = 30000.0 ** (-2 * i / 32)
        assert math.isclose(plain[i], f, rel_tol=1e-12)
        wave = 2 * math.pi / f
        if wave < 250:
            want, kind = f, "kept"
        elif wave > 1000:
            want, kind = f / 4, "stretched"
        else:
            mix = (1000 / wave - 1) / 3
            want, kind = (1 - mix) * f / 4 + mix * f, "blended"
        kinds.add(kind)
        assert math.isclose(got[i], want, rel_tol=1e-12)
    assert kinds == {"kept", "stretched", "blended"}


def test_rotation_term_by_term():
    x, f = rng(2).standard_normal((3, 2, 7)), bezadra.rotation_frequencies(4, 50.0)
    got = bezadra.rotate(x, np.arange(3), f)
    for p in range(3):
        for h in range(2):
            for i in range(2):
                a, u, v = p * f[i], x[p, h, i], x[p, h, i + 2]
                assert math.isclose(got[p, h, i], u * math.cos(a) - v * math.sin(a), rel_tol=1e-9, abs_tol=1e-12)
                assert math.isclose(got[p, h, i + 2], v * math.cos(a) + u * math.sin(a), rel_tol=1e-9, abs_tol=1e-12)
            assert np.array_equal(got[p, h, 4:], x[p, h, 4:])


def test_attention_term_by_term():
    cfg = bm.config([bm.attention(heads=4, kv_heads=2, dim=6, vdim=3, dims=4, softcap=1.5, scale=0.8)], width=9)
    p = {k: np.asarray(v, np.float64) for k, v in bezadra.sub(bezadra.random_params(cfg, "f32", 1), "l0.mix").items()}
    h = rng(3).standard_normal((7, 9))
    rot = cfg["layers"][0]["mixer"]["rot"]
    got = bezadra.attention(h, p, 4, 2, 6, 3, 0.8, 1.5, rot)
    f = bezadra.rotation_frequencies(4, rot["base"], rot["scaling"])
    turn = lambda z, t: bezadra.rotate(z[None, None], np.array([t]), f)[0, 0]
    for i in range(7):
        cat = np.zeros(12)
        for hd in range(4):
            kv = hd // 2
            q = turn(p["q"][6 * hd:6 * hd + 6] @ h[i], i)
            e = []
            for j in range(i + 1):
                s = 0.8 * float(q @ turn(p["k"][6 * kv:6 * kv + 6] @ h[j], j))
                e.append(math.exp(1.5 * math.tanh(s / 1.5)))
            total = sum(e) + math.exp(float(p["sink"][hd]))
            cat[3 * hd:3 * hd + 3] = sum(w / total * (p["v"][3 * kv:3 * kv + 3] @ h[j]) for j, w in enumerate(e))
        want = p["o"] @ (cat / (1 + np.exp(-(p["g"] @ h[i]))))
        assert np.allclose(got[i], want, rtol=1e-9)


def test_channel_delta_term_by_term():
    """Scalar loops over heads, rows and columns, the convolution over explicit earlier tokens."""
    H, G, D, E, taps, n = 4, 2, 3, 2, 3, 6
    cfg = bm.config([bm.delta(heads=H, kv_heads=G, dim=D, vdim=E, conv=taps)], width=5)
    p = {k: np.asarray(v, np.float64) for k, v in bezadra.sub(bezadra.random_params(cfg, "f32", 4, a_rank=2, g_rank=3), "l0.mix").items()}
    h = rng(5).standard_normal((n, 5))
    got = bezadra.channel_delta(h, p, H, G, D, E, 1e-5)

    def conv(name, t):
        out = []
        for c in range(len(p[name])):
            y = sum(p[name + ".conv"][c, j] * float(p[name][c] @ h[t - (taps - 1) + j]) for j in range(taps) if t - (taps - 1) + j >= 0)
            out.append(y * sig(y))
        return out

    S = np.zeros((H, D, E))
    for t in range(n):
        q, k, v = conv("q", t), conv("k", t), conv("v", t)
        cat = []
        for hd in range(H):
            g = hd // (H // G)
            qh, kh = q[D * g:D * g + D], k[D * g:D * g + D]
            qn, kn = (math.sqrt(sum(x * x for x in z) + 1e-6) for z in (qh, kh))
            qh, kh = [x / qn / math.sqrt(D) for x in qh], [x / kn for x in kh]
            beta = sig(float(p["b"][hd] @ h[t]))
            for r in range(D):
                z = float(p["a2"][hd * D + r] @ (p["a1"] @ h[t])) + p["dt_bias"][hd * D + r]
                S[hd, r] *= math.exp(-math.exp(p["A_log"][hd]) * math.log1p(math.exp(z)))
            u = [beta * (v[hd * E + c] - sum(S[hd, r, c] * kh[r] for r in range(D))) for c in range(E)]
            for r in range(D):
                for c in range(E):
                    S[hd, r, c] += kh[r] * u[c]
            o = [sum(S[hd, r, c] * qh[r] for r in range(D)) for c in range(E)]
            ms = math.sqrt(sum(x * x for x in o) / E + 1e-5)
            for c in range(E):
                cat.append(o[c] / ms * p["norm"][c] * sig(float(p["g2"][hd * E + c] @ (p["g1"] @ h[t]))))
        assert np.allclose(got[t], p["o"] @ np.array(cat), rtol=1e-8)


def test_mlp_term_by_term():
    cfg = bm.config([bm.delta(ff=4, limit=0.5)], width=6)
    p = {k: np.asarray(v, np.float64) for k, v in bezadra.sub(bezadra.random_params(cfg, "f32", 6), "l0.mlp").items()}
    h = 2 * rng(7).standard_normal((9, 6))
    got, cut = bezadra.clamped_mlp(h, p, 0.5), set()
    for t in range(9):
        y = []
        for r in range(4):
            a, b = float(p["gate"][r] @ h[t]), float(p["up"][r] @ h[t])
            cut |= {("a", a > 0.5), ("a low", a < -0.5), ("b", b > 0.5), ("b low", b < -0.5)}
            a, b = min(a, 0.5), max(-0.5, min(b, 0.5))
            y.append(a * sig(1.702 * a) * (b + 1))
        assert np.allclose(got[t], p["down"] @ np.array(y), rtol=1e-9)
    assert len(cut) == 8     # every limit met and not met; the gate's lower side is not cut


def test_order_of_a_loop():
    cfg = bm.mixed_config(loop=(1, 3, 2))
    assert bezadra.schedule(cfg) == [(0, None), (1, 0), (2, None), (1, 1), (2, None), (3, None), (4, None)]
    assert bezadra.schedule(bm.mixed_config(loop=(0, 5, 1)))[0] == (0, 0)
    del cfg["loop"]
    assert bezadra.schedule(cfg) == [(i, None) for i in range(5)]
    x, x0 = rng(8).standard_normal((2, 3, 4))
    w, s = rng(9).standard_normal((4, 8)), rng(10).standard_normal(4)
    assert np.allclose(bezadra.loop_entry(x, x0, w, s), x @ w[:, :4].T + x0 @ w[:, 4:].T + s)


@pytest.mark.parametrize("what", ["softcap", "scaling", "limit"])
def test_test_weights_show_a_mechanism_that_is_left_out(what):
    cfg = bm.mixed_config()
    p = bezadra.random_params(cfg, "f32", 11)
    ids = rng(12).integers(0, cfg["vocab"], 60)
    right, off = bezadra.Model(cfg, p).logits(ids), bezadra.Model(bm.without(cfg, what), p).logits(ids)
    assert np.abs(right - off).max() > 0.05 * np.abs(right).max()


def test_config_reader(tmp_path):
    from rai_amd import config as cf
    cfg = bm.mixed_config()
    shapes = {k: list(v) for k, v in bezadra.param_shapes(cfg, a_rank=7, g_rank=9).items()}
    assert cf.architecture(cfg) == "bezadra"
    a, b, c, d, e = cf.bezadra_layers(cfg, shapes)
    assert (a["mixer"], a["conv_taps"], a["decay_rank"], a["gate_rank"], a["mlp_kind"]) == ("channel_delta", 3, 7, 9, "dense")
    assert (b["mixer"], b["rot_dims"], b["rot_base"], b["softcap"], b["attn_scale"]) == ("attention", 16, 900.0, 2.5, 0.6)
    assert (b["rot_factor"], b["rot_low"], b["rot_high"], b["rot_original"]) == (3.0, 1.5, 5.0, 60)
    assert (b["intermediate"], b["mlp_limit"], b["mlp_alpha"]) == (88, 1.1, 1.702)
    assert c["mlp_kind"] == "none" and "rot_factor" not in d and (e["heads"], e["kv_heads"]) == (5, 1)
    with pytest.raises(cf.ConfigError):
        cf.bezadra_layers(cfg, None)                       # the ranks are nowhere
    for change in (lambda x: x["layers"][0].update(type="ssm"), lambda x: x["layers"][0]["mlp"].update(kind="moe")):
        bad = bm.mixed_config()
        change(bad)
        with pytest.raises(cf.ConfigError):
            cf.bezadra_layers(bad, shapes)
    head = json.dumps({"__metadata__": {}, "x": {"dtype": "BF16", "shape": [2, 3], "data_offsets": [0, 12]}}).encode()
    (tmp_path / "a.safetensors").write_bytes(struct.pack("<Q", len(head)) + head + bytes(12))
    assert cf.tensor_shapes([tmp_path / "a.safetensors"]) == {"x": [2, 3]}
