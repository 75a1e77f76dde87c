"""The Lelitar restatement against sums written out term by term, and the config.json reader (CPU)."""
import math

import numpy as np
import pytest

from oracle import lelitar
from tests import lelitar_models as lm


def test_grouped_norm_term_by_term():
    rng = np.random.Generator(np.random.PCG64(0))
    x, w = rng.standard_normal((2, 12)), rng.standard_normal(12)
    got = lelitar.grouped_rms_norm(x, w, 3, 0.25)
    for t in range(2):
        for g in range(3):
            ms = sum(float(v) ** 2 for v in x[t, 4 * g:4 * g + 4]) / 4
            for i in range(4 * g, 4 * g + 4):
                assert math.isclose(got[t, i], x[t, i] / math.sqrt(ms + 0.25) * w[i], rel_tol=1e-12)


def test_attention_term_by_term_and_absorbed():
    """Each position's output from its own visible keys, one head and one key at a time; and the absorbed form (query
    in the latent space, value projection after the weighted sum) gives the same."""
    cfg = lm.config([lm.layer(heads=2, dim=5, vdim=3, q_rank=4, kv_rank=6, window=4, mlp=None)], width=9)
    p = lelitar.sub(lelitar.random_params(cfg, "f32", 1), "l0.mix")
    p = {k: np.asarray(v, np.float64) for k, v in p.items()}
    h = np.random.Generator(np.random.PCG64(2)).standard_normal((11, 9))
    got = lelitar.latent_attention(h, p, 2, 5, 3, 0.7, 4, 1e-5)
    cq = lelitar.rms(h @ p["dq"].T, 1e-5) * p["dq.norm"]
    c = lelitar.rms(h @ p["dkv"].T, 1e-5) * p["dkv.norm"]
    for i in range(11):
        cat = np.zeros(6)
        for hd in range(2):
            q = p["uq"][5 * hd:5 * hd + 5] @ cq[i]
            uk, uv = p["uk"][5 * hd:5 * hd + 5], p["uv"][3 * hd:3 * hd + 3]
            keys = [j for j in range(11) if 0 <= i - j < 4]
            assert len(keys) == min(i + 1, 4)
            e = [math.exp(0.7 * float(q @ (uk @ c[j]))) for j in keys]
            e2 = [math.exp(0.7 * float((uk.T @ q) @ c[j])) for j in keys]
            assert np.allclose(e, e2, rtol=1e-10)
            lat = sum(w * c[j] for w, j in zip(e, keys)) / sum(e)
            cat[3 * hd:3 * hd + 3] = uv @ lat
        want = p["o"] @ (cat / (1 + np.exp(-(p["g"] @ h[i]))))
        assert np.allclose(got[i], want, rtol=1e-9)


def test_mixture_term_by_term():
    cfg = lm.config([lm.layer(mlp="moe", ff=5, experts=4, top=2)], width=6)
    p = {k: np.asarray(v, np.float64) for k, v in lelitar.sub(lelitar.random_params(cfg, "f32", 3), "l0.mlp").items()}
    h = np.random.Generator(np.random.PCG64(4)).standard_normal((7, 6))
    got = lelitar.mixture(h, p, 2)
    for t in range(7):
        z = [float(r @ h[t]) for r in p["router"]]
        best = sorted(range(4), key=lambda e: -z[e])[:2]
        want = np.zeros(6)
        for e in best:
            x = h[t] / (1 + math.exp(-z[e]))
            g, u = p[f"e{e}.gate"] @ x, p[f"e{e}.up"] @ x
            want += p[f"e{e}.down"] @ (g / (1 + np.exp(-g)) * u)
        assert np.allclose(got[t], want, rtol=1e-9)


def test_standout_weights_show_a_window_that_is_one_off():
    """With the standing-out key just inside (outside) the window, an off-by-one window changes the logits a lot."""
    cfg = lm.config([lm.layer(window=9, mlp=None, scale=1.0)], mult=1.0)
    p = lm.standout_params(cfg, "f32", 5, marker=7)
    ids = np.random.Generator(np.random.PCG64(6)).integers(8, cfg["vocab"], 40)
    ids[20] = 7
    right = lelitar.Model(cfg, p).logits(ids)
    scale = np.abs(right).max()
    short, long = (lelitar.Model(lm.with_window(cfg, d), p).logits(ids) for d in (-1, 1))
    assert np.abs(right - short)[28].max() > 0.1 * scale     # 28 is the last position that sees 20
    assert np.abs(right - long)[29].max() > 0.1 * scale      # 29 the first that does not


def test_config_reader():
    from rai_amd import config as cf
    cfg = lm.mixed_config()
    assert cf.architecture(cfg) == "lelitar"
    a, b, c, d = cf.lelitar_layers(cfg)
    assert (a["mlp_kind"], a["mlp_act"], a["intermediate"], a["window"]) == ("dense", "relu", 88, 19)
    assert (b["mlp_kind"], b["mlp_act"], b["experts"], b["top"]) == ("moe", "silu", 6, 2)
    assert (c["mlp_kind"], c["window"], c["qk_dim"], c["v_dim"]) == ("none", 0, 72, 24)
    assert (d["q_rank"], d["kv_rank"], d["attn_scale"]) == (72, 24, 0.2)
    for name, key in (("phi", "phi2"), ("qwen2", "qwen2"), ("gemma", "gemma"), ("phi3", "phi3")):
        assert cf.architecture({"model_type": name}) == key
    assert cf.architecture({"architectures": ["Qwen2ForCausalLM"]}) == "qwen2"
    with pytest.raises(cf.ConfigError):
        cf.architecture({"model_type": "resnet"})
    bad = lm.mixed_config()
    bad["layers"][0]["type"] = "ssm"
    with pytest.raises(cf.ConfigError):
        cf.lelitar_layers(bad)
