"""The Lelitar decoder on the device against the plain restatement (oracle/lelitar.py): each mechanism alone, prompts
whole and in portions, decoding, batches, reused caches, window edges, odd sizes, generation and the trace runner."""
import json
import os
import subprocess

import numpy as np
import pytest

from oracle import lelitar
from oracle.dtypes import rnd, to_storage
from tests import lelitar_models as lm
from tests.util import RTOL, assert_close

pytestmark = pytest.mark.gpu

DTYPES = ["f32", "bf16"]
# mixer- and MLP-only weights: what the other branch writes is zeroed
ISOLATE = {"norm": ("mix.o", "mlp.down"), "attention": ("mlp.down",), "mlp": ("mix.o",), "all": ()}


def tokens(cfg, shape, seed=1):
    return np.random.Generator(np.random.PCG64(seed)).integers(0, cfg["vocab"], shape).astype(np.uint32)


def isolate(params, what):
    p = dict(params)
    for k in p:
        if k.endswith(".down") and "mlp.down" in ISOLATE[what] or k.endswith("mix.o") and "mix.o" in ISOLATE[what]:
            p[k] = np.zeros_like(p[k])
    return p


@pytest.mark.parametrize("dt", DTYPES)
@pytest.mark.parametrize("what", list(ISOLATE))
@pytest.mark.parametrize("mlp", ["dense", "moe", None])
def test_mechanism_alone(hip, dt, what, mlp):
    cfg = lm.config([lm.layer(mlp=mlp)], mult=1.7)
    p = isolate(lm.random_params(cfg, dt, 11), what)
    ref, dec = lelitar.Model(cfg, p), lm.build(cfg, p, dt)
    ids = tokens(cfg, 45)
    want = ref.hidden(ids)[-1]
    hid, _, _ = dec.forward_hidden(ids[None])
    assert_close(hid[0], want, dt, f"{what} residual stream")
    if what == "norm":
        assert np.array_equal(hid[0], p["embed"][ids])     # both branches silent: the stream is the embedding, exactly
    assert_close(lm.run_portions(dec, ids, [45])[0], ref.logits(ids), dt, f"{what} logits")
    assert_close(lm.run_portions(dec, ids, [1])[0], ref.logits(ids), dt, f"{what} logits token by token")
    dec.close()


@pytest.mark.parametrize("dt", DTYPES)
def test_layer_by_layer(hip, dt):
    cfg = lm.mixed_config()
    p = lm.random_params(cfg, dt, 3)
    ids = tokens(cfg, 51)
    want = lelitar.Model(cfg, p).hidden(ids)
    for n in range(1, len(cfg["layers"]) + 1):
        c = dict(cfg, layers=cfg["layers"][:n])
        dec = lm.build(c, {k: p[k] for k in lelitar.param_shapes(c)}, dt)
        for portions in ([51], [20, 31], [3]):
            dec.clear_kv_cache()
            out, at = [], 0
            while at < 51:
                s = min(portions[min(len(out), len(portions) - 1)], 51 - at)
                out.append(dec.forward_hidden(ids[None, at:at + s])[0][0])
                at += s
            assert_close(np.concatenate(out), want[n - 1], dt, f"stream after layer {n - 1}, portions {portions}")
        dec.close()


SIZES = {
    "groups 1, one head": lm.config([lm.layer(heads=1, dim=64, vdim=64, q_rank=64, kv_rank=64, mlp="moe", ff=64, experts=3, top=1)],
                                    width=64, groups=1, vocab=128, mult=1.0),
    "heads wider than the flash sizes": lm.config([lm.layer(heads=2, dim=264, vdim=200, q_rank=96, kv_rank=320, scale=0.06)], width=192),
    "dim 192": lm.config([lm.layer(heads=2, dim=160, vdim=128, q_rank=128, kv_rank=128, scale=0.08, mlp="moe", ff=72, experts=9, top=4)],
                         width=256, groups=4),
    "dim 256": lm.config([lm.layer(heads=3, dim=96, vdim=256, q_rank=32, kv_rank=512, window=64, scale=0.1)], width=136, groups=17),
    "odd everything": lm.config([lm.layer(heads=3, dim=7, vdim=5, q_rank=9, kv_rank=11, window=13, ff=21, scale=0.4),
                                 lm.layer(heads=2, dim=3, vdim=9, q_rank=13, kv_rank=5, window=2, mlp="moe", ff=3, experts=5, top=5, scale=0.5)],
                                vocab=77, width=33, groups=11),
    "window 1": lm.config([lm.layer(window=1), lm.layer(window=1, mlp="moe")]),
    "130 experts": lm.config([lm.layer(mlp="moe", experts=130, top=3, ff=16), lm.layer(mlp="moe", experts=65, top=2, ff=24)]),
    "300 experts": lm.config([lm.layer(mlp="moe", experts=300, top=5, ff=16)]),
    "every expert": lm.config([lm.layer(mlp="moe", experts=4, top=4)]),
    "wide": lm.config([lm.layer(heads=20, dim=128, vdim=128, q_rank=768, kv_rank=512, window=100, ff=1024, scale=0.088)], width=2304, groups=9),
}


@pytest.mark.parametrize("dt", DTYPES)
@pytest.mark.parametrize("name", list(SIZES))
def test_sizes(hip, dt, name):
    cfg = SIZES[name]
    p = lm.random_params(cfg, dt, 21)
    dec, ids = lm.build(cfg, p, dt, max_batch=2), tokens(cfg, 70)
    want = lelitar.Model(cfg, p).logits(ids)
    for portions in ([70], [33, 2, 35], [9], [64, 1]):
        assert_close(lm.run_portions(dec, ids, portions)[0], want, dt, f"{name}, portions {portions}")
    dec.close()


@pytest.mark.parametrize("dt", DTYPES)
@pytest.mark.parametrize("portions", [[2], [3], [7], [15], [16], [17], [40], [64], [65], [100, 1], [1, 16, 2, 33], [130]])
def test_portions(hip, dt, portions):
    cfg = lm.mixed_config()
    p = lm.random_params(cfg, dt, 4)
    dec, ids = lm.build(cfg, p, dt), tokens(cfg, 130)
    assert_close(lm.run_portions(dec, ids, portions)[0], lelitar.Model(cfg, p).logits(ids), dt, f"portions {portions}")
    dec.close()


@pytest.mark.parametrize("dt", DTYPES)
def test_long_decoding_and_reused_cache(hip, dt):
    """Sequences one after the other through the same cache, long and short in turn, mostly token by token: what an
    earlier one left behind must not show."""
    cfg = lm.mixed_config()
    p = lm.random_params(cfg, dt, 5)
    ref, dec = lelitar.Model(cfg, p), lm.build(cfg, p, dt)
    for n, portions, seed in ((250, [40, 1], 1), (30, [1], 2), (200, [150, 1], 3), (3, [2, 1], 4), (90, [90], 5)):
        ids = tokens(cfg, n, seed)
        assert_close(lm.run_portions(dec, ids, portions)[0], ref.logits(ids), dt, f"sequence of {n}")
    dec.close()


@pytest.mark.parametrize("dt", DTYPES)
@pytest.mark.parametrize("batch", [2, 5, 12, 33])
def test_batch_against_each_alone(hip, dt, batch):
    cfg = lm.mixed_config()
    p = lm.random_params(cfg, dt, 6)
    dec, ids = lm.build(cfg, p, dt, max_batch=batch, max_context=64), tokens(cfg, (batch, 48))
    ref = lelitar.Model(cfg, p)
    together = lm.run_portions(dec, ids, [29, 3, 16])
    decoded = lm.run_portions(dec, ids, [40, 1])
    for b in sorted({0, 1, batch // 2, batch - 1}):
        want = ref.logits(ids[b])
        assert_close(together[b], want, dt, f"row {b} of {batch}")
        assert_close(decoded[b], want, dt, f"row {b} of {batch}, decoded")
        assert_close(lm.run_portions(dec, ids[b], [29, 3, 16])[0], together[b], dt, f"row {b} alone")
    dec.close()


def edge_cases():
    return [(w, mlp) for w in (2, 9, 64, 65, 100) for mlp in (None, "moe")]


@pytest.mark.parametrize("dt", DTYPES)
@pytest.mark.parametrize("window,mlp", edge_cases())
def test_window_edges_with_a_key_that_stands_out(hip, dt, window, mlp):
    """One key wins every query that sees it.  Its last viewer (distance window - 1) and the first that does not see it
    (distance window) are compared in prompts, in portions that end at the edge, and decoded."""
    cfg = lm.config([lm.layer(window=window, mlp=mlp, scale=1.0)], mult=1.0)
    p = lm.standout_params(cfg, dt, 8, marker=7)
    at = 37
    n = at + window + 6
    ids = np.random.Generator(np.random.PCG64(9)).integers(8, cfg["vocab"], n).astype(np.uint32)
    ids[at] = 7
    want = lelitar.Model(cfg, p).logits(ids)
    scale = np.abs(want).max()
    for delta, pos in ((-1, at + window - 1), (1, at + window)):   # a window one off would show well above the tolerance
        off = lelitar.Model(lm.with_window(cfg, delta), p).logits(ids)
        assert np.abs(off - want)[pos].max() > 5 * RTOL[dt] * scale
    dec = lm.build(cfg, p, dt)
    for portions in ([n], [at + window - 1, 1], [at + window, 2, 1], [at + 1, window - 1, 1], [at, 17], [2]):
        got = lm.run_portions(dec, ids, portions)[0]
        assert_close(got, want, dt, f"window {window}, portions {portions}")
    dec.close()


@pytest.mark.parametrize("dt", DTYPES)
@pytest.mark.parametrize("far", [1, 63, 64, 127, 200])
def test_far_key_without_a_window(hip, dt, far):
    """A single key that stands out among hundreds, found by prompts, short portions and decoded tokens; also as the
    first token of the sequence."""
    cfg = lm.config([lm.layer(window=None, mlp=None, scale=1.0)], mult=1.0)
    p = lm.standout_params(cfg, dt, 10, marker=7)
    for at in (0, 13):
        n = at + far + 1
        ids = np.random.Generator(np.random.PCG64(12)).integers(8, cfg["vocab"], n).astype(np.uint32)
        plain = lelitar.Model(cfg, p).logits(ids)[-1]
        ids[at] = 7
        want = lelitar.Model(cfg, p).logits(ids)
        if far > 1:
            assert np.abs(plain - want[-1]).max() > 3 * RTOL[dt] * np.abs(want).max()
        dec = lm.build(cfg, p, dt)
        for portions in ([n], [n - 1, 1], [max(1, n - 5), 5], [16]):
            assert_close(lm.run_portions(dec, ids, portions)[0], want, dt, f"key at {at}, {far} back, portions {portions}")
        dec.close()


@pytest.mark.parametrize("dt", DTYPES)
@pytest.mark.parametrize("batch,n", [(1, 1), (1, 6), (1, 200), (9, 40), (3, 130), (4, 1100)])
def test_uneven_experts(hip, dt, batch, n):
    """A router that sends nearly every token to the same two of many experts: full and partial row tiles, experts
    without rows, more rows than one tile."""
    cfg = lm.config([lm.layer(mlp="moe", experts=40, top=2, ff=40)], mult=1.0)
    p = lm.random_params(cfg, "f32", 13)
    p["embed"][:, 0] = 4.0
    p["l0.mlp.router"][[31, 5]] = 0.0
    p["l0.mlp.router"][31, 0] = 3.0
    p["l0.mlp.router"][5, 0] = 2.0
    p = {k: rnd(v, dt) for k, v in p.items()}
    dec, ids = lm.build(cfg, p, dt, max_batch=batch, max_context=max(64, n)), tokens(cfg, (batch, n), 14)
    got = lm.run_portions(dec, ids, [n])
    for b in range(batch):
        assert_close(got[b], lelitar.Model(cfg, p).logits(ids[b]), dt, f"row {b}")
    dec.close()


@pytest.mark.parametrize("switch", ["RAI_HIP_NO_LATENT_FUSED", "RAI_HIP_NO_LATENT_MFMA"])
def test_the_plain_forms_of_the_bf16_kernels(hip, monkeypatch, switch):
    """The launches without folded-in norms and routing, and the absorbed attention without MFMA, against the
    restatement and against the forms that normally run."""
    cfg = lm.mixed_config()
    p = lm.random_params(cfg, "bf16", 23)
    dec, ids = lm.build(cfg, p, "bf16", max_batch=3), tokens(cfg, (3, 40), 24)
    want = np.stack([lelitar.Model(cfg, p).logits(r) for r in ids])
    usual = [lm.run_portions(dec, ids, [30, 1]), lm.run_portions(dec, ids[:1], [33, 1])]
    monkeypatch.setenv(switch, "1")
    plain = [lm.run_portions(dec, ids, [30, 1]), lm.run_portions(dec, ids[:1], [33, 1])]
    for a, b in zip(usual, plain):
        assert_close(a, want[:len(a)], "bf16", "usual forms")
        assert_close(b, want[:len(b)], "bf16", f"{switch}=1")
        assert_close(b, a, "bf16", "one against the other")
    dec.close()


def check_greedy(got, tokens_ref, logits_ref, dt):
    """Tokens equal the restatement's up to a near tie of its own logits, after which a sequence may differ."""
    for t in range(len(tokens_ref)):
        if got[t] == tokens_ref[t]:
            continue
        row = logits_ref[t]
        gap = row[tokens_ref[t]] - row[got[t]]
        assert gap <= 2 * RTOL[dt] * np.abs(row).max(), f"token {t}: {got[t]} instead of {tokens_ref[t]}, gap {gap}"
        return t
    return len(tokens_ref)


@pytest.mark.parametrize("dt", DTYPES)
def test_greedy_generation(hip, dt):
    cfg = lm.mixed_config()
    p = lm.random_params(cfg, dt, 15)
    dec, ids = lm.build(cfg, p, dt, max_batch=3, max_context=128), tokens(cfg, (3, 21), 16)
    ref = lelitar.Model(cfg, p)
    got, _, _ = dec.generate(ids, 60)
    again, _, _ = dec.generate(ids, 60)          # the captured graphs, replayed after other work
    assert np.array_equal(got, again)
    for b in range(3):
        want, rows = ref.greedy(ids[b], 60)
        same = check_greedy(got[b], want, rows, dt)
        assert same == 60 or dt == "bf16"
        alone, _, _ = dec.generate(ids[b][None], 60)
        check_greedy(alone[0], want, rows, dt)
    # every generated token is the first maximum of the logits the same tokens give when fed as a prompt
    seq = np.concatenate([ids, got], axis=1)[:, :-1]
    logits = lm.run_portions(dec, seq, [seq.shape[1]])
    for b in range(3):
        for t in range(60):
            row = logits[b, 20 + t]
            assert row.max() - row[got[b, t]] <= 2 * RTOL[dt] * np.abs(row).max()
    dec.close()


def test_sampled_generation(hip):
    """The repeat penalty keeps a sequence from naming a recent token again where greedy decoding would."""
    from oracle import sampling
    cfg = lm.mixed_config()
    p = lm.random_params(cfg, "f32", 17)
    dec, ids = lm.build(cfg, p, "f32", max_context=96), tokens(cfg, (1, 9), 18)
    got, n, _, _ = dec.generate_sampled(ids, 30, repeat_penalty=1.3, repeat_last_n=16)
    ref, seq = lelitar.Model(cfg, p), list(ids[0])
    for t in range(30):
        row = sampling.apply_repeat_penalty(ref.logits(seq)[-1].astype(np.float32), 1.3, seq[-16:])
        assert row.max() - row[got[0, t]] <= 1e-4 * np.abs(row).max()
        seq.append(int(got[0, t]))
    assert n[0] == 30
    dec.close()


def write_model(path, cfg, params):
    from tests.test_gpu_safetensors import write_safetensors
    path.mkdir()
    (path / "config.json").write_text(json.dumps(cfg))
    write_safetensors(path / "model.safetensors", params, "BF16")


def test_trace_runner(hip, tmp_path):
    """bin/trace_run end to end, both precisions: several requests, portions, wanted rows, ended requests."""
    cfg = lm.mixed_config()
    p = lm.random_params(cfg, "bf16", 19)
    write_model(tmp_path / "m", cfg, p)
    root = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
    a, b = tokens(cfg, 60, 20), tokens(cfg, 25, 21)
    steps = [("a", a[:30], [0, 29], False), ("a", a[30:32], [1], False), ("a", a[32:], [], False), ("a", a[:0], [], None),
             ("b", b[:1], [0], False), ("b", b[1:], [23, 3], True)]
    steps[2] = ("a", a[32:], [], True)
    steps.pop(3)
    lines = "".join(json.dumps({"step": i, "entries": [{"id": r, "tokens": t.tolist(), "want": w}], "end": [r] if e else []}) + "\n"
                    for i, (r, t, w, e) in enumerate(steps))
    la, lb = lelitar.Model(cfg, p).logits(a), lelitar.Model(cfg, p).logits(b)
    want = {0: la[[0, 29]], 1: la[[31]], 3: lb[[0]], 4: lb[[24, 4]]}
    for name, dt in (("float32", "f32"), ("bfloat16", "bf16")):
        out = tmp_path / name
        out.mkdir()
        r = subprocess.run([os.path.join(root, "bin", "trace_run"), "--model", str(tmp_path / "m"), "--dtype", name, "--out", str(out),
                            "--max-tokens", "64"], input=lines, capture_output=True, text=True, timeout=100)
        assert r.returncode == 0, r.stderr
        assert [x for x in r.stdout.splitlines() if x.startswith("done")] == [f"done {i}" for i in range(5)]
        assert sorted(os.listdir(out)) == sorted(f"{k}.f32" for k in want)
        for k, w in want.items():
            assert_close(np.fromfile(out / f"{k}.f32", "<f4").reshape(w.shape), w, dt, f"{name} step {k}")


def test_forward_rows_serves_the_other_families(hip):
    """The rows entry point gives what forward gives for the last row, for a Phi-2 model fed in portions."""
    from oracle import phi2
    from tests.test_gpu_phi2 import small_cfg
    from tests.test_gpu_safetensors import new_decoder
    cfg = small_cfg()
    for dt in DTYPES:
        p = phi2.random_params(cfg, dt, seed=2)
        dec = new_decoder(cfg, dt)
        for n in dec.param_names():
            dec.load_param(n, to_storage(p[n], dt))
        ids = np.random.Generator(np.random.PCG64(3)).integers(0, cfg.vocab_size, (2, 12)).astype(np.uint32)
        rows = lm.run_portions(dec, ids, [5, 7])
        for n in (3, 5, 12):
            dec.clear_kv_cache()
            last, _ = dec.forward(ids[:, :n])
            assert_close(rows[:, n - 1], last, dt, f"{dt} row {n - 1}")
        dec.close()


def test_errors(hip):
    from rai_amd._lib import RaiHipError
    cfg = lm.mixed_config()
    dec = lm.build(cfg, lm.random_params(cfg, "f32", 1), "f32", max_context=16)
    with pytest.raises(RaiHipError):
        dec.forward_rows(np.zeros((1, 17), np.uint32), [0])            # longer than the context
    with pytest.raises(RaiHipError):
        dec.forward_rows(np.zeros((1, 4), np.uint32), [4])             # no such row
    with pytest.raises(RaiHipError):
        dec.forward_rows(np.full((1, 4), cfg["vocab"], np.uint32), [0])  # not a token
    dec.clear_kv_cache()
    assert dec.context_len() == 0
    dec.close()
    for bad in (dict(width=121), dict(layers=[lm.layer(mlp="moe", experts=2, top=3)])):
        c = dict(lm.mixed_config(), **bad)
        from rai_amd.config import decoder_from_config
        with pytest.raises(RaiHipError):
            decoder_from_config(c, "bf16")
