"""The Bezadra decoder on the device against the plain restatement (oracle/bezadra.py): each mechanism alone, prompts
whole and in portions, decoding, batches, reused caches and states, far keys and long memory, odd sizes, generation and
the trace runner."""
import json
import os
import subprocess

import numpy as np
import pytest

from oracle import bezadra
from oracle.dtypes import rnd
from tests import bezadra_models as bm
from tests.test_gpu_lelitar import check_greedy, tokens, write_model
from tests.util import RTOL, assert_close

pytestmark = pytest.mark.gpu

DTYPES = ["f32", "bf16"]
# what is zeroed so that one branch of a block stays alone
SILENT = {"norm": ("mix.o", "mlp.down"), "mixer": ("mlp.down",), "mlp": ("mix.o",), "all": ()}
LAYERS = {
    "attention": bm.attention(),
    "attention, no frequency scaling, all features turned": bm.attention(dims=24, scaling=None),
    "attention, one key head": bm.attention(heads=5, kv_heads=1, dim=40, vdim=8, dims=2, base=5.0),
    "attention, heads of their own, no cap": bm.attention(heads=3, kv_heads=3, dim=16, vdim=16, dims=12, softcap=0.0),
    "delta": bm.delta(),
    "delta, heads of their own": bm.delta(heads=3, kv_heads=3, dim=48, vdim=20, conv=4),
    "delta, one key head, one tap": bm.delta(heads=6, kv_heads=1, dim=36, vdim=64, conv=1),
    "delta, one head, nine taps": bm.delta(heads=1, kv_heads=1, dim=33, vdim=31, conv=9),
}


def deep_close(got, want, dt, what):
    """For models of five layers, two of them run three times: nine layer runs whose roundings to bf16 add up (measured:
    up to 2.1 % of the largest logit); f32 as everywhere."""
    assert_close(got, want, dt, what, scale=(1.5 if dt == "bf16" else 1.0) * float(np.abs(want).max()))


def silence(params, what):
    return {k: np.zeros_like(v) if k.endswith(SILENT[what]) else v for k, v in params.items()}


def portion_hidden(dec, ids, portions):
    dec.clear_kv_cache()
    out, at = [], 0
    while at < len(ids):
        s = min(portions[min(len(out), len(portions) - 1)], len(ids) - at)
        out.append(dec.forward_hidden(ids[None, at:at + s])[0][0])
        at += s
    return np.concatenate(out)


@pytest.mark.parametrize("dt", DTYPES)
@pytest.mark.parametrize("what", list(SILENT))
@pytest.mark.parametrize("name", list(LAYERS))
def test_mechanism_alone(hip, dt, what, name):
    cfg = bm.config([LAYERS[name]])
    p = silence(bezadra.random_params(cfg, dt, 11), what)
    ref, dec = bezadra.Model(cfg, p), bm.build(cfg, p, dt)
    ids = tokens(cfg, 45)
    want = ref.hidden(ids)
    hid, _, _ = dec.forward_hidden(ids[None])
    assert_close(hid[0], want[-1], dt, f"{what} residual stream")
    if what == "norm":   # both branches silent: the stream is the scaled embedding, exactly
        assert np.array_equal(hid[0], p["embed"][ids].astype(np.float32) * np.float32(cfg["embedding"]["scale"]))
    logits = ref.logits(ids, want[-1])
    assert_close(bm.run_portions(dec, ids, [45])[0], logits, dt, f"{what} logits")
    assert_close(bm.run_portions(dec, ids, [1])[0], logits, dt, f"{what} logits token by token")
    dec.close()


@pytest.mark.parametrize("dt", DTYPES)
def test_run_by_run(hip, dt):
    """The stream after every layer run of models that end there, looped layers included."""
    cfg = bm.mixed_config()
    p = bezadra.random_params(cfg, dt, 3)
    ids = tokens(cfg, 51)
    for layers, times in ((1, 0), (2, 1), (3, 1), (3, 2), (3, 3), (4, 3), (5, 3)):
        loop = (1, min(3, layers), times) if times else None
        c = bm.config(cfg["layers"][:layers], loop=loop)
        q = {k: p[k] for k in bezadra.param_shapes(c)}
        if times:
            q["loop.step"] = p["loop.step"][:times]
        want = bezadra.Model(c, q).hidden(ids)[-1]
        dec = bm.build(c, q, dt)
        for portions in ([51], [20, 31], [3], [1]):
            deep_close(portion_hidden(dec, ids, portions), want, dt, f"{layers} layers, {times} passes, portions {portions}")
        dec.close()


LOOPS = [None, (0, 1, 1), (0, 2, 2), (1, 2, 4), (0, 5, 2), (3, 5, 1), (4, 5, 2)]


@pytest.mark.parametrize("dt", DTYPES)
@pytest.mark.parametrize("loop", LOOPS)
def test_loops(hip, dt, loop):
    cfg = bm.mixed_config(loop=loop)
    p = bezadra.random_params(cfg, dt, 7)
    ids = tokens(cfg, 40)
    want = bezadra.Model(cfg, p).logits(ids)
    dec = bm.build(cfg, p, dt)
    for portions in ([40], [18, 1], [5]):
        deep_close(bm.run_portions(dec, ids, portions)[0], want, dt, f"loop {loop}, portions {portions}")
    dec.close()


SIZES = {
    "one head of 64": bm.config([bm.attention(heads=1, kv_heads=1, dim=64, vdim=64, dims=64, ff=64), bm.delta(heads=1, kv_heads=1, dim=64, vdim=64, ff=64)],
                                width=64, vocab=128, embed_scale=1.0, logit_scale=1.0),
    "eight query heads to a key head": bm.config([bm.attention(heads=16, kv_heads=2, dim=64, vdim=64, dims=48)], width=192),
    "heads wider than the flash sizes": bm.config([bm.attention(heads=2, kv_heads=1, dim=264, vdim=200, dims=130, scale=0.1)], width=192),
    "dim 192": bm.config([bm.attention(heads=4, kv_heads=2, dim=160, vdim=136, dims=160, scale=0.1)], width=136),
    "dim 256": bm.config([bm.attention(heads=4, kv_heads=1, dim=96, vdim=256, dims=32, scale=0.2)], width=128),
    "delta 128": bm.config([bm.delta(heads=4, kv_heads=2, dim=128, vdim=128, conv=4)], width=256),
    "delta 128 by 64": bm.config([bm.delta(heads=2, kv_heads=1, dim=128, vdim=64, conv=4, ff=None)], width=256),
    "delta 64 by 128": bm.config([bm.delta(heads=2, kv_heads=2, dim=64, vdim=128, conv=4)], width=256),
    "delta 256": bm.config([bm.delta(heads=2, kv_heads=1, dim=256, vdim=256, conv=4)], width=128),
    "delta 300 by 500": bm.config([bm.delta(heads=2, kv_heads=2, dim=300, vdim=500, conv=2)], width=128),
    "odd everything": bm.config([bm.attention(heads=3, kv_heads=3, dim=7, vdim=5, dims=6, ff=21), bm.delta(heads=3, kv_heads=1, dim=11, vdim=9, ff=3),
                                 bm.delta(heads=2, kv_heads=2, dim=13, vdim=15, ff=7)], loop=(0, 2, 2), vocab=77, width=33),
    "wide": bm.config([bm.attention(heads=20, kv_heads=4, dim=128, vdim=128, dims=128, scale=0.09, ff=1024),
                       bm.delta(heads=16, kv_heads=8, dim=128, vdim=128, conv=4, ff=1024)], width=2304, loop=(0, 2, 2)),
}


def test_heads_of_one(hip):
    """Unit vectors and norms of a single value are signs: f32 only, a rounding to bf16 could turn one."""
    cfg = bm.config([bm.delta(heads=4, kv_heads=2, dim=1, vdim=1, ff=7), bm.delta(heads=3, kv_heads=1, dim=3, vdim=2, ff=3), bm.attention(heads=2, kv_heads=2, dim=2, vdim=1, dims=2)], width=40)
    p = bezadra.random_params(cfg, "f32", 22, a_rank=1, g_rank=1)
    dec, ids = bm.build(cfg, p, "f32"), tokens(cfg, 80)
    for portions in ([80], [33, 1], [5]):
        assert_close(bm.run_portions(dec, ids, portions)[0], bezadra.Model(cfg, p).logits(ids), "f32", f"portions {portions}")
    dec.close()


@pytest.mark.parametrize("dt", DTYPES)
@pytest.mark.parametrize("name", list(SIZES))
def test_sizes(hip, dt, name):
    cfg = SIZES[name]
    p = bezadra.random_params(cfg, dt, 21, a_rank=19, g_rank=70)
    dec, ids = bm.build(cfg, p, dt, max_batch=2), tokens(cfg, 150)
    want = bezadra.Model(cfg, p).logits(ids)
    for portions in ([150], [33, 2, 115], [9], [64, 70, 1]):
        deep_close(bm.run_portions(dec, ids, portions)[0], want, dt, f"{name}, portions {portions}")
    dec.close()


@pytest.mark.parametrize("dt", DTYPES)
@pytest.mark.parametrize("portions", [[2], [3], [7], [15], [16], [17], [40], [63], [64], [65], [100, 1], [1, 16, 2, 33], [128], [129, 2], [200]])
def test_portions(hip, dt, portions):
    cfg = bm.mixed_config()
    p = bezadra.random_params(cfg, dt, 4)
    dec, ids = bm.build(cfg, p, dt), tokens(cfg, 200)
    deep_close(bm.run_portions(dec, ids, portions)[0], bezadra.Model(cfg, p).logits(ids), dt, f"portions {portions}")
    dec.close()


@pytest.mark.parametrize("dt", DTYPES)
def test_long_decoding_and_reused_state(hip, dt):
    """Sequences one after the other through the same caches and states, long and short in turn, mostly token by token:
    what an earlier one left behind must not show, the first tokens of a sequence included."""
    cfg = bm.mixed_config()
    p = bezadra.random_params(cfg, dt, 5)
    ref, dec = bezadra.Model(cfg, p), bm.build(cfg, p, dt)
    for n, portions, seed in ((250, [40, 1], 1), (30, [1], 2), (200, [150, 1], 3), (1, [1], 6), (3, [2, 1], 4), (90, [90], 5), (70, [2, 68], 7)):
        ids = tokens(cfg, n, seed)
        deep_close(bm.run_portions(dec, ids, portions)[0], ref.logits(ids), dt, f"sequence of {n}")
    dec.close()


@pytest.mark.parametrize("dt", DTYPES)
@pytest.mark.parametrize("batch", [2, 5, 12, 33])
def test_batch_against_each_alone(hip, dt, batch):
    cfg = bm.mixed_config()
    p = bezadra.random_params(cfg, dt, 6)
    dec, ids = bm.build(cfg, p, dt, max_batch=batch, max_context=160), tokens(cfg, (batch, 138))
    ref = bezadra.Model(cfg, p)
    together = bm.run_portions(dec, ids, [29, 3, 96, 10])
    decoded = bm.run_portions(dec, ids[:, :48], [40, 1])
    for b in sorted({0, 1, batch // 2, batch - 1}):
        want = ref.logits(ids[b])
        deep_close(together[b], want, dt, f"row {b} of {batch}")
        deep_close(decoded[b], want[:48], dt, f"row {b} of {batch}, decoded")
        deep_close(bm.run_portions(dec, ids[b], [29, 3, 96, 10])[0], together[b], dt, f"row {b} alone")
    dec.close()


def far_case(params, cfg, dt, at, far, seed):
    """Token 7 at `at`, read `far` tokens later, and how much the logits there hang on it."""
    n = at + far + 1
    ids = np.random.Generator(np.random.PCG64(seed)).integers(8, cfg["vocab"], n).astype(np.uint32)
    plain = bezadra.Model(cfg, params).logits(ids)[-1]
    ids[at] = 7
    want = bezadra.Model(cfg, params).logits(ids)
    return ids, want, np.abs(plain - want[-1]).max() / np.abs(want).max()


@pytest.mark.parametrize("dt", DTYPES)
@pytest.mark.parametrize("far", [1, 63, 64, 127, 200, 500])
def test_far_key(hip, dt, far):
    """A single key that stands out among hundreds, found by prompts, short portions and decoded tokens; also as the
    first token of the sequence."""
    cfg = bm.config([bm.attention(scale=1.0, softcap=14.0, ff=None)], embed_scale=0.3)
    p = bm.standout_key_params(cfg, dt, 10, marker=7)
    for at in (0, 13):
        ids, want, share = far_case(p, cfg, dt, at, far, 12)
        assert share > 5 * RTOL[dt]
        n = len(ids)
        dec = bm.build(cfg, p, dt, max_context=640)
        for portions in ([n], [n - 1, 1], [max(1, n - 5), 5], [max(1, n - 3), 1], [at + 1, 40]):
            assert_close(bm.run_portions(dec, ids, portions)[0], want, dt, f"key at {at}, {far} back, portions {portions}")
        dec.close()


@pytest.mark.parametrize("dt", DTYPES)
@pytest.mark.parametrize("far", [1, 15, 16, 63, 64, 65, 130])
def test_long_memory(hip, dt, far):
    """What one token wrote into the recurrent state, read many tokens later: a state that is lost or cut at any place
    shows."""
    cfg = bm.config([bm.delta(heads=3, kv_heads=3, dim=96, vdim=24, conv=4, ff=None)], embed_scale=0.5)
    p = bm.long_memory_params(cfg, dt, 14, marker=7)
    for at in (0, 30):
        ids, want, share = far_case(p, cfg, dt, at, far, 15)
        assert share > 5 * RTOL[dt]
        n = len(ids)
        dec = bm.build(cfg, p, dt)
        for portions in ([n], [n - 1, 1], [at + 1, 1], [max(1, n - 2), 2], [16], [64, 3]):
            assert_close(bm.run_portions(dec, ids, portions)[0], want, dt, f"written at {at}, {far} back, portions {portions}")
        dec.close()


@pytest.mark.parametrize("dt", DTYPES)
@pytest.mark.parametrize("dim", [32, 48, 64, 100])
@pytest.mark.parametrize("bias,rate", [(0.5, 1.0), (-12.0, 0.0), (-3.0, 1.5), (4.0, 0.0), (30.0, 3.0), (-60.0, -4.0)])
def test_decays_from_none_to_all(hip, dt, bias, rate, dim):
    """Channels that forget nothing, that forget everything at once (the decay underflows), and both next to each other."""
    cfg = bm.config([bm.delta(heads=4, kv_heads=2, dim=dim, vdim=32, conv=4, ff=None)])
    p = bezadra.random_params(cfg, "f32", 16)
    p["l0.mix.dt_bias"][::2] = bias
    p["l0.mix.A_log"][:] = rate
    p = {k: rnd(v, dt) for k, v in p.items()}
    ids = tokens(cfg, 150, 17)
    want = bezadra.Model(cfg, p).logits(ids)
    dec = bm.build(cfg, p, dt)
    for portions in ([150], [70, 80], [100, 1], [20]):
        assert_close(bm.run_portions(dec, ids, portions)[0], want, dt, f"bias {bias}, rate {rate}, portions {portions}")
    dec.close()


@pytest.mark.parametrize("dt", DTYPES)
@pytest.mark.parametrize("sink", [-8.0, 3.0, 40.0])
def test_sink(hip, dt, sink):
    """Sinks far below, among and far above the capped scores, for every head and for some of them."""
    cfg = bm.config([bm.attention(heads=8, kv_heads=2, ff=None)])
    for some in (slice(None), slice(0, None, 3)):
        p = bezadra.random_params(cfg, "f32", 18)
        p["l0.mix.sink"][some] = sink
        p = {k: rnd(v, dt) for k, v in p.items()}
        ids = tokens(cfg, 140, 19)
        want = bezadra.Model(cfg, p).logits(ids)
        dec = bm.build(cfg, p, dt)
        for portions in ([140], [130, 1], [8]):
            assert_close(bm.run_portions(dec, ids, portions)[0], want, dt, f"sink {sink}, portions {portions}")
        dec.close()


@pytest.mark.parametrize("dt", DTYPES)
def test_long_prompt(hip, dt):
    """Positions far beyond the frequency scaling's original length, more rows than the largest product tile."""
    cfg = bm.config([bm.attention(), bm.delta(heads=4, kv_heads=2, dim=64, vdim=64, conv=4)], loop=(1, 2, 2))
    p = bezadra.random_params(cfg, dt, 20)
    ids = tokens(cfg, 700, 21)
    want = bezadra.Model(cfg, p).logits(ids)
    dec = bm.build(cfg, p, dt, max_context=704)
    for portions in ([700], [300, 390, 1]):
        assert_close(bm.run_portions(dec, ids, portions)[0], want, dt, f"portions {portions}")
    dec.close()


@pytest.mark.parametrize("switch", ["RAI_HIP_NO_LATENT_FUSED", "RAI_HIP_NO_MFMA_DECODE", "RAI_HIP_FLASH_NO_KEY_SPLIT", "RAI_HIP_NO_DELTA_CHUNK"])
def test_the_plain_forms_of_the_bf16_kernels(hip, monkeypatch, switch):
    cfg = bm.config(bm.mixed_config()["layers"] + [bm.attention(heads=8, kv_heads=2, dim=64, vdim=64, dims=32)], loop=(1, 3, 2))
    p = bezadra.random_params(cfg, "bf16", 23)
    dec, ids = bm.build(cfg, p, "bf16", max_batch=3), tokens(cfg, (3, 160), 24)
    want = np.stack([bezadra.Model(cfg, p).logits(r) for r in ids])
    usual = [bm.run_portions(dec, ids, [150, 1]), bm.run_portions(dec, ids[:1], [153, 1])]
    monkeypatch.setenv(switch, "1")
    plain = [bm.run_portions(dec, ids, [150, 1]), bm.run_portions(dec, ids[:1], [153, 1])]
    for a, b in zip(usual, plain):
        deep_close(a, want[:len(a)], "bf16", "usual forms")
        deep_close(b, want[:len(b)], "bf16", f"{switch}=1")
        deep_close(b, a, "bf16", "one against the other")
    dec.close()


@pytest.mark.parametrize("dt", DTYPES)
def test_greedy_generation(hip, dt):
    cfg = bm.mixed_config()
    p = bezadra.random_params(cfg, dt, 15)
    dec, ids = bm.build(cfg, p, dt, max_batch=3, max_context=128), tokens(cfg, (3, 21), 16)
    ref = bezadra.Model(cfg, p)
    got, _, _ = dec.generate(ids, 60)
    again, _, _ = dec.generate(ids, 60)          # the captured graphs, replayed after other work
    assert np.array_equal(got, again)
    for b in range(3):
        want, rows = ref.greedy(ids[b], 60)
        check_greedy(got[b], want, rows, dt)
        alone, _, _ = dec.generate(ids[b][None], 60)
        check_greedy(alone[0], want, rows, dt)
    # every generated token is the first maximum of the logits the same tokens give when fed as a prompt
    seq = np.concatenate([ids, got], axis=1)[:, :-1]
    logits = bm.run_portions(dec, seq, [seq.shape[1]])
    for b in range(3):
        for t in range(60):
            row = logits[b, 20 + t]
            assert row.max() - row[got[b, t]] <= 2 * RTOL[dt] * np.abs(row).max()
    dec.close()


def test_sampled_generation(hip):
    from oracle import sampling
    cfg = bm.mixed_config()
    p = bezadra.random_params(cfg, "f32", 17)
    dec, ids = bm.build(cfg, p, "f32", max_context=96), tokens(cfg, (1, 9), 18)
    got, n, _, _ = dec.generate_sampled(ids, 30, repeat_penalty=1.3, repeat_last_n=16)
    ref, seq = bezadra.Model(cfg, p), list(ids[0])
    for t in range(30):
        row = sampling.apply_repeat_penalty(ref.logits(seq)[-1].astype(np.float32), 1.3, seq[-16:])
        assert row.max() - row[got[0, t]] <= 1e-4 * np.abs(row).max()
        seq.append(int(got[0, t]))
    assert n[0] == 30
    dec.close()


def test_trace_runner(hip, tmp_path):
    """bin/trace_run end to end, both precisions: the ranks read from the tensors, several requests, portions."""
    cfg = bm.mixed_config()
    p = bezadra.random_params(cfg, "bf16", 19, a_rank=5, g_rank=66)
    write_model(tmp_path / "m", cfg, p)
    root = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
    a, b = tokens(cfg, 60, 20), tokens(cfg, 25, 21)
    steps = [("a", a[:30], [0, 29], False), ("a", a[30:32], [1], False), ("a", a[32:], [], True), ("b", b[:1], [0], False), ("b", b[1:], [23, 3], True)]
    lines = "".join(json.dumps({"step": i, "entries": [{"id": r, "tokens": t.tolist(), "want": w}], "end": [r] if e else []}) + "\n"
                    for i, (r, t, w, e) in enumerate(steps))
    la, lb = bezadra.Model(cfg, p).logits(a), bezadra.Model(cfg, p).logits(b)
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
            deep_close(np.fromfile(out / f"{k}.f32", "<f4").reshape(w.shape), w, dt, f"{name} step {k}")


def test_errors(hip):
    from rai_amd._lib import RaiHipError
    from rai_amd.config import decoder_from_config
    cfg = bm.mixed_config()
    shapes = bezadra.param_shapes(cfg)
    for change in (lambda c: c["layers"][0]["mixer"].update(kv_heads=3), lambda c: c["loop"].update(stop=9),
                   lambda c: c["layers"][1]["mixer"]["rot"].update(dims=15), lambda c: c["layers"][0]["mixer"].update(dim=513)):
        bad = bm.mixed_config()
        change(bad)
        with pytest.raises(RaiHipError):
            decoder_from_config(bad, "bf16", shapes=shapes)
    dec = bm.build(cfg, bezadra.random_params(cfg, "f32", 1), "f32", max_context=16)
    with pytest.raises(RaiHipError):
        dec.forward_rows(np.zeros((1, 17), np.uint32), [0])            # longer than the context
    with pytest.raises(RaiHipError):
        dec.forward_rows(np.full((1, 4), cfg["vocab"], np.uint32), [0])  # not a token
    dec.close()
