"""The Suvazen decoder and its mechanisms on the device against the plain CPU statement (oracle/suvazen_ref.py)."""
import ctypes
import io
import json
import os
import subprocess

import numpy as np
import pytest

from candy_amd import hip, models, suvazen, trace
from oracle import suvazen_ref as ref
from tests import suvazen_models as sm

pytestmark = pytest.mark.gpu

ACTS = [pytest.param(hip.ACT_F32, id="f32"), pytest.param(hip.ACT_BF16, id="bf16")]
# whole models, root mean square of the error over that of the logits: f32 is a chain of f32 sums; bfloat16 keeps 8 bits
# of every activation
WHOLE_TOL = {hip.ACT_F32: 3e-5, hip.ACT_BF16: 4e-2}


@pytest.fixture(scope="module")
def dev():
    d = hip.Device(0)
    yield d
    d.close()


def rel(got, want):
    """Worst row: root mean square of the difference over that of all of `want`."""
    got, want = np.atleast_2d(np.asarray(got, np.float64)), np.atleast_2d(np.asarray(want, np.float64))
    assert got.shape == want.shape and np.isfinite(got).all()
    return float(np.sqrt(((got - want) ** 2).mean(1)).max() / (np.sqrt((want ** 2).mean()) + 1e-30))


# ------------------------------------------------------------------ contractions
@pytest.mark.parametrize("act", ACTS)
@pytest.mark.parametrize("rows,cols", [(64, 64), (1, 5), (300, 130), (129, 2100), (2112, 100), (4200, 72), (8256, 40), (70, 18000)])
def test_contraction(dev, rows, cols, act):
    rng = np.random.default_rng(rows + cols)
    w = sm.to_bf16(rng.standard_normal((rows, cols)) * cols ** -0.5)
    dw = dev.dense(sm.bits_of(w))
    for m in (1, 2, 3, 17, 64, 65, 150) if rows < 4000 and cols < 10000 else (1, 2, 70):
        x = rng.standard_normal((m, cols)).astype(np.float32)
        xa = sm.to_bf16(x) if act == hip.ACT_BF16 else x
        want = xa.astype(np.float64) @ w.T.astype(np.float64)
        tol = 3e-6 + 3e-8 * cols ** 0.5  # f32 sums of `cols` terms
        assert rel(dev.dense_matmul(dw, x, act), want) < tol, m
        capped = 5.0 * np.tanh(3.0 * want / 5.0)
        assert rel(dev.dense_matmul(dw, x, act, hip.EPI_SOFTCAP, 3.0, 5.0), capped) < tol, m
        assert rel(dev.dense_matmul(dw, x, act, hip.EPI_SOFTCAP, 3.0, 0.0), 3.0 * want) < tol, m
        relu2 = np.maximum(want, 0) ** 2
        got = dev.dense_matmul(dw, x, act, hip.EPI_SQUARED_RELU)
        # bfloat16 output: one rounding per value
        assert (np.abs(got - relu2) <= (0 if act == hip.ACT_F32 else 2.0 ** -8) * relu2 + 1e-4 * relu2.max()).all(), m
    dw.free()


def test_contraction_arguments(dev):
    dw = dev.dense(np.zeros((4, 8), np.uint16))
    x = dev.alloc(4 * 8)
    L = hip.lib()
    assert L.candy_hip_dense_matmul(dev.handle, None, x.ptr, 1, 0, 0, 1.0, 0.0, x.ptr) == 1
    assert L.candy_hip_dense_matmul(dev.handle, dw.handle, x.ptr, -1, 0, 0, 1.0, 0.0, x.ptr) == 1
    assert L.candy_hip_dense_matmul(dev.handle, dw.handle, x.ptr, 1, 7, 0, 1.0, 0.0, x.ptr) == 1
    assert L.candy_hip_dense_matmul(dev.handle, dw.handle, x.ptr, 1, 0, 9, 1.0, 0.0, x.ptr) == 1


# ------------------------------------------------------------------ norms
@pytest.mark.parametrize("cols", [1, 5, 64, 90, 1000, 1030, 4096, 6000, 16384])
def test_layer_norm(dev, cols):
    rng = np.random.default_rng(cols)
    x = (rng.standard_normal((3, cols)) + 3.0).astype(np.float32)  # a mean that must not leak into the variance
    y = (rng.standard_normal((3, cols)) * 0.01 - 1.0).astype(np.float32)
    w, b, step = (rng.standard_normal(cols).astype(np.float32) for _ in range(3))
    for eps in (1e-5, 0.3):
        want = ref.layer_norm(x.astype(np.float64), w, b, eps)
        assert np.abs(dev.layer_norm(x, w, b, eps) - want).max() < 2e-5 * max(1.0, np.abs(want).max())
        want = x + 0.37 * ref.layer_norm(y.astype(np.float64), w, b, eps)
        assert np.abs(dev.add_layer_norm(x, y, w, b, eps, 0.37) - want).max() < 1e-4 * max(1.0, np.abs(want).max())
        assert np.abs(dev.add_layer_norm(x, y, w, b, eps, 0.37, step) - want - step).max() < 1e-4 * max(1.0, np.abs(want).max())


# ------------------------------------------------------------------ attention
def oracle_attention(mx, q, k, sink, act):
    """q [n, H, d], k [n, G, d] as projected; bfloat16: rounded where the device stores them."""
    pos = np.arange(q.shape[0])
    qr, kr, v = ref.rotate(q, pos, mx["rot"]), ref.rotate(k, pos, mx["rot"]), k
    if act == hip.ACT_BF16:
        qr, kr, v = (sm.to_bf16(a).astype(np.float64) for a in (qr, kr, v))
    n = q.shape[0]
    return ref.attend(qr, kr, v, mx["scale"], mx["softcap"], (mx["mask"] or {}).get("size"), sink).reshape(n, -1)


def device_attention(dev, mx, q, k, sink, act, portions, max_pos=None):
    """The same through the device's kernels in portions: a number > 1 is a prompt pass, 1 a decode step."""
    n, spec = q.shape[0], suvazen.attn_spec(mx)
    max_pos = max_pos or n + 3
    bytes_ = mx["kv_heads"] * max_pos * hip.lib().candy_hip_attn_row(mx["dim"]) * (4 if act == hip.ACT_F32 else 2)
    kc, vc = dev.alloc(bytes_).zero(), dev.alloc(bytes_).zero()
    qk = np.concatenate([q.reshape(n, -1), k.reshape(n, -1)], 1).astype(np.float32)
    out, at = [], 0
    for p in portions:
        out.append(dev.window_attention(spec, act, qk[at:at + p], at, max_pos, kc, vc, sink, decode=p == 1))
        at += p
    assert at == n
    return np.concatenate(out)


MIXERS = {
    "odd": sm.mixer(6, 2, 24, 19, 10, 500.0, sm.SCALED, 0.31, 9.0),
    "full": sm.mixer(4, 4, 64, None, 64, 10000.0, None, 0.125, None),
    "one-kv": sm.mixer(7, 1, 20, 70, 20, 100.0, sm.SCALED, 0.3, 3.0),
    "hd128": sm.mixer(8, 1, 128, 64, 32, 1e6, sm.SCALED, 0.09, 30.0),
    "hd96": sm.mixer(4, 2, 96, 65, 96, 10000.0, None, 0.1, 20.0),
    "hd130": sm.mixer(2, 2, 130, 33, 2, 10.0, None, 0.1, 20.0),
    "hd256": sm.mixer(2, 1, 256, 130, 128, 10000.0, None, 0.06, 50.0),
    "window1": sm.mixer(4, 2, 32, 1, 16, 10000.0, None, 0.2, 10.0),
    "no-rope": sm.mixer(3, 1, 33, 10, 0, scale=0.2, softcap=5.0),
}


@pytest.mark.parametrize("act", ACTS)
@pytest.mark.parametrize("name", sorted(MIXERS))
def test_attention_whole_portions_and_decode(dev, name, act):
    mx, n = MIXERS[name], 150
    rng = np.random.default_rng(len(name))
    q = rng.standard_normal((n, mx["heads"], mx["dim"])) * 1.5
    k = rng.standard_normal((n, mx["kv_heads"], mx["dim"])) * 1.5
    sink = rng.standard_normal(mx["heads"]).astype(np.float32) * 2
    q, k = q.astype(np.float32), k.astype(np.float32)
    tol = 1e-5 if act == hip.ACT_F32 else 1.2e-2
    for s in (sink, None):
        want = oracle_attention(mx, q.astype(np.float64), k.astype(np.float64), s, act)
        for portions in ([n], [2, 3, 61, 64, 20], [1] * 40 + [37] + [1] * 73):
            assert rel(device_attention(dev, mx, q, k, s, act, portions), want) < tol, (s is None, portions[:3])


@pytest.mark.parametrize("act", ACTS)
@pytest.mark.parametrize("window", [1, 2, 16, 33, 63, 64, 65, 100, 128])
def test_window_edges(dev, window, act):
    """One key far louder than all others: inside the window it owns the output, one position further it is gone."""
    n, d = 230, 64
    mx = sm.mixer(2, 1, d, window, 0, scale=0.125, softcap=50.0)
    rng = np.random.default_rng(window)
    base = rng.standard_normal(d)
    q = np.tile(base, (n, 2, 1)).astype(np.float32)
    k = (rng.standard_normal((n, 1, d)) * 0.1).astype(np.float32)
    sink = np.full(2, -1.0, np.float32)
    for loud in (0, 1, 37, 63, 64, 65):
        kk = k.copy()
        kk[loud, 0] = base * 4.0
        want = oracle_attention(mx, q.astype(np.float64), kk.astype(np.float64), sink, act)
        for portions in ([n], [1] * 130 + [100], [50, 50] + [1] * 130):
            got = device_attention(dev, mx, q, kk, sink, act, portions)
            assert np.abs(got - want).max() < (1e-4 if act == hip.ACT_F32 else 0.05), (loud, portions[:2])
            along = got[:, :d] @ base / (base @ base)  # 4 where the loud key is all there is
            assert (along[loud:loud + window] > 3.5).all() and (np.abs(np.delete(along, np.s_[loud:loud + window])) < 0.5).all()


@pytest.mark.parametrize("act", ACTS)
def test_sink_is_counted_once(dev, act):
    """Equal scores: the output is the mean of the values times keys / (keys + exp(sink - score))."""
    n, d = 90, 32
    mx = sm.mixer(4, 2, d, 40, 0, scale=1.0, softcap=None)
    q = np.zeros((n, 4, d), np.float32)
    k = np.ones((n, 2, d), np.float32)
    sink = np.array([-30.0, 0.0, 2.0, 30.0], np.float32)
    cnt = np.minimum(np.arange(n) + 1, 40)[:, None]
    want = cnt / (cnt + np.exp(sink.astype(np.float64)))
    for portions in ([n], [1] * n, [30, 1, 1, 58]):
        got = device_attention(dev, mx, q, k, sink, act, portions).reshape(n, 4, d)
        assert np.abs(got - want[:, :, None]).max() < (1e-5 if act == hip.ACT_F32 else 4e-3)


@pytest.mark.parametrize("act", ACTS)
def test_long_decode_over_many_splits(dev, act):
    mx, n = sm.mixer(4, 1, 64, 1500, 32, 10000.0, None, 0.2, 20.0), 1800
    rng = np.random.default_rng(77)
    q = rng.standard_normal((n, 4, 64)).astype(np.float32)
    k = rng.standard_normal((n, 1, 64)).astype(np.float32)
    sink = np.ones(4, np.float32)
    got = device_attention(dev, mx, q, k, sink, act, [1790] + [1] * 10, max_pos=4096)[-12:]
    pos = np.arange(n)
    qr, kr = ref.rotate(q.astype(np.float64), pos, mx["rot"]), ref.rotate(k.astype(np.float64), pos, mx["rot"])
    v = k.astype(np.float64)
    want = []
    for i in range(n - 12, n):
        s = 20.0 * np.tanh(qr[i] @ kr[i - 1499:i + 1, 0].T * 0.2 / 20.0)
        e = np.exp(s - s.max(1, keepdims=True))
        want.append((e / (e.sum(1) + np.exp(1.0 - s.max(1)))[:, None] @ v[i - 1499:i + 1, 0]).reshape(-1))
    assert rel(got, np.array(want)) < (1e-5 if act == hip.ACT_F32 else 1.2e-2)


def test_attention_arguments(dev):
    buf = dev.alloc(1 << 16)
    good = suvazen.attn_spec(sm.mixer(2, 1, 32, 4, 16))
    bad = [dict(n_heads=3, n_kv_heads=2), dict(head_dim=257), dict(head_dim=0), dict(rope_dims=15), dict(rope_dims=34),
           dict(window=-1), dict(softcap=-1.0), dict(rope_original=8, rope_low=2.0, rope_high=1.0)]
    for change in bad:
        s = hip.AttnSpec.from_buffer_copy(good)
        for key, v in change.items():
            setattr(s, key, v)
        assert hip.lib().candy_hip_window_attention(dev.handle, ctypes.byref(s), 0, buf.ptr, 1, 0, 8, buf.ptr, buf.ptr, None, 0,
                                                    buf.ptr) == 1, change
    for n, pos0, decode in ((1, 8, 0), (0, 0, 0), (2, 0, 1), (9, 0, 0), (1, -1, 0)):
        assert hip.lib().candy_hip_window_attention(dev.handle, ctypes.byref(good), 0, buf.ptr, n, pos0, 8, buf.ptr, buf.ptr, None,
                                                    decode, buf.ptr) == 1


# ------------------------------------------------------------------ whole models
@pytest.fixture(scope="module")
def cases():
    """Per configuration: weights, 140 tokens, the oracle's logits and residual streams."""
    out = {}
    for i, (name, cfg) in enumerate(sorted(sm.CONFIGS.items())):
        w = sm.weights(cfg, seed=100 + i, peaky=2.0)
        tokens = [int(t) for t in np.random.default_rng(i).integers(0, cfg["vocab"], 140)]
        streams = []
        out[name] = (cfg, w, tokens, ref.forward(cfg, w, tokens, streams), streams)
    return out


def build(dev, cfg, w, act, max_pos=160):
    return suvazen.build(dev, cfg, sm.Tensors(w), max_pos, act)


@pytest.mark.parametrize("act", ACTS)
@pytest.mark.parametrize("name", sorted(sm.CONFIGS))
def test_model_prompt(dev, cases, name, act):
    cfg, w, tokens, want, streams = cases[name]
    m = build(dev, cfg, w, act)
    got = m.feed(tokens, 0, range(len(tokens)))
    assert rel(got, want) < WHOLE_TOL[act]
    assert rel(m.prompt_hidden(len(tokens)), streams[-1]) < WHOLE_TOL[act]
    nt, last = m.prefill(tokens, 0)
    assert rel(last, want[-1]) < WHOLE_TOL[act] and nt == int(np.argmax(last))
    m.free()


@pytest.mark.parametrize("act", ACTS)
@pytest.mark.parametrize("name", sorted(sm.CONFIGS))
def test_model_token_by_token(dev, cases, name, act):
    cfg, w, tokens, want, streams = cases[name]
    m = build(dev, cfg, w, act)
    got = [m.decode(t, p)[1] for p, t in enumerate(tokens)]
    assert rel(got, want) < WHOLE_TOL[act]
    assert rel(m.hidden(), streams[-1][-1]) < WHOLE_TOL[act]
    m.free()


@pytest.mark.parametrize("act", ACTS)
@pytest.mark.parametrize("name", sorted(sm.CONFIGS))
def test_model_in_portions(dev, cases, name, act):
    cfg, w, tokens, want, _ = cases[name]
    m = build(dev, cfg, w, act)
    for portions in ([2] * 70, [3, 2, 64, 1, 1, 65, 4], [1, 139], [19, 14, 31, 36, 40]):
        got, at = [], 0
        for p in portions:
            got.append(m.feed(tokens[at:at + p], at, range(p)))
            at += p
        assert rel(np.concatenate(got), want) < WHOLE_TOL[act], portions[:3]
    m.free()


@pytest.mark.parametrize("act", ACTS)
def test_layers_one_by_one(dev, cases, act):
    """Every layer of every configuration alone: the oracle's stream in front of it goes in, the one behind it comes out
    (through the decode step at position 0 and, for the stack so far, through the prompt pass)."""
    for name, (cfg, w, tokens, _, _) in cases.items():
        for i in range(len(cfg["layers"])):
            one = sm.changed(cfg, layers=[cfg["layers"][i]], loop=None)
            ww = {k.replace(f"l{i}.", "l0."): v for k, v in w.items() if k.startswith(f"l{i}.")}
            ww.update({k: w[k] for k in ("embed", "head", "final.norm", "final.norm.b")})
            trace_ = []
            ref.forward(one, ww, tokens[:80], trace_)
            m = build(dev, one, ww, act)
            m.feed(tokens[:80], 0, [79])
            assert rel(m.prompt_hidden(80), trace_[0]) < WHOLE_TOL[act] / 2, (name, i)
            x = np.random.default_rng(i).standard_normal(cfg["width"]).astype(np.float32)
            m.decode_hidden(x, 0)
            want = ref.layer(x.astype(np.float64)[None], {k: v.astype(np.float64) for k, v in ww.items()}, 0, one)
            assert rel(m.hidden(), want[0]) < WHOLE_TOL[act] / 2, (name, i)
            m.free()


@pytest.mark.parametrize("act", ACTS)
def test_sequences_share_nothing(dev, cases, act):
    """The cache is taken over by the next sequence: shorter, longer, after a long one, in other portions."""
    cfg, w, tokens, want, _ = cases["odd"]
    m = build(dev, cfg, w, act)
    other = [int(t) for t in np.random.default_rng(9).integers(0, cfg["vocab"], 150)]
    first = m.feed(tokens, 0, range(140))
    m.feed(other, 0, [])
    assert np.array_equal(m.feed(tokens, 0, range(140)), first)
    short = ref.forward(cfg, w, other[:5])
    assert rel(m.feed(other[:5], 0, range(5)), short) < WHOLE_TOL[act]
    got = [m.decode(t, p)[1] for p, t in enumerate(tokens[:30])]
    assert rel(got, want[:30]) < WHOLE_TOL[act]
    m.free()


def test_far_keys_matter_and_stop_mattering(dev):
    """A single windowed layer: changing one token changes the logits of exactly the positions whose window holds it; a
    loop of two passes doubles the reach."""
    for times, window in ((0, 24), (2, 24), (0, 64)):
        cfg = sm.config([(sm.mixer(4, 2, 32, window, 16, 10000.0, None, 0.18, 20.0), 64)], 96, 120, loop=(0, 1, times) if times else None)
        w = sm.weights(cfg, seed=5, peaky=0.3, sinks=False)
        a = [int(t) for t in np.random.default_rng(1).integers(0, 120, 130)]
        b = list(a)
        b[3] = (b[3] + 1) % 120
        reach = 3 + (window - 1) * max(times, 1)
        m = build(dev, cfg, w, hip.ACT_F32)
        for portions in ([130], [1] * 130, [70, 30] + [1] * 30):
            rows = []
            for seq in (a, b):
                got, at = [], 0
                for p in portions:
                    got.append(m.feed(seq[at:at + p], at, range(p)))
                    at += p
                rows.append(np.concatenate(got))
            diff = np.abs(rows[0] - rows[1]).max(1)
            # outside: only what other order of sums over the same values could leave, which is nothing
            assert (diff[:3] == 0).all() and (diff[reach + 1:] == 0).all(), (times, window, portions[:2])
            assert diff[3] > 0 and diff[reach] > 0 and (diff[3:reach + 1] > 0).all()
        m.free()


def test_passes_have_their_own_cache_and_row(dev):
    """The same weights run as one layer per pass without a loop (rows added by hand) give the same stream."""
    layer = (sm.mixer(4, 2, 32, 9, 16, 10000.0, None, 0.18, 20.0), 64)
    cfg = sm.config([layer], 96, 120, loop=(0, 1, 3))
    w = sm.weights(cfg, seed=6, peaky=2.0)
    tokens = [int(t) for t in np.random.default_rng(2).integers(0, 120, 60)]
    want = ref.forward(cfg, w, tokens)
    swapped = dict(w)
    swapped["loop.step"] = w["loop.step"][::-1].copy()
    for act in (hip.ACT_F32, hip.ACT_BF16):
        m, s = build(dev, cfg, w, act), build(dev, cfg, swapped, act)
        assert rel(m.feed(tokens, 0, range(60)), want) < WHOLE_TOL[act]
        assert rel(s.feed(tokens, 0, range(60)), ref.forward(cfg, swapped, tokens)) < WHOLE_TOL[act]
        assert rel(s.feed(tokens, 0, range(60)), want) > 0.1  # the order of the rows shows
        m.free()
        s.free()


def test_graph_replays_equal_eager_launches(dev, cases):
    for name, (cfg, w, tokens, _, _) in cases.items():
        m = build(dev, cfg, w, hip.ACT_BF16)
        runs = []
        for graph in (False, True):
            m.set_graph(graph)
            m.feed(tokens[:30], 0, [])
            out = []
            for p in range(30, 70):
                out.append(m.decode(tokens[p], p)[1])
                if p % 10 == 0:  # eager work and synchronizations between the replays
                    dev.layer_norm(np.ones((2, 8)), np.ones(8), np.ones(8), 1e-5)
                    m.feed(tokens[p + 1:p + 3], p + 1, [0])
            runs.append(np.array(out))
        assert np.array_equal(runs[0], runs[1]), name
        m.free()


def test_greedy_generation(dev):
    """The generation loop (token handed over on the device) against the oracle's greedy choice, as far as the two best
    logits are apart; and against a loop over single steps."""
    cfg = sm.CONFIGS["odd"]
    for seed in (1, 2):
        w = sm.weights(cfg, seed=200 + seed, peaky=1.0)
        prompt = [int(t) for t in np.random.default_rng(seed).integers(0, cfg["vocab"], 12)]
        want, gaps = ref.greedy(cfg, w, prompt, 40)
        for act, gap in ((hip.ACT_F32, 1e-3), (hip.ACT_BF16, 0.6)):
            m = build(dev, cfg, w, act)
            got = m.greedy(prompt, 40)
            sure = next((i for i, g in enumerate(gaps) if g < gap), len(gaps))
            if act == hip.ACT_F32:
                assert sure == 40
            assert got[:sure] == want[:sure]
            tok, _ = m.prefill(prompt)
            loop = [tok]
            for i in range(39):
                tok, _ = m.decode(tok, 12 + i)
                loop.append(tok)
            assert loop == got
            m.free()


def test_model_arguments(dev, cases):
    cfg, w, tokens, _, _ = cases["plain"]
    m = build(dev, cfg, w, hip.ACT_BF16, max_pos=20)
    for call in (lambda: m.feed(tokens[:21], 0, []), lambda: m.feed([cfg["vocab"], 0], 0, []), lambda: m.decode(0, 20),
                 lambda: m.decode(-1, 0), lambda: m.feed(tokens[:5], 17, [])):
        with pytest.raises(hip.CandyHipError):
            call()
    with pytest.raises(ValueError):
        m.feed(tokens[:3], 0, [3])
    with pytest.raises(hip.CandyHipError):
        m.set_matrix(hip.SV_O, 0, dev.dense(np.zeros((4, 4), np.uint16)))
    with pytest.raises(hip.CandyHipError):
        m.set_vector(hip.SV_SINK, 0, np.zeros(3, np.float32))
    with pytest.raises(hip.CandyHipError):
        hip.Suvazen(dev, *suvazen.parse_config(sm.changed(cfg, loop={"start": 0, "stop": 2, "times": 2}), 8, hip.ACT_BF16)).free()
    incomplete = hip.Suvazen(dev, *suvazen.parse_config(cfg, 8, hip.ACT_BF16))
    incomplete.set_matrix(hip.SV_EMBED, -1, dev.dense(sm.bits_of(w["embed"])))
    with pytest.raises(hip.CandyHipError):
        incomplete.feed(tokens[:2], 0, [])
    incomplete.free()
    m.free()


@pytest.mark.parametrize("act", ACTS)
def test_trace_through_the_registry(dev, cases, tmp_path, act):
    """A folder on disk, the registry's loader, the replayer: portions, single tokens and three requests in a row."""
    cfg, w, tokens, want, _ = cases["wide"]
    sm.write_folder(tmp_path / "model", cfg, w)
    m = models.load(dev, str(tmp_path / "model"), max_pos=140, act=act)
    assert models.architecture_of(str(tmp_path / "model")) == "Suvazen"
    steps, at = [], 0
    for p in (60, 2, 1, 1, 5, 1, 70):
        steps.append({"entries": [{"id": "a", "tokens": tokens[at:at + p], "want": [0, p - 1] if p > 1 else [0]}], "end": []})
        at += p
    steps[-1]["end"] = ["a"]
    steps.append({"entries": [{"id": "b", "tokens": tokens[:9], "want": []}], "end": ["b"]})
    steps.append({"entries": [{"id": "c", "tokens": tokens[:1], "want": [0]}], "end": ["c"]})
    lines = [json.dumps(dict(s, step=i)) + "\n" for i, s in enumerate(steps)]
    done = []
    trace.replay(m, io.StringIO("".join(lines)), str(tmp_path), done.append)
    assert done == list(range(len(steps)))
    at = 0
    for i, p in enumerate((60, 2, 1, 1, 5, 1, 70)):
        got = np.fromfile(tmp_path / f"{i}.f32", "<f4").reshape(-1, cfg["vocab"])
        assert rel(got, want[[at, at + p - 1] if p > 1 else [at]]) < WHOLE_TOL[act]
        at += p
    assert not (tmp_path / "7.f32").exists()
    assert rel(np.fromfile(tmp_path / "8.f32", "<f4"), want[0]) < WHOLE_TOL[act]
    m.free()


@pytest.mark.parametrize("dtype,act", [("bfloat16", hip.ACT_BF16), ("float32", hip.ACT_F32)])
def test_trace_run_program(cases, tmp_path, dtype, act):
    """The command line: its own process, steps on standard input, logits in files."""
    cfg, w, tokens, want, _ = cases["odd"]
    sm.write_folder(tmp_path / "model", cfg, w)
    steps = [{"step": 0, "entries": [{"id": "x", "tokens": tokens[:50], "want": [49, 3]}], "end": []},
             {"step": 1, "entries": [{"id": "x", "tokens": tokens[50:51], "want": [0]}], "end": ["x"]},
             {"step": 2, "entries": [{"id": "y", "tokens": tokens[:2], "want": [1]}], "end": ["y"]}]
    root = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
    r = subprocess.run([os.path.join(root, "bin", "trace_run"), "--model", str(tmp_path / "model"), "--dtype", dtype, "--out",
                        str(tmp_path / "out"), "--max-tokens", "60"], input="".join(json.dumps(s) + "\n" for s in steps),
                       capture_output=True, text=True, timeout=90)
    assert r.returncode == 0, r.stderr[-500:]
    assert [l for l in r.stdout.splitlines() if l.startswith("done")] == ["done 0", "done 1", "done 2"]
    for step, rows in ((0, [49, 3]), (1, [50]), (2, [1])):
        got = np.fromfile(tmp_path / "out" / f"{step}.f32", "<f4").reshape(-1, cfg["vocab"])
        assert rel(got, want[rows]) < WHOLE_TOL[act]
