"""No-GPU checks around the Suvazen decoder: the plain CPU statement against hand calculations, the configuration reader,
the weight file reader, the registry and the trace replayer's bookkeeping."""
import io
import json
import math

import numpy as np
import pytest

from candy_amd import hip, models, safetensors, suvazen, trace
from oracle import suvazen_ref as ref
from tests import suvazen_models as sm


def test_layer_norm_by_hand():
    got = ref.layer_norm(np.array([[1.0, 3.0]]), np.array([2.0, 2.0]), np.array([0.5, 0.0]), 3.0)
    assert np.allclose(got, [[-0.5, 1.0]])  # deviations -1, 1; variance 1; / sqrt(1 + 3)


def test_frequencies_have_three_bands():
    rot = {"base": 1000.0, "dims": 12, "scaling": sm.SCALED}
    plain = ref.rotary_frequencies({"base": 1000.0, "dims": 12, "scaling": None})
    assert np.allclose(plain, [1000.0 ** (-i / 6) for i in range(6)])
    scaled = ref.rotary_frequencies(rot)
    wave = 2 * math.pi / plain
    ratio = scaled / plain
    kept, stretched = wave < 96 / 3.0, wave > 96 / 1.0
    assert kept.any() and stretched.any() and (~kept & ~stretched).any()
    assert np.allclose(ratio[kept], 1) and np.allclose(ratio[stretched], 1 / 5.0)
    assert ((ratio < 1) & (ratio > 1 / 5.0))[~kept & ~stretched].all()


def test_rotation_turns_pairs_and_passes_the_rest():
    x = np.zeros((2, 1, 5))
    x[:, 0] = [1.0, 0.0, 0.0, 2.0, 9.0]
    got = ref.rotate(x, [0, 3], {"base": 4.0, "dims": 4, "scaling": None})
    assert np.allclose(got[0], x[0])
    # pairs (0, 2) at angle 3 and (1, 3) at angle 3 * 4^(-1/2)
    assert np.allclose(got[1, 0], [math.cos(3), -2 * math.sin(1.5), math.sin(3), 2 * math.cos(1.5), 9.0])


def test_attention_by_hand():
    q = np.array([[[1.0]], [[1.0]], [[2.0]]])
    k = np.array([[[1.0]], [[2.0]], [[3.0]]])
    out = ref.attend(q, k, k, 0.5, 4.0, 2, np.array([0.3]))
    s = [4 * math.tanh(2 * kk * 0.5 / 4) for kk in (2.0, 3.0)]
    den = math.exp(s[0]) + math.exp(s[1]) + math.exp(0.3)
    assert np.isclose(out[2, 0, 0], (2 * math.exp(s[0]) + 3 * math.exp(s[1])) / den)
    assert not ref.visible(2, 0, 2) and ref.visible(2, 1, 2) and not ref.visible(1, 2, 2) and ref.visible(9, 0, None)
    grouped = ref.attend(np.ones((1, 4, 1)), np.array([[[1.0], [5.0]]]), np.array([[[1.0], [5.0]]]), 1.0, None, None, None)
    assert np.allclose(grouped[0, :, 0], [1, 1, 5, 5])


def test_squared_relu():
    w = {"l0.mlp.up": np.array([[1.0], [-1.0]]), "l0.mlp.down": np.array([[1.0, 10.0]])}
    assert np.allclose(ref.squared_relu_mlp(np.array([[3.0], [-2.0]]), w, "l0"), [[9.0], [40.0]])


def test_layer_runs():
    cfg = {"layers": [None] * 4, "loop": {"start": 1, "stop": 3, "times": 2}}
    assert ref.layer_runs(cfg) == [(0, None), (1, 0), (2, None), (1, 1), (2, None), (3, None)]
    assert ref.layer_runs({"layers": [None] * 2, "loop": None}) == [(0, None), (1, None)]


def test_prefix_does_not_depend_on_what_follows():
    cfg = sm.CONFIGS["odd"]
    w = sm.weights(cfg, 1)
    tokens = list(range(40))
    assert np.allclose(ref.forward(cfg, w, tokens)[:25], ref.forward(cfg, w, tokens[:25]), atol=1e-12)


def test_config_reader():
    native, layers = suvazen.parse_config(sm.CONFIGS["odd"], 77, hip.ACT_F32, lambda i: i != 1)
    assert (native.n_layers, native.d_model, native.vocab, native.max_pos, native.act) == (4, 90, 173, 77, hip.ACT_F32)
    assert (native.loop_start, native.loop_stop, native.loop_times) == (1, 3, 3)
    assert [l.has_sink for l in layers] == [1, 0, 1, 1] and [l.d_ffn for l in layers] == [84, 0, 51, 130]
    a = layers[0].attn
    assert (a.n_heads, a.n_kv_heads, a.head_dim, a.window, a.rope_dims, a.rope_original) == (6, 2, 24, 19, 10, 96)
    assert (a.rope_base, a.rope_factor, a.rope_low, a.rope_high) == (500.0, 5.0, 1.0, 3.0)
    assert a.scale == np.float32(0.31) and a.softcap == 9.0 and layers[1].attn.rope_original == 0
    native, layers = suvazen.parse_config(sm.CONFIGS["plain"], 5, hip.ACT_BF16)
    assert native.loop_times == 0 and native.logit_softcap == 0
    assert layers[0].attn.window == 0 and layers[0].attn.rope_dims == 0 and layers[0].attn.softcap == 0
    missing = {k: v for k, v in sm.CONFIGS["plain"].items() if k not in ("loop", "logit_softcap")}
    assert suvazen.parse_config(missing, 5, hip.ACT_BF16)[0].loop_times == 0


@pytest.mark.parametrize("change", [{"type": "convolution"}, {"mlp": {"kind": "gated", "ff": 8}}, {"vdim": 8}])
def test_config_reader_refuses_what_it_does_not_know(change):
    cfg = json.loads(json.dumps(sm.CONFIGS["plain"]))
    if "vdim" in change:
        cfg["layers"][0]["mixer"].update(change)
    else:
        cfg["layers"][0].update(change)
    with pytest.raises(suvazen.ConfigError):
        suvazen.parse_config(cfg, 5, hip.ACT_BF16)


def test_safetensors_roundtrip(tmp_path):
    rng = np.random.default_rng(3)
    a, b = rng.standard_normal((3, 5)).astype(np.float32), np.arange(4, dtype=np.int32)
    path = str(tmp_path / "w.safetensors")
    safetensors.write(path, {"a": ("BF16", hip.bf16_bits(a)), "b": ("I32", b), "c": ("F32", a)})
    f = safetensors.SafetensorsFile(path)
    assert "a" in f and "x" not in f
    assert np.array_equal(f.f32("a"), sm.to_bf16(a)) and np.array_equal(hip.bf16_values(f.bits("a")), sm.to_bf16(a))
    assert np.array_equal(f.raw("b")[1], b) and np.array_equal(f.f32("c"), a)
    with pytest.raises(safetensors.SafetensorsError):
        f.bits("c")
    with pytest.raises(safetensors.SafetensorsError):
        f.raw("x")
    data = open(path, "rb").read()
    for cut in (4, 40, len(data) - 1):
        open(path, "wb").write(data[:cut])
        with pytest.raises(safetensors.SafetensorsError):
            safetensors.SafetensorsFile(path)


def test_rounding_to_bfloat16_is_to_nearest_even():
    x = np.array([1.0, 1.0 + 2.0 ** -8, 1.0 + 3 * 2.0 ** -8, -1.00390625 * 2, 3.3e38], np.float32)
    assert np.array_equal(hip.bf16_bits(x), sm.bits_of(sm.to_bf16(x)))
    assert hip.bf16_values(hip.bf16_bits(x))[1] == 1.0 and hip.bf16_values(hip.bf16_bits(x))[2] == 1.015625


def test_registry(tmp_path):
    sm.write_folder(tmp_path / "m", sm.CONFIGS["plain"], sm.weights(sm.CONFIGS["plain"], 1))
    assert models.architecture_of(str(tmp_path / "m")) == "Suvazen"
    json.dump({"architecture": "Unknown"}, open(tmp_path / "m" / "config.json", "w"))
    with pytest.raises(ValueError, match="unknown architecture"):
        models.architecture_of(str(tmp_path / "m"))
    with pytest.raises(models.UnsupportedFormat):
        models.ARCHITECTURES["llama"](None, "x.gguf", 8, hip.ACT_F32)


class FakeModel:
    max_pos = 10

    def __init__(self):
        self.calls = []

    def feed(self, tokens, pos0, want):
        self.calls.append((list(tokens), pos0, list(want)))
        return np.full((len(want), 3), float(pos0), np.float32)


def test_replayer_bookkeeping(tmp_path):
    m, done = FakeModel(), []
    steps = [{"step": 4, "entries": [{"id": "a", "tokens": [1, 2, 3], "want": [2]}], "end": []},
             {"step": 5, "entries": [{"id": "a", "tokens": [4], "want": []}], "end": []},
             {"step": 6, "entries": [{"id": "a", "tokens": [5], "want": [0]}], "end": ["a"]},
             {"step": 7, "entries": [{"id": "b", "tokens": [6], "want": [0]}], "end": ["b"]}]
    trace.replay(m, io.StringIO("\n".join(json.dumps(s) for s in steps) + "\n\n"), str(tmp_path), done.append)
    assert m.calls == [([1, 2, 3], 0, [2]), ([4], 3, []), ([5], 4, [0]), ([6], 0, [0])]
    assert done == [4, 5, 6, 7] and sorted(p.name for p in tmp_path.iterdir()) == ["4.f32", "6.f32", "7.f32"]
    assert np.array_equal(np.fromfile(tmp_path / "6.f32", "<f4"), [4.0] * 3)


def test_replayer_refuses_a_second_live_request_and_overlong_ones():
    s = trace.Sequences(FakeModel())
    s.feed("a", [1], [])
    with pytest.raises(ValueError, match="one sequence"):
        s.feed("b", [1], [])
    with pytest.raises(ValueError, match="more than 10"):
        s.feed("a", [1] * 10, [])
    s.end("a")
    s.feed("b", [1], [])
