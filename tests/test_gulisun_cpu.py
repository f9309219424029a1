"""No-GPU checks around the Gulisun decoder: the plain CPU statement against hand calculations, the configuration reader,
the device layouts and the registry."""
import json
import math

import numpy as np
import pytest

from candy_amd import gulisun, hip, models
from oracle import gulisun_ref as ref
from tests import gulisun_models as gm


def test_rms_norm_by_hand():
    got = ref.rms_norm(np.array([[1.0, 3.0]]), np.array([2.0, -1.0]), 4.0)
    assert np.allclose(got, [[2.0 / 3.0, -1.0]])  # mean square 5, + 4, root 3


def test_rotation_turns_pairs():
    x = np.array([[[1.0, 0.0, 0.0, 2.0]]] * 2)
    got = ref.rotate(x, [0, 3], 4.0, 4)
    assert np.allclose(got[0], x[0])
    assert np.allclose(got[1, 0], [math.cos(3), -2 * math.sin(1.5), math.sin(3), 2 * math.cos(1.5)])
    flat = ref.rotate(x[:, 0], [0, 3], 4.0, 4)   # a part without heads
    assert np.allclose(flat, got[:, 0])


def test_attention_by_hand():
    q = np.array([[[1.0, 0.0]], [[2.0, 1.0]]])
    k = np.array([[[1.0, 5.0]], [[3.0, -1.0]]])
    v = np.array([[[10.0]], [[20.0]]])
    e = [math.exp(0.5 * 7.0), math.exp(0.5 * 5.0)]
    assert np.isclose(ref.attend(q, k, v, 0.5, None)[1, 0, 0], (10 * e[0] + 20 * e[1]) / sum(e))
    assert np.isclose(ref.attend(q, k, v, 0.5, [0.3])[1, 0, 0], (10 * e[0] + 20 * e[1]) / (sum(e) + math.exp(0.3)))
    assert np.isclose(ref.attend(q, k, v, 0.5, [0.3])[0, 0, 0], 10 * math.exp(0.5) / (math.exp(0.5) + math.exp(0.3)))


def test_scalar_functions():
    assert np.isclose(ref.softplus(np.array(-3.0)), math.log1p(math.exp(-3.0))) and np.isclose(ref.softplus(np.array(800.0)), 800.0)
    assert np.isclose(ref.sigmoid(np.array(0.7)), 1 / (1 + math.exp(-0.7)))
    z = 1.3
    assert np.isclose(ref.gelu_tanh(np.array(z)), 0.5 * z * (1 + math.tanh(math.sqrt(2 / math.pi) * (z + 0.044715 * z ** 3))))


def test_causal_convolution():
    x = np.array([[1.0], [2.0], [5.0]])
    got = ref.causal_conv(x, np.array([[100.0, 10.0, 1.0]]), np.array([0.5]))
    assert np.allclose(got[:, 0], [1.5, 12.5, 125.5])


def test_recurrence_by_hand():
    lam, r, i, u = np.array([-1.0]), np.array([[0.5], [0.25]]), np.array([[1.0], [0.5]]), np.array([[2.0], [3.0]])
    sp = math.log1p(math.exp(-1.0))
    a = [math.exp(-8 * 0.5 * sp), math.exp(-8 * 0.25 * sp)]
    s0 = math.sqrt(1 - a[0] ** 2) * 2.0       # the first token is scaled like every other
    assert np.allclose(ref.recurrence(u, r, i, lam)[:, 0], [s0, a[1] * s0 + math.sqrt(1 - a[1] ** 2) * 1.5])


def test_block_gate_mixes_within_blocks_only():
    w = np.array([[[1.0, 2.0], [0.0, 1.0]], [[3.0, 0.0], [0.0, 4.0]]])
    got = ref.block_gate(np.array([[1.0, -1.0, 0.5, 0.25]]), w, np.array([[0.0, 1.0], [0.0, 0.0]]))
    assert np.allclose(got, ref.sigmoid(np.array([[-1.0, 0.0, 1.5, 1.0]])))


def test_choice_and_weights():
    h = np.array([[1.0, 2.0]])
    router = np.array([[1.0, 0.0], [0.0, 1.0], [0.5, 0.25], [1.0, 0.25]])   # scores 1, 2, 1, 1.5
    ids, w = ref.route(h, router, 3)
    assert ids.tolist() == [[1, 3, 0]]
    e = np.exp([2.0, 1.5, 1.0])
    assert np.allclose(w, e / e.sum())


def test_experts_by_hand():
    mlp = {"router": {"experts": 2, "top": 1}, "shared": {"ff": 1}}
    w = {"p.router": np.array([[1.0], [-1.0]]), "p.e0.up": np.array([[2.0], [-1.0]]), "p.e0.down": np.array([[1.0, 10.0]]),
         "p.e1.up": np.array([[1.0], [-1.0]]), "p.e1.down": np.array([[1.0, 100.0]]), "p.shared.up": np.array([[1.0]]),
         "p.shared.down": np.array([[1000.0]])}
    assert np.allclose(ref.experts(np.array([[3.0], [-2.0]]), w, "p", mlp), [[36.0 + 9000.0], [400.0]])
    assert np.allclose(ref.experts(np.array([[3.0]]), w, "p", dict(mlp, shared=None)), [[36.0]])


def test_shared_cache_is_the_source_layers():
    """Layer 2 of `odd` reads layer 0's latents: changing layer 0's key projection changes it, and it has none itself."""
    cfg = gm.CONFIGS["odd"]
    w = gm.weights(cfg, 1)
    assert "l0.mix.dkv" in w and "l2.mix.dkv" not in w and "l4.mix.dkv" not in w and "l4.mix.sink" not in w
    x = np.random.default_rng(1).standard_normal((6, cfg["width"]))
    latents = {}
    ref.mixer(x, w, 0, cfg, latents)
    a = ref.mixer(x, w, 2, cfg, latents)
    latents[0] = (latents[0][0] * 0.5, latents[0][1])
    assert list(latents) == [0] and np.abs(a - ref.mixer(x, w, 2, cfg, latents)).max() > 1e-3


@pytest.mark.parametrize("name", sorted(gm.CONFIGS))
def test_prefix_does_not_depend_on_what_follows(name):
    cfg = gm.CONFIGS[name]
    w = gm.weights(cfg, 1)
    tokens = list(range(30))
    assert np.allclose(ref.forward(cfg, w, tokens)[:17], ref.forward(cfg, w, tokens[:17]), atol=1e-10)


@pytest.mark.parametrize("name", sorted(gm.CONFIGS))
def test_steady_models_have_no_close_calls(name):
    cfg = gm.CONFIGS[name]
    w = gm.weights(cfg, 3, steady=True)
    assert gm.choice_margin(cfg, w, [int(t) for t in np.random.default_rng(0).integers(0, cfg["vocab"], 30)]) > 0.03


# ------------------------------------------------------------------ reader and layouts
def test_config_reader():
    native, layers = gulisun.parse_config(gm.CONFIGS["odd"], 77, hip.ACT_F32)
    assert (native.n_layers, native.d_model, native.vocab, native.max_pos, native.act) == (6, 90, 173, 77, hip.ACT_F32)
    assert native.norm_eps == np.float32(2e-4) and native.embed_scale == 3.0
    assert [l.mixer for l in layers] == [0, 1, 0, 0, 0, 1] and [l.has_sink for l in layers] == [1, 0, 1, 0, 0, 0]
    assert [l.kv_from for l in layers] == [-1, -1, 0, -1, 0, -1]
    a = layers[0].latent
    assert (a.n_heads, a.dim, a.rot_dim, a.vdim, a.kv_rank, a.q_rank, a.rope_base) == (5, 20, 6, 24, 40, 50, 300.0)
    assert a.scale == np.float32(0.23)
    assert (layers[5].lru.width, layers[5].lru.blocks, layers[5].lru.taps) == (65, 5, 1)
    e = layers[0].experts
    assert (e.n_experts, e.top, e.d_ff, e.shared_ff) == (5, 3, 21, 37)
    assert layers[1].experts.shared_ff == 0 and layers[2].experts.n_experts == 0


@pytest.mark.parametrize("change", [("type", "attention"), ("mlp", {"kind": "dense", "ff": 8}), ("rot", {"base": 10.0, "dims": 4})])
def test_config_reader_refuses_what_it_does_not_know(change):
    cfg = json.loads(json.dumps(gm.CONFIGS["odd"]))
    key, value = change
    (cfg["layers"][0]["mixer"] if key == "rot" else cfg["layers"][0])[key] = value
    with pytest.raises(gulisun.ConfigError):
        gulisun.parse_config(cfg, 5, hip.ACT_BF16)


def test_padded_groups():
    rows = np.arange(1, 11, dtype=np.uint16)[:, None] * np.ones((1, 2), np.uint16)
    got = gulisun.padded_groups(rows, [3, 2], 4)
    assert got[:, 0].tolist() == [1, 2, 3, 0, 4, 5, 0, 0, 6, 7, 8, 0, 9, 10, 0, 0]
    with pytest.raises(gulisun.ConfigError):
        gulisun.padded_groups(rows, [3], 4)


def test_layouts_keep_the_products():
    """Contractions with the padded matrices give the plain ones at the padded places and zeros elsewhere."""
    rng = np.random.default_rng(5)
    s = hip.LatentSpec(n_heads=3, dim=20, rot_dim=6, vdim=33, kv_rank=70, q_rank=10)
    uq, uk, uv = rng.integers(1, 9, (78, 10)), rng.integers(1, 9, (60, 70)), rng.integers(1, 9, (99, 70))
    q = (gulisun.query_rows(s, uq) @ np.ones(10)).reshape(3, 64)
    want = (uq @ np.ones(10)).reshape(3, 26)
    assert np.array_equal(q[:, :20], want[:, :20]) and np.array_equal(q[:, 32:38], want[:, 20:]) and q.sum() == want.sum()
    kv = gulisun.key_value_rows(s, uk, uv)
    assert kv.shape == (3 * 32 + 3 * 64, 70) and np.array_equal(kv[32:52], uk[20:40]) and np.array_equal(kv[96 + 64:96 + 97], uv[33:66])
    kt = gulisun.transposed_keys(s, uk)
    assert kt.shape == (3 * 128, 20) and np.array_equal(kt[128:198], uk[20:40].T) and kt.sum() == uk.sum()
    o = gulisun.value_columns(s, rng.integers(1, 9, (5, 99)))
    assert o.shape == (5, 192) and (o[:, 33:64] == 0).all() and (o[:, 64:97] > 0).all()
    down = gulisun.down_rows(s, rng.integers(1, 9, (10, 4)), rng.integers(1, 9, (76, 4)))
    assert down.shape == (64 + 128 + 32, 4) and (down[64:134] > 0).all() and (down[192:198] > 0).all() and (down[198:] == 0).all()
    assert gulisun.down_rows(s, rng.integers(1, 9, (10, 4)), None).shape == (64, 4)


def test_gate_rows():
    rng = np.random.default_rng(6)
    ra, ri = rng.integers(1, 99, (2, 70, 70)), rng.integers(1, 99, (2, 70, 70))
    g = gulisun.gate_rows(ra, ri).reshape(2, 2, 2, 64, 70)   # block, group of 64, gate, row
    assert np.array_equal(g[1, 0, 0], ra[1, :64]) and np.array_equal(g[1, 0, 1], ri[1, :64])
    assert np.array_equal(g[0, 1, 1, :6], ri[0, 64:]) and (g[0, 1, :, 6:] == 0).all()


def test_registry(tmp_path):
    gm.write_folder(tmp_path / "m", gm.CONFIGS["recurrent"], gm.weights(gm.CONFIGS["recurrent"], 1))
    assert models.architecture_of(str(tmp_path / "m")) == "Gulisun"
