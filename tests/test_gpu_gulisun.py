"""The Gulisun decoder and its mechanisms on the device against the plain CPU statement (oracle/gulisun_ref.py)."""
import ctypes
import io
import json
import os
import subprocess

import numpy as np
import pytest

from candy_amd import gulisun, hip, models, trace
from oracle import gulisun_ref as ref
from tests import gulisun_models as gm

pytestmark = pytest.mark.gpu

ACTS = [pytest.param(hip.ACT_F32, id="f32"), pytest.param(hip.ACT_BF16, id="bf16")]
# whole models, root mean square of the error over that of the logits: f32 is a chain of f32 sums; bfloat16 keeps 8 bits
# of every activation
WHOLE_TOL = {hip.ACT_F32: 3e-5, hip.ACT_BF16: 4e-2}
LAYER_TOL = {hip.ACT_F32: 1.5e-5, hip.ACT_BF16: 3e-2}
EPS = 1e-5


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


def own(got, want):
    """Worst row: root mean square of the difference over that of the row itself."""
    return max(rel(g, w) for g, w in zip(got, want))


def up(n, to):
    return -(-n // to) * to


def dense(dev, a):
    return dev.dense(gm.bits_of(a))


# ------------------------------------------------------------------ norm and epilogue
@pytest.mark.parametrize("cols", [1, 5, 90, 1030, 4096, 6000, 16384])
def test_rms_norm_of_a_result(dev, cols):
    rng = np.random.default_rng(cols)
    x, y = rng.standard_normal((3, cols)).astype(np.float32), (rng.standard_normal((3, cols)) * 0.01 - 1.0).astype(np.float32)
    w = rng.standard_normal(cols).astype(np.float32)
    for eps in (1e-5, 0.3):
        want = x + 0.37 * ref.rms_norm(y.astype(np.float64), w, eps)
        assert np.abs(dev.add_rms_norm(x, y, w, eps, 0.37) - want).max() < 2e-5 * max(1.0, np.abs(want).max())


@pytest.mark.parametrize("act", ACTS)
def test_contraction_into_the_activation_format(dev, act):
    rng = np.random.default_rng(1)
    w, x = gm.to_bf16(rng.standard_normal((130, 200))), gm.to_bf16(rng.standard_normal((150, 200)))
    want = x.astype(np.float64) @ w.T.astype(np.float64)
    for m in (1, 7, 150):
        got = dev.dense_matmul(dense(dev, w), x[:m], act, hip.EPI_ACT)
        assert (np.abs(got - want[:m]) <= (0 if act == hip.ACT_F32 else 2.0 ** -8) * np.abs(want[:m]) + 1e-5 * np.abs(want).max()).all()
        if act == hip.ACT_BF16:
            assert np.array_equal(got, gm.to_bf16(got))


# ------------------------------------------------------------------ latent attention
MIXERS = {
    "odd": gm.latent(5, 20, 6, 24, 40, 50, 300.0, 0.23),
    "one-head": gm.latent(1, 7, 2, 5, 3, 8, 10.0, 0.4),
    "even": gm.latent(20, 128, 64, 128, 512, 64),
    "dk96": gm.latent(3, 64, 18, 70, 130, 40),
    "dk256": gm.latent(2, 192, 64, 256, 256, 40),
    "wide-values": gm.latent(2, 30, 10, 300, 64, 40),
    "wide-queries": gm.latent(17, 250, 40, 33, 70, 40),
    "wide-rank": gm.latent(2, 32, 32, 32, 600, 40),
    "wide-turn": gm.latent(3, 16, 160, 16, 64, 40, 500.0),
    "no-turn": gm.latent(4, 32, 0, 32, 64, 40),
}


class Latent:
    """One layer's weights and rows, in the oracle's layout and the device's."""

    def __init__(self, dev, m, n, seed, quiet=1.0):
        rng = np.random.default_rng(seed)
        self.dev, self.m, self.n = dev, m, n
        self.spec = gulisun.latent_spec(m)
        H, s = m["heads"], np.sqrt(1.5) * (m["scale"] * np.sqrt(m["dim"] + m["rot_dim"])) ** -0.5
        self.uk = gm.to_bf16(rng.standard_normal((H * m["dim"], m["kv_rank"])) * s * m["kv_rank"] ** -0.5)
        self.uv = gm.to_bf16(rng.standard_normal((H * m["vdim"], m["kv_rank"])) * m["kv_rank"] ** -0.5)
        self.norm = gm.to_bf16(1 + 0.3 * rng.standard_normal(m["kv_rank"]))
        self.q = (rng.standard_normal((n, H, m["dim"] + m["rot_dim"])) * s).astype(np.float32)
        self.z = (rng.standard_normal((n, m["kv_rank"] + m["rot_dim"])) * s * quiet).astype(np.float32)
        self.ukv, self.ukt = dev.dense(gulisun.key_value_rows(self.spec, gm.bits_of(self.uk), gm.bits_of(self.uv))), \
            dev.dense(gulisun.transposed_keys(self.spec, gm.bits_of(self.uk)))

    def oracle(self, sink, act, rows=None):
        m, n, H = self.m, self.n, self.m["heads"]
        rounded = gm.to_bf16 if act == hip.ACT_BF16 else (lambda a: a)
        z = self.z.astype(np.float64)
        pos = np.arange(n)
        c = rounded(ref.rms_norm(z[:, :m["kv_rank"]], self.norm, EPS)).astype(np.float64)
        kr = rounded(ref.rotate(z[:, m["kv_rank"]:], pos, m["rot"]["base"], m["rot_dim"])).astype(np.float64)
        q = self.q.astype(np.float64)
        q = np.concatenate([q[..., :m["dim"]], ref.rotate(q[..., m["dim"]:], pos, m["rot"]["base"], m["rot_dim"])], -1)
        k = (c @ self.uk.T.astype(np.float64)).reshape(n, H, -1)
        k = np.concatenate([k, np.repeat(kr[:, None], H, 1)], -1)
        v = (c @ self.uv.T.astype(np.float64)).reshape(n, H, -1)
        return ref.attend(q, k, v, m["scale"], sink).reshape(n, -1)

    def device(self, sink, act, portions, max_pos=None, cache=None, own=True):
        m, n, H = self.m, self.n, self.m["heads"]
        dim, rot, kv, vd = up(m["dim"], 32), up(m["rot_dim"], 32), up(m["kv_rank"], 64), up(m["vdim"], 32)
        q = np.zeros((n, H, dim + rot), np.float32)
        q[..., :m["dim"]], q[..., dim:dim + m["rot_dim"]] = self.q[..., :m["dim"]], self.q[..., m["dim"]:]
        z = np.zeros((n, kv + rot), np.float32)
        z[:, :m["kv_rank"]], z[:, kv:kv + m["rot_dim"]] = self.z[:, :m["kv_rank"]], self.z[:, m["kv_rank"]:]
        max_pos = max_pos or n + 3
        assert hip.lib().candy_hip_latent_row(ctypes.byref(self.spec)) == kv + rot
        if cache is None:
            cache = self.dev.alloc(max_pos * (kv + rot) * 4).zero()
        out, at = [], 0
        for p in portions:
            out.append(self.dev.latent_attention(self.spec, act, q[at:at + p].reshape(p, -1), z[at:at + p] if own else None, self.norm, EPS,
                                                 self.ukv, self.ukt, at, max_pos, cache, sink, decode=p == 1))
            at += p
        assert at == n
        return np.concatenate(out).reshape(n, H, vd)[:, :, :m["vdim"]].reshape(n, -1)


ATT_TOL = {hip.ACT_F32: 1e-5, hip.ACT_BF16: 1.5e-2}


@pytest.mark.parametrize("act", ACTS)
@pytest.mark.parametrize("name", sorted(MIXERS))
def test_latent_attention_whole_portions_and_decode(dev, name, act):
    case = Latent(dev, MIXERS[name]["mixer"], 150, len(name))
    sink = np.random.default_rng(1).standard_normal(case.m["heads"]).astype(np.float32) * 2
    for s in (sink, None):
        want = case.oracle(s, act)
        for portions in ([150], [2, 3, 61, 64, 20], [1] * 40 + [37] + [1] * 73):
            assert rel(case.device(s, act, portions), want) < ATT_TOL[act], (s is None, portions[:3])


@pytest.mark.parametrize("act", ACTS)
def test_shared_cache(dev, act):
    """A layer without key projection of its own: the rows another one left, other queries, heads and values."""
    a = Latent(dev, MIXERS["odd"]["mixer"], 100, 3)
    b = Latent(dev, gm.latent(3, 36, 6, 17, 40, 70, 300.0, 0.31)["mixer"], 100, 4)
    b.z, b.norm = a.z, a.norm
    for first, portions in (([100], [100]), ([1] * 100, [30] + [1] * 70), ([64, 36], [1] * 64 + [36])):
        cache = dev.alloc(128 * 128 * 4).zero()
        a.device(None, act, first, max_pos=128, cache=cache)
        assert rel(b.device(None, act, portions, max_pos=128, cache=cache, own=False), b.oracle(None, act)) < ATT_TOL[act]


@pytest.mark.parametrize("act", ACTS)
@pytest.mark.parametrize("loud", [0, 1, 31, 32, 63, 64, 100, 127, 128])
def test_far_keys(dev, act, loud):
    """One latent that every query is drawn to, among quiet ones: from its position on it owns the output."""
    n, m = 230, gm.latent(2, 32, 8, 32, 32, 16, scale=0.3)["mixer"]
    case = Latent(dev, m, n, 9)
    case.uk = gm.to_bf16(np.tile(np.eye(32), (2, 1)))
    case.uv = case.uk
    case.ukv, case.ukt = dev.dense(gulisun.key_value_rows(case.spec, gm.bits_of(case.uk), gm.bits_of(case.uv))), \
        dev.dense(gulisun.transposed_keys(case.spec, gm.bits_of(case.uk)))
    case.norm = np.ones(32, np.float32)
    case.q[:] = 0
    case.q[..., 0] = 10.0
    case.z[:, 0] = 0
    case.z[loud] = 0
    case.z[loud, 0] = 3.0                       # normed: sqrt(32) on the first axis
    sink = np.full(2, 1.0, np.float32)
    want = case.oracle(sink, act)
    for portions in ([n], [1] * 130 + [100], [50, 50] + [1] * 130, [2] * 115):
        got = case.device(sink, act, portions)
        assert np.abs(got - want).max() < (1e-4 if act == hip.ACT_F32 else 0.05), portions[:2]
        assert (got[loud:, 0] > 5.3).all() and (np.abs(got[:loud, 0]) < 0.01).all()


@pytest.mark.parametrize("act", ACTS)
def test_sink_is_counted_once(dev, act):
    """Equal scores of 0: the output is the mean of the values times keys / (keys + exp(sink))."""
    n, m = 90, gm.latent(4, 32, 4, 32, 64, 16, scale=1.0)["mixer"]
    case = Latent(dev, m, n, 2)
    case.q[:] = 0
    case.z[:] = case.z[0]
    sink = np.array([-30.0, 0.0, 2.0, 30.0], np.float32)
    value = case.oracle(None, act)[0].reshape(4, 32)
    cnt = np.arange(1, n + 1)[:, None, None]
    want = value[None] * (cnt / (cnt + np.exp(sink.astype(np.float64))[None, :, None]))
    for portions in ([n], [1] * n, [30, 1, 1, 58]):
        got = case.device(sink, act, portions).reshape(n, 4, 32)
        assert np.abs(got - want).max() < (1e-5 if act == hip.ACT_F32 else 2e-2) * np.abs(value).max()


@pytest.mark.parametrize("act", ACTS)
@pytest.mark.parametrize("name", ["odd", "wide-rank"])
def test_long_decode_over_many_splits(dev, name, act):
    n, m = 1300, MIXERS[name]["mixer"]
    case = Latent(dev, m, n, 5)
    sink = np.ones(m["heads"], np.float32)
    got = case.device(sink, act, [1290] + [1] * 10, max_pos=5000)
    assert rel(got[-12:], case.oracle(sink, act)[-12:]) < ATT_TOL[act]


def test_latent_attention_arguments(dev):
    buf = dev.alloc(1 << 18)
    case = Latent(dev, MIXERS["odd"]["mixer"], 4, 1)

    def call(spec, n=1, pos0=0, max_pos=8, decode=0, ukv=case.ukv, act=0):
        return hip.lib().candy_hip_latent_attention(dev.handle, ctypes.byref(spec), act, buf.ptr, buf.ptr, buf.ptr, EPS, ukv.handle,
                                                    case.ukt.handle, None, n, pos0, max_pos, buf.ptr, decode, buf.ptr)

    for change in (dict(n_heads=0), dict(dim=0), dict(rot_dim=5), dict(vdim=1025), dict(kv_rank=1025), dict(q_rank=0), dict(dim=960),
                   dict(rope_base=0.0), dict(n_heads=6)):
        s = hip.LatentSpec.from_buffer_copy(case.spec)
        for key, v in change.items():
            setattr(s, key, v)
        assert call(s) == 1, change
    for kw in (dict(n=0), dict(pos0=8), dict(n=9), dict(pos0=-1), dict(n=2, decode=1), dict(ukv=case.ukt), dict(act=3)):
        assert call(case.spec, **kw) == 1, kw


# ------------------------------------------------------------------ recurrent unit
class Lru:
    def __init__(self, dev, width, blocks, taps, n, seed, lam=(-4.0, 2.0)):
        rng = np.random.default_rng(seed)
        size = width // blocks
        self.dev, self.n, self.spec = dev, n, hip.LruSpec(width=width, blocks=blocks, taps=taps)
        self.w = {"y.b": rng.standard_normal(width), "x.b": rng.standard_normal(width), "conv": rng.standard_normal((width, taps)) * taps ** -0.5,
                  "conv.b": rng.standard_normal(width) * 0.3, "ra": rng.standard_normal((blocks, size, size)) * size ** -0.5,
                  "ri": rng.standard_normal((blocks, size, size)) * size ** -0.5, "ra.b": rng.standard_normal((blocks, size)),
                  "ri.b": rng.standard_normal((blocks, size)), "lam": lam[0] + lam[1] * rng.standard_normal(width)}
        self.w = {k: gm.to_bf16(v).astype(np.float64) for k, v in self.w.items()}
        self.zy, self.zx = (rng.standard_normal((n, width)).astype(np.float32).astype(np.float64) for _ in range(2))

    def oracle(self, act):
        w = self.w
        u = ref.causal_conv(self.zx + w["x.b"], w["conv"], w["conv.b"])
        if act == hip.ACT_BF16:
            u = gm.to_bf16(u).astype(np.float64)
        s = ref.recurrence(u, ref.block_gate(u, w["ra"], w["ra.b"]), ref.block_gate(u, w["ri"], w["ri.b"]), w["lam"])
        return s * ref.gelu_tanh(self.zy + w["y.b"])

    def device(self, act, portions, state=None):
        s, w = self.spec, self.w
        wp = up(s.width, 64)

        def pad(a):
            out = np.zeros((np.atleast_2d(a).shape[0], wp), np.float32)
            out[:, :s.width] = a
            return out

        params = {"by": pad(w["y.b"]), "bx": pad(w["x.b"]), "conv": pad(w["conv"].T), "conv_b": pad(w["conv.b"]), "ra_b": pad(w["ra.b"].reshape(-1)),
                  "ri_b": pad(w["ri.b"].reshape(-1)), "lam": pad(w["lam"])}
        gates = self.dev.dense(gulisun.gate_rows(gm.bits_of(w["ra"].astype(np.float32)), gm.bits_of(w["ri"].astype(np.float32))))
        if state is None:   # what is left of another sequence must not matter
            state = self.dev.from_numpy(np.full(hip.lib().candy_hip_lru_state_floats(ctypes.byref(s)), 7.0, np.float32))
        z = np.concatenate([pad(self.zy), pad(self.zx)], 1)
        out, at = [], 0
        for p in portions:
            out.append(self.dev.lru(s, act, z[at:at + p], params, gates, state, at, decode=p == 1))
            at += p
        assert at == self.n
        return np.concatenate(out)


@pytest.mark.parametrize("act", ACTS)
@pytest.mark.parametrize("width,blocks,taps", [(84, 3, 4), (65, 5, 1), (1, 1, 2), (128, 1, 3), (600, 2, 5), (512, 2, 4), (320, 5, 20)])
def test_lru_whole_portions_and_decode(dev, width, blocks, taps, act):
    case = Lru(dev, width, blocks, taps, 150, width)
    want = case.oracle(act)
    # whole prompts multiply rounded activations with the gates, a decode step f32 ones
    tol = 1e-5 if act == hip.ACT_F32 else 2e-2
    for portions in ([150], [2] * 75, [3, 2, 64, 1, 1, 65, 14], [1] * 40 + [37] + [1] * 73, [1, 149], [33, 1, 32, 31, 1, 52]):
        assert rel(case.device(act, portions), want) < tol, portions[:3]


@pytest.mark.parametrize("act", ACTS)
def test_state_reaches_far(dev, act):
    """Decays near one and an input that is loud at one token only: what remains of it 1500 tokens later is there, however
    the tokens between are cut, and nothing of it before."""
    n, width = 1600, 64
    for loud in (0, 1, 31, 32, 33, 99):
        case = Lru(dev, width, 1, 2, n, 3, lam=(-9.0, 0.2))
        w = case.w
        w["conv"][:, 0], w["conv"][:, 1] = 0, 1
        for k in ("x.b", "conv.b", "ra", "ri"):
            w[k][:] = 0
        case.zx[:] = 0
        case.zx[loud] = 100.0
        case.zy[:] = 3.0
        want = case.oracle(act)
        assert (np.abs(want[-1]) > 0.2).any()
        for portions in ([n], [100] + [50] * 30, [200] + [1] * 30 + [2] * 5 + [1360]):
            got = case.device(act, portions)
            assert (got[:loud] == 0).all()
            assert (np.abs(got - want) <= 2e-5 * np.abs(want).max() if act == hip.ACT_F32 else np.abs(got - want) <= 6e-3 * np.abs(want) + 1e-6).all()


def test_decay_keeps_its_precision_near_one(dev):
    """sqrt(1 - a^2) where a differs from one by less than a f32 step of a."""
    case = Lru(dev, 64, 1, 1, 40, 4, lam=(-17.0, 1.0))
    got, want = case.device(hip.ACT_F32, [20] + [1] * 20), case.oracle(hip.ACT_F32)
    assert np.abs(want).max() < 0.3 and (np.abs(got - want) < 2e-5 * np.abs(want).max()).all()


def test_lru_arguments(dev):
    case = Lru(dev, 84, 3, 4, 4, 1)
    buf = dev.alloc(1 << 18)
    gates = dev.dense(gulisun.gate_rows(np.zeros((3, 28, 28), np.uint16), np.zeros((3, 28, 28), np.uint16)))
    p = hip.LruParams(*[buf.ptr] * 7)

    def call(spec, n=1, pos0=0, decode=0, params=p):
        return hip.lib().candy_hip_lru(dev.handle, ctypes.byref(spec), 0, buf.ptr, ctypes.byref(params), gates.handle, buf.ptr, n, pos0, decode,
                                       buf.ptr)

    for change in (dict(width=85), dict(blocks=0), dict(taps=0), dict(taps=65), dict(width=168)):
        s = hip.LruSpec.from_buffer_copy(case.spec)
        for key, v in change.items():
            setattr(s, key, v)
        assert call(s) == 1, change
    for kw in (dict(n=0), dict(pos0=-1), dict(n=2, decode=1), dict(params=hip.LruParams())):
        assert call(case.spec, **kw) == 1, kw


# ------------------------------------------------------------------ experts
class Experts:
    def __init__(self, dev, d, experts, top, ff, shared, seed):
        rng = np.random.default_rng(seed)
        self.dev, self.d, self.mlp = dev, d, gm.moe(experts, top, ff, shared)
        self.spec = gulisun.expert_spec(self.mlp)
        w = {"router": rng.standard_normal((experts, d)) * 1.5 * d ** -0.5}
        for e in range(experts):
            w[f"e{e}.up"], w[f"e{e}.down"] = rng.standard_normal((ff, d)) * d ** -0.5, rng.standard_normal((d, ff)) * ff ** -0.5
        if shared:
            w["shared.up"], w["shared.down"] = rng.standard_normal((shared, d)) * d ** -0.5, rng.standard_normal((d, shared)) * shared ** -0.5
        self.w = {k: gm.to_bf16(v) for k, v in w.items()}
        self.upload()

    def upload(self):
        bits = {k: gm.bits_of(v) for k, v in self.w.items()}
        E = self.spec.n_experts
        self.dense = {"router": self.dev.dense(bits["router"]), "up": self.dev.dense(gulisun.expert_rows(bits[f"e{e}.up"] for e in range(E))),
                      "down": self.dev.dense(gulisun.expert_rows(bits[f"e{e}.down"] for e in range(E)))}
        if self.spec.shared_ff:
            self.dense.update(shared_up=self.dev.dense(bits["shared.up"]), shared_down=self.dev.dense(bits["shared.down"]))

    def oracle(self, x):
        w = {"p." + k: v.astype(np.float64) for k, v in self.w.items()}
        x = x.astype(np.float64)
        return ref.experts(x, w, "p", self.mlp), *ref.route(x, w["p.router"], self.spec.top)


@pytest.mark.parametrize("act", ACTS)
@pytest.mark.parametrize("d,experts,top,ff,shared", [(90, 5, 3, 21, 37), (64, 7, 7, 30, None), (250, 64, 6, 80, 160), (320, 130, 9, 16, 65),
                                                     (70, 3, 1, 200, 10), (192, 512, 2, 8, None), (2100, 2, 1, 64, 64), (128, 1, 1, 128, None)])
def test_experts(dev, d, experts, top, ff, shared, act):
    case = Experts(dev, d, experts, top, ff, shared, d)
    x = gm.to_bf16(np.random.default_rng(d).standard_normal((200, d)) * 1.2)
    want, ids, weights = case.oracle(x)
    tol = 1e-5 if act == hip.ACT_F32 else 1.5e-2
    for n in (200, 2, 65, 1):
        got, gids, gw = dev.experts(case.spec, act, case.dense, x[:n])
        assert np.array_equal(gids, ids[:n]) and np.abs(gw - weights[:n]).max() < 2e-5
        assert own(got, want[:n]) < tol, n
    rows = np.concatenate([dev.experts(case.spec, act, case.dense, x[t:t + 1], decode=True) for t in range(12)])
    assert own(rows, want[:12]) < tol


@pytest.mark.parametrize("act", ACTS)
def test_everyone_to_one_expert_and_nobody_to_others(dev, act):
    """A router that sends every token the same way: row tiles of one expert only, more than one of them; and one that
    deals them evenly."""
    case = Experts(dev, 64, 8, 2, 40, None, 3)
    case.w["router"][:] = 0
    case.w["router"][5, 0], case.w["router"][2, 0] = 4.0, 3.0
    case.upload()
    x = gm.to_bf16(np.abs(np.random.default_rng(3).standard_normal((300, 64))) + 0.5)
    want, ids, _ = case.oracle(x)
    assert (ids == [5, 2]).all()
    got, gids, _ = dev.experts(case.spec, act, case.dense, x)
    assert np.array_equal(gids, ids) and rel(got, want) < (1e-5 if act == hip.ACT_F32 else 1e-2)
    assert rel(dev.experts(case.spec, act, case.dense, x[7:8], decode=True), want[7:8]) < 2e-2


def test_equal_scores_choose_the_lower_number(dev):
    case = Experts(dev, 64, 9, 3, 16, None, 4)
    case.w["router"][:] = 0
    case.w["router"][6, 0] = 1.0
    case.upload()
    x = np.ones((5, 64), np.float32)
    want, ids, weights = case.oracle(x)
    assert (ids == [6, 0, 1]).all()
    got, gids, gw = dev.experts(case.spec, hip.ACT_F32, case.dense, x)
    assert np.array_equal(gids, ids) and np.abs(gw - weights).max() < 1e-6 and rel(got, want) < 1e-5
    assert rel(dev.experts(case.spec, hip.ACT_F32, case.dense, x[:1], decode=True), want[:1]) < 1e-5


def test_router_sees_all_bits_of_its_input(dev):
    """Two scores that differ in the input's last bits only: their order is that of the f32 values, in both formats."""
    case = Experts(dev, 64, 2, 1, 16, None, 5)
    case.w["router"][:] = 0
    case.w["router"][0, 0], case.w["router"][1, 1] = 1.0, 1.0
    case.upload()
    x = np.zeros((40, 64), np.float32)
    a = np.float32(1.2345678)
    for t in range(40):
        x[t, 0], x[t, 1] = (a, np.nextafter(a, np.float32(9))) if t % 2 else (np.nextafter(a, np.float32(9)), a)
    for act in (hip.ACT_F32, hip.ACT_BF16):
        assert np.array_equal(dev.experts(case.spec, act, case.dense, x)[1][:, 0], np.arange(40) % 2)


def test_expert_arguments(dev):
    case = Experts(dev, 64, 4, 2, 16, 8, 6)
    buf = dev.alloc(1 << 16)
    w = hip.ExpertWeights(**{k: v.handle for k, v in case.dense.items()})

    def call(spec, n=1, decode=0, weights=w, ids=None):
        return hip.lib().candy_hip_experts(dev.handle, ctypes.byref(spec), 0, ctypes.byref(weights), buf.ptr, n, decode, buf.ptr, ids, None)

    for change in (dict(n_experts=0), dict(n_experts=5), dict(top=0), dict(top=5), dict(d_ff=0), dict(d_ff=65), dict(shared_ff=-1),
                   dict(shared_ff=9), dict(n_experts=513)):
        s = hip.ExpertSpec.from_buffer_copy(case.spec)
        for key, v in change.items():
            setattr(s, key, v)
        assert call(s) == 1, change
    for kw in (dict(n=0), dict(n=2, decode=1), dict(weights=hip.ExpertWeights()), dict(decode=1, ids=buf.ptr)):
        assert call(case.spec, **kw) == 1, kw


# ------------------------------------------------------------------ whole models
N = 140


@pytest.fixture(scope="module")
def cases():
    """Per configuration and format: weights, tokens, the oracle's logits and residual streams.  f32: any router; bfloat16:
    one without close calls."""
    out = {}
    for i, (name, cfg) in enumerate(sorted(gm.CONFIGS.items())):
        tokens = [int(t) for t in np.random.default_rng(i).integers(0, cfg["vocab"], N)]
        for act in (hip.ACT_F32, hip.ACT_BF16):
            w = gm.weights(cfg, seed=100 + i, peaky=1.5, steady=act == hip.ACT_BF16)
            streams = []
            out[name, act] = (cfg, w, tokens, ref.forward(cfg, w, tokens, streams), streams)
    return out


def build(dev, cfg, w, act, max_pos=160):
    return gulisun.build(dev, cfg, gm.Tensors(w), max_pos, act)


@pytest.mark.parametrize("act", ACTS)
@pytest.mark.parametrize("name", sorted(gm.CONFIGS))
def test_model_prompt(dev, cases, name, act):
    cfg, w, tokens, want, streams = cases[name, act]
    m = build(dev, cfg, w, act)
    got = m.feed(tokens, 0, range(N))
    assert rel(got, want) < WHOLE_TOL[act]
    assert rel(m.prompt_hidden(N), streams[-1]) < WHOLE_TOL[act]
    nt, last = m.prefill(tokens, 0)
    assert rel(last, want[-1]) < WHOLE_TOL[act] and nt == int(np.argmax(last))
    nt, last = m.prefill(tokens[:1], 0)   # a prompt pass of one token
    assert rel(last, want[0]) < WHOLE_TOL[act]
    m.free()


@pytest.mark.parametrize("act", ACTS)
@pytest.mark.parametrize("name", sorted(gm.CONFIGS))
def test_model_token_by_token(dev, cases, name, act):
    cfg, w, tokens, want, streams = cases[name, act]
    m = build(dev, cfg, w, act)
    got = [m.decode(t, p)[1] for p, t in enumerate(tokens)]
    assert rel(got, want) < WHOLE_TOL[act]
    assert rel(m.hidden(), streams[-1][-1]) < WHOLE_TOL[act]
    m.free()


@pytest.mark.parametrize("act", ACTS)
@pytest.mark.parametrize("name", sorted(gm.CONFIGS))
def test_model_in_portions(dev, cases, name, act):
    cfg, w, tokens, want, _ = cases[name, act]
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
    """Every layer with a cache of its own alone, as prompt and as a decode step from a given row."""
    for (name, a), (cfg, w, tokens, _, _) in cases.items():
        for i in range(len(cfg["layers"])):
            if a != act or cfg["layers"][i]["mixer"].get("kv_from") is not None:
                continue
            one = gm.changed(cfg, layers=[cfg["layers"][i]])
            ww = {k.replace(f"l{i}.", "l0."): v for k, v in w.items() if k.startswith(f"l{i}.")}
            ww.update({k: w[k] for k in ("embed", "final.norm")})
            trace_ = []
            ref.forward(one, ww, tokens[:80], trace_)
            m = build(dev, one, ww, act)
            m.feed(tokens[:80], 0, [79])
            assert rel(m.prompt_hidden(80), trace_[0]) < LAYER_TOL[act], (name, i)
            x = w["embed"][5] * np.float32(cfg["embedding"]["scale"] * 1.25)
            m.decode_hidden(x, 0)
            want = ref.layer(x.astype(np.float64)[None], {k: v.astype(np.float64) for k, v in ww.items()}, 0, one, {})
            assert rel(m.hidden(), want[0]) < LAYER_TOL[act], (name, i)
            m.free()


@pytest.mark.parametrize("act", ACTS)
def test_sequences_share_nothing(dev, cases, act):
    """Cache and state are taken over by the next sequence: shorter, longer, after a long one, in other portions."""
    for name in ("odd", "recurrent"):
        cfg, w, tokens, want, _ = cases[name, act]
        m = build(dev, cfg, w, act)
        other = [int(t) for t in np.random.default_rng(9).integers(0, cfg["vocab"], 150)]
        first = m.feed(tokens, 0, range(N))
        m.feed(other, 0, [])
        assert np.array_equal(m.feed(tokens, 0, range(N)), first)
        short = ref.forward(cfg, w, other[:5])
        assert rel(m.feed(other[:5], 0, range(5)), short) < WHOLE_TOL[act]
        got = [m.decode(t, p)[1] for p, t in enumerate(tokens[:30])]
        assert rel(got, want[:30]) < WHOLE_TOL[act]
        assert rel(m.feed(other[:1], 0, [0]), short[:1]) < WHOLE_TOL[act]
        m.free()


def test_recurrent_positions_come_in_order(dev, cases):
    cfg, w, tokens, want, _ = cases["recurrent", hip.ACT_F32]
    m = build(dev, cfg, w, hip.ACT_F32)
    m.feed(tokens[:10], 0, [])
    for call in (lambda: m.feed(tokens[9:12], 9, []), lambda: m.feed(tokens[11:13], 11, []), lambda: m.decode(tokens[9], 9),
                 lambda: m.decode(tokens[12], 12), lambda: m.generate(tokens[3], 3, 2),
                 lambda: m.decode_hidden(np.zeros(cfg["width"], np.float32), 11)):
        with pytest.raises(hip.CandyHipError, match="out of order"):
            call()
    assert rel(m.feed(tokens[10:13], 10, range(3)), want[10:13]) < WHOLE_TOL[hip.ACT_F32]   # a refused call changes nothing
    m.free()
    # without recurrent layers any position may be fed again
    attention = gm.config([gm.latent(2, 20, 6, 24, 40, 50)], 64, 70)
    w = gm.weights(attention, 1)
    want = ref.forward(attention, w, tokens[:12])
    m = build(dev, attention, w, hip.ACT_F32)
    m.feed(tokens[:12], 0, [])
    assert rel(m.feed(tokens[5:12], 5, range(7)), want[5:]) < WHOLE_TOL[hip.ACT_F32]
    m.free()


def test_first_token_matters_to_the_last(dev):
    """Attention over everything and long memories: changing the first token changes every position's logits, none before
    a changed one."""
    cfg = gm.config([gm.latent(4, 32, 16, 32, 64, 40, scale=0.05), gm.rglru(64, 1, 3), gm.latent(2, 16, 16, 20, 64, 30, kv_from=0)], 96, 120)
    w = gm.weights(cfg, seed=5)
    a = [int(t) for t in np.random.default_rng(1).integers(0, 120, 150)]
    for at in (0, 1, 63, 64):
        b = list(a)
        b[at] = (b[at] + 1) % 120
        m = build(dev, cfg, w, hip.ACT_F32)
        for portions in ([150], [1] * 150, [70, 50] + [1] * 30):
            rows = []
            for seq in (a, b):
                got, p0 = [], 0
                for p in portions:
                    got.append(m.feed(seq[p0:p0 + p], p0, range(p)))
                    p0 += p
                rows.append(np.concatenate(got))
            diff = np.abs(rows[0] - rows[1]).max(1)
            assert (diff[:at] == 0).all() and (diff[at:] > 1e-5).all(), (at, portions[:2])
        m.free()


def test_graph_replays_equal_eager_launches(dev, cases):
    for name in gm.CONFIGS:
        cfg, w, tokens, _, _ = cases[name, hip.ACT_BF16]
        m = build(dev, cfg, w, hip.ACT_BF16)
        runs = []
        for graph in (False, True):
            m.set_graph(graph)
            m.feed(tokens[:30], 0, [])
            out, p = [], 30
            while p < 70:
                out.append(m.decode(tokens[p], p)[1])
                p += 1
                if p % 10 == 0:  # eager work and synchronizations between the replays
                    dev.add_rms_norm(np.ones((2, 8)), np.ones((2, 8)), np.ones(8), 1e-5, 1.0)
                    out += list(m.feed(tokens[p:p + 2], p, [0, 1]))
                    p += 2
            runs.append(np.array(out))
        assert np.array_equal(runs[0], runs[1]), name
        m.free()


def test_greedy_generation(dev):
    """The generation loop (token handed over on the device) against the oracle's greedy choice, as far as the two best
    logits are apart; and against a loop over single steps."""
    cfg = gm.CONFIGS["odd"]
    for seed in (1, 2):
        prompt = [int(t) for t in np.random.default_rng(seed).integers(0, cfg["vocab"], 12)]
        for act, gap in ((hip.ACT_F32, 1e-3), (hip.ACT_BF16, 0.6)):
            w = gm.weights(cfg, seed=200 + seed, steady=act == hip.ACT_BF16)
            want, gaps = ref.greedy(cfg, w, prompt, 40)
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


@pytest.mark.parametrize("act", ACTS)
def test_long_decode_from_a_portioned_prompt(dev, act):
    cfg = gm.config([gm.latent(3, 20, 6, 24, 40, 50, 300.0, 0.2, experts=5, top=2, ff=20, shared=30), gm.rglru(64, 2, 4),
                     gm.latent(4, 24, 6, 24, 40, 30, 300.0, 0.2, kv_from=0, sink=False)], 80, 100)
    w = gm.weights(cfg, 7, steady=act == hip.ACT_BF16)
    tokens = [int(t) for t in np.random.default_rng(7).integers(0, 100, 700)]
    want = ref.forward(cfg, w, tokens)
    m = build(dev, cfg, w, act, max_pos=700)
    got = [m.feed(tokens[:200], 0, range(200)), m.feed(tokens[200:331], 200, range(131))]
    got += [m.feed([t], p, [0]) for p, t in list(enumerate(tokens))[331:]]
    assert rel(np.concatenate(got), want) < WHOLE_TOL[act]
    m.free()


def test_model_arguments(dev, cases):
    cfg, w, tokens, _, _ = cases["odd", hip.ACT_BF16]
    m = build(dev, cfg, w, hip.ACT_BF16, max_pos=20)
    for call in (lambda: m.feed(tokens[:21], 0, []), lambda: m.feed([cfg["vocab"], 0], 0, []), lambda: m.decode(0, 20),
                 lambda: m.decode(-1, 0), lambda: m.feed(tokens[:5], 17, [])):
        with pytest.raises(hip.CandyHipError):
            call()
    with pytest.raises(hip.CandyHipError):
        m.set_matrix(hip.GL_O, 0, dev.dense(np.zeros((4, 4), np.uint16)))
    with pytest.raises(hip.CandyHipError):
        m.set_matrix(hip.GL_GATES, 0, dev.dense(np.zeros((4, 4), np.uint16)))   # no recurrent layer
    with pytest.raises(hip.CandyHipError):
        m.set_vector(hip.GL_KV_NORM, 2, np.zeros(40, np.float32))               # reads another layer's cache
    with pytest.raises(hip.CandyHipError):
        m.set_vector(hip.GL_SINK, 0, np.zeros(3, np.float32))
    for layer, source in ((2, 2), (2, 3), (2, 1), (4, 2), (3, 0)):   # itself, a later one, a recurrent one, a reader, other sizes
        bad = json.loads(json.dumps(cfg))
        bad["layers"][layer]["mixer"]["kv_from"] = source
        with pytest.raises(hip.CandyHipError):
            hip.Gulisun(dev, *gulisun.parse_config(bad, 8, hip.ACT_BF16)).free()
    incomplete = hip.Gulisun(dev, *gulisun.parse_config(cfg, 8, hip.ACT_BF16))
    incomplete.set_matrix(hip.GL_EMBED, -1, dense(dev, w["embed"]))
    with pytest.raises(hip.CandyHipError):
        incomplete.feed(tokens[:2], 0, [])
    incomplete.free()
    m.free()


@pytest.mark.parametrize("act", ACTS)
def test_trace_through_the_registry(dev, cases, tmp_path, act):
    """A folder on disk, the registry's loader, the replayer: portions, single tokens and three requests in a row."""
    cfg, w, tokens, want, _ = cases["odd", act]
    gm.write_folder(tmp_path / "model", cfg, w)
    m = models.load(dev, str(tmp_path / "model"), max_pos=140, act=act)
    steps, at, cuts = [], 0, (60, 2, 1, 1, 5, 1, 70)
    for p in cuts:
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
    for i, p in enumerate(cuts):
        got = np.fromfile(tmp_path / f"{i}.f32", "<f4").reshape(-1, cfg["vocab"])
        assert rel(got, want[[at, at + p - 1] if p > 1 else [at]]) < WHOLE_TOL[act]
        at += p
    assert not (tmp_path / "7.f32").exists()
    assert rel(np.fromfile(tmp_path / "8.f32", "<f4"), want[0]) < WHOLE_TOL[act]
    m.free()


@pytest.mark.parametrize("dtype,act", [("bfloat16", hip.ACT_BF16), ("float32", hip.ACT_F32)])
def test_trace_run_program(cases, tmp_path, dtype, act):
    """The command line: its own process, steps on standard input, logits in files."""
    cfg, w, tokens, want, _ = cases["recurrent", act]
    gm.write_folder(tmp_path / "model", cfg, w)
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
