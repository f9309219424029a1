"""Small random Gulisun models for the tests: configurations, weights rounded to bfloat16."""
from __future__ import annotations

import numpy as np

from tests.suvazen_models import Tensors, bits_of, changed, to_bf16, write_folder  # noqa: F401  (used through this module)


def latent(heads, dim, rot_dim, vdim, kv_rank, q_rank, base=10000.0, scale=None, kv_from=None, sink=True, **mlp):
    m = {"heads": heads, "dim": dim, "rot_dim": rot_dim, "vdim": vdim, "kv_rank": kv_rank, "q_rank": q_rank,
         "scale": (dim + rot_dim) ** -0.5 if scale is None else scale, "rot": {"base": base, "dims": rot_dim}}
    if kv_from is not None:
        m["kv_from"] = kv_from
    return {"type": "latent_attention" if sink else "latent_attention_2", "mixer": m, "mlp": moe(**mlp) if mlp else None}


def rglru(width, blocks, taps, **mlp):
    return {"type": "rglru", "mixer": {"width": width, "blocks": blocks, "conv": taps}, "mlp": moe(**mlp) if mlp else None}


def moe(experts, top, ff, shared=None):
    out = {"kind": "moe", "router": {"experts": experts, "top": top}, "expert": {"ff": ff}}
    out["shared"] = {"ff": shared} if shared else None
    return out


def config(layers, width, vocab, eps=1e-5, scale=3.0):
    return {"architecture": "Gulisun", "vocab": vocab, "width": width, "layers": layers, "norm": {"eps": eps},
            "embedding": {"scale": scale}}


CONFIGS = {
    # sizes that are multiples of nothing, per-layer differences, a cache that two other layers read, both optional parts
    # of the feed-forward absent somewhere, one tap, everything chosen, one chosen
    "odd": config([latent(5, 20, 6, 24, 40, 50, 300.0, 0.23, experts=5, top=3, ff=21, shared=37),
                   rglru(84, 3, 4, experts=7, top=7, ff=30),
                   latent(3, 36, 6, 17, 40, 70, 300.0, 0.31, kv_from=0),
                   latent(2, 70, 34, 50, 100, 33, 2e4, 0.1, sink=False, experts=6, top=1, ff=65, shared=20),
                   latent(4, 9, 6, 40, 40, 20, 300.0, 0.4, kv_from=0, sink=False, experts=4, top=2, ff=64, shared=64),
                   rglru(65, 5, 1, experts=3, top=2, ff=10, shared=130)], 90, 173, eps=2e-4),
    # a recurrent layer first and alone
    "recurrent": config([rglru(128, 1, 3), rglru(192, 2, 9, experts=8, top=2, ff=48, shared=16)], 64, 64, scale=0.5),
    # heads, ranks and numbers of experts past what the tile kernels take
    "wide": config([latent(2, 200, 64, 300, 600, 130, experts=70, top=6, ff=32, shared=64),
                    latent(3, 40, 160, 33, 200, 90, 500.0, sink=False, experts=130, top=9, ff=16),
                    rglru(600, 2, 5)], 192, 300),
    # the shape of a common decoder layer
    "even": config([latent(20, 128, 64, 128, 512, 256, experts=16, top=4, ff=128, shared=256),
                    rglru(512, 2, 4, experts=16, top=4, ff=128, shared=256),
                    latent(20, 128, 64, 128, 512, 256, kv_from=0, experts=16, top=4, ff=128, shared=256),
                    latent(8, 64, 32, 64, 256, 128, sink=False, experts=16, top=4, ff=128, shared=256)], 320, 512),
}


def weights(cfg, seed, peaky=1.0, steady=False):
    """{name: float32 array of bfloat16 values}.  peaky scales queries and keys: larger values make single keys dominate.
    steady: routers read columns of the residual stream that hold a permutation of levels per token and that the layers
    hardly touch, so that no choice is a close call (which 8-bit activations may decide either way)."""
    rng = np.random.default_rng(seed)
    d, V, out = cfg["width"], cfg["vocab"], {}

    def put(name, *shape, std=1.0, mean=0.0):
        out[name] = to_bf16(mean + std * rng.standard_normal(shape))

    put("embed", V, d, std=1.5 * d ** -0.5)
    sizes = sorted({l["mlp"]["router"]["experts"] for l in cfg["layers"] if l["mlp"]})
    levels = max(sizes, default=0)
    assert levels <= d
    if steady and levels:
        gap = 0.6 / cfg["embedding"]["scale"] * min(1.0, 12.0 / levels)
        order = np.argsort(rng.random((V, levels)), axis=1)
        out["embed"][:, :levels] = to_bf16(gap * (order - levels / 2))
    quiet = np.ones(d, np.float32)
    if steady:
        quiet[:levels] = 2.0 ** -9
    put("final.norm", d, std=0.3, mean=1.0)
    for i, layer in enumerate(cfg["layers"]):
        m, p = layer["mixer"], f"l{i}"
        for n in ("norm1", "norm2") if layer["mlp"] else ("norm1",):
            put(f"{p}.{n}", d, std=0.3, mean=1.0)
            out[f"{p}.{n}"] = to_bf16(out[f"{p}.{n}"] * quiet)
        x = 1.0 / cfg["embedding"]["scale"]   # brings the residual stream back to about one
        if layer["type"] == "rglru":
            w, b = m["width"], m["blocks"]
            size = w // b
            put(p + ".mix.y", w, d, std=x * d ** -0.5)
            put(p + ".mix.x", w, d, std=x * d ** -0.5)
            put(p + ".mix.conv", w, m["conv"], std=m["conv"] ** -0.5)
            put(p + ".mix.ra", b, size, size, std=size ** -0.5)
            put(p + ".mix.ri", b, size, size, std=size ** -0.5)
            for n, shape in (("y.b", (w,)), ("x.b", (w,)), ("conv.b", (w,)), ("ra.b", (b, size)), ("ri.b", (b, size))):
                put(f"{p}.mix.{n}", *shape, std=0.3)
            put(p + ".mix.lam", w, std=2.0, mean=-4.0)   # memories from one token to thousands
            put(p + ".mix.o", d, w, std=w ** -0.5)
        else:
            H, dk = m["heads"], m["dim"] + m["rot_dim"]
            s = np.sqrt(peaky) * (m["scale"] * np.sqrt(dk)) ** -0.5
            put(p + ".mix.dq", m["q_rank"], d, std=d ** -0.5)
            put(p + ".mix.dq.norm", m["q_rank"], std=0.3, mean=1.0)
            put(p + ".mix.uq", H * dk, m["q_rank"], std=1.5 * s * m["q_rank"] ** -0.5)
            if m.get("kv_from") is None:
                put(p + ".mix.dkv", m["kv_rank"] + m["rot_dim"], d, std=1.5 * s * x * d ** -0.5)
                put(p + ".mix.dkv.norm", m["kv_rank"], std=0.3, mean=1.0)
            put(p + ".mix.uk", H * m["dim"], m["kv_rank"], std=1.5 * s * m["kv_rank"] ** -0.5)
            put(p + ".mix.uv", H * m["vdim"], m["kv_rank"], std=m["kv_rank"] ** -0.5)
            if layer["type"] == "latent_attention":
                put(p + ".mix.sink", H, std=1.5, mean=1.0)
            put(p + ".mix.o", d, H * m["vdim"], std=(H * m["vdim"]) ** -0.5)
        if layer["mlp"]:
            r, ff, sh = layer["mlp"]["router"], layer["mlp"]["expert"]["ff"], layer["mlp"]["shared"]
            put(p + ".mlp.router", r["experts"], d, std=1.5 * x * d ** -0.5)
            if steady:
                out[p + ".mlp.router"] = np.eye(r["experts"], d, dtype=np.float32)
            for e in range(r["experts"]):
                put(f"{p}.mlp.e{e}.up", ff, d, std=d ** -0.5)
                put(f"{p}.mlp.e{e}.down", d, ff, std=ff ** -0.5)
            if sh:
                put(p + ".mlp.shared.up", sh["ff"], d, std=d ** -0.5)
                put(p + ".mlp.shared.down", d, sh["ff"], std=sh["ff"] ** -0.5)
    return out


def choice_margin(cfg, w, tokens):
    """Smallest gap between the last chosen score's logarithm and the first one left out, over layers and tokens."""
    from oracle import gulisun_ref as ref
    seen, route = [], ref.route

    def watched(h, router, top):
        z = np.sort(h @ router.T, axis=1)[:, ::-1]
        if top < z.shape[1]:
            seen.append((z[:, top - 1] - z[:, top]).min())
        return route(h, router, top)

    ref.route = watched
    try:
        ref.forward(cfg, w, tokens)
    finally:
        ref.route = route
    return min(seen, default=np.inf)
