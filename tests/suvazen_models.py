"""Small random Suvazen models for the tests: configurations, weights rounded to bfloat16, files on disk."""
from __future__ import annotations

import copy
import json
import os
import struct

import numpy as np


def to_bf16(x):
    """float32 values rounded to the nearest bfloat16 (ties to even), as float32."""
    u = np.ascontiguousarray(x, np.float32).view(np.uint32).astype(np.uint64)
    u = (u + 0x7FFF + ((u >> 16) & 1)) & 0xFFFF0000
    return u.astype(np.uint32).view(np.float32)


def bits_of(x):
    return (np.ascontiguousarray(x, np.float32).view(np.uint32) >> 16).astype(np.uint16)


def mixer(heads, kv_heads, dim, window=None, rope_dims=0, base=10000.0, scaling=None, scale=None, softcap=None):
    out = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": dim, "scale": dim ** -0.5 if scale is None else scale,
           "softcap": softcap}
    out["mask"] = {"size": window} if window else None
    out["rot"] = {"base": base, "dims": rope_dims, "scaling": scaling} if rope_dims else None
    return out


def config(layers, width, vocab, loop=None, eps=1e-5, mult=0.7, logit_scale=1.5, logit_softcap=20.0):
    """layers: [(mixer, ff or None)]; loop: (start, stop, times)."""
    return {"architecture": "Suvazen", "vocab": vocab, "width": width,
            "layers": [{"type": "attention", "mixer": m, "mlp": {"kind": "dense", "ff": ff} if ff else None} for m, ff in layers],
            "loop": dict(zip(("start", "stop", "times"), loop)) if loop else None, "norm": {"eps": eps},
            "residual_mult": mult, "logit_scale": logit_scale, "logit_softcap": logit_softcap}


SCALED = {"factor": 5.0, "low": 1.0, "high": 3.0, "original": 96}

# sizes that are multiples of nothing, per-layer differences, every optional part present and absent somewhere
CONFIGS = {
    # three query heads per kv head, partial rotation, three frequency bands, a loop that is neither first nor last
    "odd": config([(mixer(6, 2, 24, 19, 10, 500.0, SCALED, 0.31, 9.0), 84),
                   (mixer(4, 4, 40, 33, 40, 10000.0, None, 0.2, 4.0), None),
                   (mixer(5, 1, 20, 7, 4, 100.0, SCALED, 0.5, 15.0), 51),
                   (mixer(3, 3, 36, 50, 18, 2000.0, None, 0.11, 6.0), 130)], width=90, vocab=173, loop=(1, 3, 3)),
    # one layer, no loop, no rotation, no cap, all positions visible
    "plain": config([(mixer(4, 2, 32), 96)], width=64, vocab=64, logit_softcap=None, mult=1.0, logit_scale=1.0),
    # wide heads, a window of one position, a loop over everything with a single pass
    "wide": config([(mixer(2, 1, 130, 1, 64, 10000.0, None, 0.1, 30.0), 64),
                    (mixer(8, 1, 96, 65, 96, 1e6, SCALED, 0.12, 12.0), 200)], width=192, vocab=300, loop=(0, 2, 1)),
    # the shape of a common decoder layer, eight query heads per kv head
    "even": config([(mixer(8, 1, 128, 64, 64, 10000.0, SCALED, 0.09, 25.0), 512),
                    (mixer(12, 4, 64, 128, 64, 10000.0, None, 0.125, 25.0), 384)], width=320, vocab=512, loop=(0, 1, 2)),
}


def weights(cfg, seed, peaky=1.0, sinks=True):
    """{name: float32 array of bfloat16 values}.  peaky scales q and k: larger values make single keys dominate."""
    rng = np.random.default_rng(seed)
    d, out = cfg["width"], {}

    def put(name, *shape, std=1.0, mean=0.0):
        out[name] = to_bf16(mean + std * rng.standard_normal(shape))

    put("embed", cfg["vocab"], d)
    put("head", cfg["vocab"], d, std=1.5 * d ** -0.5)
    norms = ["final.norm"]
    for i, layer in enumerate(cfg["layers"]):
        m, p = layer["mixer"], f"l{i}"
        q = np.sqrt(peaky) * (m["scale"] * np.sqrt(m["dim"])) ** -0.5 * d ** -0.5
        put(p + ".mix.q", m["heads"] * m["dim"], d, std=1.5 * q)
        put(p + ".mix.k", m["kv_heads"] * m["dim"], d, std=1.5 * q)
        put(p + ".mix.o", d, m["heads"] * m["dim"], std=(m["heads"] * m["dim"]) ** -0.5)
        if sinks:
            put(p + ".mix.sink", m["heads"], std=1.5, mean=1.0)
        norms += [p + ".norm1", p + ".norm1b"]
        if layer["mlp"]:
            ff = layer["mlp"]["ff"]
            put(p + ".mlp.up", ff, d, std=d ** -0.5)
            put(p + ".mlp.down", d, ff, std=ff ** -0.5)
            norms += [p + ".norm2", p + ".norm2b"]
    for n in norms:
        put(n, d, std=0.3, mean=1.0)
        put(n + ".b", d, std=0.2)
    if cfg["loop"]:
        put("loop.step", cfg["loop"]["times"], d, std=0.5)
    return out


class Tensors:
    """The interface of a weight file over a dict of arrays."""

    def __init__(self, w):
        self.w = w

    def __contains__(self, name):
        return name in self.w

    def bits(self, name):
        return bits_of(self.w[name])

    def f32(self, name):
        return np.asarray(self.w[name], np.float32)


def write_folder(path, cfg, w):
    """config.json and model.safetensors, written by hand."""
    os.makedirs(path, exist_ok=True)
    with open(os.path.join(path, "config.json"), "w") as f:
        json.dump(cfg, f)
    header, blob = {}, b""
    for name, a in w.items():
        b = bits_of(a).tobytes()
        header[name] = {"dtype": "BF16", "shape": list(np.shape(a)), "data_offsets": [len(blob), len(blob) + len(b)]}
        blob += b
    head = json.dumps(header).encode()
    with open(os.path.join(path, "model.safetensors"), "wb") as f:
        f.write(struct.pack("<Q", len(head)) + head + blob)


def changed(cfg, **kw):
    out = copy.deepcopy(cfg)
    out.update(kw)
    return out
