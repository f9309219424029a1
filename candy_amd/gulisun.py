"""Gulisun: configuration and weights of a model folder (config.json, model.safetensors) -> the device decoder.

config.json: `vocab`, `width`, `embedding.scale`, `norm.eps`, and `layers`, per layer `type`, `mixer` and `mlp`:
  "latent_attention" (softmax with a sink) and "latent_attention_2" (without): heads, dim, rot_dim, vdim, kv_rank, q_rank,
      scale, rot.{base, dims}, and optionally kv_from, the layer whose cache this one reads;
  "rglru": width, blocks, conv (taps);
  mlp = {kind: "moe", router.{experts, top}, expert.ff, shared.ff} or null; absent or null `shared`: no shared expert.

Tensors: embed, final.norm, and per layer l<i>: norm1, norm2, mix.* (dq, dq.norm, uq, dkv, dkv.norm, uk, uv, sink, o; or y, x
with biases, conv, conv.b, ra, ri with biases, lam, o), mlp.router, mlp.e<k>.{up, down}, mlp.shared.{up, down}.

The device wants head widths padded to multiples of 32 and ranks and inner widths to multiples of 64 (zeros); the functions
below lay the matrices out that way.
"""
from __future__ import annotations

import json
import os

import numpy as np

from . import hip
from .safetensors import SafetensorsFile


class ConfigError(ValueError):
    pass


def _up(n: int, to: int) -> int:
    return -(-n // to) * to


# ------------------------------------------------------------------ configuration
def latent_spec(mixer: dict) -> hip.LatentSpec:
    rot, rot_dim = mixer.get("rot") or {}, int(mixer["rot_dim"])
    if int(rot.get("dims", 0)) != rot_dim:
        raise ConfigError(f"the rotated part turns as a whole: rot.dims {rot.get('dims')} must equal rot_dim {rot_dim}")
    return hip.LatentSpec(n_heads=int(mixer["heads"]), dim=int(mixer["dim"]), rot_dim=rot_dim, vdim=int(mixer["vdim"]),
                          kv_rank=int(mixer["kv_rank"]), q_rank=int(mixer["q_rank"]), scale=float(mixer["scale"]),
                          rope_base=float(rot.get("base", 1.0)))


def lru_spec(mixer: dict) -> hip.LruSpec:
    return hip.LruSpec(width=int(mixer["width"]), blocks=int(mixer["blocks"]), taps=int(mixer["conv"]))


def expert_spec(mlp: dict | None) -> hip.ExpertSpec:
    if mlp is None:
        return hip.ExpertSpec()
    if mlp["kind"] != "moe":
        raise ConfigError(f"no feed-forward of kind {mlp['kind']!r}")
    return hip.ExpertSpec(n_experts=int(mlp["router"]["experts"]), top=int(mlp["router"]["top"]), d_ff=int(mlp["expert"]["ff"]),
                          shared_ff=int((mlp.get("shared") or {}).get("ff", 0)))


def parse_config(cfg: dict, max_pos: int, act: int):
    """config.json -> (GulisunConfig, [GulisunLayer])."""
    layers = []
    for i, entry in enumerate(cfg["layers"]):
        kind, mixer, experts = entry["type"], entry["mixer"], expert_spec(entry.get("mlp"))
        if kind == "rglru":
            layers.append(hip.GulisunLayer(mixer=hip.GL_LRU, kv_from=-1, lru=lru_spec(mixer), experts=experts))
        elif kind in ("latent_attention", "latent_attention_2"):
            source = mixer.get("kv_from")
            layers.append(hip.GulisunLayer(mixer=hip.GL_LATENT, kv_from=-1 if source is None else int(source),
                                           has_sink=int(kind == "latent_attention"), latent=latent_spec(mixer), experts=experts))
        else:
            raise ConfigError(f"layer {i}: no mixer of type {kind!r}")
    return hip.GulisunConfig(n_layers=len(layers), d_model=int(cfg["width"]), vocab=int(cfg["vocab"]), max_pos=int(max_pos), act=act,
                             norm_eps=float(cfg["norm"]["eps"]), embed_scale=float(cfg["embedding"]["scale"])), layers


# ------------------------------------------------------------------ device layouts
def padded_groups(bits: np.ndarray, sizes, to: int) -> np.ndarray:
    """Rows in groups of the given sizes, over and over; every group padded with zero rows to a multiple of `to`."""
    per = sum(sizes)
    times, cols = bits.shape[0] // per, bits.shape[1]
    if times * per != bits.shape[0]:
        raise ConfigError(f"{bits.shape[0]} rows do not divide into groups of {per}")
    src = bits.reshape(times, per, cols)
    out = np.zeros((times, sum(_up(s, to) for s in sizes), cols), bits.dtype)
    a = b = 0
    for s in sizes:
        out[:, b:b + s] = src[:, a:a + s]
        a, b = a + s, b + _up(s, to)
    return out.reshape(-1, cols)


def down_rows(spec: hip.LatentSpec, dq: np.ndarray, dkv: np.ndarray | None) -> np.ndarray:
    parts = [padded_groups(dq, [spec.q_rank], 64)]
    if dkv is not None:
        parts += [padded_groups(dkv[:spec.kv_rank], [spec.kv_rank], 64)]
        if spec.rot_dim:
            parts += [padded_groups(dkv[spec.kv_rank:], [spec.rot_dim], 32)]
    return np.concatenate(parts)


def query_rows(spec: hip.LatentSpec, uq: np.ndarray) -> np.ndarray:
    return padded_groups(uq, [spec.dim, spec.rot_dim], 32)


def key_value_rows(spec: hip.LatentSpec, uk: np.ndarray, uv: np.ndarray) -> np.ndarray:
    return np.concatenate([padded_groups(uk, [spec.dim], 32), padded_groups(uv, [spec.vdim], 32)])


def transposed_keys(spec: hip.LatentSpec, uk: np.ndarray) -> np.ndarray:
    heads = uk.reshape(spec.n_heads, spec.dim, spec.kv_rank).transpose(0, 2, 1)
    return padded_groups(heads.reshape(-1, spec.dim), [spec.kv_rank], 64)


def value_columns(spec: hip.LatentSpec, o: np.ndarray) -> np.ndarray:
    return np.ascontiguousarray(padded_groups(np.ascontiguousarray(o.T), [spec.vdim], 32).T)


def branch_rows(y: np.ndarray, x: np.ndarray) -> np.ndarray:
    return np.concatenate([padded_groups(y, [y.shape[0]], 64), padded_groups(x, [x.shape[0]], 64)])


def gate_rows(ra: np.ndarray, ri: np.ndarray) -> np.ndarray:
    """[blocks, size, size] twice -> per block, 64 rows of the one and the same 64 of the other in turn."""
    blocks, size, _ = ra.shape
    both = np.zeros((blocks, _up(size, 64) // 64, 2, 64, size), ra.dtype)
    for k, m in enumerate((ra, ri)):
        padded = np.zeros((blocks, _up(size, 64), size), ra.dtype)
        padded[:, :size] = m
        both[:, :, k] = padded.reshape(blocks, -1, 64, size)
    return both.reshape(-1, size)


def expert_rows(matrices) -> np.ndarray:
    return np.concatenate([padded_groups(m, [m.shape[0]], 64) for m in matrices])


# ------------------------------------------------------------------ weights
def build(dev, cfg: dict, tensors, max_pos: int, act: int = hip.ACT_BF16) -> hip.Gulisun:
    """tensors: .bits(name) and .f32(name), as SafetensorsFile has them."""
    native, layers = parse_config(cfg, max_pos, act)
    model = hip.Gulisun(dev, native, layers)
    bits, f32 = tensors.bits, tensors.f32
    for i, layer in enumerate(layers):
        p, m = f"l{i}", f"l{i}.mix."
        matrices, vectors = [], [(hip.GL_NORM1, f32(p + ".norm1"))]
        if layer.mixer == hip.GL_LATENT:
            s, own = layer.latent, layer.kv_from < 0
            uk, uv = bits(m + "uk"), bits(m + "uv")
            matrices += [(hip.GL_IN, down_rows(s, bits(m + "dq"), bits(m + "dkv") if own else None)),
                         (hip.GL_UQ, query_rows(s, bits(m + "uq"))), (hip.GL_UKV, key_value_rows(s, uk, uv)),
                         (hip.GL_UKT, transposed_keys(s, uk)), (hip.GL_O, value_columns(s, bits(m + "o")))]
            vectors += [(hip.GL_Q_NORM, f32(m + "dq.norm"))]
            if own:
                vectors += [(hip.GL_KV_NORM, f32(m + "dkv.norm"))]
            if layer.has_sink:
                vectors += [(hip.GL_SINK, f32(m + "sink"))]
        else:
            matrices += [(hip.GL_IN, branch_rows(bits(m + "y"), bits(m + "x"))), (hip.GL_GATES, gate_rows(bits(m + "ra"), bits(m + "ri"))),
                         (hip.GL_O, bits(m + "o"))]
            vectors += [(hip.GL_Y_BIAS, f32(m + "y.b")), (hip.GL_X_BIAS, f32(m + "x.b")), (hip.GL_CONV, f32(m + "conv").T),
                        (hip.GL_CONV_BIAS, f32(m + "conv.b")), (hip.GL_RA_BIAS, f32(m + "ra.b")), (hip.GL_RI_BIAS, f32(m + "ri.b")),
                        (hip.GL_LAM, f32(m + "lam"))]
        e = layer.experts
        if e.n_experts:
            q = p + ".mlp."
            matrices += [(hip.GL_ROUTER, bits(q + "router")), (hip.GL_UP, expert_rows(bits(f"{q}e{k}.up") for k in range(e.n_experts))),
                         (hip.GL_DOWN, expert_rows(bits(f"{q}e{k}.down") for k in range(e.n_experts)))]
            if e.shared_ff:
                matrices += [(hip.GL_SHARED_UP, bits(q + "shared.up")), (hip.GL_SHARED_DOWN, bits(q + "shared.down"))]
            vectors += [(hip.GL_NORM2, f32(p + ".norm2"))]
        for which, rows in matrices:
            model.set_matrix(which, i, dev.dense(rows))
        for which, values in vectors:
            model.set_vector(which, i, values)
    model.set_vector(hip.GL_FINAL, -1, f32("final.norm"))
    model.set_matrix(hip.GL_EMBED, -1, dev.dense(bits("embed")))
    return model


def load(dev, path: str, max_pos: int, act: int = hip.ACT_BF16) -> hip.Gulisun:
    with open(os.path.join(path, "config.json")) as f:
        cfg = json.load(f)
    return build(dev, cfg, SafetensorsFile(os.path.join(path, "model.safetensors")), max_pos, act)
