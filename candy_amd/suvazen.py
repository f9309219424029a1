"""Suvazen: configuration and weights of a model folder (config.json, model.safetensors) -> the device decoder.

config.json: `vocab`, `width`, `layers` (per layer `type` = "attention", `mixer` with heads, kv_heads, dim, vdim, scale,
softcap, mask.size, rot.{base, dims, scaling.{factor, low, high, original}}, and `mlp` = {kind: "dense", ff} or null),
`loop` = {start, stop, times}, `norm.eps`, `residual_mult`, `logit_scale`, `logit_softcap`.  Absent or null `loop`,
`softcap`, `mask`, `rot` and `scaling` switch the mechanism off.

Tensors: embed, head, final.norm(.b), loop.step [times, width], and per layer l<i>: norm1, norm1b, norm2, norm2b (each
with .b), mix.q, mix.k, mix.o, mix.sink, mlp.up, mlp.down.  q and k share their input: their rows go to the device as one
matrix.
"""
from __future__ import annotations

import json
import os

import numpy as np

from . import hip
from .safetensors import SafetensorsFile


class ConfigError(ValueError):
    pass


def attn_spec(mixer: dict) -> hip.AttnSpec:
    dim = int(mixer["dim"])
    if int(mixer.get("vdim", dim)) != dim:
        raise ConfigError(f"the values are the keys: vdim {mixer['vdim']} must equal dim {dim}")
    rot = mixer.get("rot") or {}
    scaling = rot.get("scaling") or {}
    mask = mixer.get("mask") or {}
    return hip.AttnSpec(n_heads=int(mixer["heads"]), n_kv_heads=int(mixer["kv_heads"]), head_dim=dim,
                        window=int(mask.get("size") or 0), rope_dims=int(rot.get("dims") or 0),
                        rope_original=int(scaling.get("original") or 0), scale=float(mixer["scale"]),
                        softcap=float(mixer.get("softcap") or 0.0), rope_base=float(rot.get("base") or 1.0),
                        rope_factor=float(scaling.get("factor") or 1.0), rope_low=float(scaling.get("low") or 1.0),
                        rope_high=float(scaling.get("high") or 2.0))


def parse_config(cfg: dict, max_pos: int, act: int, has_sink=lambda layer: True):
    """config.json -> (SuvazenConfig, [SuvazenLayer])."""
    layers = []
    for i, entry in enumerate(cfg["layers"]):
        if entry["type"] != "attention":
            raise ConfigError(f"layer {i}: no mixer of type {entry['type']!r}")
        mlp = entry.get("mlp")
        if mlp is not None and mlp["kind"] != "dense":
            raise ConfigError(f"layer {i}: no feed-forward of kind {mlp['kind']!r}")
        layers.append(hip.SuvazenLayer(attn=attn_spec(entry["mixer"]), d_ffn=int(mlp["ff"]) if mlp else 0,
                                       has_sink=int(has_sink(i))))
    loop = cfg.get("loop") or {}
    return hip.SuvazenConfig(n_layers=len(layers), d_model=int(cfg["width"]), vocab=int(cfg["vocab"]), max_pos=int(max_pos),
                             loop_start=int(loop.get("start", 0)), loop_stop=int(loop.get("stop", 0)),
                             loop_times=int(loop.get("times", 0)), act=act, norm_eps=float(cfg["norm"]["eps"]),
                             residual_mult=float(cfg["residual_mult"]), logit_scale=float(cfg["logit_scale"]),
                             logit_softcap=float(cfg.get("logit_softcap") or 0.0)), layers


NORMS = (("norm1", hip.SV_NORM1), ("norm1b", hip.SV_NORM1B), ("norm2", hip.SV_NORM2), ("norm2b", hip.SV_NORM2B))


def build(dev, cfg: dict, tensors, max_pos: int, act: int = hip.ACT_BF16) -> hip.Suvazen:
    """tensors: `in`, .bits(name) and .f32(name), as SafetensorsFile has them."""
    native, layers = parse_config(cfg, max_pos, act, lambda i: f"l{i}.mix.sink" in tensors)
    model = hip.Suvazen(dev, native, layers)
    for i, layer in enumerate(layers):
        p = f"l{i}"
        matrices = [(hip.SV_QK, np.concatenate([tensors.bits(p + ".mix.q"), tensors.bits(p + ".mix.k")])),
                    (hip.SV_O, tensors.bits(p + ".mix.o"))]
        norms = NORMS[:2]
        if layer.d_ffn:
            matrices += [(hip.SV_UP, tensors.bits(p + ".mlp.up")), (hip.SV_DOWN, tensors.bits(p + ".mlp.down"))]
            norms = NORMS
        for which, bits in matrices:
            model.set_matrix(which, i, dev.dense(bits))
        for name, which in norms:
            model.set_vector(which, i, tensors.f32(f"{p}.{name}"))
            model.set_vector(which + 1, i, tensors.f32(f"{p}.{name}.b"))
        if layer.has_sink:
            model.set_vector(hip.SV_SINK, i, tensors.f32(p + ".mix.sink"))
    for t in range(native.loop_times):
        model.set_vector(hip.SV_STEP, t, tensors.f32("loop.step")[t])
    model.set_vector(hip.SV_FINAL, -1, tensors.f32("final.norm"))
    model.set_vector(hip.SV_FINAL_BIAS, -1, tensors.f32("final.norm.b"))
    model.set_matrix(hip.SV_EMBED, -1, dev.dense(tensors.bits("embed")))
    model.set_matrix(hip.SV_HEAD, -1, dev.dense(tensors.bits("head")))
    return model


def load(dev, path: str, max_pos: int, act: int = hip.ACT_BF16) -> hip.Suvazen:
    with open(os.path.join(path, "config.json")) as f:
        cfg = json.load(f)
    return build(dev, cfg, SafetensorsFile(os.path.join(path, "model.safetensors")), max_pos, act)
