"""Plain CPU statement of the Suvazen decoder, one function per mechanism, in float64.

TEST INFRASTRUCTURE ONLY; nothing here is shared with the product path.  Shapes: a sequence is [tokens, width]; heads
are [tokens, heads, dim].  Everything is evaluated for whole sequences from position 0, by direct sums: a position's
result does not depend on any cache, and token-by-token or portioned runs of the device are compared with the rows of
one such evaluation.

`weights` is {tensor name: array}; `cfg` is the parsed config.json.
"""
from __future__ import annotations

import math

import numpy as np


def layer_norm(x, w, b, eps):
    """(x - mean) / sqrt(mean((x - mean)^2) + eps) * w + b over the last axis."""
    mean = x.mean(axis=-1, keepdims=True)
    dev = x - mean
    return dev / np.sqrt((dev * dev).mean(axis=-1, keepdims=True) + eps) * w + b


def rotary_frequencies(rot):
    """f_i = base^(-2i/dims), i = 0 .. dims/2 - 1, with the wavelength-dependent stretch where `scaling` asks for it."""
    out = []
    for i in range(rot["dims"] // 2):
        f = float(rot["base"]) ** (-2.0 * i / rot["dims"])
        s = rot.get("scaling")
        if s:
            wavelength = 2.0 * math.pi / f
            if wavelength > s["original"] / s["low"]:
                f = f / s["factor"]
            elif wavelength >= s["original"] / s["high"]:
                mix = (s["original"] / wavelength - s["low"]) / (s["high"] - s["low"])
                f = (1.0 - mix) * f / s["factor"] + mix * f
        out.append(f)
    return np.array(out, np.float64)


def rotate(x, positions, rot):
    """Pairs (i, i + dims/2) of the first `dims` values of each head, x [tokens, heads, dim]."""
    if not rot:
        return x
    half = rot["dims"] // 2
    ang = np.asarray(positions, np.float64)[:, None] * rotary_frequencies(rot)[None, :]
    c, s = np.cos(ang)[:, None, :], np.sin(ang)[:, None, :]
    u, v = x[..., :half], x[..., half:2 * half]
    return np.concatenate([u * c - v * s, v * c + u * s, x[..., 2 * half:]], axis=-1)


def visible(i, j, window):
    """Whether position i attends to position j."""
    return j <= i and (window is None or i - j < window)


def capped(scores, cap):
    return scores if cap is None else cap * np.tanh(scores / cap)


def attend(q, k, v, scale, cap, window, sink):
    """Sliding-window softmax attention whose denominator also holds exp(sink) per query head.
    q [tokens, H, dim], k / v [tokens, G, dim]; returns [tokens, H, dim]."""
    n, H, _ = q.shape
    G = k.shape[1]
    out = np.zeros((n, H, v.shape[2]))
    for h in range(H):
        g = h // (H // G)
        for i in range(n):
            lo = 0 if window is None else max(0, i - window + 1)
            s = capped(k[lo:i + 1, g] @ q[i, h] * scale, cap)
            top = s.max() if sink is None else max(s.max(), sink[h])
            e = np.exp(s - top)
            den = e.sum() + (0.0 if sink is None else math.exp(sink[h] - top))
            out[i, h] = (e / den) @ v[lo:i + 1, g]
    return out


def attention_mixer(x, w, prefix, mixer):
    """q / k projections, values = unrotated keys, rotary positions, attention, output projection."""
    n = x.shape[0]
    H, G, d = mixer["heads"], mixer["kv_heads"], mixer["dim"]
    q = (x @ w[prefix + ".mix.q"].T).reshape(n, H, d)
    k = (x @ w[prefix + ".mix.k"].T).reshape(n, G, d)
    pos = np.arange(n)
    mask = mixer.get("mask") or {}
    a = attend(rotate(q, pos, mixer.get("rot")), rotate(k, pos, mixer.get("rot")), k, mixer["scale"],
               mixer.get("softcap"), mask.get("size"), w.get(prefix + ".mix.sink"))
    return a.reshape(n, H * d) @ w[prefix + ".mix.o"].T


def squared_relu_mlp(x, w, prefix):
    """down . max(up . x, 0)^2"""
    u = np.maximum(x @ w[prefix + ".mlp.up"].T, 0.0)
    return (u * u) @ w[prefix + ".mlp.down"].T


def norm_of(w, name, x, eps):
    return layer_norm(x, w[name], w[name + ".b"], eps)


def layer(x, w, i, cfg):
    """Both sublayers with a norm in front and behind, the result scaled into the residual sum."""
    p, eps, m = f"l{i}", cfg["norm"]["eps"], cfg["residual_mult"]
    y = attention_mixer(norm_of(w, p + ".norm1", x, eps), w, p, cfg["layers"][i]["mixer"])
    x = x + m * norm_of(w, p + ".norm1b", y, eps)
    if cfg["layers"][i]["mlp"] is not None:
        y = squared_relu_mlp(norm_of(w, p + ".norm2", x, eps), w, p)
        x = x + m * norm_of(w, p + ".norm2b", y, eps)
    return x


def layer_runs(cfg):
    """The order in which layers run, as (layer, step row to add in front or None)."""
    n, loop = len(cfg["layers"]), cfg.get("loop")
    if not loop:
        return [(i, None) for i in range(n)]
    runs = [(i, None) for i in range(loop["start"])]
    for t in range(loop["times"]):
        runs += [(i, t if i == loop["start"] else None) for i in range(loop["start"], loop["stop"])]
    return runs + [(i, None) for i in range(loop["stop"], n)]


def forward(cfg, weights, tokens, trace=None):
    """Logits [tokens, vocab]; trace (optional list) receives the residual stream behind every layer run."""
    w = {k: np.asarray(v, np.float64) for k, v in weights.items()}
    x = w["embed"][np.asarray(tokens, np.int64)]
    for i, t in layer_runs(cfg):
        if t is not None:
            x = x + w["loop.step"][t]
        x = layer(x, w, i, cfg)
        if trace is not None:
            trace.append(x.copy())
    z = norm_of(w, "final.norm", x, cfg["norm"]["eps"]) @ w["head"].T * cfg["logit_scale"]
    return capped(z, cfg["logit_softcap"])


def greedy(cfg, weights, prompt, n_steps):
    """The tokens greedy decoding chooses, and the gap between the two best logits at each step."""
    tokens, gaps = [int(t) for t in prompt], []
    for _ in range(n_steps):
        z = forward(cfg, weights, tokens)[-1]
        best = np.sort(z)[-2:]
        gaps.append(float(best[1] - best[0]))
        tokens.append(int(np.argmax(z)))
    return tokens[len(prompt):], gaps
