"""Plain CPU statement of the Gulisun decoder, one function per mechanism, in float64.

TEST INFRASTRUCTURE ONLY; nothing here is shared with the product path.  Shapes: a sequence is [tokens, width]; heads
are [tokens, heads, dim].  Everything is evaluated for whole sequences from position 0, by direct sums and a plain loop
over tokens for the recurrence: a position's result does not depend on any cache, and token-by-token or portioned runs of
the device are compared with the rows of one such evaluation.

`weights` is {tensor name: array}; `cfg` is the parsed config.json.
"""
from __future__ import annotations

import numpy as np


def rms_norm(x, w, eps):
    """x / sqrt(mean(x^2) + eps) * w over the last axis."""
    return x / np.sqrt((x * x).mean(axis=-1, keepdims=True) + eps) * w


def sigmoid(z):
    return 1.0 / (1.0 + np.exp(-z))


def softplus(z):
    return np.log1p(np.exp(-np.abs(z))) + np.maximum(z, 0.0)


def gelu_tanh(z):
    return 0.5 * z * (1.0 + np.tanh(np.sqrt(2.0 / np.pi) * (z + 0.044715 * z ** 3)))


# ------------------------------------------------------------------ latent attention
def rotate(x, positions, base, dims):
    """Pairs (i, i + dims/2) of the first `dims` values of the last axis; x [tokens, ..., d]."""
    if not dims:
        return x
    half = dims // 2
    f = np.array([float(base) ** (-2.0 * i / dims) for i in range(half)], np.float64)
    ang = np.asarray(positions, np.float64)[:, None] * f[None, :]
    ang = ang.reshape((len(positions),) + (1,) * (x.ndim - 2) + (half,))
    u, v = x[..., :half], x[..., half:2 * half]
    return np.concatenate([u * np.cos(ang) - v * np.sin(ang), v * np.cos(ang) + u * np.sin(ang), x[..., 2 * half:]], axis=-1)


def latent_of(h, w, p, m, eps):
    """What a layer's cache holds: the normed latent [tokens, kv_rank] and the rotated key part [tokens, rot_dim]."""
    z = h @ w[p + ".dkv"].T
    c = rms_norm(z[:, :m["kv_rank"]], w[p + ".dkv.norm"], eps)
    k_rot = z[:, m["kv_rank"]:]
    return c, rotate(k_rot, np.arange(len(h)), m["rot"]["base"], m["rot"]["dims"])


def queries_of(h, w, p, m, eps):
    """[tokens, heads, dim + rot_dim], the last rot_dim rotated."""
    cq = rms_norm(h @ w[p + ".dq"].T, w[p + ".dq.norm"], eps)
    q = (cq @ w[p + ".uq"].T).reshape(len(h), m["heads"], m["dim"] + m["rot_dim"])
    turned = rotate(q[..., m["dim"]:], np.arange(len(h)), m["rot"]["base"], m["rot"]["dims"])
    return np.concatenate([q[..., :m["dim"]], turned], axis=-1)


def attend(q, k, v, scale, sink):
    """Causal softmax attention, one key and value per head; the denominator also holds exp(sink) per head if given.
    q, k [tokens, H, dk], v [tokens, H, dv]."""
    n, H, _ = q.shape
    out = np.zeros((n, H, v.shape[2]))
    for h in range(H):
        for i in range(n):
            s = k[:i + 1, h] @ q[i, h] * scale
            top = s.max() if sink is None else max(s.max(), sink[h])
            e = np.exp(s - top)
            den = e.sum() + (0.0 if sink is None else np.exp(sink[h] - top))
            out[i, h] = (e / den) @ v[:i + 1, h]
    return out


def latent_attention(h, w, p, m, eps, latent, sink):
    """latent: this layer's own (c, rotated key part), or another layer's."""
    n, H = len(h), m["heads"]
    c, k_rot = latent
    k = (c @ w[p + ".uk"].T).reshape(n, H, m["dim"])
    k = np.concatenate([k, np.repeat(k_rot[:, None, :], H, axis=1)], axis=-1)
    v = (c @ w[p + ".uv"].T).reshape(n, H, m["vdim"])
    return attend(queries_of(h, w, p, m, eps), k, v, m["scale"], sink).reshape(n, -1) @ w[p + ".o"].T


# ------------------------------------------------------------------ gated linear recurrence
def causal_conv(x, w, b):
    """Per channel; w [channels, taps], the last column weighs the current token; zeros before the start."""
    n, taps = x.shape[0], w.shape[1]
    padded = np.concatenate([np.zeros((taps - 1, x.shape[1])), x])
    return sum(padded[j:j + n] * w[:, j] for j in range(taps)) + b


def block_gate(u, w, b):
    """sigmoid of a block-diagonal product; w [blocks, size, size] as [out, in], b [blocks, size]."""
    n, blocks = u.shape[0], w.shape[0]
    parts = u.reshape(n, blocks, -1)
    return np.concatenate([sigmoid(parts[:, i] @ w[i].T + b[i]) for i in range(blocks)], axis=1)


def recurrence(u, r, i, lam):
    """S_t = a S_(t-1) + sqrt(1 - a^2) i u with log a = -8 r softplus(lam), S_(-1) = 0."""
    log_a = -8.0 * r * softplus(lam)
    a, b = np.exp(log_a), np.sqrt(-np.expm1(2.0 * log_a)) * i * u
    s, out = np.zeros(u.shape[1]), []
    for t in range(len(u)):
        s = a[t] * s + b[t]
        out.append(s)
    return np.array(out)


def rglru(h, w, p):
    y = gelu_tanh(h @ w[p + ".y"].T + w[p + ".y.b"])
    u = causal_conv(h @ w[p + ".x"].T + w[p + ".x.b"], w[p + ".conv"], w[p + ".conv.b"])
    s = recurrence(u, block_gate(u, w[p + ".ra"], w[p + ".ra.b"]), block_gate(u, w[p + ".ri"], w[p + ".ri.b"]), w[p + ".lam"])
    return (s * y) @ w[p + ".o"].T


# ------------------------------------------------------------------ experts
def expert(h, up, down):
    u = np.maximum(h @ up.T, 0.0)
    return (u * u) @ down.T


def route(h, router, top):
    """(expert numbers, weights), both [tokens, top], largest score first."""
    z = h @ router.T
    e = np.exp(z - z.max(axis=1, keepdims=True))
    s = e / e.sum(axis=1, keepdims=True)
    ids = np.argsort(-s, axis=1, kind="stable")[:, :top]
    chosen = np.take_along_axis(s, ids, axis=1)
    return ids, chosen / (chosen.sum(axis=1, keepdims=True) + 1e-20)


def experts(h, w, p, mlp):
    ids, weights = route(h, w[p + ".router"], mlp["router"]["top"])
    out = np.zeros_like(h)
    for e in range(mlp["router"]["experts"]):
        for t, k in zip(*np.nonzero(ids == e)):
            out[t] += weights[t, k] * expert(h[t], w[f"{p}.e{e}.up"], w[f"{p}.e{e}.down"])
    if mlp.get("shared"):
        out = out + expert(h, w[p + ".shared.up"], w[p + ".shared.down"])
    return out


# ------------------------------------------------------------------ the model
def mixer(x, w, i, cfg, latents):
    entry, p, eps = cfg["layers"][i], f"l{i}.mix", cfg["norm"]["eps"]
    m = entry["mixer"]
    if entry["type"] == "rglru":
        return rglru(x, w, p)
    if m.get("kv_from") is None:
        latents[i] = latent_of(x, w, p, m, eps)
        source = i
    else:
        source = m["kv_from"]
    sink = w[p + ".sink"] if entry["type"] == "latent_attention" else None
    return latent_attention(x, w, p, m, eps, latents[source], sink)


def layer(x, w, i, cfg, latents):
    """Both sublayers read x itself; a norm of their result enters the sum."""
    p, eps = f"l{i}", cfg["norm"]["eps"]
    x = x + rms_norm(mixer(x, w, i, cfg, latents), w[p + ".norm1"], eps)
    mlp = cfg["layers"][i].get("mlp")
    if mlp is not None:
        x = x + rms_norm(experts(x, w, p + ".mlp", mlp), w[p + ".norm2"], eps)
    return x


def forward(cfg, weights, tokens, trace=None):
    """Logits [tokens, vocab]; trace (optional list) receives the residual stream behind every layer."""
    w = {k: np.asarray(v, np.float64) for k, v in weights.items()}
    x = w["embed"][np.asarray(tokens, np.int64)] * cfg["embedding"]["scale"]
    latents = {}
    for i in range(len(cfg["layers"])):
        x = layer(x, w, i, cfg, latents)
        if trace is not None:
            trace.append(x.copy())
    return rms_norm(x, w["final.norm"], cfg["norm"]["eps"]) @ w["embed"].T


def greedy(cfg, weights, prompt, n_steps):
    """The tokens greedy decoding chooses, and the gap between the two best logits at each step."""
    tokens, gaps = [int(t) for t in prompt], []
    for _ in range(n_steps):
        z = forward(cfg, weights, tokens)[-1]
        best = np.sort(z)[-2:]
        gaps.append(float(best[1] - best[0]))
        tokens.append(int(np.argmax(z)))
    return tokens[len(prompt):], gaps
