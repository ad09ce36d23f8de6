"""Kisepel written plainly: float64 numpy, one function per mechanism, token by token where a mechanism is
sequential.  It shares nothing with the library: the tests hold the library to it.

``weights`` maps checkpoint names to float64 arrays (the experts' table to integers), ``cfg`` is the dictionary of
config.json.  A mixer's ``state`` is a dictionary it keeps between calls for one sequence and one run.
"""
from __future__ import annotations

import math

import numpy as np


def sigmoid(z):
    return 1.0 / (1.0 + np.exp(-z))


def silu(z):
    return z * sigmoid(z)


def softplus(z):
    return np.logaddexp(0.0, z)


def rms_unit(x, eps):
    """x / sqrt(mean(x^2) + eps) over the last axis."""
    return x / np.sqrt((x * x).mean(-1, keepdims=True) + eps)


def norm_from_one(x, stored, eps):
    return rms_unit(x, eps) * (1.0 + stored)


def rotate_halves(x, positions, dims, base, factor):
    """x [T, heads, dim]: the elements (i, i + dims / 2) of every head turn by positions * base^(-2i / dims) / factor;
    what lies behind ``dims`` stays."""
    out = x.copy()
    half = dims // 2
    for i in range(half):
        a = positions * (base ** (-2.0 * i / dims) / factor)
        c, s = np.cos(a)[:, None], np.sin(a)[:, None]
        u, v = x[:, :, i], x[:, :, i + half]
        out[:, :, i] = u * c - v * s
        out[:, :, i + half] = v * c + u * s
    return out


def short_conv(x, taps, bias, state, key):
    """x [T, channels] through a causal convolution per channel: taps [channels, n], the last the current token's."""
    n = taps.shape[1]
    before = state.get(key, np.zeros((n - 1, x.shape[1])))
    line = np.concatenate([before, x])
    out = np.zeros_like(x)
    for i in range(x.shape[0]):
        for j in range(n):
            out[i] += taps[:, j] * line[i + j]
    state[key] = line[len(line) - (n - 1):].copy()
    return out if bias is None else out + bias


# ---------------------------------------------------------------- linear attention with a fixed decay a head
def lightning_mixer(h, w, p, m, eps, state):
    t = h.shape[0]
    heads, dim, vdim = m["heads"], m["dim"], m["vdim"]
    q = silu(h @ w[p + "q"].T).reshape(t, heads, dim)
    k = silu(h @ w[p + "k"].T).reshape(t, heads, dim)
    v = silu(h @ w[p + "v"].T).reshape(t, heads, vdim)
    s = state.get("S", np.zeros((heads, dim, vdim)))
    out = np.zeros((t, heads, vdim))
    for i in range(t):
        for hd in range(heads):
            s[hd] = m["decay"][hd] * s[hd] + np.outer(k[i, hd], v[i, hd])
            out[i, hd] = s[hd].T @ q[i, hd]
    state["S"] = s
    y = rms_unit(out.reshape(t, -1), eps) * w[p + "norm"] * sigmoid(h @ w[p + "g"].T)
    return y @ w[p + "o"].T


# ---------------------------------------------------------------- the state-space mixer
def mamba2_mixer(h, w, p, m, eps, state):
    t = h.shape[0]
    heads, vdim, n, groups, parts = m["heads"], m["vdim"], m["state"], m["groups"], m["norm_groups"]
    inner, gn = heads * vdim, groups * n
    proj = h @ w[p + "in"].T
    z, xbc, dt = proj[:, :inner], proj[:, inner:2 * inner + 2 * gn], proj[:, 2 * inner + 2 * gn:]
    xbc = silu(short_conv(xbc, w[p + "conv"], w[p + "conv.b"], state, "tail"))
    x = xbc[:, :inner].reshape(t, heads, vdim)
    b = xbc[:, inner:inner + gn].reshape(t, groups, n)
    c = xbc[:, inner + gn:].reshape(t, groups, n)
    dt = softplus(dt + w[p + "dt_bias"])
    s = state.get("S", np.zeros((heads, n, vdim)))
    y = np.zeros((t, heads, vdim))
    for i in range(t):
        for hd in range(heads):
            g = hd // (heads // groups)
            s[hd] = math.exp(-math.exp(w[p + "A_log"][hd]) * dt[i, hd]) * s[hd] + dt[i, hd] * np.outer(b[i, g], x[i, hd])
            y[i, hd] = s[hd].T @ c[i, g] + w[p + "D"][hd] * x[i, hd]
    state["S"] = s
    y = y.reshape(t, inner) * silu(z)
    y = rms_unit(y.reshape(t, parts, inner // parts), eps).reshape(t, inner) * w[p + "norm"]
    return y @ w[p + "o"].T


# ---------------------------------------------------------------- softmax attention in chunks of the sequence
def attention_core(q, keys, values, start, size, scale):
    """q [T, heads, dim] at positions start ..; keys and values [start + T, groups, .] from position 0 on; a query sees the keys
    of its own run of ``size`` positions up to itself."""
    heads, groups = q.shape[1], keys.shape[1]
    out = np.zeros((q.shape[0], heads, values.shape[2]))
    for i in range(q.shape[0]):
        at = start + i
        lo = at // size * size                       # the first position of the query's chunk
        for hd in range(heads):
            g = hd // (heads // groups)
            s = keys[lo:at + 1, g] @ q[i, hd] * scale
            e = np.exp(s - s.max())
            out[i, hd] = (e / e.sum()) @ values[lo:at + 1, g]
    return out


def chunked_attention(h, w, p, m, eps, state):
    t = h.shape[0]
    heads, groups, dim, vdim = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    size = m["mask"]["size"] if m.get("mask") else 1 << 40
    start = state.get("len", 0)
    pos = np.arange(start, start + t, dtype=np.float64)
    rot = (m["rot"]["dims"], m["rot"]["base"], (m["rot"].get("scaling") or {"factor": 1.0})["factor"]) if m.get("rot") else (0, 1.0, 1.0)
    q = rms_unit((h @ w[p + "q"].T).reshape(t, heads, dim), eps) * w[p + "q.norm"]
    k = rms_unit((h @ w[p + "k"].T).reshape(t, groups, dim), eps) * w[p + "k.norm"]
    q, k = rotate_halves(q, pos, *rot), rotate_halves(k, pos, *rot)
    v = (h @ w[p + "v"].T).reshape(t, groups, vdim)
    state["k"] = np.concatenate([state["k"], k]) if "k" in state else k
    state["v"] = np.concatenate([state["v"], v]) if "v" in state else v
    state["len"] = start + t
    out = attention_core(q, state["k"], state["v"], start, size, m["scale"])
    return out.reshape(t, heads * vdim) @ w[p + "o"].T


# ---------------------------------------------------------------- the delta rule with a decay a key channel
def unit(x):
    return x / np.sqrt((x * x).sum(-1, keepdims=True) + 1e-6)


def decays(z, a_log, dt_bias):
    """z [T, heads * dim] -> a factor per head and key channel."""
    heads = a_log.shape[0]
    return np.exp(-np.exp(a_log)[None, :, None] * softplus(z + dt_bias).reshape(len(z), heads, -1))


def delta_walk(q, k, v, beta, g, s):
    """q, k [T, kv, dim], v [T, heads, vdim], beta [T, heads], g [T, heads, dim]; the states s [heads, dim, vdim] change in place."""
    out = np.zeros(v.shape)
    share = v.shape[1] // q.shape[1]
    for i in range(v.shape[0]):
        for hd in range(v.shape[1]):
            qi, ki = q[i, hd // share], k[i, hd // share]
            s[hd] = g[i, hd][:, None] * s[hd]
            u = beta[i, hd] * (v[i, hd] - s[hd].T @ ki)
            s[hd] = s[hd] + np.outer(ki, u)
            out[i, hd] = s[hd].T @ qi                # the read-out sees the token's own write
    return out


def delta_mixer(h, w, p, m, eps, state):
    t = h.shape[0]
    heads, kv, dim, vdim = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    conv = lambda n: silu(short_conv(h @ w[p + n].T, w[p + n + ".conv"], None, state, n))
    q = unit(conv("q").reshape(t, kv, dim)) * dim ** -0.5
    k = unit(conv("k").reshape(t, kv, dim))
    v = conv("v").reshape(t, heads, vdim)
    beta = sigmoid(h @ w[p + "b"].T)
    g = decays((h @ w[p + "a1"].T) @ w[p + "a2"].T, w[p + "A_log"], w[p + "dt_bias"])
    s = state.get("S", np.zeros((heads, dim, vdim)))
    out = delta_walk(q, k, v, beta, g, s)
    state["S"] = s
    gate = sigmoid((h @ w[p + "g1"].T) @ w[p + "g2"].T)
    y = (rms_unit(out, eps) * w[p + "norm"]).reshape(t, heads * vdim) * gate
    return y @ w[p + "o"].T


def parallel_mixer(h, w, p, m, eps, state):
    left = chunked_attention(h, w, p + "left.", m["left"], eps, state.setdefault("left", {}))
    right = delta_mixer(h, w, p + "right.", m["right"], eps, state.setdefault("right", {}))
    return 0.5 * (rms_unit(left, eps) * w[p + "left.out"] + rms_unit(right, eps) * w[p + "right.out"])


MIXERS = {"lightning": lightning_mixer, "mamba2": mamba2_mixer, "parallel": parallel_mixer}


# ---------------------------------------------------------------- feed-forward
def gated(h, w, p):
    return (silu(h @ w[p + "gate"].T) * (h @ w[p + "up"].T)) @ w[p + "down"].T


def table_experts(h, w, p, mlp, tokens):
    top = mlp["router"]["top"]
    out = np.zeros_like(h)
    for i, tok in enumerate(tokens):
        for e in w[p + "table"][tok][:top]:
            out[i] += gated(h[i:i + 1], w, f"{p}e{int(e)}.")[0] / top
    if mlp.get("shared") is not None:
        out += gated(h, w, p + "shared.")
    return out


# ---------------------------------------------------------------- the model
def order(cfg):
    """(layer, whether the embedding output is added before it) for every run, in their order."""
    n = len(cfg["layers"])
    loop = cfg.get("loop") or {"start": 0, "stop": 0, "times": 1}
    a, b = loop["start"], loop["stop"]
    runs = [(i, False) for i in range(a)]
    for turn in range(loop["times"]):
        runs += [(i, turn > 0 and i == a) for i in range(a, b)]
    return runs + [(i, False) for i in range(b, n)]


def forward(cfg, w, tokens, state=None, layers=None):
    """Logits [T, vocab] of one sequence's next tokens; ``state`` carries it on; ``layers`` collects the residual after
    every layer run."""
    state = {} if state is None else state
    eps = cfg["norm"]["eps"]
    embedded = w["embed"][np.asarray(tokens)] * cfg["embedding"]["scale"]
    x = embedded
    for run, (i, again) in enumerate(order(cfg)):
        layer, p = cfg["layers"][i], f"l{i}."
        if again:
            x = x + embedded
        h = norm_from_one(x, w[p + "norm1"], eps)
        y = MIXERS[layer["type"]](h, w, p + "mix.", layer["mixer"], eps, state.setdefault(run, {}))
        if layer.get("mlp") is not None:
            y = y + table_experts(h, w, p + "mlp.", layer["mlp"], tokens)
        x = x + y
        if layers is not None:
            layers.append(x)
    return norm_from_one(x, w["final.norm"], eps) @ w["embed"].T * cfg["logit_scale"]
