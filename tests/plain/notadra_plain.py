"""Notadra written plainly: float64 numpy, one function per mechanism, token by token where the order matters.  It
shares nothing with the library: the tests hold the library to it.

``weights`` maps checkpoint names to float64 arrays, ``cfg`` is the dictionary of config.json.
"""
from __future__ import annotations

import math

import numpy as np


def rms_norm(x, w, eps):
    """The norm whose stored weight is the gain's distance from one."""
    return x / np.sqrt((x * x).mean(-1, keepdims=True) + eps) * (1.0 + w)


# ---------------------------------------------------------------- the embedding
def bigram_rows(tokens, before, bigram):
    """The rows of the pair table for ``tokens``; ``before`` is the token ahead of the first one, or None at a sequence's
    start."""
    rows = []
    for t in tokens:
        rows.append(bigram["buckets"] if before is None
                    else (int(before) * bigram["mul_prev"] + int(t) * bigram["mul_cur"]) % bigram["buckets"])
        before = t
    return rows


def embed(tokens, w, bigram, state):
    rows = bigram_rows(tokens, state.get("before"), bigram)
    if len(tokens):
        state["before"] = int(tokens[-1])
    return w["embed"][np.asarray(tokens)] + w["bigram"][np.asarray(rows)]


# ---------------------------------------------------------------- the rotation
def frequencies(rot):
    """One frequency a pair and the factor on cosine and sine."""
    dims, base = rot["dims"], rot["base"]
    plain = [base ** (-2.0 * i / dims) for i in range(dims // 2)]
    sc = rot.get("scaling")
    if not sc:
        return np.array(plain), 1.0

    def turns_at(t):                                          # the (real) pair index that turns t times in `original` tokens
        return dims * math.log(sc["original"] / (2.0 * math.pi * t)) / (2.0 * math.log(base))

    lo = max(math.floor(turns_at(sc["fast"])), 0)
    hi = min(math.ceil(turns_at(sc["slow"])), dims - 1)
    out = []
    for i, f in enumerate(plain):
        r = (i - lo) / max(hi - lo, 0.001)
        r = min(max(r, 0.0), 1.0)
        out.append(f / sc["factor"] * r + f * (1.0 - r))
    return np.array(out), 0.1 * math.log(sc["factor"]) + 1.0


def rotate_half(x, positions, rot):
    """x [T, heads, dim]: elements i and i + dims/2 of the first ``dims`` turn together; the rest stays."""
    out = x.copy()
    dims = rot["dims"]
    freq, mult = frequencies(rot)
    for i in range(dims // 2):
        a = positions * freq[i]
        c, s = np.cos(a)[:, None] * mult, np.sin(a)[:, None] * mult
        u, v = x[:, :, i], x[:, :, i + dims // 2]
        out[:, :, i] = u * c - v * s
        out[:, :, i + dims // 2] = v * c + u * s
    return out


# ---------------------------------------------------------------- attention
def capped_attention(q, keys, vals, start, scale, cap):
    """q [T, heads, dim] at positions start .. start + T - 1, keys and values of positions 0 on; [T, heads, vdim]."""
    t, heads, _ = q.shape
    share = heads // keys.shape[1]
    out = np.zeros((t, heads, vals.shape[2]))
    for i in range(t):
        n = start + i + 1                                     # keys 0 .. start + i
        for hd in range(heads):
            s = keys[:n, hd // share] @ q[i, hd] * scale
            if cap:
                s = cap * np.tanh(s / cap)
            top = max(s.max(), 0.0)
            e = np.exp(s - top)
            out[i, hd] = e @ vals[:n, hd // share] / (math.exp(-top) + e.sum())     # a sink of score 0, in the denominator alone
    return out


def attention(h, w, p, m, own, shared):
    """``own``: what this layer keeps of the sequence; ``shared``: that of the layer whose keys and values it reads, or
    None where it makes its own."""
    t = h.shape[0]
    heads, groups, dim = m["heads"], m["kv_heads"], m["dim"]
    vdim = m.get("vdim", dim)
    start = own.get("len", 0)
    pos = np.arange(start, start + t, dtype=np.float64)
    rot = m.get("rot")
    turn = (lambda x: rotate_half(x, pos, rot)) if rot and rot["dims"] else (lambda x: x)
    q = turn((h @ w[p + "q"].T + w[p + "q.b"]).reshape(t, heads, dim))
    if shared is None:
        k = turn((h @ w[p + "k"].T + w[p + "k.b"]).reshape(t, groups, dim))
        v = (h @ w[p + "v"].T + w[p + "v.b"]).reshape(t, groups, vdim)
        own["k"] = np.concatenate([own["k"], k]) if "k" in own else k
        own["v"] = np.concatenate([own["v"], v]) if "v" in own else v
        shared = own
    own["len"] = start + t
    o = capped_attention(q, shared["k"], shared["v"], start, m["scale"], m.get("softcap"))
    return o.reshape(t, heads * vdim) @ w[p + "o"].T


# ---------------------------------------------------------------- experts
def route(h, w, p, router):
    """The chosen experts and their weights for every token, and every token's distance to another choice."""
    s = 1.0 / (1.0 + np.exp(-(h @ w[p + "router"].T)))
    choice = s + w[p + "correction"]
    n, top = choice.shape[1], router["top"]
    groups = router.get("groups") or {"count": 1, "keep": 1}
    count, keep = groups["count"], groups["keep"]
    per = n // count
    ids, gaps = [], []
    for row in choice:
        score = [np.sort(row[g * per:(g + 1) * per])[-2:].sum() for g in range(count)]
        order = sorted(range(count), key=lambda g: (-score[g], g))
        kept = set(order[:keep])
        gap = score[order[keep - 1]] - score[order[keep]] if keep < count else np.inf
        open_to = sorted((e for e in range(n) if e // per in kept), key=lambda e: (-row[e], e))
        ids.append(open_to[:top])
        if top < len(open_to):
            gap = min(gap, row[open_to[top - 1]] - row[open_to[top]])
        gaps.append(gap)
    ids = np.array(ids)
    return ids, np.take_along_axis(s, ids, -1), np.array(gaps)


def expert(x, w, p, e):
    return w[f"{p}e{e}.down"] @ np.maximum(w[f"{p}e{e}.up"] @ x, 0.0) ** 2


def moe(h, w, p, mlp, gaps=None):
    ids, weights, gap = route(h, w, p, mlp["router"])
    if gaps is not None:
        gaps.append(gap)
    out = np.zeros_like(h)
    for i in range(h.shape[0]):
        for e, a in zip(ids[i], weights[i]):
            out[i] += a * expert(h[i], w, p, e)
    return out


# ---------------------------------------------------------------- the model
def forward(cfg, w, tokens, state=None, gaps=None, layers_out=None):
    """Logits [T, vocab] of the next ``tokens`` of one sequence; ``state`` (a dict, empty at the start) carries the
    sequence from call to call.  ``layers_out``: a list that receives the residual after every layer."""
    state = {} if state is None else state
    eps = cfg["norm"]["eps"]
    x = embed(tokens, w, cfg["embedding"]["bigram"], state.setdefault("embedding", {}))
    for i, layer in enumerate(cfg["layers"]):
        p, m = f"l{i}.", layer["mixer"]
        own = state.setdefault(i, {})
        shared = state[m["kv_from"]] if m.get("kv_from") is not None else None
        y = attention(rms_norm(x, w[p + "norm1"], eps), w, p + "mix.", m, own, shared)
        x = x + rms_norm(y, w[p + "norm1b"], eps)
        if layer.get("mlp") is not None:
            y = moe(rms_norm(x, w[p + "norm2"], eps), w, p + "mlp.", layer["mlp"], gaps)
            x = x + rms_norm(y, w[p + "norm2b"], eps)
        if layers_out is not None:
            layers_out.append(x.copy())
    x = rms_norm(x, w["final.norm"], eps)
    return x @ w["head"].T * cfg["logit_scale"]
