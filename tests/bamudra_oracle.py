"""Plain float64 implementation of the Bamudra design: whole sequences, no cache, one function
per mechanism. It reads a configuration dict (the layout of the design's ``config.json``) and a
dict of checkpoint-named float64 arrays, and shares no code with the package.

    x = E[tok]
    per layer run:  x <- x + mixer(norm1(x));  x <- x + ff(norm2(x))
    loop:           passes 2, 3, ... start with x <- x + E[tok]
    output:         logits = W_head norm(x)
"""
import math

import numpy as np


def rms(x, eps):
    return x / np.sqrt((x * x).mean(-1, keepdims=True) + eps)


def norm(x, w, eps):
    return rms(x, eps) * w


def sigmoid(z):
    return 1.0 / (1.0 + np.exp(-z))


def silu(z):
    return z * sigmoid(z)


def rotate_half(x, positions, rot):
    """x [T, heads, n]: dimension i < dims/2 of every head turns with dimension i + dims/2 by
    position * base^(-2i/dims); dimensions from ``dims`` on stay."""
    dims = int((rot or {}).get("dims") or 0)
    if not dims:
        return x
    half = dims // 2
    f = float(rot["base"]) ** (-2.0 * np.arange(half) / dims)
    ang = np.asarray(positions, np.float64)[:, None, None] * f[None, None, :]
    c, s = np.cos(ang), np.sin(ang)
    u, v = x[..., :half], x[..., half:dims]
    return np.concatenate([u * c - v * s, v * c + u * s, x[..., dims:]], -1)


# ----------------------------------------------------------------------------- mixers
def retention(h, w, p, mx, eps):
    """Linear attention with one fixed decay per head over rotated queries and keys; every
    head's read-out is divided by its own RMS and the concatenation gated."""
    T = h.shape[0]
    H, d, dv = int(mx["heads"]), int(mx["dim"]), int(mx["vdim"])
    pos = np.arange(T)
    q = rotate_half((h @ w[p + "q"].T).reshape(T, H, d), pos, mx.get("rot"))
    k = rotate_half((h @ w[p + "k"].T).reshape(T, H, d), pos, mx.get("rot")) * d ** -0.5
    v = (h @ w[p + "v"].T).reshape(T, H, dv)
    o = np.zeros((T, H, dv))
    for hh in range(H):
        S = np.zeros((d, dv))
        for t in range(T):
            S = float(mx["decay"][hh]) * S + np.outer(k[t, hh], v[t, hh])
            o[t, hh] = S.T @ q[t, hh]
    o = rms(o, eps).reshape(T, H * dv) * silu(h @ w[p + "g"].T)
    return o @ w[p + "o"].T


def visible(T, mask):
    """[T, T] bool: position i sees j <= i inside the window or among the kept first tokens."""
    i, j = np.arange(T)[:, None], np.arange(T)[None, :]
    ok = j <= i
    if mask:
        ok = ok & ((i - j < int(mask["size"])) | (j < int(mask.get("keep_first") or 0)))
    return ok


def attention(h, w, p, mx, eps):
    """Windowed grouped-query attention with kept first tokens; the values are the projected
    keys before their rotation; biased projections."""
    T = h.shape[0]
    H, G, d = int(mx["heads"]), int(mx["kv_heads"]), int(mx["dim"])
    pos = np.arange(T)
    kraw = (h @ w[p + "k"].T + w[p + "k.b"]).reshape(T, G, d)
    q = rotate_half((h @ w[p + "q"].T + w[p + "q.b"]).reshape(T, H, d), pos, mx.get("rot"))
    k = rotate_half(kraw, pos, mx.get("rot"))
    ok = visible(T, mx.get("mask"))
    out = np.zeros((T, H, d))
    for hh in range(H):
        g = hh // (H // G)
        sc = np.where(ok, (q[:, hh] @ k[:, g].T) * float(mx["scale"]), -np.inf)
        e = np.exp(sc - sc.max(-1, keepdims=True))
        out[:, hh] = (e / e.sum(-1, keepdims=True)) @ kraw[:, g]
    return out.reshape(T, H * d) @ w[p + "o"].T + w[p + "o.b"]


MIXERS = {"retention": retention, "attention": attention}


# ----------------------------------------------------------------------------- feed-forward
def dense_ff(h, w, p, limit):
    g = np.minimum(h @ w[p + "gate"].T, limit)
    u = np.clip(h @ w[p + "up"].T, -limit, limit)
    return (g * sigmoid(1.702 * g) * (u + 1.0)) @ w[p + "down"].T


# ----------------------------------------------------------------------------- the model
def layer_runs(c):
    """(layer, starts a pass after the first) in execution order."""
    n = len(c["layers"])
    lp = c.get("loop")
    if not lp:
        return [(i, False) for i in range(n)]
    a, b, times = int(lp["start"]), int(lp["stop"]), int(lp["times"])
    body = [(i, t > 0 and i == a) for t in range(times) for i in range(a, b)]
    return [(i, False) for i in range(a)] + body + [(i, False) for i in range(b, n)]


def forward(c, w, tokens, trace=None):
    """Logits [T, vocab] of one sequence; ``trace`` (a list) receives the residual stream after
    every layer run."""
    eps = float(c["norm"]["eps"])
    x0 = w["embed"][np.asarray(tokens)]
    x = x0.copy()
    for i, again in layer_runs(c):
        L, a = c["layers"][i], f"l{i}."
        if again:
            x = x + x0
        x = x + MIXERS[L["type"]](norm(x, w[a + "norm1"], eps), w, a + "mix.", L["mixer"], eps)
        if L.get("mlp"):
            x = x + dense_ff(norm(x, w[a + "norm2"], eps), w, a + "mlp.", float(L["mlp"]["limit"]))
        if trace is not None:
            trace.append(x.copy())
    return norm(x, w["final.norm"], eps) @ w["head"].T


# ----------------------------------------------------------------------------- test weights
def bf16_exact(a):
    """Round to values bfloat16 holds exactly (so that every precision sees the same weights)."""
    import torch
    return torch.as_tensor(np.asarray(a, np.float64)).to(torch.bfloat16).double().numpy()


def random_weights(c, seed=0):
    """Checkpoint-named float64 arrays (bfloat16-exact) for configuration ``c``."""
    rng = np.random.default_rng(seed)
    D, V = int(c["width"]), int(c["vocab"])
    w = {}

    def lin(name, o, i, gain=1.0):
        w[name] = rng.standard_normal((o, i)) * gain / math.sqrt(i)

    w["embed"] = rng.standard_normal((V, D))
    lin("head", V, D)
    w["final.norm"] = 1.0 + 0.2 * rng.standard_normal(D)
    for i, L in enumerate(c["layers"]):
        a, mx = f"l{i}.", L["mixer"]
        m = a + "mix."
        w[a + "norm1"] = 1.0 + 0.2 * rng.standard_normal(D)
        H, d = int(mx["heads"]), int(mx["dim"])
        if L["type"] == "retention":
            dv = int(mx["vdim"])
            lin(m + "q", H * d, D), lin(m + "k", H * d, D), lin(m + "v", H * dv, D)
            # a token's key leans towards its query: a read-out close to zero (a first token's
            # above all) would magnify every rounding when it is divided by its RMS
            w[m + "k"] = 0.8 * w[m + "q"] + 0.6 * w[m + "k"]
            lin(m + "g", H * dv, D, 1.5), lin(m + "o", D, H * dv)
        else:
            G = int(mx["kv_heads"])
            lin(m + "q", H * d, D), lin(m + "k", G * d, D), lin(m + "o", D, H * d)
            for n, rows in (("q", H * d), ("k", G * d), ("o", D)):
                w[m + n + ".b"] = 0.3 * rng.standard_normal(rows)
        if L.get("mlp"):
            F, f = int(L["mlp"]["ff"]), a + "mlp."
            w[a + "norm2"] = 1.0 + 0.2 * rng.standard_normal(D)
            lin(f + "gate", F, D, 1.5), lin(f + "up", F, D, 1.5), lin(f + "down", D, F)
    return {k: bf16_exact(v) for k, v in w.items()}
