"""Plain float64 implementation of the Lutovik design: whole sequences, no cache, one function
per mechanism. It reads a configuration dict (the layout of the design's ``config.json``) and a
dict of checkpoint-named float64 arrays, and shares no code with the package.

    x = scale * E[tok]
    per layer:  x <- x + post1(mixer(pre1(x)));  x <- x + post2(ff(pre2(x)))
    output:     logits = W_head norm(x)
"""
import math

import numpy as np


def rms(x, eps):
    return x / np.sqrt((x * x).mean(-1, keepdims=True) + eps)


def norm(x, w, eps):
    """RMS norm whose weight is stored as an offset from one."""
    return rms(x, eps) * (1.0 + w)


def sigmoid(z):
    return np.exp(-np.logaddexp(0.0, -z))


def silu(z):
    return z * sigmoid(z)


def softplus(z):
    return np.logaddexp(0.0, z)


# ----------------------------------------------------------------------------- rotation
def frequencies(rot):
    """Angle per position of every rotated pair; with ``scaling`` long waves are slowed by the
    factor, short ones kept, and those between blended by how many turns fit the length."""
    dims = int(rot["dims"])
    f = [float(rot["base"]) ** (-2.0 * i / dims) for i in range(dims // 2)]
    sc = rot.get("scaling")
    if not sc:
        return np.array(f)
    factor, low, high, orig = (float(sc[k]) for k in ("factor", "low", "high", "original"))
    out = []
    for v in f:
        turns = orig / (2.0 * math.pi / v)
        if turns > high:
            out.append(v)
        elif turns < low:
            out.append(v / factor)
        else:
            s = (turns - low) / (high - low)
            out.append((1.0 - s) * v / factor + s * v)
    return np.array(out)


def rotate(x, rot, half):
    """x [T, heads, n], row t at position t. ``half``: dimension i turns with i + dims/2, else
    2i with 2i + 1; dimensions from ``dims`` on stay."""
    dims = int((rot or {}).get("dims") or 0)
    if not dims:
        return x
    ang = np.arange(x.shape[0])[:, None, None] * frequencies(rot)[None, None, :]
    c, s = np.cos(ang), np.sin(ang)
    y = x.copy()
    a, b = (slice(0, dims // 2), slice(dims // 2, dims)) if half else (slice(0, dims, 2), slice(1, dims, 2))
    y[..., a] = x[..., a] * c - x[..., b] * s
    y[..., b] = x[..., b] * c + x[..., a] * s
    return y


# ----------------------------------------------------------------------------- attention
def heads_of(h, w, n):
    y = h @ w.T
    return y.reshape(h.shape[0], n, -1)


def keys_values(h, w, p, mx, half):
    G = int(mx["kv_heads"])
    return rotate(heads_of(h, w[p + "k"], G), mx.get("rot"), half), heads_of(h, w[p + "v"], G)


def attend(h, w, p, mx, half, kv):
    """Causal grouped-query softmax attention; the concatenated heads [T, H * vdim]."""
    T, H, G = h.shape[0], int(mx["heads"]), int(mx["kv_heads"])
    q = rotate(heads_of(h, w[p + "q"], H), mx.get("rot"), half)
    k, v = kv
    seen = np.tril(np.ones((T, T), bool))
    out = []
    for hh in range(H):
        g = hh // (H // G)
        sc = np.where(seen, q[:, hh] @ k[:, g].T * float(mx["scale"]), -np.inf)
        e = np.exp(sc - sc.max(-1, keepdims=True))
        out.append(e / e.sum(-1, keepdims=True) @ v[:, g])
    return np.concatenate(out, -1)


def attention(h, w, p, mx, eps, shared):
    """``shared``: layer -> (keys, values) of the attention layers so far."""
    kv = shared.get(mx.get("kv_from"))
    if kv is None:
        kv = keys_values(h, w, p, mx, False)
    return attend(h, w, p, mx, False, kv) @ w[p + "o"].T, kv


# ----------------------------------------------------------------------------- state space
def causal_conv(u, taps, bias):
    """Every channel's own filter over its last tokens (zeros before the start), then SiLU."""
    T, n = u.shape[0], taps.shape[1]
    pad = np.concatenate([np.zeros((n - 1, u.shape[1])), u])
    y = sum(pad[i:i + T] * taps[:, i] for i in range(n)) + bias
    return silu(y)


def ssd_scan(x, B, C, dt, A_log, D):
    """x [T, H, P], B / C [T, G, N], dt [T, H] (positive): y [T, H, P]."""
    T, H, P = x.shape
    G, N = B.shape[1:]
    y = np.zeros_like(x)
    for h in range(H):
        g = h // (H // G)
        S = np.zeros((N, P))
        for t in range(T):
            S = np.exp(-np.exp(A_log[h]) * dt[t, h]) * S + dt[t, h] * np.outer(B[t, g], x[t, h])
            y[t, h] = S.T @ C[t, g] + D[h] * x[t, h]
    return y


def ssd(h, w, p, mx, eps):
    T = h.shape[0]
    H, P, N, G = (int(mx[k]) for k in ("heads", "vdim", "state", "groups"))
    inner, parts = H * P, int(mx["norm_groups"])
    z, xbc, dt = np.split(h @ w[p + "in"].T, [inner, 2 * inner + 2 * G * N], axis=1)
    xbc = causal_conv(xbc, w[p + "conv"], w[p + "conv.b"])
    x, B, C = np.split(xbc, [inner, inner + G * N], axis=1)
    y = ssd_scan(x.reshape(T, H, P), B.reshape(T, G, N), C.reshape(T, G, N),
                 softplus(dt + w[p + "dt_bias"]), w[p + "A_log"], w[p + "D"])
    y = y.reshape(T, inner) * silu(z)
    y = rms(y.reshape(T, parts, inner // parts), eps).reshape(T, inner) * w[p + "norm"]
    return y @ w[p + "o"].T


# ----------------------------------------------------------------------------- side by side
def parallel_sides(h, w, p, mx, eps):
    l = p + "left."
    o = attend(h, w, l, mx["left"], True, keys_values(h, w, l, mx["left"], True))
    return (o * sigmoid(h @ w[l + "g"].T)) @ w[l + "o"].T, ssd(h, w, p + "right.", mx["right"], eps)


def parallel(h, w, p, mx, eps):
    a, b = parallel_sides(h, w, p, mx, eps)
    return 0.5 * (rms(a, eps) * w[p + "left.out"] + rms(b, eps) * w[p + "right.out"])


# ----------------------------------------------------------------------------- feed-forward
def dense_ff(h, w, p):
    return (np.maximum(h @ w[p + "gate"].T, 0.0) * (h @ w[p + "up"].T)) @ w[p + "down"].T


def expert(h, w, p):
    return (silu(h @ w[p + "gate"].T) * (h @ w[p + "up"].T)) @ w[p + "down"].T


def router(h, w, p, top):
    """(chosen experts, their sigmoid scores) [T, top]."""
    s = sigmoid(h @ w[p + "router"].T)
    ids = np.argsort(-s, -1, kind="stable")[:, :top]
    return ids, np.take_along_axis(s, ids, -1)


def moe(h, w, p, mlp):
    """The score of a chosen expert multiplies what goes into it."""
    ids, s = router(h, w, p, int(mlp["router"]["top"]))
    out = np.zeros_like(h)
    for t in range(h.shape[0]):
        for e, v in zip(ids[t], s[t]):
            out[t] += expert(v * h[t:t + 1], w, f"{p}e{e}.")[0]
    if mlp.get("shared"):
        out = out + expert(h, w, p + "shared.")
    return out


def router_margin(h, w, p, top):
    """By how much the least chosen score beats the best one that was not chosen."""
    s = np.sort(sigmoid(h @ w[p + "router"].T), -1)[:, ::-1]
    return s[:, top - 1] - s[:, top] if top < s.shape[1] else np.full(h.shape[0], np.inf)


# ----------------------------------------------------------------------------- the model
def forward(c, w, tokens, trace=None, margins=None):
    """Logits [T, vocab] of one sequence; ``trace`` (a list) receives the residual stream after
    every layer, ``margins`` the routers' margins per routed layer."""
    eps = float(c["norm"]["eps"])
    x = w["embed"][np.asarray(tokens)] * float(c["embedding"]["scale"])
    shared = {}
    for i, L in enumerate(c["layers"]):
        a, mx = f"l{i}.", L["mixer"]
        h = norm(x, w[a + "norm1"], eps)
        if L["type"] == "attention":
            y, shared[i] = attention(h, w, a + "mix.", mx, eps, shared)
        else:
            y = parallel(h, w, a + "mix.", mx, eps)
        x = x + norm(y, w[a + "norm1b"], eps)
        if L.get("mlp"):
            h = norm(x, w[a + "norm2"], eps)
            if L["mlp"]["kind"] == "dense":
                y = dense_ff(h, w, a + "mlp.")
            else:
                y = moe(h, w, a + "mlp.", L["mlp"])
                if margins is not None:
                    margins.append(router_margin(h, w, a + "mlp.", int(L["mlp"]["router"]["top"])))
            x = x + norm(y, w[a + "norm2b"], eps)
        if trace is not None:
            trace.append(x.copy())
    return norm(x, w["final.norm"], eps) @ w["head"].T
