"""Plain float64 implementation of the Generax decoder, one function per mechanism, whole
sequences at a time.  It shares no code with the package: numpy only, weights as a dict of
float64 arrays under the checkpoint's tensor names, the configuration as the dict that
config.json holds.

  x = embed[token]
  per layer:  h = rms(x) * norm1;   x += mixer(h) + ff(h)
  logits = c * tanh(head @ (rms(x) * final.norm) / c)              (c: logit_softcap)
with rms(v) = v / sqrt(mean(v^2) + eps).
"""
from __future__ import annotations

import numpy as np


def rms(v, eps):
    return v / np.sqrt((v * v).mean(-1, keepdims=True) + eps)


def sigmoid(z):
    return 1.0 / (1.0 + np.exp(-z))


def silu(z):
    return z * sigmoid(z)


def softplus(z):
    return np.logaddexp(0.0, z)


def softcap(z, c):
    return c * np.tanh(z / c) if c else z


def gated_ff(h, W, p):
    return (silu(h @ W[p + "gate"].T) * (h @ W[p + "up"].T)) @ W[p + "down"].T


# ------------------------------------------------------------------ attention
def rotate_halves(x, pos, dims, base, factor=1.0, sign=1.0):
    """x [T, heads, n]: dimension i < dims/2 of a head pairs with i + dims/2 and turns by
    sign * pos * base^(-2 i / dims) / factor; dimensions from ``dims`` on pass unchanged."""
    half = dims // 2
    f = base ** (-2.0 * np.arange(half) / dims) / factor
    a = sign * pos[:, None, None] * f
    u, v = x[..., :half], x[..., half:dims]
    return np.concatenate([u * np.cos(a) - v * np.sin(a), v * np.cos(a) + u * np.sin(a),
                           x[..., dims:]], -1)


def visible_window(T, size):
    """[T, T] bool: i sees j when 0 <= i - j < size (size 0: every j <= i)."""
    d = np.arange(T)[:, None] - np.arange(T)[None, :]
    return (d >= 0) & ((d < size) if size else True)


def pooled_blocks(x, pool):
    """x [T, G, n] -> [T // pool, G, n]: means of whole blocks of ``pool`` tokens."""
    n = x.shape[0] // pool
    return x[: n * pool].reshape(n, pool, *x.shape[1:]).mean(1)


def visible_blocks(T, size, pool):
    """[T, T // pool] bool: i sees block b when its last token lies before i's window."""
    last = np.arange(T // pool) * pool + pool - 1
    return last[None, :] <= np.arange(T)[:, None] - size


def attend(q, k, v, vis, scale):
    """q [T, H, d]; k [N, G, d], v [N, G, dv], vis [T, N]; scale a number or [H]."""
    T, H, _ = q.shape
    g = np.arange(H) // (H // k.shape[1])
    s = np.einsum("thd,nhd->htn", q, k[:, g]) * np.broadcast_to(scale, (H,))[:, None, None]
    s = np.where(vis[None], s, -np.inf)
    w = np.exp(s - s.max(-1, keepdims=True))
    w /= w.sum(-1, keepdims=True)
    return np.einsum("htn,nhv->thv", w, v[:, g])


def queries(h, W, p, m, eps):
    return (rms(h @ W[p + "q"].T, eps) * W[p + "q.norm"]).reshape(-1, m["heads"], m["dim"])


def keys(h, W, p, m, eps):
    return (rms(h @ W[p + "k"].T, eps) * W[p + "k.norm"]).reshape(-1, m["kv_heads"], m["dim"])


def pooled_attention(h, W, p, m, eps):
    T = h.shape[0]
    q, k = queries(h, W, p, m, eps), keys(h, W, p, m, eps)
    v = (h @ W[p + "v"].T).reshape(T, m["kv_heads"], m["vdim"])
    size, pool = m["mask"]["size"], m["mask"]["pool"]
    o = attend(q, np.concatenate([k, pooled_blocks(k, pool)]),
               np.concatenate([v, pooled_blocks(v, pool)]),
               np.concatenate([visible_window(T, size), visible_blocks(T, size, pool)], 1),
               m["scale"])
    return o.reshape(T, -1) @ W[p + "o"].T


def rotary_attention(h, W, p, m, eps, kv):
    """kv: None, or the rotated (k, v) of the layer whose cache this one reads.  Returns
    (output, (k, v))."""
    T = h.shape[0]
    pos = np.arange(T, dtype=np.float64)
    rot = m["rot"]
    base, factor = rot["base"], rot.get("scaling", {}).get("factor", 1.0)
    q = rotate_halves(queries(h, W, p, m, eps), pos, rot["dims"], base, factor)
    if kv is None:
        k = rotate_halves(keys(h, W, p, m, eps), pos, rot["dims"], base, factor)
        v = (h @ W[p + "v"].T).reshape(T, m["kv_heads"], m["vdim"])
        kv = k, rotate_halves(v, pos, m["vdim"], base)
    o = attend(q, *kv, visible_window(T, m["mask"]["size"]), m["scale"] * W[p + "temp"])
    o = rotate_halves(o, pos, m["vdim"], base, sign=-1.0)
    return o.reshape(T, -1) @ W[p + "o"].T, kv


# ------------------------------------------------------------------ gated delta rule
def causal_conv(u, w):
    """u [T, C], w [C, K]: y[t] = sum_j w[:, j] * u[t - (K - 1) + j], zeros before t = 0."""
    T, C = u.shape
    K = w.shape[1]
    pad = np.concatenate([np.zeros((K - 1, C)), u], 0)
    y = np.zeros((T, C))
    for j in range(K):
        y += pad[j:j + T] * w[:, j]
    return y


def unit(x):
    return x / np.sqrt((x * x).sum(-1, keepdims=True) + 1e-6)


def delta_scan(q, k, v, beta, g):
    """q, k [T, H, d], v [T, H, dv], beta [T, H], g [T, H, d]:
    S = diag(g) S;  u = beta (v - S^T k);  S = S + k u^T;  o = S^T q  ->  [T, H, dv]."""
    T, H, d = q.shape
    S = np.zeros((H, d, v.shape[2]))
    o = np.zeros((T, H, v.shape[2]))
    for t in range(T):
        S = g[t][:, :, None] * S
        u = beta[t][:, None] * (v[t] - np.einsum("hdv,hd->hv", S, k[t]))
        S = S + k[t][:, :, None] * u[:, None, :]
        o[t] = np.einsum("hdv,hd->hv", S, q[t])
    return o


def channel_decay(h, W, p, m):
    z = (h @ W[p + "a1"].T) @ W[p + "a2"].T + W[p + "dt_bias"]
    return np.exp(-np.exp(W[p + "A_log"])[:, None] *
                  softplus(z).reshape(-1, m["heads"], m["dim"]))


def delta_mixer(h, W, p, m, eps):
    T = h.shape[0]
    H, G, d, dv = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q, k, v = (silu(causal_conv(h @ W[p + n].T, W[p + n + ".conv"])) for n in "qkv")
    of = np.arange(H) // (H // G)
    q = unit(q.reshape(T, G, d))[:, of] * d ** -0.5
    k = unit(k.reshape(T, G, d))[:, of]
    o = delta_scan(q, k, v.reshape(T, H, dv), sigmoid(h @ W[p + "b"].T), channel_decay(h, W, p, m))
    gate = sigmoid((h @ W[p + "g1"].T) @ W[p + "g2"].T)
    return ((rms(o, eps) * W[p + "norm"]).reshape(T, H * dv) * gate) @ W[p + "o"].T


# ------------------------------------------------------------------ the model
def forward(cfg, W, tokens, taps=None):
    """-> logits [T, vocab]; ``taps``: the stream after every layer is appended."""
    eps = cfg["norm"]["eps"]
    x = W["embed"][np.asarray(tokens)]
    cached = {}
    for i, L in enumerate(cfg["layers"]):
        p, m = f"l{i}.", L["mixer"]
        h = rms(x, eps) * W[p + "norm1"]
        if L["type"] == "parallel":
            left = pooled_attention(h, W, p + "mix.left.", m["left"], eps)
            right = delta_mixer(h, W, p + "mix.right.", m["right"], eps)
            y = 0.5 * (rms(left, eps) * W[p + "mix.left.out"] + rms(right, eps) * W[p + "mix.right.out"])
        else:
            y, cached[i] = rotary_attention(h, W, p + "mix.", m, eps, cached.get(m.get("kv_from")))
        if L.get("mlp"):
            y = y + gated_ff(h, W, p + "mlp.")
        x = x + y
        if taps is not None:
            taps.append(x.copy())
    return softcap((rms(x, eps) * W["final.norm"]) @ W["head"].T, cfg.get("logit_softcap", 0.0))


# ------------------------------------------------------------------ random weights
def random_weights(cfg, seed):
    """float64 arrays under the checkpoint's names, rounded to bfloat16 values.  The ranks of
    the low-rank projections come from the mixer's "_a_rank" / "_g_rank" entries."""
    rng = np.random.default_rng(seed)
    W = {}

    def put(name, shape, scale, base=0.0):
        v = (rng.standard_normal(shape) * scale + base).astype(np.float32)
        u = v.view(np.uint32)
        u = (u + 0x7FFF + ((u >> 16) & 1)) & np.uint32(0xFFFF0000)
        W[name] = u.view(np.float32).astype(np.float64)
    w = cfg["width"]
    lin = w ** -0.5
    put("embed", (cfg["vocab"], w), 1.0)
    put("head", (cfg["vocab"], w), 3.0 * lin)
    put("final.norm", (w,), 0.2, 1.0)

    def attention(p, m, own_kv, temp):
        H, G, d, dv = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
        put(p + "q", (H * d, w), lin)
        put(p + "q.norm", (H * d,), 0.3, 1.0)
        if own_kv:
            put(p + "k", (G * d, w), lin)
            put(p + "k.norm", (G * d,), 0.3, 1.0)
            put(p + "v", (G * dv, w), lin)
        if temp:
            put(p + "temp", (H,), 0.3, 1.2)
        put(p + "o", (w, H * dv), (H * dv) ** -0.5)
    for i, L in enumerate(cfg["layers"]):
        p, m = f"l{i}.", L["mixer"]
        put(p + "norm1", (w,), 0.2, 1.0)
        if L["type"] == "parallel":
            attention(p + "mix.left.", m["left"], True, False)
            r, q = m["right"], p + "mix.right."
            H, G, d, dv, K = r["heads"], r["kv_heads"], r["dim"], r["vdim"], r["conv"]
            for n, c in (("q", G * d), ("k", G * d), ("v", H * dv)):
                put(q + n, (c, w), 2.0 * lin)
                put(q + n + ".conv", (c, K), 0.6)
            put(q + "b", (H, w), lin)
            put(q + "A_log", (H,), 0.5)
            put(q + "norm", (dv,), 0.2, 1.0)
            ra, rg = r["_a_rank"], r["_g_rank"]
            put(q + "a1", (ra, w), lin)
            put(q + "a2", (H * d, ra), ra ** -0.5)
            put(q + "dt_bias", (H * d,), 1.0, -3.0)
            put(q + "g1", (rg, w), lin)
            put(q + "g2", (H * dv, rg), rg ** -0.5)
            put(q + "o", (w, H * dv), (H * dv) ** -0.5)
            put(p + "mix.left.out", (w,), 0.2, 1.0)
            put(p + "mix.right.out", (w,), 0.2, 1.0)
        else:
            attention(p + "mix.", m, m.get("kv_from") is None, True)
        if L.get("mlp"):
            ff = L["mlp"]["ff"]
            put(p + "mlp.gate", (ff, w), lin)
            put(p + "mlp.up", (ff, w), lin)
            put(p + "mlp.down", (w, ff), ff ** -0.5)
    return W
