"""Plain float64 implementation of the Ratizen decoder, one function per mechanism, whole
sequences at a time.  It shares no code with the package: numpy only, weights as a dict of
float64 arrays under the checkpoint's tensor names, the configuration as the dict that
config.json holds.

  X[s] = embed[token] * scale for every stream s
  per sublayer (mixer, then feed-forward; hc = hc1 / hc2, norm = norm1 / norm2):
    u = sum_s in[s] X[s];   y = sublayer(rms(u) (1 + norm))
    X'[t] = sum_s mix[s, t] X[s] + m out[t] y
  logits = logit_scale * head (rms(sum_s X[s]) (1 + final.norm))
with rms(v) = v / sqrt(mean(v^2) + eps).
"""
from __future__ import annotations

import math

import numpy as np


def rms(v, eps):
    return v / np.sqrt((v * v).mean(-1, keepdims=True) + eps)


def sigmoid(z):
    return 1.0 / (1.0 + np.exp(-z))


def silu(z):
    return z * sigmoid(z)


# ------------------------------------------------------------------ hyper-connections
def combine_in(X, w):
    """X [S, T, W], w [S] -> what a sublayer reads."""
    return np.tensordot(w, X, axes=(0, 0))


def combine_out(X, y, mix, out, m):
    """Every stream anew from all old ones (mix [from, to]) and the sublayer's result."""
    return np.stack([np.tensordot(mix[:, t], X, axes=(0, 0)) + m * out[t] * y
                     for t in range(X.shape[0])])


# ------------------------------------------------------------------ visibility
def visible_chunks(T, size):
    """[T, T] bool: i sees j <= i in the same chunk of ``size`` positions (0: every j <= i)."""
    i, j = np.arange(T)[:, None], np.arange(T)[None, :]
    return (j <= i) & ((i // size == j // size) if size else True)


def visible_window(T, size):
    """[T, T] bool: i sees j when 0 <= i - j < size (size 0: every j <= i)."""
    d = np.arange(T)[:, None] - np.arange(T)[None, :]
    return (d >= 0) & ((d < size) if size else True)


def weights_with_sink(s):
    """Softmax over the last axis with 1 added to the denominator (hidden scores are -inf)."""
    top = np.maximum(s.max(-1, keepdims=True), 0.0)
    e = np.exp(s - top)
    return e / (np.exp(-top) + e.sum(-1, keepdims=True))


def weights_plain(s):
    e = np.exp(s - s.max(-1, keepdims=True))
    return e / e.sum(-1, keepdims=True)


# ------------------------------------------------------------------ mixers
def mask_size(m):
    return m["mask"]["size"] if m.get("mask") else 0


def attention(h, wts, P, m, eps):
    T = h.shape[0]
    H, G, d, dv = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q = rms((h @ wts[P + "q"].T).reshape(T, H, d), eps) * wts[P + "q.norm"]
    k = rms((h @ wts[P + "k"].T).reshape(T, G, d), eps) * wts[P + "k.norm"]
    v = (h @ wts[P + "v"].T).reshape(T, G, dv)
    vis = visible_chunks(T, mask_size(m))
    o = np.zeros((T, H, dv))
    for a in range(H):
        g = a // (H // G)
        s = np.where(vis, q[:, a] @ k[:, g].T * m["scale"], -np.inf)
        o[:, a] = weights_with_sink(s) @ v[:, g]
    return o.reshape(T, H * dv) @ wts[P + "o"].T


def yarn_frequencies(dims, base, scaling):
    """Angular frequency of every pair, and the factor on cos and sin."""
    i = np.arange(dims // 2)
    f = float(base) ** (-2.0 * i / dims)
    if not scaling:
        return f, 1.0

    def dim_of(turns):
        return dims * math.log(scaling["original"] / (2 * math.pi * turns)) / (2 * math.log(base))
    lo = max(math.floor(dim_of(scaling["fast"])), 0)
    hi = min(math.ceil(dim_of(scaling["slow"])), dims - 1)
    ramp = np.clip((i - lo) / max(hi - lo, 0.001), 0.0, 1.0)
    return f / scaling["factor"] * ramp + f * (1.0 - ramp), 0.1 * math.log(scaling["factor"]) + 1.0


def rotate_pairs(x, pos, rot):
    """x [T, ..., dims]: (x[2i], x[2i + 1]) turns by pos * f_i."""
    f, mag = yarn_frequencies(rot["dims"], rot["base"], rot.get("scaling"))
    a = (pos[:, None] * f).reshape((x.shape[0],) + (1,) * (x.ndim - 2) + (-1,))
    c, s = np.cos(a) * mag, np.sin(a) * mag
    u, v = x[..., 0::2], x[..., 1::2]
    out = np.empty_like(x)
    out[..., 0::2] = u * c - v * s
    out[..., 1::2] = v * c + u * s
    return out


def latent_attention(h, wts, P, m, eps):
    T = h.shape[0]
    H, d, r, dv, rank = m["heads"], m["dim"], m["rot_dim"], m["vdim"], m["kv_rank"]
    pos = np.arange(T, dtype=np.float64)
    cq = rms(h @ wts[P + "dq"].T, eps) * wts[P + "dq.norm"]
    q = (cq @ wts[P + "uq"].T).reshape(T, H, d + r)
    down = h @ wts[P + "dkv"].T
    c = rms(down[:, :rank], eps) * wts[P + "dkv.norm"]
    kr = rotate_pairs(down[:, rank:], pos, m["rot"])
    qr = rotate_pairs(q[..., d:], pos, m["rot"])
    k = (c @ wts[P + "uk"].T).reshape(T, H, d)
    v = (c @ wts[P + "uv"].T).reshape(T, H, dv)
    gate = sigmoid(h @ wts[P + "g"].T)
    vis = visible_window(T, mask_size(m))
    o = np.zeros((T, H, dv))
    for a in range(H):
        s = np.where(vis, (q[:, a, :d] @ k[:, a].T + qr[:, a] @ kr.T) * m["scale"], -np.inf)
        o[:, a] = weights_plain(s) @ v[:, a] * gate[:, a: a + 1]
    return o.reshape(T, H * dv) @ wts[P + "o"].T


# ------------------------------------------------------------------ feed-forward
def gated(h, wts, p):
    return (silu(h @ wts[p + "gate"].T) * (h @ wts[p + "up"].T)) @ wts[p + "down"].T


def route(h, router, top):
    """-> ids [T, top] of the largest scores (the lower index first among equals), scores
    [T, top], and how close each token's decision was: the gap between the last chosen and the
    first unchosen logit over the largest logit."""
    z = h @ router.T
    order = np.argsort(-z, axis=-1, kind="stable")
    ranked = np.take_along_axis(z, order, -1)
    gap = np.full(len(z), np.inf)
    if top < z.shape[1]:
        gap = (ranked[:, top - 1] - ranked[:, top]) / np.abs(z).max(-1)
    return order[:, :top], sigmoid(ranked[:, :top]), gap


def experts(h, wts, P, mlp, gaps=None):
    ids, w, gap = route(h, wts[P + "router"], mlp["router"]["top"])
    if gaps is not None:
        gaps.append(gap)
    out = np.zeros_like(h)
    for e in range(mlp["router"]["experts"]):
        t, j = np.nonzero(ids == e)
        if len(t):
            out[t] += gated(h[t] * w[t, j][:, None], wts, P + "e%d." % e)
    if mlp.get("shared"):
        out += gated(h, wts, P + "shared.")
    return out


# ------------------------------------------------------------------ the model
MIXERS = {"attention": attention, "latent_attention": latent_attention}


def forward(cfg, wts, tokens, taps=None, gaps=None):
    """-> logits [T, vocab]; ``taps`` receives the sum of the streams after every layer,
    ``gaps`` the routing gaps of every routed layer."""
    eps, m = cfg["norm"]["eps"], cfg["residual_mult"]
    e = wts["embed"][np.asarray(tokens)] * cfg["embedding"]["scale"]
    X = np.stack([e] * cfg["streams"])
    for i, lay in enumerate(cfg["layers"]):
        L = "l%d." % i
        subs = [("1", lambda h: MIXERS[lay["type"]](h, wts, L + "mix.", lay["mixer"], eps))]
        if lay.get("mlp"):
            subs.append(("2", lambda h: experts(h, wts, L + "mlp.", lay["mlp"], gaps)))
        for n, f in subs:
            u = combine_in(X, wts[L + "hc%s.in" % n])
            y = f(rms(u, eps) * (1.0 + wts[L + "norm" + n]))
            X = combine_out(X, y, wts[L + "hc%s.mix" % n], wts[L + "hc%s.out" % n], m)
        if taps is not None:
            taps.append(X.sum(0))
    return (rms(X.sum(0), eps) * (1.0 + wts["final.norm"])) @ wts["head"].T * cfg["logit_scale"]


# ------------------------------------------------------------------ random checkpoints
def tensor_shapes(cfg):
    """Checkpoint names -> shapes."""
    W, S = cfg["width"], cfg["streams"]
    out = {"embed": (cfg["vocab"], W), "head": (cfg["vocab"], W), "final.norm": (W,)}
    for i, lay in enumerate(cfg["layers"]):
        L, m, f = "l%d." % i, lay["mixer"], lay.get("mlp")
        for n in ("1", "2") if f else ("1",):
            out.update({L + "norm" + n: (W,), L + "hc%s.in" % n: (S,), L + "hc%s.out" % n: (S,),
                        L + "hc%s.mix" % n: (S, S)})
        P, H = L + "mix.", m["heads"]
        if lay["type"] == "attention":
            G, d, dv = m["kv_heads"], m["dim"], m["vdim"]
            out.update({P + "q": (H * d, W), P + "k": (G * d, W), P + "v": (G * dv, W),
                        P + "q.norm": (d,), P + "k.norm": (d,), P + "o": (W, H * dv)})
        else:
            d, r, dv, rank, qr = m["dim"], m["rot_dim"], m["vdim"], m["kv_rank"], m["q_rank"]
            out.update({P + "dq": (qr, W), P + "dq.norm": (qr,), P + "uq": (H * (d + r), qr),
                        P + "dkv": (rank + r, W), P + "dkv.norm": (rank,), P + "uk": (H * d, rank),
                        P + "uv": (H * dv, rank), P + "g": (H, W), P + "o": (W, H * dv)})
        if f:
            P, E = L + "mlp.", f["router"]["experts"]
            out[P + "router"] = (E, W)
            ffs = [("e%d." % e, f["expert"]["ff"]) for e in range(E)]
            if f.get("shared"):
                ffs.append(("shared.", f["shared"]["ff"]))
            for n, ff in ffs:
                out.update({P + n + "gate": (ff, W), P + n + "up": (ff, W), P + n + "down": (W, ff)})
    return out


def bf16(a):
    """Round-to-nearest-even bf16 values, as float64."""
    b = np.ascontiguousarray(a, dtype=np.float32).view(np.uint32)
    b = (b + 0x7FFF + ((b >> 16) & 1)) & np.uint32(0xFFFF0000)
    return b.view(np.float32).astype(np.float64)


def random_weights(cfg, seed):
    """bf16-valued random weights.  The routers decide on a code of the token: the first
    columns of the stream (as many as the largest router has outputs) hold a permutation of
    spaced levels that no sublayer writes to, so no routing decision is close and rounding cannot
    turn one; all other mechanisms see random data."""
    rng = np.random.default_rng(seed)
    S, V = cfg["streams"], cfg["vocab"]
    C = max([lay["mlp"]["router"]["experts"] for lay in cfg["layers"] if lay.get("mlp")] or [0])
    wts = {}
    for name, shape in tensor_shapes(cfg).items():
        leaf = name.split(".", 1)[-1]
        z = rng.normal(size=shape)
        if leaf in ("hc1.in", "hc2.in"):
            w = rng.uniform(0.4, 1.6, shape) / S
        elif leaf in ("hc1.out", "hc2.out"):
            w = 1.0 + 0.4 * z
        elif leaf in ("hc1.mix", "hc2.mix"):
            w = 0.75 * np.eye(S) + rng.uniform(0.0, 0.5, shape) / S
        elif leaf in ("norm1", "norm2") or name == "final.norm":
            w = 0.2 * z
            w[:C] = 0.0
        elif len(shape) == 1:
            w = 1.0 + 0.3 * z
        elif name == "embed":
            w = z
            w[:, :C] = np.stack([rng.permutation(np.linspace(-2.0, 2.0, C)) for _ in range(V)]) if C else 0
        elif leaf.endswith("router"):
            w = np.zeros(shape)
            w[np.arange(shape[0]), rng.permutation(C)[: shape[0]]] = 2.5
        else:
            w = 1.3 * z / np.sqrt(shape[1])
            if C and shape[0] == cfg["width"] and (leaf.endswith(".o") or leaf.endswith("down")):
                w[:C] = 0.0
        wts[name] = bf16(w)
    return wts
