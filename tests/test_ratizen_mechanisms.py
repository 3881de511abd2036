"""Each mechanism of the Ratizen decoder alone (the product's op or module) against the numpy
oracle's function for it, on the CPU reference ops and, with ``-m gpu``, on the HIP kernels:
hyper-connections, per-head norms, chunks and the sink with a planted stand-out key at every
edge, YaRN frequencies, latent attention over portions of every size, one matrix per head,
routing, experts on scaled inputs in both of their forms."""
import types

import numpy as np
import pytest
import torch

import ratizen_oracle as oracle
from kubernetes_gpu_cluster_amd import ops
from kubernetes_gpu_cluster_amd.models.attention import (AttentionCore, ForwardContext,
                                                         LatentQueryAttention)
from kubernetes_gpu_cluster_amd.models.configs import (FeedForwardSpec, MixerSpec, RotarySpec,
                                                       WindowSpec)
from kubernetes_gpu_cluster_amd.models.moe import InputScaledExperts

DEV = [pytest.param("cpu", id="cpu"), pytest.param("cuda", marks=pytest.mark.gpu, id="gpu")]
GPU = [pytest.param("cuda", marks=pytest.mark.gpu, id="gpu")]
KINDS = [pytest.param("cpu", torch.float32, id="cpu-fp32"),
         pytest.param("cuda", torch.float32, marks=pytest.mark.gpu, id="gpu-fp32"),
         pytest.param("cuda", torch.bfloat16, marks=pytest.mark.gpu, id="gpu-bf16")]


def dev_of(name):
    if name == "cuda" and not torch.cuda.is_available():
        pytest.skip("no GPU")
    return torch.device(name)


def f32(a, dev):
    return torch.tensor(np.ascontiguousarray(a), dtype=torch.float32, device=dev).contiguous()


def rel(got, want):
    """Largest row error: rms of the difference over the rms of all of ``want``."""
    got = got.float().cpu().numpy() if torch.is_tensor(got) else got
    want = np.asarray(want, dtype=np.float64)
    d = (got.astype(np.float64) - want).reshape(want.shape[0], -1)
    return np.sqrt((d ** 2).mean(-1)).max() / np.sqrt((want ** 2).mean())


def tol(dtype, fp32=3e-6, bf16=2e-2):
    return fp32 if dtype == torch.float32 else bf16


def meta_for(lo, hi, table, slots, dev):
    """One sequence's positions [lo, hi): a prefill chunk, or a decode row."""
    m = types.SimpleNamespace()
    i32 = lambda v: torch.tensor(v, dtype=torch.int32, device=dev)   # noqa: E731
    dec = hi - lo == 1 and lo > 0
    m.num_prefills, m.num_decodes, m.num_prefill_tokens = int(not dec), int(dec), 0 if dec else hi - lo
    m.query_start_loc = None if dec else i32([0, hi - lo])
    m.prefill_seq_lens = None if dec else i32([hi])
    m.prefill_block_tables = None if dec else table
    m.decode_ctx_lens = i32([hi]) if dec else None
    m.decode_block_tables = table if dec else None
    m.state_slots = m.work_seq = m.work_mblk = None
    m.slot_mapping = slots
    return m, torch.arange(lo, hi, dtype=torch.int64, device=dev)


def portions(n, cuts):
    out, lo, i = [], 0, 0
    while lo < n:
        hi = min(n, lo + cuts[min(i, len(cuts) - 1)])
        out.append((lo, hi))
        lo, i = hi, i + 1
    return out


class Pages:
    """Pages handed out in a scrambled order, filled with leftovers of other requests."""

    def __init__(self, n, page, dev):
        self.page, self.dev = page, dev
        k = -(-n // page)
        self.n = k + 1
        self.order = np.random.default_rng(5).permutation(k) + 1
        self.table = torch.tensor([self.order.tolist()], dtype=torch.int32, device=dev)

    def cache(self, groups, width, dtype, fill):
        return torch.full((self.n, groups, self.page, width), fill, dtype=dtype, device=self.dev)

    def slots(self, lo, hi):
        return torch.tensor([int(self.order[p // self.page]) * self.page + p % self.page
                             for p in range(lo, hi)], dtype=torch.int64, device=self.dev)


# ---------------------------------------------------------------- hyper-connections
@pytest.mark.parametrize("device,dtype", KINDS)
@pytest.mark.parametrize("S,W", [(1, 64), (2, 72), (3, 70), (4, 256), (4, 1500), (4, 3000), (4, 5000),
                                 (6, 96), (9, 33)])
def test_hyper_connection(device, dtype, S, W):
    """Reading, writing back and the norm, over signed and asymmetric mixes; the result comes as
    one row per token, as several, and as fp32 partial sums."""
    dev, T, rng = dev_of(device), 5, np.random.default_rng(S * W)
    X, mix = rng.normal(size=(S, T, W)), rng.normal(size=(S, S))
    w_in, w_out, w = rng.normal(size=S), rng.normal(size=S), rng.normal(size=W)
    rows = oracle.bf16(rng.normal(size=(T, 3, W)))
    parts = rng.normal(size=(2, T * 2, W))
    y = rows.sum(1) + parts.sum(0).reshape(T, 2, W).sum(1)
    adds = [(f32(rows.reshape(T * 3, W), dev).to(dtype), 3), (f32(parts, dev), 2)]
    new = oracle.combine_out(X, y, mix, w_out, 1.0)
    want = oracle.rms(oracle.combine_in(new, w_in), 1e-5) * w
    x = f32(X.transpose(1, 0, 2), dev)
    args = (adds, f32(mix, dev), f32(w_out, dev), f32(w_in, dev), f32(w, dev), 1e-5, dtype)
    dst = torch.full_like(x, 7.0)
    h = ops.hyper_norm(x, dst, *args)
    assert rel(dst.permute(1, 0, 2).contiguous(), new) < 1e-6
    assert rel(h, want) < tol(dtype, bf16=1e-2)
    # without a place to write, and in place
    before = x.clone()
    h2 = ops.hyper_norm(x, None, *args)
    assert torch.equal(x, before) and torch.equal(h2, h)
    ops.hyper_norm(x, x, *args)
    assert torch.equal(x, dst)
    # only one addend; the plain combination in fp32, and no output at all
    x2 = before.clone()
    u = ops.hyper_norm(x2, x2, adds[:1], *args[1:4], None, 1e-5, torch.float32)
    new1 = oracle.combine_out(X, rows.sum(1), mix, w_out, 1.0)
    assert rel(u, oracle.combine_in(new1, w_in)) < 1e-6
    assert ops.hyper_norm(before.clone(), x2, adds[:1], *args[1:4], None, 1e-5, None) is None
    assert rel(x2.permute(1, 0, 2).contiguous(), new1) < 1e-6


@pytest.mark.parametrize("device,dtype", KINDS)
def test_streams_that_start_alike(device, dtype):
    """All streams equal at the start: one row per token read S times."""
    dev, rng, T, S, W = dev_of(device), np.random.default_rng(4), 6, 4, 96
    e, w_in, w = rng.normal(size=(T, W)), rng.normal(size=S), rng.normal(size=W)
    mix, w_out, y = rng.normal(size=(S, S)), rng.normal(size=S), oracle.bf16(rng.normal(size=(T, W)))
    src = f32(e, dev)[:, None, :].expand(T, S, W)
    X = np.stack([e] * S)
    h = ops.hyper_norm(src, None, [], None, None, f32(w_in, dev), f32(w, dev), 1e-6, dtype)
    assert rel(h, oracle.rms(oracle.combine_in(X, w_in), 1e-6) * w) < tol(dtype)
    dst = torch.empty(T, S, W, device=dev)
    ops.hyper_norm(src, dst, [(f32(y, dev).to(dtype), 1)], f32(mix, dev), f32(w_out, dev), f32(w_in, dev),
                   f32(w, dev), 1e-6, dtype)
    assert rel(dst.permute(1, 0, 2).contiguous(), oracle.combine_out(X, y, mix, w_out, 1.0)) < 1e-6


# ---------------------------------------------------------------- chunked attention, head norms, sink
class Chunked:
    """AttentionCore over scrambled pages; q | k | v are given, the layer's output comes back."""

    def __init__(self, H, G, dk, dv, size, scale, dev, dtype, page=8, n=400, eps=1e-5, sink=0.0):
        sp = MixerSpec("attention", H, dk, dv, kv_heads=G, scale=scale, head_norm=True, sink=sink,
                       window=WindowSpec(size, chunked=True) if size else None)
        self.core, self.dtype, self.dev = AttentionCore(sp, 1.0, eps, dev), dtype, dev
        self.pages = Pages(n, page, dev)
        self.kv = (self.pages.cache(G, dk, dtype, 3.0), self.pages.cache(G, dv, dtype, -2.0))

    def run(self, q, k, v, qw, kw, cuts):
        self.core.q_norm.data.copy_(f32(qw, self.dev))
        self.core.k_norm.data.copy_(f32(kw, self.dev))
        proj = f32(np.concatenate([q, k, v], 1), self.dev).to(self.dtype)
        out = torch.empty(q.shape[0], self.core.n_out, dtype=self.dtype, device=self.dev)
        for lo, hi in portions(q.shape[0], cuts):
            m, pos = meta_for(lo, hi, self.pages.table, self.pages.slots(lo, hi), self.dev)
            self.core(proj[lo:hi], 0, pos, ForwardContext(m, [self.kv], block_size=self.pages.page), 0,
                      out[lo:hi])
        return out


def chunk_oracle(q, k, v, qw, kw, H, G, dk, dv, size, scale, eps=1e-5, sink=True):
    T = q.shape[0]
    q = oracle.rms(q.reshape(T, H, dk), eps) * qw
    k = oracle.rms(k.reshape(T, G, dk), eps) * kw
    v = v.reshape(T, G, dv)
    vis = oracle.visible_chunks(T, size)
    weigh = oracle.weights_with_sink if sink else oracle.weights_plain
    o = np.zeros((T, H, dv))
    for a in range(H):
        s = np.where(vis, q[:, a] @ k[:, a // (H // G)].T * scale, -np.inf)
        o[:, a] = weigh(s) @ v[:, a // (H // G)]
    return o.reshape(T, H * dv)


def qkv(rng, n, H, G, dk, dv):
    bf = lambda *s: oracle.bf16(rng.normal(size=s))      # noqa: E731
    return (bf(n, H * dk), bf(n, G * dk), bf(n, G * dv), rng.normal(size=dk) * 0.3 + 1,
            rng.normal(size=dk) * 0.3 + 1)


@pytest.mark.parametrize("device,dtype", KINDS)
@pytest.mark.parametrize("H,G,dk,dv,size,page", [(4, 2, 12, 10, 13, 8), (3, 3, 7, 5, 9, 5), (8, 2, 64, 32, 70, 16),
                                                 (8, 1, 56, 48, 64, 8), (16, 2, 128, 128, 50, 32),
                                                 (2, 2, 16, 16, 1, 8), (6, 2, 24, 16, 0, 8), (1, 1, 200, 64, 33, 8)])
def test_chunked_attention_with_sink(device, dtype, H, G, dk, dv, size, page):
    dev, rng, n, scale = dev_of(device), np.random.default_rng(dk + size), 170, 0.7 / np.sqrt(dk)
    data = qkv(rng, n, H, G, dk, dv)
    want = chunk_oracle(*data, H, G, dk, dv, size, scale)
    # the sink and the chunk's edges show in what is compared
    assert rel(chunk_oracle(*data, H, G, dk, dv, size, scale, sink=False), want) > 0.05
    if size:
        assert rel(chunk_oracle(*data, H, G, dk, dv, size + 1, scale), want) > 0.05
    for cuts in ([n], [70, 65, 3, 1], [2], [1]) if device == "cuda" else ([n], [61, 2, 40, 1]):
        att = Chunked(H, G, dk, dv, size, scale, dev, dtype, page=page)
        assert rel(att.run(*data, cuts), want) < tol(dtype), cuts


@pytest.mark.parametrize("device,dtype", KINDS)
@pytest.mark.parametrize("dk,size", [(16, 13), (64, 64), (64, 100)])
def test_planted_key_at_chunk_edges(device, dtype, dk, size):
    """One key whose score stands far above all others, at the first and the last place of a
    chunk and at page borders: the rows that see it, and only they, return its value."""
    dev, H, G, dv, n = dev_of(device), 4, 2, 16, 3 * size + 5
    rng = np.random.default_rng(size)
    q, k, v, qw, kw = qkv(rng, n, H, G, dk, dv)
    q = oracle.bf16(0.2 * q.reshape(n, H, dk) + 1.0).reshape(n, H * dk)      # all queries alike
    k = oracle.bf16(0.2 * k + np.tile([1.0, -1.0], G * dk // 2))
    one = np.ones(dk)
    for at in (size, 2 * size - 1, size + 8, size + 7, 0):
        k2 = k.copy()
        k2[at] = 1.0
        want = chunk_oracle(q, k2, v, one, one, H, G, dk, dv, size, 1.5)
        seen = [i for i in range(n) if at <= i < at // size * size + size]
        for cuts in ([n], [at + 1, 1], [size - 1, 2, size, 1]):
            got = Chunked(H, G, dk, dv, size, 1.5, dev, dtype).run(q, k2, v, one, one, cuts)
            assert rel(got, want) < tol(dtype, bf16=4e-2), (at, cuts)
            g = got.float().cpu().numpy().reshape(n, H, dv)
            for h in range(H):
                dist = np.abs(g[:, h] - v.reshape(n, G, dv)[at, h // 2]).max(-1)
                assert dist[seen].max() < 0.05
                assert dist[[i for i in range(n) if i not in seen]].min() > 0.2


@pytest.mark.parametrize("device,dtype", KINDS)
@pytest.mark.parametrize("sink", [0.0, 1.75, -3.0])
def test_sink_of_any_score_against_high_and_low_scores(device, dtype, sink):
    """Scores far below the sink give almost nothing, scores far above it ignore it."""
    dev, H, G, dk, dv, n = dev_of(device), 2, 1, 32, 16, 90
    rng = np.random.default_rng(7)
    _, _, v, _, _ = qkv(rng, n, H, G, dk, dv)
    for sign in (-1.0, 1.0):
        q, k = np.ones((n, H * dk)), np.tile(sign * np.ones(dk), (n, 1))
        vals = v.reshape(n, 1, dv)
        s = sign * dk * 0.3                                 # every visible key's score
        want = np.zeros((n, H, dv))
        for i in range(n):
            lo = i // 40 * 40
            m = i - lo + 1
            top = max(s, sink)
            p = np.exp(s - top) / (m * np.exp(s - top) + np.exp(sink - top))
            want[i] = p * vals[lo:i + 1].sum(0)
        for cuts in ([n], [33, 1]):
            att = Chunked(H, G, dk, dv, 40, 0.3, dev, dtype, sink=sink, eps=1e-9)
            got = att.run(q, k, v, np.ones(dk), np.ones(dk), cuts)
            assert rel(got, want.reshape(n, -1)) < tol(dtype, fp32=2e-5)


@pytest.mark.parametrize("device", GPU)
@pytest.mark.parametrize("size", [48, 100])
def test_fast_and_simple_attention_kernels_agree(device, size, monkeypatch):
    dev, H, G, dk, dv, n = dev_of(device), 8, 2, 72, 64, 300
    data = qkv(np.random.default_rng(1), n, H, G, dk, dv)
    for cuts in ([n], [150, 1]):
        fast = Chunked(H, G, dk, dv, size, 0.1, dev, torch.bfloat16).run(*data, cuts)
        monkeypatch.setenv("KGC_WINDOW_ATTN", "simple")
        simple = Chunked(H, G, dk, dv, size, 0.1, dev, torch.bfloat16).run(*data, cuts)
        monkeypatch.delenv("KGC_WINDOW_ATTN")
        assert rel(fast, simple.float().cpu().numpy()) < 5e-3


@pytest.mark.parametrize("device,dtype", KINDS)
@pytest.mark.parametrize("H,G,dk,dv", [(4, 2, 16, 8), (3, 1, 48, 40), (5, 5, 6, 9), (2, 2, 520, 16)])
def test_head_norms_and_padding_rows(device, dtype, H, G, dk, dv):
    """Per-head norms with one weight per dimension; a row without a slot leaves the cache alone."""
    dev, n = dev_of(device), 6
    q, k, v, qw, kw = qkv(np.random.default_rng(dk), n, H, G, dk, dv)
    proj = f32(np.concatenate([np.full((n, 8), 9.0), q, k, v], 1), dev).to(dtype)[:, 8:]
    kc = torch.zeros(2, G, 8, dk, dtype=dtype, device=dev)
    vc = torch.zeros(2, G, 8, dv, dtype=dtype, device=dev)
    slots = torch.tensor([9, 8, -1, 15, 3, 12], dtype=torch.int64, device=dev)
    pos = torch.arange(n, device=dev)
    got = ops.norm_kv_store(proj, pos, kc, vc, slots, H, G, dk, dv, 1e-4, True, False, None, dtype,
                            f32(qw, dev), f32(kw, dev))
    assert rel(got, oracle.rms(q.reshape(n, H, dk), 1e-4) * qw) < tol(dtype, bf16=1e-2)
    kn, vn = oracle.rms(k.reshape(n, G, dk), 1e-4) * kw, v.reshape(n, G, dv)
    for i, s in enumerate(slots.tolist()):
        if s >= 0:
            assert rel(kc[s // 8, :, s % 8], kn[i]) < tol(dtype, bf16=1e-2)
            assert rel(vc[s // 8, :, s % 8], vn[i]) < tol(dtype, bf16=1e-2)
    used = {s for s in slots.tolist() if s >= 0}
    for s in set(range(16)) - used:
        assert float(kc[s // 8, :, s % 8].float().abs().max()) == 0


# ---------------------------------------------------------------- latent attention
@pytest.mark.parametrize("dims,base,scaling", [
    (16, 1e4, None), (8, 500.0, (4.0, 128, 16.0, 1.0)), (64, 5e5, (8.0, 4096, 32.0, 1.0)),
    (2, 50.0, (3.0, 10, 2.0, 1.0)), (32, 100.0, (2.0, 16, 64.0, 32.0)), (12, 1e4, (1.0, 64, 32.0, 1.0))])
def test_yarn_table(dims, base, scaling):
    sc = dict(zip(("factor", "original", "fast", "slow"), scaling)) if scaling else None
    f, mag = oracle.yarn_frequencies(dims, base, sc)
    a = np.arange(5000)[:, None] * f
    got = ops.ref.rope_table_yarn(dims, 5000, base, scaling).double().numpy()
    np.testing.assert_allclose(got, np.concatenate([np.cos(a), np.sin(a)], 1) * mag, atol=2e-7)


LATENT = [dict(H=3, d=10, r=6, dv=14, rank=18, qr=22, size=11, W=40),
          dict(H=1, d=1, r=2, dv=3, rank=5, qr=1, size=1, W=24),
          dict(H=8, d=32, r=8, dv=48, rank=64, qr=40, size=37, W=128),
          dict(H=4, d=64, r=64, dv=64, rank=192, qr=96, size=70, W=128),
          dict(H=2, d=24, r=16, dv=16, rank=272, qr=64, size=0, W=64),
          dict(H=20, d=16, r=8, dv=16, rank=48, qr=32, size=50, W=64),
          dict(H=6, d=16, r=32, dv=24, rank=224, qr=32, size=33, W=64)]


def latent_module(c, scaling, dev, dtype, scale):
    rs = RotarySpec(c["r"], 300.0, interleaved=True, yarn=scaling)
    sp = MixerSpec("latent_attention", c["H"], c["d"], c["dv"], kv_heads=1, scale=scale, rot_dims=c["r"],
                   rotary=rs, window=WindowSpec(c["size"]) if c["size"] else None, kv_rank=c["rank"],
                   q_rank=c["qr"], head_gate=True)
    m = LatentQueryAttention(c["W"], sp, 1e-5, dtype, dev)
    m.prepare({}, 500, dev)
    return m


def latent_weights(c, seed):
    rng = np.random.default_rng(seed)
    H, d, r, dv, rank, qr, W = (c[k] for k in ("H", "d", "r", "dv", "rank", "qr", "W"))
    lin = lambda o, i: oracle.bf16(1.5 * rng.normal(size=(o, i)) / np.sqrt(i))      # noqa: E731
    return {"dq": lin(qr, W), "dq.norm": 1 + 0.3 * rng.normal(size=qr), "uq": lin(H * (d + r), qr),
            "dkv": lin(rank + r, W), "dkv.norm": 1 + 0.3 * rng.normal(size=rank), "uk": lin(H * d, rank),
            "uv": lin(H * dv, rank), "g": 2 * lin(H, W), "o": lin(W, H * dv)}


def load_latent(m, c, w, dev):
    H, d, rank = c["H"], c["d"], c["rank"]
    for k in ("dq", "dkv", "g"):
        m.proj.weight.data.narrow(0, *m.rows[k]).copy_(f32(w[k], dev))
    m.uq_proj.weight.data.copy_(f32(w["uq"], dev))
    m.o_proj.weight.data.copy_(f32(w["o"], dev))
    m.w_uk.data.copy_(f32(w["uk"].reshape(H, d, rank).transpose(0, 2, 1), dev))
    m.w_uv.data.copy_(f32(w["uv"].reshape(H, c["dv"], rank), dev))
    m.q_norm.data.copy_(f32(w["dq.norm"], dev))
    m.kv_norm.data.copy_(f32(w["dkv.norm"], dev))


@pytest.mark.parametrize("device,dtype", KINDS)
@pytest.mark.parametrize("scaling", [None, (5.0, 40, 6.0, 1.0)], ids=["plain", "yarn"])
@pytest.mark.parametrize("i", range(len(LATENT)))
def test_latent_attention(device, dtype, i, scaling):
    dev, c, n = dev_of(device), LATENT[i], 150
    scale = 0.9 / np.sqrt(c["d"] + c["r"])
    w = latent_weights(c, 20 + i)
    h = oracle.bf16(np.random.default_rng(i).normal(size=(n, c["W"])))
    cfg = {"heads": c["H"], "dim": c["d"], "rot_dim": c["r"], "vdim": c["dv"], "kv_rank": c["rank"],
           "q_rank": c["qr"], "scale": scale, "rot": {"dims": c["r"], "base": 300.0}}
    if c["size"]:
        cfg["mask"] = {"size": c["size"]}
    if scaling:
        cfg["rot"]["scaling"] = dict(zip(("factor", "original", "fast", "slow"), scaling))
    want = oracle.latent_attention(h, w, "", cfg, 1e-5)
    if c["size"] > 1:                                  # an edge that is one off shows
        assert rel(oracle.latent_attention(h, w, "", {**cfg, "mask": {"size": c["size"] - 1}}, 1e-5), want) > 0.01
    m = latent_module(c, scaling, dev, dtype, scale)
    load_latent(m, c, w, dev)
    for cuts in ([n], [70, 65, 3, 1], [2], [1]) if device == "cuda" else ([n], [31, 2, 80, 1]):
        pages = Pages(n, 8, dev)
        cache = pages.cache(1, c["rank"] + c["r"], dtype, 5.0)
        got = []
        for lo, hi in portions(n, cuts):
            meta, pos = meta_for(lo, hi, pages.table, pages.slots(lo, hi), dev)
            y = m(f32(h[lo:hi], dev).to(dtype), pos,
                  ForwardContext(meta, [(cache, cache[..., :0])], block_size=8), 0)
            got.append(y.float().sum(0) if y.dim() == 3 else y.float())       # (K-slices)
        assert rel(torch.cat(got), want) < tol(dtype, fp32=1e-5, bf16=3e-2), cuts


@pytest.mark.parametrize("device,dtype", KINDS)
@pytest.mark.parametrize("T,H,N,K,r", [(5, 4, 24, 16, 8), (1, 3, 10, 7, 6), (70, 8, 48, 32, 16), (200, 16, 192, 128, 64),
                                       (33, 2, 256, 256, 0), (130, 5, 20, 200, 4), (17, 2, 64, 300, 2)])
def test_one_matrix_per_head(device, dtype, T, H, N, K, r):
    dev, rng = dev_of(device), np.random.default_rng(N + K)
    x, w = oracle.bf16(rng.normal(size=(T, H, K + r))), oracle.bf16(rng.normal(size=(H, N, K)) / np.sqrt(K))
    pos = rng.integers(0, 90, T)
    rot = {"dims": r, "base": 70.0}
    want = np.einsum("thk,hnk->thn", x[..., :K], w)
    if r:
        want = np.concatenate([want, oracle.rotate_pairs(x[..., K:], pos.astype(np.float64), rot)], -1)
    xt = f32(x, dev).to(dtype)
    out = torch.full((T, H, N + r), 5.0, dtype=dtype, device=dev)
    table = ops.ref.rope_table_yarn(r, 90, 70.0).to(dev) if r else None
    ops.head_gemm(xt[..., :K], f32(w, dev).to(dtype), out, xt[..., K:] if r else None,
                  torch.tensor(pos, device=dev), table)
    assert rel(out, want) < tol(dtype, bf16=1e-2)


# ---------------------------------------------------------------- routing and experts
@pytest.mark.parametrize("device", DEV)
@pytest.mark.parametrize("E,top", [(5, 2), (12, 1), (3, 3), (24, 6), (64, 16), (70, 4), (300, 9), (40, 20)])
def test_raw_sigmoid_routing(device, E, top):
    dev, T, rng = dev_of(device), 40, np.random.default_rng(E)
    h, router = oracle.bf16(rng.normal(size=(T, 64))), oracle.bf16(0.3 * rng.normal(size=(E, 64)))
    ids, w, _ = oracle.route(h, router, top)
    s = ops.gate_proj(f32(h, dev), f32(router, dev), None, ops.GATE_SIGMOID)
    gw, gi = ops.moe_route_sigmoid(s, None, top, 1.0, False)
    assert np.array_equal(gi.cpu().numpy(), ids)
    np.testing.assert_allclose(gw.cpu().numpy(), w, rtol=1e-5)
    # the router's product and the choice in one launch (16-bit activations), or both ops
    for dt in (torch.float32, torch.bfloat16):
        for n in (T, 17, 1):
            gw, gi = ops.moe_gate_sigmoid(f32(h[:n], dev).to(dt), f32(router, dev).to(dt), None, top, 1.0, False)
            assert np.array_equal(gi.cpu().numpy(), ids[:n])
            np.testing.assert_allclose(gw.cpu().numpy(), w[:n], rtol=1e-4)
    corr = f32(rng.normal(size=E), dev)
    want = ops.moe_route_sigmoid(s, corr, top, 2.5)
    got = ops.moe_gate_sigmoid(f32(h, dev).to(torch.bfloat16), f32(router, dev).to(torch.bfloat16), corr, top, 2.5)
    assert torch.equal(got[1], want[1])
    np.testing.assert_allclose(got[0].cpu().numpy(), want[0].cpu().numpy(), rtol=1e-4)
    # equal scores: the lowest index; and the correction still only steers the choice
    flat = torch.full((3, E), 0.25, device=dev)
    gw, gi = ops.moe_route_sigmoid(flat, None, top, 1.0, False)
    assert gi.cpu().tolist() == [list(range(top))] * 3 and float((gw - 0.25).abs().max()) == 0
    corr = torch.zeros(E, device=dev)
    corr[E - 1] = 1.0
    gw, gi = ops.moe_route_sigmoid(flat, corr, top, 1.0, False)
    assert gi[:, 0].cpu().tolist() == [E - 1] * 3 and float((gw - 0.25).abs().max()) == 0


def experts_module(W, E, top, ff, shared, dev, dtype, seed):
    spec = FeedForwardSpec("moe", ff, act="silu", gated=True, experts=E, top=top, router="sigmoid_raw",
                           weight_input=True, shared_ff=shared, shared_gate=False)
    m = InputScaledExperts(W, spec, dtype, dev)
    rng = np.random.default_rng(seed)
    wts = {"router": oracle.bf16(0.4 * rng.normal(size=(E, W)))}
    for e in range(E + (1 if shared else 0)):
        n, f = ("e%d." % e, ff) if e < E else ("shared.", shared)
        for k, shape in (("gate", (f, W)), ("up", (f, W)), ("down", (W, f))):
            wts[n + k] = oracle.bf16(1.5 * rng.normal(size=shape) / np.sqrt(shape[1]))
        m.expert_in(e).copy_(f32(np.concatenate([wts[n + "gate"], wts[n + "up"]]), dev))
        m.expert_down(e).copy_(f32(wts[n + "down"], dev))
    m.router.data.copy_(f32(wts["router"], dev))
    return m, wts


def summed(adds, T, W):
    out = 0
    for a, k in adds:
        a = a.float().sum(0) if a.dim() == 3 else a.float()
        out = out + a.view(T, k, W).sum(1)
    return out


@pytest.mark.parametrize("device,dtype", KINDS)
@pytest.mark.parametrize("W,E,top,ff,shared", [(64, 5, 2, 24, 20), (70, 3, 3, 13, 0), (128, 4, 1, 64, 72),
                                               (256, 8, 2, 128, 128), (128, 6, 4, 192, 0)])
def test_experts_on_scaled_inputs(device, dtype, W, E, top, ff, shared):
    """Both forms (one GEMM pair over all experts, grouped rows) against the oracle; a weight on
    the output instead of the input, or renormalised weights, would show."""
    dev, T = dev_of(device), 90
    m, wts = experts_module(W, E, top, ff, shared, dev, dtype, W + E)
    h = oracle.bf16(np.random.default_rng(9).normal(size=(T, W)))
    mlp = {"router": {"experts": E, "top": top}, "shared": {"ff": shared} if shared else None}
    gaps = []
    want = oracle.experts(h, wts, "", mlp, gaps)
    ids, w, _ = oracle.route(h, wts["router"], top)
    late = want.copy()
    for e in range(E):
        t, j = np.nonzero(ids == e)
        late[t] += oracle.gated(h[t], wts, "e%d." % e) * w[t, j][:, None] - \
            oracle.gated(h[t] * w[t, j][:, None], wts, "e%d." % e)
    assert rel(late, want) > 0.1
    x = f32(h, dev).to(dtype)
    forms = [True, False] if m.native else [True]
    assert m.native == (device == "cuda" and dtype == torch.bfloat16 and W % 128 == 0)
    for dense in forms:
        m.dense_step = lambda T, d=dense: d
        for n in (T, 3, 1):
            got = summed(m(x[:n].contiguous()), n, W)
            assert rel(got, want[:n]) < tol(dtype, fp32=1e-5), (dense, n)


@pytest.mark.parametrize("device", GPU)
def test_grouped_experts_split_k(device):
    """A down projection cut into fp32 partial sums (few rows, long rows)."""
    dev, W, E, top, ff = dev_of(device), 128, 3, 2, 2048
    m, wts = experts_module(W, E, top, ff, 0, dev, torch.bfloat16, 8)
    h = oracle.bf16(np.random.default_rng(9).normal(size=(20, W)))
    m.dense_step = lambda T: False
    adds = m(f32(h, dev).to(torch.bfloat16))
    assert adds[0][0].dim() == 3 and adds[0][0].dtype == torch.float32
    want = oracle.experts(h, wts, "", {"router": {"experts": E, "top": top}})
    assert rel(summed(adds, 20, W), want) < 2e-2


def test_which_form_a_step_takes():
    def form(E, top, ff, T, native=True):
        spec = FeedForwardSpec("moe", ff, gated=True, experts=E, top=top, router="sigmoid_raw",
                               weight_input=True, shared_gate=False)
        m = InputScaledExperts(4096, spec, torch.bfloat16, "meta")
        m.native = native
        return ["grouped", "dense"][m.dense_step(T)]
    assert form(8, 2, 1792, 5000, native=False) == "dense"     # sizes or types without tiles
    assert [form(8, 2, 1792, t) for t in (2, 64, 256, 257)] == ["dense"] * 3 + ["grouped"]
    # many large experts of which a step touches few
    assert [form(64, 2, 4096, t) for t in (1, 4, 64, 5000)] == ["grouped", "grouped", "dense", "grouped"]
