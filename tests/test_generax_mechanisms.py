"""Each mechanism of the Generax decoder alone (the product's op or module) against the numpy
oracle's function for it, on the CPU reference ops and, with ``-m gpu``, on the HIP kernels:
whole-projection norms with rotation and rotated values, windows and pooled blocks with a
planted stand-out key at every edge, shared keys, the channel-wise delta rule and its gates
over portions of every size with state carried in slots, results joining the stream, the
strided gated activation, the logit cap."""
import types

import numpy as np
import pytest
import torch

import generax_oracle as oracle
from kubernetes_gpu_cluster_amd import ops
from kubernetes_gpu_cluster_amd.models.attention import ForwardContext
from kubernetes_gpu_cluster_amd.models.configs import MixerSpec
from kubernetes_gpu_cluster_amd.models.recurrent import ChannelDeltaCore

DEV = [pytest.param("cpu", id="cpu"), pytest.param("cuda", marks=pytest.mark.gpu, id="gpu")]
GPU = [pytest.param("cuda", marks=pytest.mark.gpu, id="gpu")]


def dev_of(name):
    if name == "cuda" and not torch.cuda.is_available():
        pytest.skip("no GPU")
    return torch.device(name)


def f32(a, dev):
    return torch.tensor(np.asarray(a), dtype=torch.float32, device=dev)


def bf(a, dev):
    return f32(a, dev).to(torch.bfloat16)


def meta_for(chunks, decodes, tables, dev, slots=None, slot_mapping=None):
    """chunks: [(first position, length)], decodes: [position] -> (metadata, positions)."""
    m = types.SimpleNamespace()
    i32 = lambda v: torch.tensor(v, dtype=torch.int32, device=dev)   # noqa: E731
    P, D = len(chunks), len(decodes)
    qsl = np.concatenate([[0], np.cumsum([n for _, n in chunks])]).astype(int).tolist()
    m.num_prefills, m.num_decodes, m.num_prefill_tokens = P, D, qsl[-1]
    m.query_start_loc = i32(qsl) if P else None
    m.prefill_seq_lens = i32([a + n for a, n in chunks]) if P else None
    m.prefill_block_tables = tables[:P].contiguous().to(dev) if P and tables is not None else None
    m.decode_ctx_lens = i32([p + 1 for p in decodes]) if D else None
    m.decode_block_tables = tables[P:P + D].contiguous().to(dev) if D and tables is not None else None
    m.state_slots = i32(slots) if slots is not None else None
    m.work_seq = m.work_mblk = None
    m.slot_mapping = slot_mapping
    pos = [p for a, n in chunks for p in range(a, a + n)] + list(decodes)
    return m, torch.tensor(pos, dtype=torch.int64, device=dev)


def steps_of(n, cuts):
    """[(lo, hi, is a decode row)] for a sequence fed in portions `cuts` (the last repeats)."""
    out, lo, i = [], 0, 0
    while lo < n:
        c = cuts[min(i, len(cuts) - 1)]
        i += 1
        hi = min(n, lo + c)
        out.append((lo, hi, hi - lo == 1 and lo > 0))
        lo = hi
    return out


# ---------------------------------------------------------------- attention
class Attention:
    """qk_norm_store + window_attention over pages handed out in a scrambled order."""

    def __init__(self, H, G, dk, dv, dev, page=8, size=0, pool=0, rot=0, base=50.0, factor=1.0,
                 values=False, inter=False, scale=0.5, dtype=torch.float32, n=400, eps=1e-6):
        self.a = (H, G, dk, dv)
        self.dev, self.page, self.size, self.pool, self.inter = dev, page, size, pool, inter
        self.scale, self.dtype, self.eps = scale, dtype, eps
        pages = -(-n // page)
        self.order = np.random.default_rng(5).permutation(pages) + 1
        self.table = torch.tensor([self.order.tolist()], dtype=torch.int32, device=dev)
        rows = page + (-(-page // pool) if pool else 0)
        # leftovers of other requests everywhere
        self.kc = torch.full((pages + 1, G, rows, dk), 3.0, dtype=dtype, device=dev)
        self.vc = torch.full((pages + 1, G, rows, dv), -2.0, dtype=dtype, device=dev)
        self.rope = ops.ref.rope_table_linear(rot, n, base, factor).to(dev) if rot else None
        self.vrope = ops.ref.rope_table_linear(dv, n, base).to(dev) if values else None

    def slots(self, lo, hi):
        return torch.tensor([int(self.order[p // self.page]) * self.page + p % self.page
                             for p in range(lo, hi)], dtype=torch.int64, device=self.dev)

    def step(self, qkv, lo, hi, dec, qw, kw, store=True):
        H, G, dk, dv = self.a
        sl = self.slots(lo, hi)
        m, pos = meta_for([] if dec else [(lo, hi - lo)], [lo] if dec else [], self.table, self.dev,
                          slot_mapping=sl)
        q = ops.qk_norm_store(qkv, pos, qw, kw if store else None, self.eps, self.rope, self.vrope,
                              self.kc if store else None, self.vc if store else None, sl, H, G, dk,
                              dv, self.page, self.inter)
        out = torch.zeros(hi - lo, H * dv + 8, dtype=self.dtype, device=self.dev)
        ops.window_attention(q, self.kc, self.vc, pos, m, self.scale, self.size, 0, None,
                             out=out[:, 8:], pool=self.pool, block_size=self.page,
                             v_table=self.vrope, interleaved=self.inter)
        assert float(out[:, :8].float().abs().max()) == 0
        return out[:, 8:].float().cpu().numpy()

    def run(self, q, k, v, qw, kw, cuts):
        rng = np.random.default_rng(1)
        n = q.shape[0]
        wide = f32(np.concatenate([rng.normal(size=(n, 8)), q, k, v], 1), self.dev).to(self.dtype)
        return np.concatenate([self.step(wide[lo:hi, 8:], lo, hi, dec, f32(qw, self.dev), f32(kw, self.dev))
                               for lo, hi, dec in steps_of(n, cuts)])


def attention_oracle(q, k, v, qw, kw, H, G, dk, dv, size, pool, rot, base, factor, values, scale, eps=1e-6):
    n = q.shape[0]
    pos = np.arange(n, dtype=np.float64)
    q = (oracle.rms(q, eps) * qw).reshape(n, H, dk)
    k = (oracle.rms(k, eps) * kw).reshape(n, G, dk)
    v = v.reshape(n, G, dv)
    if rot:
        q, k = (oracle.rotate_halves(x, pos, rot, base, factor) for x in (q, k))
    if values:
        v = oracle.rotate_halves(v, pos, dv, base)
    vis = oracle.visible_window(n, size)
    if pool:
        k = np.concatenate([k, oracle.pooled_blocks(k, pool)])
        v = np.concatenate([v, oracle.pooled_blocks(v, pool)])
        vis = np.concatenate([vis, oracle.visible_blocks(n, size, pool)], 1)
    o = oracle.attend(q, k, v, vis, scale)
    if values:
        o = oracle.rotate_halves(o, pos, dv, base, sign=-1.0)
    return o.reshape(n, H * dv)


def qkv_for(n, H, G, dk, dv, seed=0):
    rng = np.random.default_rng(seed)
    return (rng.normal(size=(n, H * dk)), rng.normal(size=(n, G * dk)), rng.normal(size=(n, G * dv)),
            rng.normal(size=H * dk) * 0.4 + 1.0, rng.normal(size=G * dk) * 0.4 + 1.0)


ACUTS = [[400], [1], [2], [7, 1, 2, 9, 1, 1, 30, 2]]


@pytest.mark.parametrize("dev", DEV)
@pytest.mark.parametrize("H,G,dk,dv,rot,factor,values", [
    (4, 2, 12, 10, 8, 3.0, True), (3, 1, 16, 16, 16, 1.0, True), (2, 2, 10, 14, 6, 8.0, True),
    (4, 1, 8, 24, 0, 1.0, False), (8, 2, 64, 32, 32, 4.0, True), (2, 1, 32, 48, 32, 2.0, True)])
def test_rotary_window_attention(dev, H, G, dk, dv, rot, factor, values):
    """Norms over the whole q and k rows, partly rotated heads, values turned by their
    positions and turned back, any portions."""
    dev = dev_of(dev)
    n, size = 60, 13
    q, k, v, qw, kw = qkv_for(n, H, G, dk, dv)
    want = attention_oracle(q, k, v, qw, kw, H, G, dk, dv, size, 0, rot, 50.0, factor, values, 0.5)
    for cuts in ACUTS:
        a = Attention(H, G, dk, dv, dev, size=size, rot=rot, factor=factor, values=values)
        np.testing.assert_allclose(a.run(q, k, v, qw, kw, cuts), want, rtol=1e-4, atol=2e-5, err_msg=str(cuts))


@pytest.mark.parametrize("dev", DEV)
@pytest.mark.parametrize("page,pool,size", [(8, 1, 1), (8, 2, 1), (8, 3, 7), (8, 4, 13), (8, 8, 8),
                                            (8, 11, 5), (8, 16, 30), (8, 20, 9), (5, 7, 11), (16, 6, 3)])
def test_pooled_blocks(dev, page, pool, size):
    """Blocks shorter and longer than pages and than the window, block borders on and off
    page borders."""
    dev = dev_of(dev)
    H, G, dk, dv, n = 4, 2, 8, 6, 75
    q, k, v, qw, kw = qkv_for(n, H, G, dk, dv, seed=pool)
    want = attention_oracle(q, k, v, qw, kw, H, G, dk, dv, size, pool, 0, 1.0, 1.0, False, 0.9)
    for cuts in ACUTS:
        a = Attention(H, G, dk, dv, dev, page=page, size=size, pool=pool, scale=0.9)
        np.testing.assert_allclose(a.run(q, k, v, qw, kw, cuts), want, rtol=1e-4, atol=2e-5, err_msg=str(cuts))


@pytest.mark.parametrize("dev", DEV)
@pytest.mark.parametrize("where", ["first", "page_border", "block"])
def test_planted_key_at_every_edge(dev, where):
    """One key (or one block's keys) stands far above all others for every query: whether it
    is visible decides the output at each position, just inside and just outside the window,
    in the gap between leaving the window and its block's turn, and from then on."""
    dev = dev_of(dev)
    H, G, dk, dv, n, size, pool = 2, 1, 8, 6, 70, 13, 6
    rng = np.random.default_rng(4)
    q = rng.normal(size=(n, H * dk)) * 0.1 + np.tile([2.0, 0, 0, 0, 0, 0, 0, 0], H)
    k = rng.normal(size=(n, dk)) * 0.1 + np.array([0, 2.0, 0, 0, 0, 0, 0, 0])
    v = rng.normal(size=(n, dv))
    at = {"first": [0], "page_border": [15, 16], "block": list(range(18, 24))}[where]
    k[at] = [3.0] + [0.0] * 7
    v[at] += 40.0
    one = np.ones
    args = (q, k, v, one(H * dk), one(dk))
    want = attention_oracle(*args, H, G, dk, dv, size, pool, 0, 1.0, 1.0, False, 6.0)
    # the oracle itself tells the positions apart: seen, then not, then seen as a block
    seen = np.abs(want).max(1) > 4.5
    last, blk = max(at), max(at) // pool * pool + pool - 1
    assert seen[last: last + size].all() and seen[blk + size:].all()
    if blk > last:
        assert not seen[last + size: blk + size].any()
    for cuts in ACUTS:
        got = Attention(H, G, dk, dv, dev, size=size, pool=pool, scale=6.0).run(*args, cuts)
        np.testing.assert_allclose(got, want, rtol=2e-4, atol=2e-4, err_msg=str(cuts))


@pytest.mark.parametrize("dev", GPU)
@pytest.mark.parametrize("H,G,dk,dv,size,pool,rot,values", [
    (8, 2, 64, 32, 70, 16, 0, False), (4, 1, 128, 128, 100, 0, 128, True),
    (4, 2, 32, 64, 33, 5, 0, False), (2, 1, 64, 256, 50, 0, 32, True),
    (4, 2, 64, 64, 1, 3, 0, False), (4, 4, 96, 96, 40, 0, 96, True),
    (2, 1, 64, 48, 40, 0, 64, True), (16, 1, 64, 64, 130, 24, 0, False)])
def test_matrix_core_prefill_and_decode(dev, H, G, dk, dv, size, pool, rot, values):
    """bf16 heads of the sizes the matrix-core prefill kernel and the 8-wave decode kernel
    take, over several key tiles, row blocks and tiles of pooled rows (values of 48 columns
    rotate in pairs that straddle its tiles: the one-wave kernel)."""
    dev = dev_of(dev)
    n = 330
    q, k, v, qw, kw = qkv_for(n, H, G, dk, dv, seed=dk)
    r = lambda x: torch.tensor(x).to(torch.bfloat16).double().numpy()   # noqa: E731
    q, k, v = r(q), r(k), r(v)
    scale = 2.5 * dk ** -0.5
    want = attention_oracle(q, k, v, qw, kw, H, G, dk, dv, size, pool, rot, 50.0, 2.0, values, scale)
    for cuts in ([400], [200, 1], [70, 3, 65, 2, 1, 100]):
        a = Attention(H, G, dk, dv, dev, page=32, size=size, pool=pool, rot=rot, factor=2.0, values=values,
                      scale=scale, dtype=torch.bfloat16)
        got = a.run(q, k, v, qw, kw, cuts)
        err = np.sqrt(((got - want) ** 2).mean(1)) / np.sqrt((want ** 2).mean())
        # rounding of q, the cached rows and the result
        assert err.max() < 0.035, (cuts, err.max(), int(err.argmax()))
        assert np.median(err) < 0.012, cuts


@pytest.mark.parametrize("dev", GPU)
@pytest.mark.parametrize("dk,dv,rot,values,inter", [(64, 64, 0, False, False), (64, 64, 64, True, False),
                                                    (64, 64, 64, True, True), (32, 48, 32, True, True)])
def test_simple_and_fast_attention_agree(dev, dk, dv, rot, values, inter, monkeypatch):
    dev = dev_of(dev)
    H, G, n = 4, 2, 200
    q, k, v, qw, kw = qkv_for(n, H, G, dk, dv, seed=9)
    got = {}
    for kind in ("fast", "simple"):
        monkeypatch.setenv("KGC_WINDOW_ATTN", kind)
        got[kind] = np.concatenate([
            Attention(H, G, dk, dv, dev, size=45, pool=0 if rot else 7, rot=rot, values=values, inter=inter,
                      scale=0.3, dtype=torch.bfloat16).run(q, k, v, qw, kw, cuts) for cuts in ([150, 1], [1])])
    np.testing.assert_allclose(got["fast"], got["simple"], rtol=2e-2, atol=2e-2)


@pytest.mark.parametrize("dev", DEV)
@pytest.mark.parametrize("inter", [False, True])
def test_rotated_values_cancel_in_a_window_of_one(dev, inter):
    """A query that sees only its own token gets its value back unturned, while the cache
    holds it turned."""
    dev = dev_of(dev)
    H, G, dk, dv, n = 2, 2, 8, 12, 40
    q, k, v, qw, kw = qkv_for(n, H, G, dk, dv, seed=2)
    for cuts in ([40], [11, 1]):
        a = Attention(H, G, dk, dv, dev, size=1, rot=8, values=True, inter=inter)
        got = a.run(q, k, v, qw, kw, cuts)
        np.testing.assert_allclose(got, v, rtol=1e-5, atol=1e-5)
        sl = a.slots(0, n)
        cached = a.vc[sl // 8, :, sl % 8].cpu().numpy()
        assert np.abs(cached[5:] - v.reshape(n, G, dv)[5:]).max() > 0.5
        if not inter:
            np.testing.assert_allclose(cached, oracle.rotate_halves(v.reshape(n, G, dv), np.arange(n) * 1.0, dv, 50.0),
                                       rtol=1e-4, atol=1e-5)


@pytest.mark.parametrize("dev", GPU)
@pytest.mark.parametrize("H,G,dk,dv,inter", [(120, 8, 128, 64, True), (140, 4, 127, 30, False), (128, 8, 128, 128, False),
                                             (32, 8, 128, 128, False), (32, 4, 64, 64, True)])
def test_wide_rows_of_heads(dev, H, G, dk, dv, inter):
    """Rows longer than the LDS staging and than one unit per thread, in both pair layouts,
    against the reference op."""
    dev = dev_of(dev)
    n, page = 9, 4
    q, k, v, qw, kw = qkv_for(n, H, G, dk, dv)
    x = torch.tensor(np.concatenate([q, k, v], 1), dtype=torch.float32)
    rot = dk // 2 // 16 * 16
    tab, vtab = ops.ref.rope_table_linear(rot, n, 50.0, 2.0), ops.ref.rope_table_linear(dv, n, 50.0)
    qw, kw = torch.tensor(qw, dtype=torch.float32), torch.tensor(kw, dtype=torch.float32)
    slots = torch.tensor([4, 5, 6, 7, -1, 8, 9, 10, 11])
    pos = torch.arange(n)
    want = torch.zeros(4, G, page, dk), torch.zeros(4, G, page, dv)
    wq = ops.ref.qk_norm_store(x, pos, qw, kw, 1e-6, tab, vtab, *want, slots, H, G, dk, dv, page, inter)
    got = want[0].clone().zero_().to(dev), want[1].clone().zero_().to(dev)
    gq = ops.qk_norm_store(x.to(dev), pos.to(dev), qw.to(dev), kw.to(dev), 1e-6, tab.to(dev), vtab.to(dev), *got,
                           slots.to(dev), H, G, dk, dv, page, inter)
    for a, b in ((gq, wq), (got[0], want[0]), (got[1], want[1])):
        np.testing.assert_allclose(a.cpu().numpy(), b.numpy(), rtol=1e-4, atol=1e-5)


@pytest.mark.parametrize("dev", DEV)
def test_queries_on_another_layers_cache(dev):
    """A layer without keys and values of its own: q columns only, the cache left as it is."""
    dev = dev_of(dev)
    H, G, dk, dv, n = 4, 2, 12, 10, 50
    q, k, v, qw, kw = qkv_for(n, H, G, dk, dv)
    q2, _, _, qw2, _ = qkv_for(n, H, G, dk, dv, seed=8)
    a = Attention(H, G, dk, dv, dev, size=13, rot=8, values=True)
    a.run(q, k, v, qw, kw, [n])
    kc, vc = a.kc.clone(), a.vc.clone()
    a.size = 29
    want = attention_oracle(q2, k, v, qw2, kw, H, G, dk, dv, 29, 0, 8, 50.0, 1.0, True, 0.5)
    got = np.concatenate([a.step(f32(q2[lo:hi], dev), lo, hi, dec, f32(qw2, dev), None, store=False)
                          for lo, hi, dec in steps_of(n, [20, 1, 1, 5])])
    np.testing.assert_allclose(got, want, rtol=1e-4, atol=2e-5)
    assert torch.equal(a.kc, kc) and torch.equal(a.vc, vc)


@pytest.mark.parametrize("dev", DEV)
@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
def test_pooled_rows_in_a_batch(dev, dtype):
    """Two prompts' portions and decode rows of two sequences in one step, over pages with
    stale rows; a padding row (context 0) pools and stores nothing."""
    if dtype != torch.float32 and dev == "cpu":
        pytest.skip("one dtype is enough on the CPU")
    dev = dev_of(dev)
    H, G, dk, dv, page, pool, size = 2, 1, 16, 16, 8, 5, 6
    lens = [33, 21, 30, 40]
    data = [qkv_for(n, H, G, dk, dv, seed=20 + i) for i, n in enumerate(lens)]
    one = np.ones
    mb = 5
    order = np.random.default_rng(6).permutation(4 * mb) + 1
    tables = torch.tensor(order.reshape(4, mb), dtype=torch.int32)
    rows = page + -(-page // pool)
    kc = torch.full((4 * mb + 1, G, rows, dk), 9.0, dtype=dtype, device=dev)
    vc = torch.full((4 * mb + 1, G, rows, dv), 9.0, dtype=dtype, device=dev)
    want = [attention_oracle(q, k, v, one(H * dk), one(G * dk), H, G, dk, dv, size, pool, 0, 1.0, 1.0, False, 0.7)
            for q, k, v, _, _ in data]

    def step(parts, pad=False):
        """parts: [(sequence, lo, hi, decode)], chunks first."""
        ch = [(lo, hi - lo) for _, lo, hi, d in parts if not d]
        de = [lo for _, lo, _, d in parts if d] + ([-1] if pad else [])
        tab = torch.cat([tables[[s for s, *_ in parts]]] + ([torch.zeros(1, mb, dtype=torch.int32)] if pad else []))
        sl = [int(tables[s, p // page]) * page + p % page for s, lo, hi, _ in parts for p in range(lo, hi)]
        sl = torch.tensor(sl + ([-1] if pad else []), dtype=torch.int64, device=dev)
        m, pos = meta_for(ch, de, tab, dev, slot_mapping=sl)
        x = [np.concatenate(data[s][:3], 1)[lo:hi] for s, lo, hi, _ in parts]
        x = f32(np.concatenate(x + ([np.ones((1, x[0].shape[1]))] if pad else [])), dev).to(dtype)
        q = ops.qk_norm_store(x, pos, f32(one(H * dk), dev), f32(one(G * dk), dev), 1e-6, None, None, kc, vc,
                              sl, H, G, dk, dv, page)
        o = ops.window_attention(q, kc, vc, pos, m, 0.7, size, 0, None, pool=pool, block_size=page)
        o = o.float().cpu().numpy()
        a = 0
        for s, lo, hi, _ in parts:
            tol = 1e-4 if dtype == torch.float32 else 0.06
            np.testing.assert_allclose(o[a:a + hi - lo], want[s][lo:hi], rtol=tol, atol=tol)
            a += hi - lo
        assert not pad or np.all(o[-1] == 0)
    page0 = kc[0].clone()
    step([(0, 0, 17, False), (1, 0, 2, False), (2, 0, 29, False), (3, 0, 9, False)])
    step([(0, 17, 31, False), (1, 2, 20, False), (2, 29, 30, True), (3, 9, 10, True)], pad=True)
    step([(0, 31, 32, True), (1, 20, 21, True), (3, 10, 11, True)], pad=True)
    step([(3, 11, 40, False), (0, 32, 33, True)])
    assert torch.equal(kc[0], page0)


# ---------------------------------------------------------------- channel-wise delta rule
def delta_inputs(n, H, G, d, V, seed):
    rng = np.random.default_rng(seed)
    return rng.normal(size=(n, 2 * G * d + H * V)), rng.normal(size=(n, H)), rng.uniform(0.5, 1.0, size=(n, H * d))


def delta_want(qkv, b, g, H, G, d, V):
    n = qkv.shape[0]
    of = np.arange(H) // (H // G)
    q = oracle.unit(qkv[:, :G * d].reshape(n, G, d))[:, of] * d ** -0.5
    k = oracle.unit(qkv[:, G * d:2 * G * d].reshape(n, G, d))[:, of]
    return oracle.delta_scan(q, k, qkv[:, 2 * G * d:].reshape(n, H, V), oracle.sigmoid(b),
                             g.reshape(n, H, d)).reshape(n, H * V)


CUTS = [[200], [1], [2], [3, 1, 2, 70, 1, 1, 40, 2], [64, 65, 1], [17, 16, 15, 1]]


@pytest.mark.parametrize("dev", DEV)
@pytest.mark.parametrize("H,G,d,V", [(4, 2, 10, 6), (2, 2, 24, 72), (6, 3, 7, 3), (2, 1, 64, 20), (2, 1, 128, 64),
                                     (1, 1, 256, 5)])
def test_channel_delta_scan_over_steps(dev, H, G, d, V):
    dev = dev_of(dev)
    n = 120
    qkv, b, g = delta_inputs(n, H, G, d, V, H * d)
    want = delta_want(qkv, b, g, H, G, d, V)
    bw = f32(np.concatenate([np.full((n, 3), 7.0), b], 1), dev)
    for cuts in CUTS[1:4] if d >= 128 else CUTS:
        state = torch.full((4, H, d, V), 5.0, device=dev)       # another request's leftovers
        got = []
        for lo, hi, dec in steps_of(n, cuts):
            m, _ = meta_for([] if dec else [(lo, hi - lo)], [lo] if dec else [], None, dev, [2])
            got.append(ops.channel_delta_scan(f32(qkv[lo:hi], dev), bw[lo:hi, 3:], f32(g[lo:hi], dev),
                                              state, m, H, G, d, V).cpu().numpy())
        np.testing.assert_allclose(np.concatenate(got), want, rtol=2e-4, atol=2e-4 * np.abs(want).max(),
                                   err_msg=str(cuts))
        assert float(state[1].min()) == 5.0 and float(state[3].max()) == 5.0


@pytest.mark.parametrize("dev", DEV)
@pytest.mark.parametrize("V", [24, 64, 80])
def test_channel_delta_scan_with_many_sequences(dev, V):
    """Sixteen prompts and sixteen decode rows (one of them padding) of 32 heads: the grid size
    at which the GPU kernel keeps 16 value columns per wave (smaller steps keep 4)."""
    dev = dev_of(dev)
    H, G, d = 32, 8, 20
    lens = [1, 2, 3, 5, 8, 13, 16, 17, 21, 30, 31, 32, 33, 34, 40, 47]
    rng = np.random.default_rng(13)
    off = np.concatenate([[0], np.cumsum(lens)])
    T = int(off[-1])
    qkv, b, g = delta_inputs(T, H, G, d, V, 14)
    st = torch.full((32, H, d, V), 2.0, device=dev)
    before = rng.normal(size=(16, H, d, V)) * 0.3
    st[16:] = f32(before, dev)
    q2, b2, g2 = delta_inputs(16, H, G, d, V, 15)
    m, _ = meta_for([(0, n) for n in lens], [9] * 15 + [-1], None, dev, list(range(16)) + list(range(16, 31)) + [-1])
    got = ops.channel_delta_scan(f32(np.concatenate([qkv, q2]), dev), f32(np.concatenate([b, b2]), dev),
                                 f32(np.concatenate([g, g2]), dev), st, m, H, G, d, V).cpu().numpy()
    for i in (0, 1, 7, 12, 15):
        s = slice(off[i], off[i + 1])
        want = delta_want(qkv[s], b[s], g[s], H, G, d, V)
        np.testing.assert_allclose(got[s], want, rtol=2e-4, atol=2e-4 * np.abs(want).max())
    of = np.arange(H) // (H // G)
    for i in (0, 6, 14):                                   # a decode row continues its state
        q = oracle.unit(q2[i, :G * d].reshape(G, d))[of] * d ** -0.5
        k = oracle.unit(q2[i, G * d:2 * G * d].reshape(G, d))[of]
        S = g2[i].reshape(H, d)[:, :, None] * before[i]
        u = oracle.sigmoid(b2[i])[:, None] * (q2[i, 2 * G * d:].reshape(H, V) - np.einsum("hdv,hd->hv", S, k))
        S = S + k[:, :, None] * u[:, None]
        np.testing.assert_allclose(got[T + i], np.einsum("hdv,hd->hv", S, q).ravel(), rtol=1e-4, atol=1e-4)
        np.testing.assert_allclose(st[16 + i].cpu().numpy(), S, rtol=1e-4, atol=1e-5)
    assert np.all(got[T + 15] == 0)
    np.testing.assert_array_equal(st[31].cpu().numpy(), before[15].astype(np.float32))


@pytest.mark.parametrize("dev", DEV)
def test_one_channel_remembers_while_another_forgets(dev):
    """Key channel 0 never decays, channel 1 forgets at once: after fifty steps that write
    nothing, a query of channel 0 reads its value whole and one of channel 1 reads nothing."""
    dev = dev_of(dev)
    d, V, n = 4, 3, 52
    e = np.eye(d)
    v0, v1 = np.array([1.0, 2.0, 3.0]), np.array([5.0, 6.0, 7.0])
    z = np.zeros(V)
    rows = [np.concatenate([e[2], e[0], v0]), np.concatenate([e[2], e[1], v1])]
    rows += [np.concatenate([e[0] if t % 2 else e[1], e[3], z]) for t in range(n - 2)]
    b = np.full((n, 1), 40.0)
    b[2:] = -40.0                                              # write strength 0
    g = np.tile([1.0, 0.0, 1.0, 1.0], (n, 1))
    for cuts in ([n], [3, 1]):
        st = torch.zeros(1, 1, d, V, device=dev)
        got = []
        for lo, hi, dec in steps_of(n, cuts):
            m, _ = meta_for([] if dec else [(lo, hi - lo)], [lo] if dec else [], None, dev, [0])
            got.append(ops.channel_delta_scan(f32(np.stack(rows[lo:hi]), dev), f32(b[lo:hi], dev), f32(g[lo:hi], dev),
                                              st, m, 1, 1, d, V).cpu().numpy())
        got = np.concatenate(got)
        np.testing.assert_allclose(got[51], v0 / 2.0, rtol=1e-4)
        np.testing.assert_allclose(got[50], 0.0, atol=1e-6)


@pytest.mark.parametrize("dev", DEV)
def test_delta_rule_overwrites_a_key(dev):
    """With full write strength and no decay, writing key k twice leaves only the second
    value under it."""
    dev = dev_of(dev)
    d, V = 16, 8
    rng = np.random.default_rng(3)
    k, v1, v2 = rng.normal(size=d), rng.normal(size=V), rng.normal(size=V)
    qkv = np.stack([np.concatenate([k, k, v1]), np.concatenate([k, k, v2])])
    st = torch.zeros(1, 1, d, V, device=dev)
    m, _ = meta_for([(0, 2)], [], None, dev, [0])
    got = ops.channel_delta_scan(f32(qkv, dev), f32([[40.0], [40.0]], dev), f32(np.ones((2, d)), dev), st, m,
                                 1, 1, d, V).cpu().numpy()
    np.testing.assert_allclose(got[0], v1 / np.sqrt(d), rtol=1e-4, atol=1e-5)
    np.testing.assert_allclose(got[1], v2 / np.sqrt(d), rtol=1e-4, atol=1e-5)


@pytest.mark.parametrize("dev", DEV)
@pytest.mark.parametrize("T,Nd,Ng,ra,rg", [(1, 20, 12, 3, 5), (70, 96, 64, 32, 64), (5, 70, 35, 32, 32),
                                           (33, 256, 130, 64, 32), (130, 128, 128, 128, 96)])
@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
def test_delta_gates(dev, T, Nd, Ng, ra, rg, dtype):
    dev = dev_of(dev)
    rng = np.random.default_rng(Nd)
    r = lambda *s: f32(rng.normal(size=s), dev).to(dtype)           # noqa: E731
    wide, a2, g2 = r(T, ra + rg + 24), r(Nd, ra), r(Ng, rg)
    low = wide[:, 8:8 + ra + rg]
    neg_a, dtb = f32(-np.exp(rng.normal(size=Nd)), dev), f32(rng.normal(size=Nd) * 3 - 2, dev)
    decay, gate = ops.delta_gates(low, a2, g2, neg_a, dtb)
    l64, n = low.double().cpu().numpy(), lambda t: t.double().cpu().numpy()      # noqa: E731
    want = np.exp(n(neg_a) * oracle.softplus(l64[:, :ra] @ n(a2).T + n(dtb)))
    np.testing.assert_allclose(decay.cpu().numpy(), want, rtol=2e-4, atol=1e-5)
    wg = l64[:, ra:] @ n(g2).T
    tol = 1e-4 if dtype == torch.float32 else 1e-2
    np.testing.assert_allclose(gate.float().cpu().numpy(), wg, rtol=tol, atol=tol * np.abs(wg).max())


@pytest.mark.parametrize("dev", DEV)
@pytest.mark.parametrize("H,G,d,V,K,ra,rg", [(4, 2, 8, 6, 3, 5, 3), (2, 1, 16, 32, 4, 32, 40), (3, 3, 5, 7, 1, 1, 1)])
def test_delta_core_over_steps(dev, H, G, d, V, K, ra, rg):
    """Everything between the projections: convolutions, gates, scan, head norm and gate."""
    dev = dev_of(dev)
    rng = np.random.default_rng(K)
    n, eps = 90, 1e-5
    spec = MixerSpec("channel_delta", H, d, V, kv_heads=G, conv=K, decay_rank=ra, gate_rank=rg)
    core = ChannelDeltaCore(spec, eps, dev, torch.float32)
    W = {"norm": rng.normal(size=V) * 0.3 + 1, "A_log": rng.normal(size=H) * 0.5,
         "dt_bias": rng.normal(size=H * d) - 2, "a2": rng.normal(size=(H * d, ra)), "g2": rng.normal(size=(H * V, rg))}
    proj = np.zeros((n, 8 + core.n_in))
    conv = []
    for name, (a, c) in core.cols.items():
        proj[:, 8 + a:8 + a + c] = rng.normal(size=(n, c))
        W[name] = np.eye(c)
        if name in "qkv":
            W[name + ".conv"] = rng.normal(size=(c, K))
            conv.append(W[name + ".conv"])
    core.conv_w.data.copy_(f32(np.concatenate(conv), dev))
    core.neg_a.data.copy_(f32(-np.repeat(np.exp(W["A_log"]), d), dev))
    core.dt_bias.data.copy_(f32(W["dt_bias"], dev))
    core.norm_weight.data.copy_(f32(np.tile(W["norm"], H), dev))
    core.a2.data[:, :ra] = f32(W["a2"], dev)
    core.g2.data[:, :rg] = f32(W["g2"], dev)
    # the oracle's mixer reads its projections of h: give it selector matrices
    off, total = {}, 0
    for name, (a, c) in core.cols.items():
        off[name] = (total, c)
        total += c
    h = np.concatenate([proj[:, 8 + a:8 + a + c] for a, c in core.cols.values()], 1)
    for name, (a, c) in off.items():
        W[name] = np.zeros((c, total))
        W[name][:, a:a + c] = np.eye(c)
    W["o"] = np.eye(H * V)
    want = oracle.delta_mixer(h, W, "", {"heads": H, "kv_heads": G, "dim": d, "vdim": V}, eps)
    for cuts in CUTS:
        state = tuple(torch.full((3, *s), 4.0, device=dev) for s in core.state_shapes())
        got = []
        for lo, hi, dec in steps_of(n, cuts):
            m, _ = meta_for([] if dec else [(lo, hi - lo)], [lo] if dec else [], None, dev, [1])
            got.append(core(f32(proj[lo:hi], dev), 8, ForwardContext(m, []), state).cpu().numpy())
        np.testing.assert_allclose(np.concatenate(got), want, rtol=3e-4, atol=3e-4, err_msg=str(cuts))


# ---------------------------------------------------------------- stream, activation, logits
@pytest.mark.parametrize("dev", DEV)
@pytest.mark.parametrize("W", [70, 64, 1030, 2048, 4096, 4608])
@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
def test_residual_sum_norm(dev, W, dtype):
    dev = dev_of(dev)
    rng = np.random.default_rng(W)
    T, eps = 5, 1e-3
    x0, adds = rng.normal(size=(T, W)), [f32(rng.normal(size=(T, W)) * s, dev).to(dtype) for s in (0.3, 3.0, 1.0)]
    ws = [f32(rng.normal(size=W), dev) for _ in range(3)]
    w = f32(rng.normal(size=W), dev)
    n = lambda t: t.double().cpu().numpy()                          # noqa: E731
    for pick in ([], [(0, False)], [(0, True), (1, True), (2, False)], [(2, True)], [(0, False), (1, True)]):
        want = x0.astype(np.float32).astype(np.float64)
        for j, normed in pick:
            want = want + (oracle.rms(n(adds[j]), eps) * n(ws[j]) if normed else n(adds[j]))
        for odt in (dtype, torch.float32, None):
            x = f32(x0, dev)
            got = ops.residual_sum_norm(x, [(adds[j], ws[j] if normed else None) for j, normed in pick],
                                        w if odt is not None else None, eps, odt)
            np.testing.assert_allclose(n(x), want, rtol=1e-5, atol=1e-5)
            if odt is None:
                assert got is None
                continue
            tol = 1e-2 if odt == torch.bfloat16 else 2e-5
            assert got.dtype == odt
            np.testing.assert_allclose(n(got), oracle.rms(want, eps) * n(w), rtol=tol, atol=tol)


@pytest.mark.parametrize("dev", DEV)
@pytest.mark.parametrize("I,a,b", [(48, 8, 16), (37, 3, 5), (2056, 0, 24)])
@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
def test_silu_mul_between_column_slices(dev, I, a, b, dtype):
    dev = dev_of(dev)
    rng = np.random.default_rng(I)
    x = f32(rng.normal(size=(7, a + 2 * I + 8)), dev).to(dtype)
    out = torch.zeros(7, b + I + 8, dtype=dtype, device=dev)
    ops.silu_mul(x[:, a:a + 2 * I], out[:, b:b + I])
    g, u = (x[:, a + s:a + s + I].double().cpu().numpy() for s in (0, I))
    tol = 1e-2 if dtype == torch.bfloat16 else 2e-5
    np.testing.assert_allclose(out[:, b:b + I].double().cpu().numpy(), oracle.silu(g) * u, rtol=tol, atol=tol)
    assert float(out[:, :b].float().abs().sum()) == 0 and float(out[:, b + I:].float().abs().sum()) == 0


@pytest.mark.parametrize("dev", DEV)
@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
def test_logit_softcap(dev, dtype):
    dev = dev_of(dev)
    x = f32(np.random.default_rng(0).normal(size=(3, 300)) * 30, dev).to(dtype)
    got = ops.logit_softcap(x[:, 5:262], 7.5)
    assert got.dtype == torch.float32
    np.testing.assert_allclose(got.cpu().numpy(), oracle.softcap(x[:, 5:262].double().cpu().numpy(), 7.5),
                               rtol=1e-5, atol=1e-5)


def test_rope_table_is_exact_far_out():
    t = ops.ref.rope_table_linear(8, 200001, 50000.0, 4.0)[200000].double().numpy()
    a = 200000 * 50000.0 ** (-2.0 * np.arange(4) / 8) / 4.0
    np.testing.assert_allclose(t, np.concatenate([np.cos(a), np.sin(a)]), atol=1e-6)
