"""Ratizen through the engine (registry, safetensors loading, block manager, step packing,
kernels) against the plain numpy oracle in ``ratizen_oracle.py``.

Every test writes its own small config.json + model.safetensors (random bf16 weights) and
drives the engine with the teacher-forced replayer or the generation entry points.  CPU runs
use the reference ops in fp32; ``-m gpu`` runs use the HIP kernels in fp32 and bf16.  Pages
are 8 tokens, so prompts cross many page, window and chunk borders."""
import json
import os

import numpy as np
import pytest
import torch

import ratizen_oracle as oracle
from kubernetes_gpu_cluster_amd.engine.config import EngineConfig
from kubernetes_gpu_cluster_amd.engine.llm_engine import LLM, LLMEngine
from kubernetes_gpu_cluster_amd.engine.replay import TraceReplayer
from kubernetes_gpu_cluster_amd.engine.sequence import SamplingParams
from kubernetes_gpu_cluster_amd.models.configs import PRESETS, ratizen_config, resolve_model

CPU = pytest.param("cpu", "float32", id="cpu-fp32")
GPU32 = pytest.param("cuda", "float32", marks=pytest.mark.gpu, id="gpu-fp32")
GPU16 = pytest.param("cuda", "bfloat16", marks=pytest.mark.gpu, id="gpu-bf16")
DEVICES = [CPU, GPU32, GPU16]
# Row error: rms of the logit difference over the rms of the logits, means taken off
TOL = {"float32": 5e-5, "bfloat16": 0.12}
TOL_MEDIAN = {"float32": 2e-5, "bfloat16": 0.04}


def moe(experts=5, top=2, ff=24, shared=20):
    m = {"kind": "moe", "expert": {"ff": ff}, "router": {"experts": experts, "top": top}}
    if shared:
        m["shared"] = {"ff": shared}
    return m


def att(heads=4, kv=2, dim=12, vdim=10, size=13, scale=0.9, mlp=True):
    m = {"heads": heads, "kv_heads": kv, "dim": dim, "vdim": vdim, "scale": scale}
    if size:
        m["mask"] = {"size": size}
    return {"type": "attention", "mixer": m, "mlp": moe() if mlp is True else mlp}


def lat(heads=3, dim=10, rot=6, vdim=14, rank=18, q_rank=22, size=11, base=400.0, scale=0.4,
        yarn=(6.0, 64, 8.0, 1.0), mlp=True):
    m = {"heads": heads, "dim": dim, "rot_dim": rot, "vdim": vdim, "kv_rank": rank, "q_rank": q_rank,
         "scale": scale, "rot": {"dims": rot, "base": base}}
    if size:
        m["mask"] = {"size": size}
    if yarn:
        m["rot"]["scaling"] = dict(zip(("factor", "original", "fast", "slow"), yarn))
    return {"type": "latent_attention", "mixer": m, "mlp": moe() if mlp is True else mlp}


def config(layers, width=64, vocab=160, eps=1e-6, streams=3, mult=0.45, logit=1.7, scale=2.5):
    return {"architecture": "Ratizen", "vocab": vocab, "width": width, "layers": layers,
            "norm": {"eps": eps}, "streams": streams, "residual_mult": mult, "logit_scale": logit,
            "embedding": {"scale": scale}}


# layers without a feed-forward or a shared expert, other masks, heads and ranks in every layer,
# one plain causal layer of each type
MIXED = config([att(), lat(), att(size=21, heads=6, kv=3, mlp=moe(7, 3, 16, 0)), lat(size=5, mlp=None),
                att(size=8, heads=2, kv=2, dim=16, vdim=6, mlp=None), att(size=0, dim=8),
                lat(heads=4, rank=24, q_rank=10, size=30, base=90.0, yarn=(3.0, 20, 2.0, 0.5)),
                lat(size=0, rot=8, dim=4, yarn=None, mlp=moe(4, 1, 30, 12))])
# values a model may make equal or 1: one stream, one head, chunks and windows of one token, one
# expert, all experts chosen, no frequency scaling, unit constants, value size = key size
PLAIN = config([lat(heads=1, dim=16, rot=4, vdim=16, rank=16, q_rank=16, size=20, yarn=None, scale=1.0,
                    mlp=moe(1, 1, 32, 32)),
                att(heads=1, kv=1, dim=16, vdim=16, size=1, scale=1.0, mlp=moe(3, 3, 32, 32)),
                att(heads=2, kv=1, dim=8, vdim=8, size=2, scale=1.0, mlp=moe(2, 1, 8, 0)),
                lat(heads=2, dim=2, rot=2, vdim=2, rank=8, q_rank=8, size=1, scale=1.0, mlp=None)],
               width=48, vocab=96, streams=1, mult=1.0, logit=1.0, scale=1.0)
# sizes the matrix-core kernels take (attention, grouped experts, one matrix per head), keys of
# 72 and 56 dimensions that their tiles pad; prompts over several key tiles and row blocks
WIDE = config([att(heads=8, kv=2, dim=56, vdim=32, size=70, scale=0.3, mlp=moe(4, 2, 64, 40)),
               lat(heads=8, dim=32, rot=8, vdim=48, rank=64, q_rank=40, size=37, base=1e4, scale=0.3,
                   yarn=(8.0, 256, 16.0, 1.0), mlp=moe(6, 1, 128, 64)),
               att(heads=8, kv=4, dim=64, vdim=64, size=90, scale=0.2, mlp=moe(3, 2, 64, 0)),
               lat(heads=4, dim=64, rot=64, vdim=64, rank=128, q_rank=96, size=90, base=1e4, scale=0.2,
                   yarn=(4.0, 512, 32.0, 2.0), mlp=moe(8, 3, 64, 72))],
              width=128, vocab=200, eps=1e-5, streams=2)
# sizes that are multiples of nothing, more streams than the kernel unrolls exactly, one chunk
# that is longer than a page by one
ODD = config([att(heads=6, kv=2, dim=7, vdim=5, size=9, scale=0.8, mlp=moe(5, 2, 13, 11)),
              lat(heads=3, dim=5, rot=2, vdim=9, rank=11, q_rank=7, size=23, base=37.0, scale=0.6,
                  mlp=moe(3, 1, 18, 7)),
              att(heads=3, kv=1, dim=10, vdim=14, size=17, mlp=moe(2, 2, 26, 0))],
             width=70, vocab=251, streams=5)


def write_model(path, cfg, seed):
    """Random bf16 weights in the checkpoint's naming; returns them as float64 arrays."""
    wts = oracle.random_weights(cfg, seed)
    save_model(path, cfg, wts)
    return wts


def save_model(path, cfg, wts):
    from safetensors.torch import save_file
    os.makedirs(path, exist_ok=True)
    with open(os.path.join(path, "config.json"), "w") as f:
        json.dump(cfg, f)
    save_file({k: torch.tensor(v, dtype=torch.float32).to(torch.bfloat16).contiguous()
               for k, v in wts.items()}, os.path.join(path, "model.safetensors"))


NAMES = ["mixed", "plain", "wide", "odd"]


@pytest.fixture(scope="module")
def models(tmp_path_factory):
    root = tmp_path_factory.mktemp("ratizen")
    out = {}
    for name, cfg, seed in zip(NAMES, (MIXED, PLAIN, WIDE, ODD), (61, 62, 63, 64)):
        d = str(root / name)
        out[name] = (d, cfg, write_model(d, cfg, seed))
    return out


_engines = {}


@pytest.fixture(scope="module", autouse=True)
def _release_engines():
    """Engines are shared by the tests of this module and released after the last one."""
    yield
    for eng in _engines.values():
        eng.shutdown()
    _engines.clear()
    import gc
    gc.collect()
    if torch.cuda.is_available():
        torch.cuda.empty_cache()


def engine(models, name, device, dtype, pages=24, page=8, seqs=4, **kw):
    if device == "cuda" and not torch.cuda.is_available():
        pytest.skip("no GPU")
    key = (name, device, dtype, pages, page, seqs, tuple(sorted(kw.items())))
    if key not in _engines:
        d = models[name][0]
        _engines[key] = LLMEngine(EngineConfig(
            model=d, dtype=dtype, device=device, block_size=page, max_num_seqs=seqs,
            max_model_len=pages * page, max_num_batched_tokens=pages * page,
            num_gpu_blocks_override=pages + 1, cuda_graph_max_bs=seqs, **kw))
    return _engines[key]


def row_errs(got, want):
    got, want = np.asarray(got, dtype=np.float64), np.asarray(want, dtype=np.float64)
    d = got - want
    d = d - d.mean(-1, keepdims=True)
    w = want - want.mean(-1, keepdims=True)
    return np.sqrt((d ** 2).mean(-1) / (w ** 2).mean(-1))


class Verdict:
    def __init__(self, ok, text):
        self.ok, self.text = ok, text

    def __bool__(self):
        return self.ok

    def __repr__(self):
        return self.text


_expected = {}


def expected(cfg, wts, toks):
    """Oracle logits; no routing decision among them is close."""
    key = (id(wts), tuple(toks))
    if key not in _expected:
        gaps = []
        _expected[key] = oracle.forward(cfg, wts, toks, gaps=gaps)
        assert not gaps or min(g.min() for g in gaps) > 0.1
    return _expected[key]


def close(got, want, dtype):
    e = row_errs(got, want)
    ok = e.max() < TOL[dtype] and (len(e) < 8 or np.median(e) < TOL_MEDIAN[dtype])
    return Verdict(bool(ok), "rows %d: median %.2g, worst %.2g at %d" % (
        len(e), np.median(e), e.max(), int(e.argmax())))


def tokens_for(cfg, n, seed):
    return np.random.default_rng(seed).integers(0, cfg["vocab"], n).tolist()


def run_alone(rp, rid, toks, cuts):
    """Feed `toks` in portions of the sizes `cuts` (the last size repeats); all logits."""
    out, lo, i = [], 0, 0
    while lo < len(toks):
        n = cuts[min(i, len(cuts) - 1)]
        i += 1
        hi = min(len(toks), lo + n)
        lg = rp.step([{"id": rid, "tokens": toks[lo:hi], "want": list(range(hi - lo))}],
                     [rid] if hi == len(toks) else [])
        out.append(lg.cpu().numpy())
        lo = hi
    return np.concatenate(out)


# ---------------------------------------------------------------- whole prompts, decode, portions
@pytest.mark.parametrize("device,dtype", DEVICES)
@pytest.mark.parametrize("name", NAMES)
def test_whole_prompt_matches_oracle(models, name, device, dtype):
    _, cfg, wts = models[name]
    rp = TraceReplayer(engine(models, name, device, dtype))
    toks = tokens_for(cfg, 190 if name == "wide" else 75, 1)
    want = expected(cfg, wts, toks)
    got = run_alone(rp, "w", toks, [len(toks)])
    assert close(got, want, dtype)
    # the first tokens of a sequence, and a one-token prompt
    assert close(got[:3], want[:3], dtype)
    assert close(run_alone(rp, "o", toks[:1], [1]), want[:1], dtype)


@pytest.mark.parametrize("device,dtype", DEVICES)
@pytest.mark.parametrize("name", NAMES)
def test_prefill_then_token_by_token(models, name, device, dtype):
    _, cfg, wts = models[name]
    rp = TraceReplayer(engine(models, name, device, dtype))
    toks = tokens_for(cfg, 150 if name == "wide" else 70, 2)
    want = expected(cfg, wts, toks)
    if name == "wide":                             # portions across 64-row blocks and key tiles
        assert close(run_alone(rp, "c", toks, [70, 3, 65, 2, 1]), want, dtype)
    assert close(run_alone(rp, "d", toks, [20, 1]), want, dtype)
    if name != "wide" or device != "cpu":          # decoding from the very first token
        assert close(run_alone(rp, "e", toks, [1]), want, dtype)


@pytest.mark.parametrize("device,dtype", DEVICES)
@pytest.mark.parametrize("cuts", [[2], [3, 2, 7, 2, 11, 5, 1], [8], [9, 16, 2, 1], [1, 2, 1, 3]])
def test_portions(models, device, dtype, cuts):
    """Portions down to two tokens, cut inside pages, windows and chunks."""
    for name, n in (("mixed", 45), ("odd", 52)):
        _, cfg, wts = models[name]
        rp = TraceReplayer(engine(models, name, device, dtype))
        toks = tokens_for(cfg, n, 3)
        assert close(run_alone(rp, "p", toks, cuts), expected(cfg, wts, toks), dtype), name


@pytest.mark.parametrize("device,dtype", DEVICES)
def test_long_decode(models, device, dtype):
    """Windows, chunks and pages pass over decoded tokens many times."""
    _, cfg, wts = models["odd"]
    rp = TraceReplayer(engine(models, "odd", device, dtype, pages=40))
    toks = tokens_for(cfg, 160, 4)
    want = expected(cfg, wts, toks)
    got = run_alone(rp, "l", toks, [5, 1])
    assert close(got[-20:], want[-20:], dtype)
    assert close(got, want, dtype)


@pytest.mark.parametrize("device,dtype", DEVICES)
@pytest.mark.parametrize("name", ["mixed", "wide"])
def test_long_prompt(models, name, device, dtype):
    """A prompt of several hundred tokens in one step, then a second portion and decoded tokens."""
    _, cfg, wts = models[name]
    rp = TraceReplayer(engine(models, name, device, dtype, pages=60))
    toks = tokens_for(cfg, 440, 6)
    want = expected(cfg, wts, toks)
    got = run_alone(rp, "L", toks, [300, 130, 1])
    assert close(got[-40:], want[-40:], dtype)
    assert close(got, want, dtype)


@pytest.mark.parametrize("page", [16, 5])
@pytest.mark.parametrize("device,dtype", [CPU, GPU32])
def test_page_sizes(models, device, dtype, page):
    _, cfg, wts = models["odd"]
    rp = TraceReplayer(engine(models, "odd", device, dtype, pages=26, page=page))
    toks = tokens_for(cfg, 90, 8)
    assert close(run_alone(rp, "g", toks, [40, 13, 1]), expected(cfg, wts, toks), dtype)


# ---------------------------------------------------------------- batches, pages and slots reused
@pytest.mark.parametrize("device,dtype", DEVICES)
@pytest.mark.parametrize("name", ["mixed", "wide", "odd"])
def test_mixed_batches_and_reuse(models, name, device, dtype):
    """Four live requests of unequal length, portions beside decode rows, requests that sit out
    steps; the pool (14 pages) and the four slots are used again by later requests.  Every row
    must match the request run alone (the oracle)."""
    _, cfg, wts = models[name]
    rp = TraceReplayer(engine(models, name, device, dtype, pages=14))
    lens = {"a": 30, "b": 9, "c": 41, "d": 2, "e": 25, "f": 17, "g": 33}
    toks = {k: tokens_for(cfg, n, 10 + i) for i, (k, n) in enumerate(lens.items())}
    want = {k: expected(cfg, wts, v) for k, v in toks.items()}
    at = {k: 0 for k in lens}
    got = {k: [] for k in lens}
    # (request, tokens) per step; a request is freed when its tokens are used up
    plan = [[("a", 7), ("b", 3)], [("a", 1), ("b", 1), ("c", 12)], [("a", 1), ("c", 2), ("d", 2)],
            [("b", 5), ("c", 1), ("a", 9)], [("a", 1), ("c", 1)], [("a", 11), ("c", 25), ("e", 4)],
            [("e", 1), ("f", 17)], [("e", 1), ("g", 8)], [("e", 19), ("g", 1)], [("g", 24)]]
    used_pages = []
    for step in plan:
        entries, end = [], []
        for k, n in step:
            lo = at[k]
            entries.append({"id": k, "tokens": toks[k][lo:lo + n], "want": list(range(n))})
            at[k] += n
            if at[k] == lens[k]:
                end.append(k)
        lg = rp.step(entries, end).cpu().numpy()
        assert len(rp.seqs) <= 4
        for s in rp.seqs.values():
            used_pages += s.block_ids
        o = 0
        for k, n in step:
            got[k].append(lg[o:o + n])
            o += n
    assert len(used_pages) > len(set(used_pages))          # pages were handed out again
    for k in lens:
        assert at[k] == lens[k]
        assert close(np.concatenate(got[k]), want[k], dtype), k


@pytest.mark.parametrize("device,dtype", DEVICES)
def test_page_reuse_starts_clean(models, device, dtype):
    """A request that takes over the pages of a finished one must not see anything of it."""
    _, cfg, wts = models["mixed"]
    rp = TraceReplayer(engine(models, "mixed", device, dtype, pages=8, seqs=1))
    for i in range(3):
        toks = tokens_for(cfg, 47 + i, 20 + i)
        assert close(run_alone(rp, "r%d" % i, toks, [11, 1]), expected(cfg, wts, toks), dtype), i


@pytest.mark.parametrize("device,dtype", [CPU, GPU32])
@pytest.mark.parametrize("name", NAMES)
def test_streams_after_every_layer(models, name, device, dtype):
    """The sum of the streams after every layer, and with it the forward pass that hands it out."""
    _, cfg, wts = models[name]
    eng = engine(models, name, device, dtype)
    toks = tokens_for(cfg, 33, 9)
    want = []
    logits = oracle.forward(cfg, wts, toks, taps=want)
    model = eng.executor.runner.model
    taps = []
    orig = model.forward
    model.forward = lambda *a, **k: orig(*a, taps=taps, **k)
    try:
        got = run_alone(TraceReplayer(eng), "t", toks, [len(toks)])
    finally:
        model.forward = orig
    assert len(taps) == len(want) == len(cfg["layers"])
    for i, (g, w) in enumerate(zip(taps, want)):
        np.testing.assert_allclose(g.cpu().numpy(), w, rtol=2e-4, atol=2e-4 * np.abs(w).max(),
                                   err_msg="layer %d" % i)
    assert close(got, logits, dtype)


# ---------------------------------------------------------------- planted visibility
def planted(layer, width=48, vocab=40):
    """One layer in which token 39 is what every query asks for: its score stands far above all
    others while it is visible.  -> (config, weights)."""
    cfg = config([layer], width=width, vocab=vocab, streams=2, scale=1.0, mult=1.0)
    wts = oracle.random_weights(cfg, 78)
    E = wts["embed"]
    E[:, 0] = 0.0
    E[:39, 1] = 2.0
    E[39] = 0.0
    E[39, 0] = 6.0
    m, P = layer["mixer"], "l0.mix."
    if layer["type"] == "attention":
        H, G, d = m["heads"], m["kv_heads"], m["dim"]
        wts[P + "q"] *= 0.25
        wts[P + "k"] *= 0.25
        wts[P + "q"][:, 1] = np.tile([2.0, -2.0], H * d // 2)
        wts[P + "k"][:, 0] = np.tile([2.0, -2.0], G * d // 2)
    else:
        H, d, r = m["heads"], m["dim"], m["rot_dim"]
        wts[P + "dq"] *= 0.25
        wts[P + "dkv"] *= 0.25
        wts[P + "dq"][:, 1] = 2.0
        wts[P + "dkv"][: m["kv_rank"], 0] = 2.0
        wts[P + "uq"][:] = 0.1 * wts[P + "uq"]
        wts[P + "uk"][:] = 0.1 * wts[P + "uk"]
        uq = wts[P + "uq"].reshape(H, d + r, -1)
        uq[:, 0, :] = 0.6
        wts[P + "uk"].reshape(H, d, -1)[:, 0, :] = 0.6
    return cfg, {k: oracle.bf16(v) for k, v in wts.items()}


@pytest.mark.parametrize("device,dtype", DEVICES)
@pytest.mark.parametrize("cuts", [[62], [30, 1], [17, 9, 2, 1]], ids=["prompt", "decode", "portions"])
@pytest.mark.parametrize("kind,size", [("attention", 13), ("attention", 24), ("latent_attention", 13),
                                       ("latent_attention", 21)])
def test_planted_key_decides_the_output(tmp_path, device, dtype, cuts, kind, size):
    """The queries just inside and just outside the planted token's chunk or window see it, or do
    not: an edge that is one position off changes the logits there."""
    if device == "cuda" and not torch.cuda.is_available():
        pytest.skip("no GPU")
    make = (lambda n: att(heads=2, kv=1, dim=16, vdim=16, size=n, scale=2.0, mlp=None)) \
        if kind == "attention" else (lambda n: lat(heads=2, dim=8, rot=8, vdim=16, rank=16, q_rank=16, size=n,
                                                   scale=0.5, mlp=None))
    cfg, wts = planted(make(size))
    at = 26 if kind == "attention" else 20
    toks = np.random.default_rng(3).integers(0, 39, 62).tolist()
    toks[at] = 39
    want = oracle.forward(cfg, wts, toks)
    # the last position that sees the planted token, and the next one
    last = at // size * size + size - 1 if kind == "attention" else at + size - 1
    for other in (size - 1, size + 1):
        wrong = oracle.forward({**cfg, "layers": [make(other)]}, wts, toks)
        assert max(row_errs(wrong, want)[last: last + 2]) > 0.1
    save_model(str(tmp_path), cfg, wts)
    eng = LLMEngine(EngineConfig(model=str(tmp_path), dtype=dtype, device=device, block_size=8,
                                 max_num_seqs=2, max_model_len=72, max_num_batched_tokens=72,
                                 num_gpu_blocks_override=12, cuda_graph_max_bs=2))
    try:
        got = run_alone(TraceReplayer(eng), "f", toks, cuts)
    finally:
        eng.shutdown()
    assert close(got, want, dtype)


# ---------------------------------------------------------------- generation, presets, config
def greedy_follows(cfg, wts, prompt, gen):
    """Every generated token is the oracle's arg-max where that is clear."""
    seq = list(prompt)
    for tok in gen:
        lg = oracle.forward(cfg, wts, seq)[-1]
        top2 = np.sort(lg)[-2:]
        if top2[1] - top2[0] > 1e-3 * np.abs(lg).max():
            assert tok == int(np.argmax(lg))
        seq.append(tok)


@pytest.mark.parametrize("device,dtype", [CPU, GPU32])
def test_greedy_generation_through_the_scheduler(models, device, dtype):
    """LLM.generate (scheduler, chunked prefill, sampling kernel at temperature 0, decode
    graphs on the GPU) picks the oracle's arg-max token at every step."""
    if device == "cuda" and not torch.cuda.is_available():
        pytest.skip("no GPU")
    d, cfg, wts = models["mixed"]
    llm = LLM(model=d, dtype=dtype, device=device, block_size=8, max_num_seqs=3, max_model_len=96,
              max_num_batched_tokens=16, num_gpu_blocks_override=40, cuda_graph_max_bs=3)
    try:
        prompts = [tokens_for(cfg, n, 30 + n) for n in (19, 5, 33)]
        outs = llm.generate(prompts, SamplingParams(temperature=0.0, max_tokens=12, ignore_eos=True))
        for p, o in zip(prompts, outs):
            assert len(o.output_token_ids) == 12
            greedy_follows(cfg, wts, p, o.output_token_ids)
    finally:
        llm.shutdown()


@pytest.mark.parametrize("device,dtype", [CPU, GPU32])
def test_cached_prefixes(models, device, dtype):
    """Everything a prefix leaves behind lies in its pages: a second prompt with the same
    beginning starts from them."""
    if device == "cuda" and not torch.cuda.is_available():
        pytest.skip("no GPU")
    d, cfg, wts = models["mixed"]
    llm = LLM(model=d, dtype=dtype, device=device, block_size=8, max_num_seqs=2, max_model_len=96,
              num_gpu_blocks_override=30, cuda_graph_max_bs=2)
    try:
        assert not llm.engine.mcfg.has_recurrent_state
        head = tokens_for(cfg, 33, 5)
        for tail in ([7, 9], [3], [11, 2, 5, 1]):
            out = llm.generate([head + tail], SamplingParams(temperature=0.0, max_tokens=6, ignore_eos=True))[0]
            greedy_follows(cfg, wts, head + tail, out.output_token_ids)
        assert llm.engine.bm.hit_tokens >= 2 * 32
    finally:
        llm.shutdown()


@pytest.mark.parametrize("device,dtype", [CPU, GPU16])
def test_preset_runs_through_sampling(device, dtype):
    if device == "cuda" and not torch.cuda.is_available():
        pytest.skip("no GPU")
    llm = LLM(model="tiny-ratizen", dtype=dtype, device=device, random_init=True, seed=3,
              block_size=8, max_num_seqs=4, max_model_len=64, num_gpu_blocks_override=40)
    try:
        outs = llm.generate([[1, 5, 9, 200], [7] * 11],
                            SamplingParams(temperature=0.8, top_k=20, max_tokens=6, ignore_eos=True))
        assert len(outs) == 2 and all(len(o.output_token_ids) == 6 for o in outs)
        assert all(0 <= t < 1024 for o in outs for t in o.output_token_ids)
    finally:
        llm.shutdown()


def test_config_reader(models):
    d, cfg, wts = models["mixed"]
    mc, wdir = resolve_model(d)
    assert wdir == d and mc.arch == "ratizen" and not mc.has_recurrent_state
    assert (mc.streams, mc.residual_mult, mc.logit_scale, mc.embed_scale) == (3, 0.45, 1.7, 2.5)
    a, l = mc.layer_specs[0], mc.layer_specs[1]
    assert (a.window.size, a.window.chunked, a.head_norm, a.sink, a.rot_dims) == (13, True, True, 0.0, 0)
    assert (l.window.size, l.window.chunked, l.q_rank, l.kv_rank, l.head_gate) == (11, False, 22, 18, True)
    assert l.rotary.yarn == (6.0, 64.0, 8.0, 1.0) and l.rotary.interleaved and l.sink is None
    assert (a.mlp.router, a.mlp.weight_input, a.mlp.shared_ff, a.mlp.top) == ("sigmoid_raw", True, 20, 2)
    assert mc.layer_specs[2].mlp.shared_ff == 0 and mc.layer_specs[3].mlp is None
    assert mc.layer_specs[5].window is None and mc.layer_specs[7].rotary.yarn is None
    # a latent layer's pages hold one row of latent and rotary key part per token
    runner = engine(models, "mixed", "cpu", "float32").executor.runner
    assert [tuple(c[0].shape[1:]) for c in runner.kv_caches[:2]] == [(2, 8, 12), (1, 8, 24)]
    assert runner.kv_bytes_per_block() == 8 * mc.kv_bytes_per_token(4)
    # the parameter count: every matrix of the checkpoint but the stream mixes
    assert mc.num_params() == sum(v.size for k, v in wts.items() if v.ndim == 2 and not k.endswith(".mix"))
    assert PRESETS["tiny-ratizen"].layer_specs[2].q_rank == 48
    bad = json.loads(json.dumps(cfg))
    bad["layers"][0]["mixer"]["kv_heads"] = 3
    with pytest.raises(ValueError):
        ratizen_config(bad, "bad")
    bad = json.loads(json.dumps(cfg))
    bad["layers"][1]["mlp"]["router"]["top"] = 9
    with pytest.raises(ValueError):
        ratizen_config(bad, "bad")


def test_unknown_or_misshapen_tensors_are_refused(models):
    from kubernetes_gpu_cluster_amd.models import build_model
    mc, _ = resolve_model(models["mixed"][0])
    m = build_model(mc, torch.float32)
    for name, shape in (("l3.norm2", (64,)), ("l3.mlp.router", (5, 64)), ("l0.mix.dq", (22, 64)),
                        ("l2.mlp.shared.up", (20, 64)), ("l0.mlp.e5.up", (24, 64)), ("l9.norm1", (64,))):
        with pytest.raises(KeyError):
            m.load_weights([(name, torch.zeros(*shape))])
    for name, shape in (("l1.mix.uq", (47, 22)), ("l1.mix.uk", (18, 30)), ("l0.hc1.mix", (3, 4)),
                        ("l0.mlp.e1.down", (24, 64)), ("embed", (160, 63))):
        with pytest.raises(ValueError):
            m.load_weights([(name, torch.zeros(*shape))])
