"""Generax through the engine (registry, safetensors loading, block manager, pooled cache rows,
state slots, step packing, kernels) against the plain numpy oracle in ``generax_oracle.py``.

Every test writes its own small config.json + model.safetensors (random bf16 weights) and
drives the engine with the teacher-forced replayer or the generation entry points.  CPU runs
use the reference ops in fp32; ``-m gpu`` runs use the HIP kernels in fp32 and bf16.  Pages
are 8 tokens, so prompts cross many page, window and pooled-block borders."""
import json
import os

import numpy as np
import pytest
import torch

import generax_oracle as oracle
from kubernetes_gpu_cluster_amd.engine.config import EngineConfig
from kubernetes_gpu_cluster_amd.engine.llm_engine import LLM, LLMEngine
from kubernetes_gpu_cluster_amd.engine.replay import TraceReplayer
from kubernetes_gpu_cluster_amd.engine.sequence import SamplingParams
from kubernetes_gpu_cluster_amd.models.configs import PRESETS, generax_config, resolve_model

CPU = pytest.param("cpu", "float32", id="cpu-fp32")
GPU32 = pytest.param("cuda", "float32", marks=pytest.mark.gpu, id="gpu-fp32")
GPU16 = pytest.param("cuda", "bfloat16", marks=pytest.mark.gpu, id="gpu-bf16")
DEVICES = [CPU, GPU32, GPU16]
# Row error: rms of the logit difference over the rms of the logits, means taken off
TOL = {"float32": 5e-5, "bfloat16": 0.12}
TOL_MEDIAN = {"float32": 2e-5, "bfloat16": 0.04}


def att(heads=4, kv=2, dim=12, vdim=10, size=13, rot=8, base=500.0, factor=4.0, scale=0.5, kv_from=None):
    m = {"heads": heads, "kv_heads": kv, "dim": dim, "vdim": vdim, "scale": scale,
         "mask": {"size": size}, "rot": {"dims": rot, "base": base}}
    if factor is not None:
        m["rot"]["scaling"] = {"factor": factor}
    if kv_from is not None:
        m["kv_from"] = kv_from
    return m


def left(heads=4, kv=2, dim=12, vdim=10, size=13, pool=4, scale=0.5):
    return {"heads": heads, "kv_heads": kv, "dim": dim, "vdim": vdim, "scale": scale,
            "mask": {"size": size, "pool": pool}}


def delta(heads=4, kv=2, dim=8, vdim=6, conv=3, ra=5, rg=3):
    return {"heads": heads, "kv_heads": kv, "dim": dim, "vdim": vdim, "conv": conv,
            "_a_rank": ra, "_g_rank": rg}


def attl(m, ff=48):
    return {"type": "attention", "mixer": m, "mlp": {"kind": "dense", "ff": ff} if ff else None}


def par(l, r, ff=48):
    return {"type": "parallel", "mixer": {"left": l, "right": r},
            "mlp": {"kind": "dense", "ff": ff} if ff else None}


def config(layers, width=64, vocab=160, eps=1e-6, cap=9.0):
    return {"architecture": "Generax", "vocab": vocab, "width": width, "layers": layers,
            "norm": {"eps": eps}, "logit_softcap": cap}


# shared keys and values with another window, two sources, layers without a feed-forward
MIXED = config([par(left(), delta()), attl(att()), attl(att(size=21, base=90.0, heads=6, kv=3)),
                par(left(size=9, pool=3, heads=2, kv=1), delta(heads=2, kv=2, vdim=9, conv=4, ra=2, rg=7), 0),
                attl(att(kv_from=1, size=5)), attl(att(size=30, kv_from=2, base=90.0, heads=6, kv=3), 0),
                attl(att(), 0), attl(att(kv_from=1, size=40), 40)])
# values a model may make equal or 1: one head, blocks and windows of one token, one tap, ranks
# of one, no frequency scaling, a partly rotated head, value size = key size, attention first
PLAIN = config([attl(att(heads=1, kv=1, dim=16, vdim=16, size=20, rot=4, factor=None, scale=1.0)),
                par(left(heads=1, kv=1, dim=16, vdim=16, size=1, pool=1, scale=1.0),
                    delta(heads=1, kv=1, dim=16, vdim=16, conv=1, ra=1, rg=1)),
                attl(att(heads=1, kv=1, dim=16, vdim=16, size=1, rot=4, factor=None, scale=1.0, kv_from=0), 0),
                par(left(heads=2, kv=2, dim=8, vdim=8, size=1, pool=2, scale=0.3),
                    delta(heads=2, kv=1, dim=4, vdim=4, conv=2, ra=3, rg=1), 0)],
               width=48, vocab=96, cap=30.0)
# sizes the matrix-core prefill kernel, the 16-byte decode paths and the matrix-core gate
# projections take; prompts over several key tiles and row blocks
WIDE = config([par(left(heads=8, kv=2, dim=64, vdim=32, size=70, pool=16, scale=0.2),
                   delta(heads=4, kv=2, dim=64, vdim=64, conv=4, ra=24, rg=40), 96),
               attl(att(heads=8, kv=2, dim=64, vdim=64, size=37, rot=64, base=1e4, factor=8.0, scale=0.2), 96),
               attl(att(heads=8, kv=2, dim=64, vdim=64, size=90, rot=64, base=1e4, factor=8.0, scale=0.2,
                        kv_from=1), 64)],
              width=128, vocab=200, eps=1e-5, cap=12.0)
# sizes that are multiples of nothing, blocks that straddle pages, blocks longer than the
# window and than a page
ODD = config([par(left(heads=6, kv=2, dim=6, vdim=5, size=5, pool=11, scale=0.8),
                  delta(heads=3, kv=1, dim=7, vdim=10, conv=5, ra=4, rg=6), 26),
              attl(att(heads=3, kv=3, dim=10, vdim=14, size=11, rot=6, base=37.0, factor=1.7, scale=0.6), 18),
              par(left(heads=3, kv=1, dim=10, vdim=14, size=23, pool=7, scale=0.4),
                  delta(heads=6, kv=3, dim=10, vdim=3, conv=2, ra=9, rg=1), 30)],
             width=70, vocab=251, cap=5.0)


def clean(cfg):
    """The config as a checkpoint has it: only the tensors' shapes give the ranks."""
    c = json.loads(json.dumps(cfg))
    for L in c["layers"]:
        for k in ("_a_rank", "_g_rank"):
            L["mixer"].get("right", {}).pop(k, None)
    return c


def write_model(path, cfg, seed):
    """Random bf16 weights in the checkpoint's naming; returns them as float64 arrays."""
    from safetensors.torch import save_file
    wts = oracle.random_weights(cfg, seed)
    os.makedirs(path, exist_ok=True)
    with open(os.path.join(path, "config.json"), "w") as f:
        json.dump(clean(cfg), f)
    save_file({k: torch.tensor(v, dtype=torch.float32).to(torch.bfloat16).contiguous()
               for k, v in wts.items()}, os.path.join(path, "model.safetensors"))
    return wts


NAMES = ["mixed", "plain", "wide", "odd"]


@pytest.fixture(scope="module")
def models(tmp_path_factory):
    root = tmp_path_factory.mktemp("generax")
    out = {}
    for name, cfg, seed in zip(NAMES, (MIXED, PLAIN, WIDE, ODD), (51, 52, 53, 54)):
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
    key = (id(wts), tuple(toks))
    if key not in _expected:
        _expected[key] = oracle.forward(cfg, wts, toks)
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
    """Portions down to two tokens (shorter than the convolutions' taps - 1), cut inside
    pages, windows and pooled blocks."""
    for name, n in (("mixed", 45), ("odd", 52)):
        _, cfg, wts = models[name]
        rp = TraceReplayer(engine(models, name, device, dtype))
        toks = tokens_for(cfg, n, 3)
        assert close(run_alone(rp, "p", toks, cuts), expected(cfg, wts, toks), dtype), name


@pytest.mark.parametrize("device,dtype", DEVICES)
def test_long_decode(models, device, dtype):
    """Windows, blocks and pages pass over decoded tokens many times."""
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
    """A prompt of several hundred tokens in one step, then a second portion and decoded
    tokens that continue its state and its pooled rows."""
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
    """Pooled rows per page differ with the page: blocks of 11 and 7 tokens in pages of 16
    and of 5."""
    _, cfg, wts = models["odd"]
    rp = TraceReplayer(engine(models, "odd", device, dtype, pages=26, page=page))
    toks = tokens_for(cfg, 90, 8)
    assert close(run_alone(rp, "g", toks, [40, 13, 1]), expected(cfg, wts, toks), dtype)


# ---------------------------------------------------------------- batches, pages and slots reused
@pytest.mark.parametrize("device,dtype", DEVICES)
@pytest.mark.parametrize("name", ["mixed", "wide", "odd"])
def test_mixed_batches_and_reuse(models, name, device, dtype):
    """Four live requests of unequal length, portions beside decode rows, requests that
    sit out steps; the pool (14 pages) and the four slots are used again by later
    requests.  Every row must match the request run alone (the oracle)."""
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
def test_slot_and_page_reuse_starts_clean(models, device, dtype):
    """A request that takes over the slot and the pages (token rows and pooled rows) of a
    finished one must not see anything of it."""
    _, cfg, wts = models["mixed"]
    rp = TraceReplayer(engine(models, "mixed", device, dtype, pages=8, seqs=1))
    for i in range(3):
        toks = tokens_for(cfg, 47 + i, 20 + i)
        assert close(run_alone(rp, "r%d" % i, toks, [11, 1]), expected(cfg, wts, toks), dtype), i


@pytest.mark.parametrize("device,dtype", [CPU, GPU32])
@pytest.mark.parametrize("name", NAMES)
def test_residual_stream_after_every_layer(models, name, device, dtype):
    _, cfg, wts = models[name]
    eng = engine(models, name, device, dtype)
    toks = tokens_for(cfg, 33, 9)
    want = []
    oracle.forward(cfg, wts, toks, taps=want)
    model = eng.executor.runner.model
    taps = []
    orig = model.forward
    model.forward = lambda *a, **k: orig(*a, taps=taps, **k)
    try:
        run_alone(TraceReplayer(eng), "t", toks, [len(toks)])
    finally:
        model.forward = orig
    assert len(taps) == len(want) == len(cfg["layers"])
    for i, (g, w) in enumerate(zip(taps, want)):
        np.testing.assert_allclose(g.cpu().numpy(), w, rtol=2e-4, atol=2e-4, err_msg="layer %d" % i)


# ---------------------------------------------------------------- planted long-range visibility
@pytest.mark.parametrize("device,dtype", DEVICES)
@pytest.mark.parametrize("cuts", [[62], [30, 1], [17, 9, 2, 1]], ids=["prompt", "decode", "portions"])
def test_far_block_decides_the_output(tmp_path, device, dtype, cuts):
    """A token that appears in one block only is what every later query asks for: the score of
    that block's mean key stands far above all others from the position it becomes visible on,
    so a block seen one position early or late, or lost, changes every logit."""
    if device == "cuda" and not torch.cuda.is_available():
        pytest.skip("no GPU")
    cfg = config([par(left(heads=2, kv=1, dim=16, vdim=16, size=13, pool=4, scale=3.0),
                      delta(heads=1, kv=1, dim=8, vdim=8, ra=2, rg=2), 0)], width=48, vocab=40, cap=20.0)
    wts = write_model(str(tmp_path), cfg, 77)
    # token 39 maps to a direction of its own, which W_k turns into a key all queries match
    E, Q, K = wts["embed"], wts["l0.mix.left.q"], wts["l0.mix.left.k"]
    E[:, 0] = 0.0
    E[:39, 1] = 2.0
    E[39] = 0.0
    E[39, 0] = 6.0
    Q[:], K[:] = 0.25 * Q, 0.25 * K
    Q[:, 1] = np.tile([2.0, -2.0], 16)
    K[:, 0] = np.tile([2.0, -2.0], 8)
    bf = lambda a: torch.tensor(a, dtype=torch.float32).to(torch.bfloat16)      # noqa: E731
    wts = {k: bf(v).double().numpy() for k, v in wts.items()}
    from safetensors.torch import save_file
    save_file({k: bf(v) for k, v in wts.items()}, str(tmp_path / "model.safetensors"))
    toks = np.random.default_rng(3).integers(0, 39, 62).tolist()
    toks[20:22] = [39] * 2                                  # the first half of block 5
    want = oracle.forward(cfg, wts, toks)
    # those tokens leave the window at 33 and 34; the block (last token 23) is seen from 36 on
    early = oracle.forward({**cfg, "layers": [{**cfg["layers"][0], "mixer": {
        **cfg["layers"][0]["mixer"], "left": left(heads=2, kv=1, dim=16, vdim=16, size=12, pool=4, scale=3.0)}}]},
        wts, toks)
    assert row_errs(early, want)[35] > 0.1
    eng = LLMEngine(EngineConfig(model=str(tmp_path), dtype=dtype, device=device, block_size=8,
                                 max_num_seqs=2, max_model_len=72, max_num_batched_tokens=72,
                                 num_gpu_blocks_override=12, cuda_graph_max_bs=2))
    try:
        got = run_alone(TraceReplayer(eng), "f", toks, cuts)
    finally:
        eng.shutdown()
    assert close(got, want, dtype)


# ---------------------------------------------------------------- generation, presets, config
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
            seq = list(p)
            gen = list(o.output_token_ids)
            assert len(gen) == 12
            for tok in gen:
                lg = oracle.forward(cfg, wts, seq)[-1]
                top2 = np.sort(lg)[-2:]
                if top2[1] - top2[0] > 1e-3 * np.abs(lg).max():      # a clear arg-max
                    assert tok == int(np.argmax(lg))
                seq.append(tok)
    finally:
        llm.shutdown()


@pytest.mark.parametrize("device,dtype", [CPU, GPU16])
def test_preset_runs_through_sampling(device, dtype):
    if device == "cuda" and not torch.cuda.is_available():
        pytest.skip("no GPU")
    llm = LLM(model="tiny-generax", dtype=dtype, device=device, random_init=True, seed=3,
              block_size=8, max_num_seqs=4, max_model_len=64, num_gpu_blocks_override=40)
    try:
        outs = llm.generate([[1, 5, 9, 200], [7] * 11],
                            SamplingParams(temperature=0.8, top_k=20, max_tokens=6, ignore_eos=True))
        assert len(outs) == 2 and all(len(o.output_token_ids) == 6 for o in outs)
        assert all(0 <= t < 1024 for o in outs for t in o.output_token_ids)
    finally:
        llm.shutdown()


@pytest.mark.parametrize("device,dtype", [CPU, GPU32])
def test_cached_prefixes_of_a_model_without_recurrences(tmp_path, device, dtype):
    """Only attention layers: everything a prefix leaves behind lies in its pages, so a second
    prompt with the same beginning starts from them (keys and values turned by the same
    positions, shared by the layers that read them)."""
    if device == "cuda" and not torch.cuda.is_available():
        pytest.skip("no GPU")
    cfg = config([attl(att()), attl(att(kv_from=0, size=40)), attl(att(size=25, rot=12, vdim=6))])
    wts = write_model(str(tmp_path), cfg, 61)
    llm = LLM(model=str(tmp_path), dtype=dtype, device=device, block_size=8, max_num_seqs=2, max_model_len=96,
              num_gpu_blocks_override=30, cuda_graph_max_bs=2)
    try:
        assert not llm.engine.mcfg.has_recurrent_state
        head = tokens_for(cfg, 33, 5)
        for tail in ([7, 9], [3], [11, 2, 5, 1]):
            seq = head + tail
            out = llm.generate([seq], SamplingParams(temperature=0.0, max_tokens=6, ignore_eos=True))[0]
            for tok in out.output_token_ids:
                lg = oracle.forward(cfg, wts, seq)[-1]
                top2 = np.sort(lg)[-2:]
                if top2[1] - top2[0] > 1e-3 * np.abs(lg).max():
                    assert tok == int(np.argmax(lg))
                seq = seq + [tok]
        assert llm.engine.bm.hit_tokens >= 2 * 32
    finally:
        llm.shutdown()


def test_config_reader(models):
    d, cfg, wts = models["mixed"]
    mc, wdir = resolve_model(d)
    assert wdir == d and mc.arch == "generax" and mc.logit_softcap == 9.0 and mc.has_recurrent_state
    p, a, s = mc.layer_specs[0], mc.layer_specs[1], mc.layer_specs[4]
    assert (p.left.window.size, p.left.window.pool, p.left.qk_norm, p.left.rot_dims) == (13, 4, True, 0)
    assert (p.right.kind, p.right.decay_rank, p.right.gate_rank, p.right.conv) == ("channel_delta", 5, 3, 3)
    assert (a.rotary.factor, a.rotary.values, a.head_temp, a.kv_from) == (4.0, True, True, None)
    assert s.kv_from == 1 and s.window.size == 5 and mc.layer_specs[5].mlp is None
    # a layer on another's keys and values has no cache; pooled rows count into the pages
    model = engine(models, "mixed", "cpu", "float32").executor.runner
    assert model.model.cache_of == [0, 1, 2, 3, 1, 2, 4, 1]
    assert [c[0].shape[2] for c in model.kv_caches] == [10, 8, 8, 11, 8]
    rows = [c[0].shape[1] * c[0].shape[2] * (c[0].shape[3] + c[1].shape[3]) for c in model.kv_caches]
    assert model.kv_bytes_per_block() == 4 * sum(rows)
    # the parameter count: every 2-D tensor of the checkpoint but the convolutions
    n = sum(v.size for k, v in wts.items() if v.ndim == 2 and not k.endswith(".conv"))
    assert mc.num_params() == n
    assert PRESETS["tiny-generax"].layer_specs[3].kv_from == 1
    for layer, key, val in ((4, "kv_from", 4), (4, "kv_from", 0), (7, "kv_from", 4), (4, "kv_heads", 4)):
        bad = clean(cfg)
        bad["layers"][layer]["mixer"][key] = val
        with pytest.raises(ValueError):
            generax_config(bad, "bad", {k: v.shape for k, v in wts.items()})
    with pytest.raises(ValueError):                        # the ranks are nowhere
        generax_config(clean(cfg), "bad", {})


def test_unknown_or_misshapen_tensors_are_refused(models):
    from kubernetes_gpu_cluster_amd.models import build_model
    mc, _ = resolve_model(models["mixed"][0])
    m = build_model(mc, torch.float32)
    with pytest.raises(KeyError):
        m.load_weights([("l4.mix.k", torch.zeros(24, 64))])          # reads layer 1's keys
    with pytest.raises(KeyError):
        m.load_weights([("l5.mlp.up", torch.zeros(48, 64))])
    with pytest.raises(ValueError):
        m.load_weights([("l1.mix.q", torch.zeros(47, 64))])
