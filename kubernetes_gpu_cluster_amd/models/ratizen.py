"""Ratizen: chunked attention with a sink and gated latent attention over hyper-connected
residual streams, with routed experts whose input carries the routing weight.

S residual streams X_1 .. X_S (fp32, width W), all embed[token] * embed_scale at the start; per
sublayer (mixer, then the feed-forward where there is one) with its learned in [S], out [S] and
mix [from, to]:
  u = sum_s in[s] X_s;   y = sublayer(RMSNorm(u) (1 + w))
  X_t <- sum_s mix[s, t] X_s + m out[t] y          (all at once from the old streams)
  logits = logit_scale * head(RMSNorm(sum_s X_s) (1 + w_f))
Layer type "attention": grouped-query attention, q and k RMS-normed per head, no rotation, a
query sees its own chunk, a sink of score 0 joins the softmax.  Type "latent_attention": queries
and keys through normed latents, YaRN rotation of a part of each head, a sliding window, a
sigmoid gate per head.  Feed-forward: the ``top`` experts by sigmoid score, each on the input
times its score, and a shared expert.  Norm weights are kept as 1 + w; m rides on ``out``, the
logit scale on the final norm's weight.  Projections run in the activation dtype with fp32
accumulation; the streams, norms, rotation, softmax and routing are fp32.

Kernel sequence per layer (ops/__init__.py, "Ratizen-style decoders"):
  hyper_norm (the previous result joins the streams, which are mixed and combined; norm) ->
  attention:         q | k | v GEMM -> norm_kv_store -> window_attention -> output GEMM
  latent_attention:  merged GEMM -> latent_down_store -> query GEMM -> head_gemm (with the
                     rotation) -> window_attention (gate in its epilogue) -> head_gemm -> GEMM
  -> hyper_norm -> moe_gate_sigmoid -> all experts as one GEMM pair around expert_silu_all
  (decode sizes), or the grouped expert GEMMs beside the shared expert's; K-slices of the
  projections and a token's expert rows are summed by the next hyper_norm.
One GPU per replica (TP = PP = 1).
"""
from __future__ import annotations

import re
from typing import Iterable, Optional

import torch
import torch.nn as nn

from .. import ops
from ..ops.gemm import linear_slices
from ..parallel.layers import ParallelLMHead, ReplicatedLinear, VocabParallelEmbedding
from ..parallel.state import get_state
from .attention import AttentionCore, ForwardContext, LatentQueryAttention
from .configs import ModelConfig
from .moe import InputScaledExperts


def _f32(shape, device, fill=0.0):
    return nn.Parameter(torch.full(shape, fill, dtype=torch.float32, device=device),
                        requires_grad=False)


class CoreAttention(nn.Module):
    """A mixer that is one attention core between its own projections; the result may come as
    K-slices (``linear_slices``)."""

    def __init__(self, hidden: int, spec, eps: float, dtype, device):
        super().__init__()
        self.core = AttentionCore(spec, 1.0, eps, device)
        self.qkv_proj = ReplicatedLinear(hidden, self.core.n_in, dtype=dtype, device=device)
        self.o_proj = ReplicatedLinear(self.core.n_out, hidden, dtype=dtype, device=device)

    def prepare(self, tables: dict, max_pos: int, device) -> None:
        self.core.prepare(tables, max_pos, device)

    def cache_shape(self) -> tuple:
        return self.core.cache_shape()

    def forward(self, h: torch.Tensor, positions: torch.Tensor, ctx: ForwardContext,
                cache_idx: int) -> torch.Tensor:
        o = torch.empty(h.shape[0], self.core.n_out, dtype=h.dtype, device=h.device)
        self.core(self.qkv_proj(h), 0, positions, ctx, cache_idx, o)
        return linear_slices(o, self.o_proj.weight)


class HyperConnection(nn.Module):
    """The learned weights of one sublayer's connection to the residual streams."""

    def __init__(self, streams: int, width: int, device):
        super().__init__()
        self.w_in = _f32((streams,), device, 1.0 / streams)
        self.w_out = _f32((streams,), device, 1.0)      # times the residual multiplier
        self.mix = _f32((streams, streams), device)     # [from, to]
        self.mix.data.fill_diagonal_(1.0)
        self.norm = _f32((width,), device, 1.0)         # 1 + the checkpoint's weight


class RatizenLayer(nn.Module):
    def __init__(self, cfg: ModelConfig, idx: int, dtype, device):
        super().__init__()
        sp, W = cfg.layer_specs[idx], cfg.hidden_size
        self.idx, self.spec = idx, sp
        cls = CoreAttention if sp.kind == "attention" else LatentQueryAttention
        self.mix = cls(W, sp, cfg.rms_eps, dtype, device)
        self.hc1 = HyperConnection(cfg.streams, W, device)
        self.hc2 = self.mlp = None
        if sp.mlp is not None:
            self.hc2 = HyperConnection(cfg.streams, W, device)
            self.mlp = InputScaledExperts(W, sp.mlp, dtype, device)


class RatizenForCausalLM(nn.Module):
    def __init__(self, cfg: ModelConfig, dtype=torch.bfloat16, device=None):
        super().__init__()
        s = get_state()
        assert s.tp_size == 1 and s.pp_size == 1, "Ratizen runs on one GPU per replica"
        self.cfg, self.dtype = cfg, dtype
        self.start, self.end = 0, cfg.num_layers
        self.first = self.last = True
        W, L = cfg.hidden_size, cfg.num_layers
        self.embed_tokens = VocabParallelEmbedding(cfg.vocab_size, W, dtype, device)
        self.layers = nn.ModuleList([RatizenLayer(cfg, i, dtype, device) for i in range(L)])
        self.final_norm = _f32((W,), device, cfg.logit_scale)   # (1 + w) * logit_scale
        self.sum_in = _f32((cfg.streams,), device, 1.0)
        self.lm_head = ParallelLMHead(cfg.vocab_size, W, dtype, device)
        self.streams = self.embed_out = None        # [Tcap, S, W] / [Tcap, W] fp32 step buffers

    # ------------------------------------------------------------------ engine hooks
    @property
    def num_local_layers(self) -> int:
        return len(self.layers)

    def local_kv_heads(self) -> int:
        return max(l.spec.kv_heads for l in self.layers)

    def cache_layout(self) -> list:
        return [l.mix.cache_shape() for l in self.layers]

    def sum_shapes(self) -> set:
        """(N, K) of the projections whose results ``hyper_norm`` sums."""
        ws = [l.mix.o_proj.weight for l in self.layers]
        ws += [l.mlp.down_proj.weight for l in self.layers if l.mlp is not None]
        return {tuple(w.shape) for w in ws}

    def stream_shapes(self) -> set:
        """(N, K) of all other projections."""
        return {tuple(p.shape) for n, p in self.named_parameters()
                if p.dim() == 2 and n.endswith("proj.weight")} - self.sum_shapes()

    def sum_consumer(self, M: int, N: int):
        """A ``hyper_norm`` over scratch rows, for timing a projection with what follows it."""
        hc, dev = self.layers[0].hc1, self.final_norm.device
        X = torch.zeros(M, self.cfg.streams, N, dtype=torch.float32, device=dev)
        return lambda y: ops.hyper_norm(X, X, [(y, 1)], hc.mix, hc.w_out, hc.w_in, hc.norm,
                                        self.cfg.rms_eps, self.dtype)

    def prepare(self, max_pos: int, max_tokens: int, device) -> None:
        """Rotary tables for ``max_pos`` positions and the step buffers for ``max_tokens`` rows
        (static, so captured decode graphs replay over them)."""
        tables: dict = {}
        for l in self.layers:
            l.mix.prepare(tables, max_pos, device)
        W, S = self.cfg.hidden_size, self.cfg.streams
        self.streams = torch.zeros(max_tokens, S, W, dtype=torch.float32, device=device)
        self.embed_out = torch.zeros(max_tokens, W, dtype=torch.float32, device=device)

    @torch.no_grad()
    def init_random(self, seed: int = 0, std: float = 0.02) -> None:
        """Random weights for benchmarking: projections ~ N(0, std), norm weights near 1, stream
        mixes near the identity."""
        g = torch.Generator(device="cpu").manual_seed(seed)

        def rnd(p, scale, base=0.0):
            if p.numel() > 1 << 24:             # large matrices: on the parameter's device
                dg = torch.Generator(device=p.device).manual_seed(seed + p.numel())
                p.copy_(torch.empty(p.shape, dtype=p.dtype, device=p.device).normal_(
                    base, scale, generator=dg))
                return
            p.copy_((torch.randn(p.shape, generator=g) * scale + base).to(p.device, p.dtype))
        S = self.cfg.streams
        for name, p in self.named_parameters():
            leaf = name.rsplit(".", 1)[-1]
            if leaf == "final_norm":
                rnd(p, 0.05 * self.cfg.logit_scale, self.cfg.logit_scale)
            elif leaf in ("norm", "q_norm", "k_norm", "kv_norm"):
                rnd(p, 0.05, 1.0)
            elif leaf == "w_in":
                rnd(p, 0.05, 1.0 / S)
            elif leaf == "w_out":
                rnd(p, 0.1 * self.cfg.residual_mult, self.cfg.residual_mult)
            elif leaf == "mix":
                rnd(p, 0.05 / S)
                p.diagonal().add_(1.0)
            elif leaf == "sum_in":
                pass
            elif leaf == "router":
                rnd(p, 0.1)
            else:
                rnd(p, std)
        for l in self.layers:       # padding rows are zeros, as in a loaded model
            if isinstance(l.mix, LatentQueryAttention):
                l.mix.proj.weight.data[sum(l.mix.rows["g"]):] = 0

    # ------------------------------------------------------------------ forward
    def forward(self, input_ids: torch.Tensor, positions: torch.Tensor, ctx: ForwardContext,
                hidden=None, residual=None, taps: Optional[list] = None):
        """-> the final-normed hidden rows.  ``taps``: the sum of the streams after every layer
        is appended (fp32; debugging and tests)."""
        cfg = self.cfg
        T = input_ids.shape[0]
        if self.streams is None or self.streams.shape[0] < T:
            self.prepare(cfg.max_position, max(T, 1), input_ids.device)
        eps, dt = cfg.rms_eps, self.dtype
        X, emb = self.streams[:T], self.embed_out[:T]
        ops.embed_pos(input_ids, positions, self.embed_tokens.weight, cfg.embed_scale, None, emb)
        src = emb[:, None, :].expand(T, cfg.streams, cfg.hidden_size)   # all streams alike
        hc = self.layers[0].hc1
        h = ops.hyper_norm(src, None, [], None, None, hc.w_in, hc.norm, eps, dt)
        for i, layer in enumerate(self.layers):
            last = i + 1 == len(self.layers)
            subs = [(hc, lambda h: [(layer.mix(h, positions, ctx, i), 1)])]
            if layer.mlp is not None:
                subs.append((layer.hc2, layer.mlp))
            for n, (hc, sub) in enumerate(subs):
                y = sub(h)
                if n + 1 < len(subs):
                    nxt = subs[n + 1][0]
                elif taps is not None:          # the layer's result is wanted by itself
                    taps.append(ops.hyper_norm(src, X, y, hc.mix, hc.w_out, self.sum_in, None,
                                               eps, torch.float32))
                    src, y = X, None
                    nxt = None if last else self.layers[i + 1].hc1
                else:
                    nxt = None if last else self.layers[i + 1].hc1
                w_in, norm = (nxt.w_in, nxt.norm) if nxt else (self.sum_in, self.final_norm)
                if y is None:
                    h = ops.hyper_norm(src, None, [], None, None, w_in, norm, eps, dt)
                else:
                    h = ops.hyper_norm(src, X if nxt else None, y, hc.mix, hc.w_out, w_in, norm,
                                       eps, dt)
                src, hc = X, nxt
        return h

    def compute_logits(self, hidden: torch.Tensor, gather: bool = True) -> torch.Tensor:
        return self.lm_head(hidden, gather)

    # ------------------------------------------------------------------ weights
    def load_weights(self, weights: Iterable[tuple[str, torch.Tensor]]) -> int:
        """Checkpoint names: ``embed``, ``head``, ``final.norm`` and per layer i
        ``l<i>.norm1|norm2``, ``l<i>.hc1|hc2.in|out|mix``, ``l<i>.mix.*`` (attention: q k v o
        q.norm k.norm; latent: dq dq.norm uq dkv dkv.norm uk uv g o), ``l<i>.mlp.router``,
        ``l<i>.mlp.e<j>|shared.gate|up|down``.  Returns the number loaded and raises on a name or
        a shape it does not know."""
        n = 0
        for name, w in weights:
            if not self._load_one(name, w):
                raise KeyError(f"unexpected tensor {name!r} in a Ratizen checkpoint")
            n += 1
        return n

    @staticmethod
    def _put(tgt: torch.Tensor, w: torch.Tensor) -> bool:
        if tuple(tgt.shape) != tuple(w.shape):
            raise ValueError(f"shape {tuple(w.shape)} does not fit {tuple(tgt.shape)}")
        tgt.copy_(w.to(tgt.dtype))
        return True

    def _load_one(self, name: str, w: torch.Tensor) -> bool:
        put = self._put
        if name == "embed":
            return put(self.embed_tokens.weight.data, w)
        if name == "head":
            return put(self.lm_head.weight.data, w)
        if name == "final.norm":
            return put(self.final_norm.data, (1.0 + w.float()) * self.cfg.logit_scale)
        mm = re.match(r"l(\d+)\.(.*)", name)
        if mm is None or int(mm.group(1)) >= len(self.layers):
            return False
        layer, rest = self.layers[int(mm.group(1))], mm.group(2)
        m2 = re.match(r"(norm|hc)([12])(?:\.(in|out|mix))?$", rest)
        if m2:
            hc = layer.hc1 if m2.group(2) == "1" else layer.hc2
            leaf = m2.group(3)
            if hc is None or (m2.group(1) == "hc") != (leaf is not None):
                return False
            if leaf is None:
                return put(hc.norm.data, 1.0 + w.float())
            if leaf == "out":
                return put(hc.w_out.data, w.float() * self.cfg.residual_mult)
            return put((hc.w_in if leaf == "in" else hc.mix).data, w)
        if rest.startswith("mix."):
            load = self._load_attention if layer.spec.kind == "attention" else self._load_latent
            return load(layer.mix, layer.spec, rest[4:], w)
        if rest.startswith("mlp.") and layer.mlp is not None:
            return self._load_mlp(layer.mlp, layer.spec.mlp, rest[4:], w)
        return False

    def _load_attention(self, mix: CoreAttention, sp, leaf: str, w: torch.Tensor) -> bool:
        put = self._put
        H, G, dk, dv = sp.heads, sp.kv_heads, sp.dim, sp.vdim
        off = {"q": (0, H * dk), "k": (H * dk, G * dk), "v": ((H + G) * dk, G * dv)}
        if leaf in off:
            return put(mix.qkv_proj.weight.data.narrow(0, *off[leaf]), w)
        tgt = {"o": mix.o_proj.weight, "q.norm": mix.core.q_norm, "k.norm": mix.core.k_norm}.get(leaf)
        return tgt is not None and put(tgt.data, w)

    def _load_latent(self, mix: LatentQueryAttention, sp, leaf: str, w: torch.Tensor) -> bool:
        put = self._put
        if leaf in mix.rows:
            return put(mix.proj.weight.data.narrow(0, *mix.rows[leaf]), w)
        if leaf == "uk":                    # [H d, rank] -> [H, rank, d]
            if tuple(w.shape) != (sp.heads * sp.dim, sp.kv_rank):
                raise ValueError(f"shape {tuple(w.shape)} of uk")
            return put(mix.w_uk.data, w.view(sp.heads, sp.dim, sp.kv_rank).transpose(1, 2))
        if leaf == "uv":                    # [H dv, rank] = [H, dv, rank]
            return put(mix.w_uv.data.view(sp.heads * sp.vdim, sp.kv_rank), w)
        tgt = {"uq": mix.uq_proj.weight, "o": mix.o_proj.weight, "dq.norm": mix.q_norm,
               "dkv.norm": mix.kv_norm}.get(leaf)
        return tgt is not None and put(tgt.data, w)

    def _load_mlp(self, mlp: InputScaledExperts, f, leaf: str, w: torch.Tensor) -> bool:
        if leaf == "router":
            return self._put(mlp.router.data, w)
        me = re.match(r"(e(\d+)|shared)\.(gate|up|down)$", leaf)
        if me is None:
            return False
        shared = me.group(2) is None
        e, ff = (f.experts, f.shared_ff) if shared else (int(me.group(2)), f.ff)
        if (shared and not ff) or (not shared and e >= f.experts):
            return False
        if me.group(3) == "down":
            return self._put(mlp.expert_down(e), w)
        return self._put(mlp.expert_in(e).narrow(0, 0 if me.group(3) == "gate" else ff, ff), w)
