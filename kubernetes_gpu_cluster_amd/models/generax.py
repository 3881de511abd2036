"""Generax: a decoder whose mixer and feed-forward read one norm and join the stream together.

On an fp32 residual stream x (width W):
  x = embed[token]
  per layer:  h = RMSNorm(x) w_1;   x += mixer(h) + down(silu(gate h) * up h)
  logits = cap * tanh(head(RMSNorm(x) w_f) / cap)
Layer type "attention": RMS norms over the whole q and k rows, rotation with linearly scaled
frequencies, a factor per query head on the scores, a sliding window, and values that are
cached turned by their positions (each head's output is turned back); a layer may read
another layer's cached keys and values with queries of its own.  Type "parallel": windowed
attention without rotation that also sees one mean key and value per block of tokens behind
the window, beside the gated delta rule with a decay per key channel; the result is half the
sum of the two, each RMS-normed over the width.  Any feed-forward may be absent.  Projections
run in the activation dtype with fp32 accumulation; the stream, every norm, rotation, softmax
and everything of the recurrence past its convolutions are fp32.

Kernel sequence per layer (ops/__init__.py, "Generax-style decoders"):
  residual_sum_norm (the previous layer's results join x, the normed ones normed in the same
  pass; norm) -> ONE projection GEMM for the mixer and the feed-forward ->
  attention: qk_norm_store -> window_attention | silu_mul into the two parts of one buffer ->
             ONE GEMM [o | down]
  parallel:  qk_norm_store -> window_attention (pooled rows written on the way) -> GEMM |
             causal_conv -> delta_gates -> channel_delta_scan -> head_norm_gate -> GEMM |
             silu_mul -> GEMM
One GPU per replica (TP = PP = 1).
"""
from __future__ import annotations

import re
from typing import Iterable, Optional

import torch
import torch.nn as nn

from .. import ops
from ..parallel.layers import ParallelLMHead, ReplicatedLinear, VocabParallelEmbedding
from ..parallel.state import get_state
from .attention import AttentionCore, ForwardContext
from .configs import ModelConfig
from .recurrent import ChannelDeltaCore


def _f32(shape, device, fill=0.0):
    return nn.Parameter(torch.full(shape, fill, dtype=torch.float32, device=device),
                        requires_grad=False)


def _up8(n: int) -> int:
    return -(-n // 8) * 8


class GeneraxLayer(nn.Module):
    """One layer: the merged input projection (attention | recurrence | gate | up columns,
    each part on a 16-byte border), the mixer cores, and the output projections."""

    def __init__(self, cfg: ModelConfig, idx: int, dtype, device):
        super().__init__()
        sp, W, eps = cfg.layer_specs[idx], cfg.hidden_size, cfg.rms_eps
        self.idx, self.spec = idx, sp
        self.parallel = sp.kind == "parallel"
        self.ff = sp.mlp.ff if sp.mlp else 0
        self.norm1 = _f32((W,), device, 1.0)
        self.att = AttentionCore(sp.left if self.parallel else sp, 1.0, eps, device)
        n = self.delta0 = _up8(self.att.n_in)
        self.delta = None
        if self.parallel:
            self.delta = ChannelDeltaCore(sp.right, eps, device, dtype)
            n = _up8(n + self.delta.n_in)
        self.ff0 = n
        n = -(-(n + 2 * self.ff) // 64) * 64
        lin = lambda i, o: ReplicatedLinear(i, o, dtype=dtype, device=device)   # noqa: E731
        self.in_proj = lin(W, n)
        if self.parallel:
            self.o_proj = lin(self.att.n_out, W)
            self.delta_o_proj = lin(self.delta.n_out, W)
            self.down_proj = lin(self.ff, W) if self.ff else None
            # the checkpoint's weights times the half of the sum
            self.out_norm = _f32((W,), device, 0.5)
            self.delta_out_norm = _f32((W,), device, 0.5)
        else:
            self.o_proj = lin(self.att.n_out + self.ff, W)      # [o | down]

    @property
    def own_cache(self) -> bool:
        return self.att.own_kv

    def state_shapes(self) -> tuple:
        return self.delta.state_shapes() if self.parallel else ()

    def forward(self, h: torch.Tensor, positions: torch.Tensor, ctx: ForwardContext,
                cache_idx: int, state: tuple) -> list:
        """-> [(result [T, W], norm weight or None)]: what joins the stream."""
        T, na, ff = h.shape[0], self.att.n_out, self.ff
        proj = self.in_proj(h)
        gate_up = proj[:, self.ff0: self.ff0 + 2 * ff]
        feats = torch.empty(T, na if self.parallel else na + ff, dtype=h.dtype, device=h.device)
        self.att(proj, 0, positions, ctx, cache_idx, feats[:, :na])
        if not self.parallel:
            if ff:
                ops.silu_mul(gate_up, feats[:, na:])
            return [(self.o_proj(feats), None)]
        adds = [(self.o_proj(feats), self.out_norm),
                (self.delta_o_proj(self.delta(proj, self.delta0, ctx, state)), self.delta_out_norm)]
        if ff:
            adds.append((self.down_proj(ops.silu_mul(gate_up)), None))
        return adds


class GeneraxForCausalLM(nn.Module):
    def __init__(self, cfg: ModelConfig, dtype=torch.bfloat16, device=None):
        super().__init__()
        s = get_state()
        assert s.tp_size == 1 and s.pp_size == 1, "Generax runs on one GPU per replica"
        self.cfg, self.dtype = cfg, dtype
        self.start, self.end = 0, cfg.num_layers
        self.first = self.last = True
        W, L = cfg.hidden_size, cfg.num_layers
        self.embed_tokens = VocabParallelEmbedding(cfg.vocab_size, W, dtype, device)
        self.layers = nn.ModuleList([GeneraxLayer(cfg, i, dtype, device) for i in range(L)])
        self.final_norm = _f32((W,), device, 1.0)
        self.lm_head = ParallelLMHead(cfg.vocab_size, W, dtype, device)
        # the cache every layer reads: its own, or that of the layer it names
        self.cache_of, n = [], 0
        for i, l in enumerate(self.layers):
            self.cache_of.append(n if l.own_cache else self.cache_of[l.spec.kv_from])
            n += l.own_cache
        self.stream = None          # [Tcap, W] fp32 step buffer

    # ------------------------------------------------------------------ engine hooks
    @property
    def num_local_layers(self) -> int:
        return len(self.layers)

    def local_kv_heads(self) -> int:
        return max(l.att.spec.kv_heads for l in self.layers)

    def cache_layout(self) -> list:
        """(kv heads, key size, value size, tokens per pooled row) of every layer with keys
        and values of its own."""
        return [l.att.cache_shape() for l in self.layers if l.own_cache]

    def state_layout(self) -> list:
        """Per layer, the per-slot shapes of its state tensors (parallel: convolution inputs,
        delta-rule state; attention: none)."""
        return [l.state_shapes() for l in self.layers]

    def prepare(self, max_pos: int, max_tokens: int, device) -> None:
        """Rotary tables for ``max_pos`` positions and the step buffer for ``max_tokens`` rows
        (static, so captured decode graphs replay over it)."""
        tables: dict = {}
        for l in self.layers:
            l.att.prepare(tables, max_pos, device)
        self.stream = torch.zeros(max_tokens, self.cfg.hidden_size, dtype=torch.float32,
                                  device=device)

    @torch.no_grad()
    def init_random(self, seed: int = 0, std: float = 0.02) -> None:
        """Random weights for benchmarking: projections ~ N(0, std), norm weights near 1,
        decays in the range trained models use."""
        g = torch.Generator(device="cpu").manual_seed(seed)

        def rnd(p, scale, base=0.0):
            p.copy_((torch.randn(p.shape, generator=g) * scale + base).to(p.device, p.dtype))
        for name, p in self.named_parameters():
            leaf = name.rsplit(".", 1)[-1]
            if leaf in ("norm1", "final_norm", "norm_weight", "q_norm", "k_norm"):
                rnd(p, 0.05, 1.0)
            elif leaf in ("out_norm", "delta_out_norm"):
                rnd(p, 0.02, 0.25)
            elif leaf == "neg_a":
                p.copy_(-(1.0 + 7.0 * torch.rand(p.shape, generator=g)).to(p.device))
            elif leaf == "dt_bias":
                rnd(p, 0.5, -4.0)
            elif leaf == "conv_w":
                rnd(p, 0.3)
            elif leaf in ("a2", "g2"):
                rnd(p, 0.1)
            else:
                rnd(p, std)
        for l in self.layers:       # padding columns are zeros, as in a loaded model
            if l.delta is not None:
                l.delta.a2[:, l.delta.spec.decay_rank:] = 0
                l.delta.g2[:, l.delta.spec.gate_rank:] = 0

    # ------------------------------------------------------------------ forward
    def forward(self, input_ids: torch.Tensor, positions: torch.Tensor, ctx: ForwardContext,
                hidden=None, residual=None, taps: Optional[list] = None):
        """-> the final-normed hidden rows.  ``taps``: the residual stream after every layer
        is appended (fp32 copies; debugging and tests)."""
        cfg = self.cfg
        T = input_ids.shape[0]
        if self.stream is None or self.stream.shape[0] < T:
            self.prepare(cfg.max_position, max(T, 1), input_ids.device)
        eps, dt = cfg.rms_eps, self.dtype
        x = self.stream[:T]
        ops.embed_pos(input_ids, positions, self.embed_tokens.weight, 1.0, None, x)
        adds: list = []                     # results that have not joined x yet
        for i, layer in enumerate(self.layers):
            h = ops.residual_sum_norm(x, adds, layer.norm1, eps, dt)
            adds = layer(h, positions, ctx, self.cache_of[i], ctx.states[i])
            if taps is not None:
                ops.residual_sum_norm(x, adds, None, eps, None)
                adds = []
                taps.append(x.clone())
        return ops.residual_sum_norm(x, adds, self.final_norm, eps, dt)

    def compute_logits(self, hidden: torch.Tensor, gather: bool = True) -> torch.Tensor:
        logits, cap = self.lm_head(hidden, gather), self.cfg.logit_softcap
        return ops.logit_softcap(logits, cap) if cap > 0 else logits

    # ------------------------------------------------------------------ weights
    def load_weights(self, weights: Iterable[tuple[str, torch.Tensor]]) -> int:
        """Checkpoint names: ``embed``, ``head``, ``final.norm`` and per layer i ``l<i>.norm1``,
        ``l<i>.mlp.gate|up|down``, and ``l<i>.mix.*``: an attention layer's q k v o q.norm
        k.norm temp (no k, v, k.norm where it reads another layer's), or left.q|k|v|o|q.norm|
        k.norm|out and right.q|k|v (+ .conv), right.b|A_log|a1|a2|dt_bias|g1|g2|norm|o|out.
        Returns the number loaded and raises on a name or a shape it does not know."""
        with torch.no_grad():
            for l in self.layers:
                # q.norm and temp multiply into one parameter, in whatever order they come
                l.att.q_norm.fill_(1.0)
                l.in_proj.weight.zero_()            # padding columns stay zero
        n = 0
        for name, w in weights:
            if not self._load_one(name, w):
                raise KeyError(f"unexpected tensor {name!r} in a Generax checkpoint")
            n += 1
        return n

    @staticmethod
    def _put(tgt: torch.Tensor, w: torch.Tensor) -> bool:
        if tuple(tgt.shape) != tuple(w.shape):
            raise ValueError(f"shape {tuple(w.shape)} does not fit {tuple(tgt.shape)}")
        tgt.copy_(w.to(tgt.dtype))
        return True

    def _load_one(self, name: str, w: torch.Tensor) -> bool:
        put, dt = self._put, self.dtype
        if name == "embed":
            self.embed_tokens.weight.weight_loader(self.embed_tokens.weight, w.to(dt))
            return True
        if name == "head":
            self.lm_head.weight.weight_loader(self.lm_head.weight, w.to(dt))
            return True
        if name == "final.norm":
            return put(self.final_norm.data, w)
        mm = re.match(r"l(\d+)\.(.*)", name)
        if mm is None or int(mm.group(1)) >= len(self.layers):
            return False
        layer, rest = self.layers[int(mm.group(1))], mm.group(2)
        if rest == "norm1":
            return put(layer.norm1.data, w)
        if rest.startswith("mlp.") and layer.ff:
            return self._load_mlp(layer, rest[4:], w)
        if layer.parallel and rest.startswith("mix.left."):
            return self._load_attention(layer, rest[9:], w)
        if layer.parallel and rest.startswith("mix.right."):
            return self._load_delta(layer, rest[10:], w)
        if not layer.parallel and rest.startswith("mix."):
            return self._load_attention(layer, rest[4:], w)
        return False

    def _load_mlp(self, layer: GeneraxLayer, leaf: str, w: torch.Tensor) -> bool:
        ff = layer.ff
        if leaf in ("gate", "up"):
            a = layer.ff0 + (ff if leaf == "up" else 0)
            return self._put(layer.in_proj.weight.data.narrow(0, a, ff), w)
        if leaf != "down":
            return False
        return self._put(layer.down_proj.weight.data if layer.parallel
                         else layer.o_proj.weight.data[:, layer.att.n_out:], w)

    def _load_attention(self, layer: GeneraxLayer, leaf: str, w: torch.Tensor) -> bool:
        put, att = self._put, layer.att
        sp = att.spec
        H, G, dk, dv = sp.heads, sp.kv_heads, sp.dim, sp.vdim
        off = {"q": (0, H * dk)}
        if att.own_kv:
            off.update(k=(H * dk, G * dk), v=((H + G) * dk, G * dv))
        if leaf in off:
            return put(layer.in_proj.weight.data.narrow(0, *off[leaf]), w)
        if leaf == "o":
            return put(layer.o_proj.weight.data[:, : att.n_out], w)
        if leaf == "q.norm":
            return put(att.q_norm.data, w.float().to(att.q_norm.device) * att.q_norm.data)
        if leaf == "temp" and sp.head_temp:
            f = w.float().to(att.q_norm.device).repeat_interleave(dk)
            return put(att.q_norm.data, f * att.q_norm.data)
        if leaf == "k.norm" and att.own_kv:
            return put(att.k_norm.data, w)
        if leaf == "out" and layer.parallel:
            return put(layer.out_norm.data, _share(layer.spec.left_scale, w))
        return False

    def _load_delta(self, layer: GeneraxLayer, leaf: str, w: torch.Tensor) -> bool:
        put, core = self._put, layer.delta
        sp = core.spec
        if leaf in core.cols:
            a, n = core.cols[leaf]
            return put(layer.in_proj.weight.data.narrow(0, layer.delta0 + a, n), w)
        if leaf in ("q.conv", "k.conv", "v.conv"):
            return put(core.conv_w.data.narrow(0, *core.cols[leaf[0]]), w)
        if leaf == "A_log":
            return put(core.neg_a.data, (-torch.exp(w.float())).repeat_interleave(sp.dim))
        if leaf == "norm":
            return put(core.norm_weight.data, w.float().repeat(sp.heads))
        if leaf == "out":
            return put(layer.delta_out_norm.data, _share(layer.spec.right_scale, w))
        tgt = {"a2": core.a2.data[:, : sp.decay_rank], "g2": core.g2.data[:, : sp.gate_rank],
               "dt_bias": core.dt_bias.data, "o": layer.delta_o_proj.weight.data}.get(leaf)
        return tgt is not None and put(tgt, w)


def _share(scale: float, w: torch.Tensor) -> torch.Tensor:
    """A mixer's share of the parallel sum, carried by its output norm's weight."""
    return w.float() * scale
