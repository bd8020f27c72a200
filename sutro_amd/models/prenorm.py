"""Layer-list decoders of pre-norm layers,

    x <- x + mixer(n1(x));   x <- x + ff(n2(x))            (ff optional)

with weighted RMS norms: the block and the model that the designs of this form
share (which mixers, feed-forwards, embedding and head a model has is in its
spec). A run of layers may be passed several times with the same weights
(`spec.loop`): every pass has pages and state of its own, and (by default) the
embedding output is added to the stream before each pass but the first.

The residual stream is fp32. Per sublayer: one merged input GEMM, the mixer's
kernels, one output GEMM, and ONE kernel that adds the sublayer's result (for
routed experts: the weighted gather of a token's expert rows, the identity
share of its input and the shared expert; at the end of a pass: the embedding
output) to the stream and emits the next sublayer's normed input.

With `spec.streams` the residual is a bundle of streams (hyper-connections,
`layers.HyperConnection`): a sublayer reads a weighted sum of them, and the
same one kernel mixes the streams, adds the result to all of them and emits the
next sublayer's normed input. The bundle is [T, streams, W] fp32; it is first
written by the first layer's mixer (before that all streams are the embedding
output) and the last sublayer of a step only makes the final normed sum.
"""

from __future__ import annotations

import math
import zlib
from typing import Dict, Optional

import torch
import torch.nn as nn
import torch.nn.functional as F

from ..engine.batch import ForwardBatch
from ..engine.kv_cache import PagedKVCache
from ..ops import hybrid as hops
from ..parallel.tp import TPContext
from .hybrid_spec import (AttnMixerSpec, DecayAttnMixerSpec, DeltaMixerSpec,
                          HybridLayerSpec, HybridSpec, LatentAttnMixerSpec,
                          SSDMixerSpec)
from .layers import (DecayAttention, GatedDeltaRule, HyperConnection,
                     LatentAttention, LocalAttention, RoutedExperts,
                     SectionedLinear, SSDMixer, _pad)


class PreNormBlock(nn.Module):
    """One layer: norm, merged input projection, mixer, output projection;
    norm, feed-forward (dense, gated or squared-ReLU, or routed experts)."""

    def __init__(self, spec: HybridSpec, layer: HybridLayerSpec, idx: int,
                 dtype: torch.dtype):
        super().__init__()
        W = spec.hidden_size
        self.idx = idx
        self.eps = spec.norm_eps
        m = layer.mixer
        if isinstance(m, AttnMixerSpec):
            self.mixer = LocalAttention(m, spec.norm_eps, idx)
        elif isinstance(m, DecayAttnMixerSpec):
            self.mixer = DecayAttention(m, spec.norm_eps, idx)
        elif isinstance(m, SSDMixerSpec):
            self.mixer = SSDMixer(m, spec.norm_eps, idx)
        elif isinstance(m, LatentAttnMixerSpec):
            self.mixer = LatentAttention(m, spec.norm_eps, idx, dtype)
        elif isinstance(m, DeltaMixerSpec):
            self.mixer = GatedDeltaRule(m, spec.norm_eps, idx)
        else:
            raise ValueError(f"layer {idx}: unsupported mixer "
                             f"{type(m).__name__}")
        f32 = torch.float32
        self.norm1 = nn.Parameter(torch.ones(W, dtype=f32))
        self.in_proj = SectionedLinear(W, self.mixer.in_sections(""), dtype)
        k = _pad(self.mixer.out_width)
        self.out_padded = k != self.mixer.out_width
        self.out_proj = nn.Linear(k, W, bias=False, dtype=dtype)
        self.ff = layer.ff
        self.relu2 = layer.ff_kind == "relu2"
        self.experts: Optional[RoutedExperts] = None
        if layer.ff or layer.moe is not None:
            self.norm2 = nn.Parameter(torch.ones(W, dtype=f32))
        if layer.ff:
            self.ff_in = SectionedLinear(
                W, [("up", layer.ff, False)] if self.relu2 else
                [("gate", layer.ff, False), ("up", layer.ff, False)], dtype)
            self.ff_out = nn.Linear(layer.ff, W, bias=False, dtype=dtype)
        if layer.moe is not None:
            self.experts = RoutedExperts(layer.moe, W, dtype)
        self.streams = spec.streams
        self.hc1 = self.hc2 = None
        if spec.streams:
            self.hc1 = HyperConnection(spec.streams)
            if self.has_ff:
                self.hc2 = HyperConnection(spec.streams)
            if layer.moe is not None and (
                    layer.moe.identity
                    or (layer.moe.shared_ff and layer.moe.shared_gate)):
                raise ValueError(f"layer {idx}: several streams go with "
                                 f"ungated shared experts, not with identity "
                                 f"experts")

    @property
    def has_ff(self) -> bool:
        return bool(self.ff) or self.experts is not None

    def checkpoint_targets(self, prefix: str,
                           norm_offset: float) -> Dict[str, tuple]:
        lp = f"l{self.idx}"
        ck = lp + ".mix"
        W = self.norm1.numel()
        t = {lp + ".norm1": (prefix + "norm1", 0, 0, W, 1.0, norm_offset)}
        t.update(self.in_proj.section_targets(
            prefix + "in_proj.", self.mixer.section_names("", ck)))
        if hasattr(self.mixer, "param_targets"):
            t.update(self.mixer.param_targets(prefix + "mixer.", ck))
        if isinstance(self.mixer, LocalAttention):
            # a layer that does not blend may still carry the (unused) weight
            t[ck + ".vmix"] = (prefix + "mixer.v_lambda", None, 0, 0, 1.0) \
                if self.mixer.spec.v_mix else None
        t[ck + ".o"] = (prefix + "out_proj.weight", 1, 0,
                        self.mixer.out_width, 1.0)
        # a layer without a feed-forward may still carry its (unused) norm and
        # stream weights
        t[lp + ".norm2"] = (prefix + "norm2", 0, 0, W, 1.0, norm_offset) \
            if self.has_ff else None
        for n, hc in (("hc1", self.hc1), ("hc2", self.hc2)):
            if self.streams:
                t.update(HyperConnection.targets(
                    f"{prefix}{n}.", f"{lp}.{n}", self.streams)
                    if hc is not None else
                    {f"{lp}.{n}.{k}": None for k in ("in", "out", "mix")})
        if self.ff:
            t.update(self.ff_in.section_targets(
                prefix + "ff_in.",
                {n: f"{lp}.mlp.{n}" for n in self.ff_in.offsets}))
            t[lp + ".mlp.down"] = (prefix + "ff_out.weight", 1, 0, self.ff, 1.0)
        if self.experts is not None:
            t.update(self.experts.param_targets(prefix + "experts.",
                                                lp + ".mlp"))
        return t

    def _join(self, x: torch.Tensor, h: torch.Tensor,
              hc: Optional[HyperConnection], norm_w: torch.Tensor,
              next_in: Optional[torch.Tensor], x_in=None, extra=None,
              write: bool = True, y=None, rows=None, padpos=None, wts=None,
              idw=None, y2=None, proj2=None, sg: int = -1) -> None:
        """Take a sublayer's result (y, expert rows, shared expert y2) into
        the residual and make the next sublayer's input in h. One kernel."""
        if hc is None:
            # h is read (identity experts) and rewritten row by row
            hops.add_rmsnorm(x, y, rows, padpos, wts, idw,
                             h if idw is not None else None, y2, proj2, sg,
                             norm_w, self.eps, h, x_in=x_in, extra=extra)
        else:
            hops.hyper_rmsnorm(x, x_in, y, rows, padpos, wts, y2, hc.w_mix,
                               hc.w_out, next_in, norm_w, self.eps, h, write)

    def forward(self, x: torch.Tensor, h: torch.Tensor, fb: ForwardBatch,
                kv: PagedKVCache, next_norm: torch.Tensor,
                cache_idx: Optional[int] = None,
                x_in: Optional[torch.Tensor] = None,
                extra: Optional[torch.Tensor] = None,
                next_in: Optional[torch.Tensor] = None,
                write: bool = True) -> None:
        """x fp32 [T, W]: the stream, updated in place (read from `x_in`
        instead, if given); with several streams [T, streams, W], each of
        which is x_in, if given. h [T, W] activation type: this layer's normed
        input, overwritten with the next layer's (normed with the weight
        `next_norm`; with several streams their sum weighted by `next_in`).
        `cache_idx`: which pages or state this run uses. `extra` fp32 [T, W]:
        joins the stream behind the layer (single streams). `write` off:
        nobody reads the streams behind this layer."""
        T = h.shape[0]
        proj = self.in_proj(h)
        alloc = torch.zeros if self.out_padded else torch.empty
        mix_in = alloc((T, self.out_proj.in_features), dtype=h.dtype,
                       device=h.device)
        # one run per layer: the mixer's own layer index is its cache
        kw = {} if cache_idx is None or cache_idx == self.idx \
            else {"cache_idx": cache_idx}
        self.mixer(proj, self.in_proj.offsets, "", fb, kv, mix_in, 0, 1.0, **kw)
        y = self.out_proj(mix_in)
        if not self.has_ff:
            self._join(x, h, self.hc1, next_norm, next_in, x_in, extra, write,
                       y=y)
            return
        self._join(x, h, self.hc1, self.norm2,
                   self.hc2.w_in if self.streams else None, x_in, y=y)
        if self.ff:
            proj = self.ff_in(h)
            off = self.ff_in.offsets
            if self.relu2:
                act = hops.relu_sq(proj)[:, :self.ff]
            else:
                act = hops.glu_mul(proj, off["gate"], off["up"], self.ff,
                                   hops.GLU_SILU)
            self._join(x, h, self.hc2, next_norm, next_in, None, extra, write,
                       y=self.ff_out(act))
            return
        ex = self.experts
        rows, padpos, wts, idw = ex(h, fb.input_ids, fb.aux)
        y2 = proj2 = None
        sg = -1
        if ex.spec.shared_ff:
            y2, proj2, sg = ex.shared_forward(h)
        self._join(x, h, self.hc2, next_norm, next_in, None, extra, write,
                   rows=rows, padpos=padpos, wts=wts, idw=idw, y2=y2,
                   proj2=proj2, sg=sg)


class PreNormModel(nn.Module):
    """Scaled token rows (+ hashed-bigram rows), the layers, a final norm, a
    tied or untied head, scaled logits. Same engine-facing surface as the other models: forward(fb, kv) ->
    hidden rows, compute_logits(hidden), cache_layout(),
    checkpoint_targets(), init_random_weights()."""

    def __init__(self, spec: HybridSpec, dtype: torch.dtype, max_len: int,
                 tp: Optional[TPContext] = None):
        super().__init__()
        self.spec = spec
        self.tp = tp or TPContext()
        if self.tp.size > 1:
            raise NotImplementedError(
                "layer-list decoders run on one GPU per replica (the "
                "recurrent state is not sharded); use data parallelism")
        W = spec.hidden_size
        self.embed_tokens = nn.Embedding(spec.vocab_size, W, dtype=dtype)
        # with a bigram table the embedding looks at (previous token, token)
        # pairs: the engine fills ForwardBatch.prev_ids
        self.uses_prev_ids = spec.bigram is not None
        if spec.bigram:
            self.bigram = nn.Embedding(spec.bigram[0] + 1, W, dtype=dtype)
        self.layers = nn.ModuleList(
            [PreNormBlock(spec, layer, i, dtype)
             for i, layer in enumerate(spec.layers)])
        self.final_norm = nn.Parameter(torch.ones(W, dtype=torch.float32))
        if spec.streams:   # the model's output is the plain sum of the streams
            self.register_buffer("sum_in", torch.ones(spec.streams),
                                 persistent=False)
        if not spec.tie_embeddings:
            self.lm_head = nn.Linear(W, spec.vocab_size, bias=False, dtype=dtype)
        self.act_dtype = dtype
        # debugging aid: when set to a list, the fp32 residual stream after
        # every layer run is appended to it
        self.layer_taps: Optional[list] = None

    def cache_layout(self):
        """(KV shapes, recurrent state shapes) of every layer run."""
        mixers = [self.layers[i].mixer for i, _ in self.spec.runs]
        return ([m.kv_shape() for m in mixers],
                [m.state_shape() for m in mixers])

    def checkpoint_targets(self) -> Dict[str, tuple]:
        s = self.spec
        t = {"embed": ("embed_tokens.weight", 0, 0, s.vocab_size, 1.0),
             "final.norm": ("final_norm", 0, 0, s.hidden_size, 1.0,
                            s.norm_offset)}
        if not s.tie_embeddings:
            t["head"] = ("lm_head.weight", 0, 0, s.vocab_size, 1.0)
        if s.bigram:
            t["bigram"] = ("bigram.weight", 0, 0, s.bigram[0] + 1, 1.0)
        for i, blk in enumerate(self.layers):
            t.update(blk.checkpoint_targets(f"layers.{i}.", s.norm_offset))
        return t

    def check_loaded(self) -> None:
        for blk in self.layers:
            if blk.experts is not None:
                blk.experts.check_loaded()

    @torch.no_grad()
    def forward(self, fb: ForwardBatch, kv: PagedKVCache) -> torch.Tensor:
        # per-step scratch (rotation tables, the first blending layer's
        # values, expert layouts) is rebuilt on every pass
        fb.aux.clear()
        s = self.spec
        T = fb.input_ids.shape[0]
        big = s.bigram or (0, 0, 0)
        e0 = hops.token_embed(fb.input_ids, fb.prev_ids if s.bigram else None,
                              fb.positions, self.embed_tokens.weight,
                              self.bigram.weight if s.bigram else None,
                              big[0], big[1], big[2], None,
                              scale=s.embed_scale)
        h = torch.empty((T, s.hidden_size), dtype=self.act_dtype,
                        device=e0.device)
        runs = s.runs
        n = len(runs)
        if s.streams and n:
            return self._forward_streams(e0, h, fb, kv)
        hops.add_rmsnorm(e0, norm_w=self.layers[runs[0][0]].norm1 if n
                         else self.final_norm, eps=s.norm_eps, h_out=h)
        # a looped model needs the embedding output again: the stream then
        # gets a buffer of its own
        x = torch.empty_like(e0) if s.loop else e0
        for j, (i, _) in enumerate(runs):
            nxt, extra = self.final_norm, None
            if j + 1 < n:
                ni, npass = runs[j + 1]
                nxt = self.layers[ni].norm1
                if npass and ni == s.loop[0] and s.loop_reenter:
                    extra = e0
            self.layers[i](x, h, fb, kv, nxt, cache_idx=j,
                           x_in=e0 if j == 0 and s.loop else None, extra=extra)
            if self.layer_taps is not None:
                self.layer_taps.append(x.clone() if extra is None
                                       else x - extra)
        return h

    def _forward_streams(self, e0: torch.Tensor, h: torch.Tensor,
                         fb: ForwardBatch, kv: PagedKVCache) -> torch.Tensor:
        """The layer runs over a bundle of streams (all of them e0 at first)."""
        s = self.spec
        runs = s.runs
        x = torch.empty((e0.shape[0], s.streams, s.hidden_size),
                        dtype=torch.float32, device=e0.device)
        first = self.layers[runs[0][0]]
        hops.hyper_rmsnorm(x, e0, in_w=first.hc1.w_in, norm_w=first.norm1,
                           eps=s.norm_eps, h_out=h)
        taps = self.layer_taps
        for j, (i, _) in enumerate(runs):
            last = j + 1 == len(runs)
            nxt = None if last else self.layers[runs[j + 1][0]]
            self.layers[i](
                x, h, fb, kv, self.final_norm if last else nxt.norm1,
                cache_idx=j, x_in=e0 if j == 0 else None,
                next_in=self.sum_in if last else nxt.hc1.w_in,
                write=not last or taps is not None)
            if taps is not None:
                taps.append(x.sum(dim=1))
        return h

    @torch.no_grad()
    def compute_logits(self, hidden: torch.Tensor) -> torch.Tensor:
        logits = F.linear(hidden, self.embed_tokens.weight
                          if self.spec.tie_embeddings
                          else self.lm_head.weight).float()
        if self.spec.logit_scale != 1.0:
            logits = logits * self.spec.logit_scale
        return logits

    @torch.no_grad()
    def init_random_weights(self, seed: int = 0) -> None:
        """Deterministic random init on the parameters' own device, scaled so
        activations, decays and router scores stay in a sane range at any
        width."""
        for name, p in sorted(self.named_parameters()):
            gen = torch.Generator(device=p.device)
            gen.manual_seed(seed * 1000003 + zlib.crc32(name.encode()))

            def rnd(shape, std):
                return torch.randn(shape, generator=gen, dtype=torch.float32,
                                   device=p.device) * std

            leaf = name.rsplit(".", 1)[-1]
            if leaf in ("norm1", "norm2", "final_norm", "norm_w", "dkv_norm",
                        "dq_norm"):
                p.copy_(1.0 + rnd(p.shape, 0.05))
            elif leaf == "v_lambda":
                p.fill_(0.3)
            elif leaf == "sink_w":
                p.copy_(rnd(p.shape, 0.5))
            elif leaf == "w_in":    # streams: read about their mean,
                p.copy_((1.0 + rnd(p.shape, 0.2)) / p.shape[0])
            elif leaf == "w_out":   # written with about the full result,
                p.copy_(1.0 + rnd(p.shape, 0.2))
            elif leaf == "w_mix":   # mixed a little
                S = p.shape[0]
                p.copy_((torch.eye(S, device=p.device) + rnd(p.shape, 0.1))
                        / (1.0 + 0.1 * S ** 0.5))
            elif leaf == "a_log":
                p.copy_(rnd(p.shape, 0.3) - 0.5)
            elif leaf == "dt_bias":
                p.copy_(rnd(p.shape, 0.5) - 1.0)
            elif leaf == "skip":
                p.copy_(1.0 + rnd(p.shape, 0.1))
            elif leaf == "conv_w":
                p.copy_(rnd(p.shape, 0.4))
            elif leaf in ("conv_b", "correction"):
                p.copy_(rnd(p.shape, 0.02))
            elif leaf == "bias":
                p.copy_(rnd(p.shape, 0.02).to(p.dtype))
            elif leaf == "router":
                p.copy_(rnd(p.shape, 2.0 / math.sqrt(p.shape[-1])))
            elif leaf == "table":   # `top` neighbours from a random expert on
                E = self.layers[int(name.split(".")[1])].experts.spec.experts
                first = torch.randint(E, (p.shape[0], 1), generator=gen,
                                      device=p.device)
                step = torch.arange(p.shape[1], device=p.device)
                p.copy_(((first + step) % E).to(p.dtype))
            elif name.startswith(("embed_tokens", "bigram")):
                # a tied head reads the table as an output projection
                std = 1.0 / math.sqrt(p.shape[1]) if self.spec.tie_embeddings \
                    and name.startswith("embed_tokens") else 1.0
                p.copy_(rnd(p.shape, std).to(p.dtype))
            else:
                p.copy_(rnd(p.shape, 1.0 / math.sqrt(p.shape[-1])).to(p.dtype))
        # padding rows/columns of merged projections stay zero
        for blk in self.layers:
            lins = [blk.in_proj]
            if blk.ff:
                lins.append(blk.ff_in)
            if blk.experts is not None and blk.experts.spec.shared_ff:
                lins.append(blk.experts.shared_in)
            for lin in lins:
                keep = torch.zeros(lin.out_features, dtype=torch.bool,
                                   device=lin.weight.device)
                for sec, o in lin.offsets.items():
                    keep[o:o + lin.sizes[sec]] = True
                lin.weight[~keep] = 0
                if lin.bias is not None:
                    lin.bias[~keep] = 0
            blk.out_proj.weight[:, blk.mixer.out_width:] = 0
