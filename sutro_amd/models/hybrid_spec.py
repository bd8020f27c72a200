"""Specs for layer-list ("hybrid") decoders: every layer names its own token
mixer and feed-forward, so attention layers, recurrent layers and layers that
run both side by side can be ordered freely.

A spec is built from a checkpoint's ``config.json`` (see :func:`vodinex_spec`,
:func:`ruludra_spec`, :func:`vukotar_spec`, :func:`nosalorn_spec`,
:func:`vanulorn_spec` and :func:`tubepel_spec`) or directly in code (tests,
benchmarks). Nothing here fixes a size: widths, head counts, mask sizes, filter
lengths and the order of layers all come from the config.
"""

from __future__ import annotations

from dataclasses import dataclass
from typing import Optional, Tuple, Union


@dataclass(frozen=True)
class AttnMixerSpec:
    """Softmax attention with grouped key/value heads over a local mask.

    ``chunk``: a query at position i sees keys j <= i with
    ``j // chunk == i // chunk`` (0 = no chunking). ``window``: a query sees
    at most the last ``window`` keys (0 = unlimited). Both may be combined.
    ``keep_first``: with a window, keys at positions below `keep_first` stay
    visible to every later query (at their true positions).
    ``rot_dims``: how many leading dimensions of each head are rotated
    (rotate-half pairing inside that prefix); 0 = no rotation.
    ``rot_scaling``: (factor, original length, fast turns, slow turns) of a
    YaRN frequency blend: frequencies that turn fewer than `slow` times over
    the original length are divided by `factor`, those that turn more than
    `fast` times are kept, a linear ramp over the pair index lies between,
    and cos / sin are multiplied by 0.1 ln(factor) + 1.
    ``v_mix``: the values of every such layer but the first are blended with
    the first such layer's values of the same token, v <- (1 - l) v + l v1,
    with a learned scalar l; the blend is what the cache holds."""

    heads: int
    kv_heads: int
    dim: int                 # per-head query/key size
    vdim: int                # per-head value size
    scale: float
    rot_dims: int = 0
    rot_base: float = 10000.0
    chunk: int = 0
    window: int = 0
    qk_norm: bool = True
    bias: bool = True        # q/k/v/o projections carry biases
    out_gate: bool = True    # sigmoid gate on the attention output
    gate_elements: bool = False  # one gate per element instead of one per head
    # a silent sink: a key of score 0 without a value takes part in the
    # normalisation, p_j = exp(s_j) / (1 + sum_j exp(s_j))
    sink: bool = False
    # the sink's score is a learned number per head instead of 0
    sink_learned: bool = False
    keep_first: int = 0
    rot_scaling: Optional[Tuple[float, float, float, float]] = None
    v_mix: bool = False
    out_bias: bool = True    # with `bias`: the output projection has one too


@dataclass(frozen=True)
class DeltaMixerSpec:
    """Gated delta rule fed through short causal depthwise filters.

    ``decay`` "channel": one decay per head and key channel from a low-rank
    projection of inner size ``decay_rank``; "head": one decay per head from a
    plain projection. ``gate`` "low_rank": the read-out is gated by the
    sigmoid of a low-rank projection of inner size ``gate_rank``; "silu": by
    the silu of a full projection. (The ranks are read from the
    checkpoint.)"""

    heads: int
    kv_heads: int
    dim: int
    vdim: int
    conv: int                # filter taps (the last tap is the current token)
    decay_rank: int = 0
    gate_rank: int = 0
    decay: str = "channel"
    gate: str = "low_rank"


@dataclass(frozen=True)
class ParallelMixerSpec:
    """An attention mixer and a delta-rule mixer reading the same input; the
    result is ``left_scale * left + right_scale * right``."""

    left: AttnMixerSpec
    right: DeltaMixerSpec
    left_scale: float
    right_scale: float


@dataclass(frozen=True)
class TiedAttnMixerSpec:
    """Windowed softmax attention whose values are its raw keys (no value
    projection): q and k are RMS-normed over the whole projection (all heads
    at once), q is scaled by 1 + temp_coef * ln(floor((p+1)/temp_every) + 1)
    at position p (temp_every 0 = off), and with `dist_bias` the score of
    query i and key j is lowered by r1[h] * ln(1 + r2[h] * (i - j)). No
    rotation. ``window``: a query sees itself and the window-1 keys before it
    (0 = unlimited)."""

    heads: int
    kv_heads: int
    dim: int
    scale: float
    window: int = 0
    temp_coef: float = 0.0
    temp_every: int = 0
    dist_bias: bool = True


@dataclass(frozen=True)
class LatentAttnMixerSpec:
    """Attention through low-rank latents: queries are up-projected from a
    normed latent of size q_rank (0: projected directly); keys and values are
    up-projected per head from one normed latent of size kv_rank, which is all
    the cache holds. ``out_gate``: the concatenated heads pass an elementwise
    sigmoid gate. ``kv_from``: index of an earlier layer whose cached latent
    this layer reads instead of making its own.
    ``rot_dim``: that many further query dimensions per head are rotated and
    meet one rotated key part shared by all heads (projected beside the
    latent, not normed, cached beside it); 0 = no positions. ``rot_base`` and
    ``rot_scaling`` as in :class:`AttnMixerSpec`. ``rot_adjacent``: dimensions
    2i and 2i + 1 of the rotated part turn together instead of i and i +
    rot_dim / 2."""

    heads: int
    dim: int
    vdim: int
    q_rank: int
    kv_rank: int
    scale: float
    window: int = 0
    kv_from: Optional[int] = None
    rot_dim: int = 0
    rot_base: float = 10000.0
    rot_scaling: Optional[Tuple[float, float, float, float]] = None
    out_gate: bool = True
    rot_adjacent: bool = False


@dataclass(frozen=True)
class MLSTMMixerSpec:
    """mLSTM matrix memory: per head a [dim, vdim] state with exponential
    input gate, sigmoid forget gate (both soft-capped at ``gate_cap`` in log
    space) and a running-maximum stabiliser; read-out normed per head and
    gated elementwise."""

    heads: int
    dim: int
    vdim: int
    gate_cap: float


@dataclass(frozen=True)
class DecayAttnMixerSpec:
    """Linear attention with one fixed decay per head: S_t = decay_h S_(t-1)
    + k_t v_t^T, o_t = S_t^T q_t.

    ``act`` "silu" ("lightning" attention): q, k, v pass silu. "none"
    (retention): q and k are rotated on their first ``rot_dims`` dimensions
    (0 = not at all) and k is multiplied by ``k_scale``.
    ``norm`` "all": the concatenated heads pass one weighted RMS norm; "head":
    every head is divided by its own root mean square, without a weight.
    ``gate``: elementwise "sigmoid" or "silu" gate after the norm."""

    heads: int
    dim: int
    vdim: int
    decay: Tuple[float, ...]
    act: str = "silu"
    rot_dims: int = 0
    rot_base: float = 10000.0
    rot_scaling: Optional[Tuple[float, float, float, float]] = None
    k_scale: float = 1.0
    norm: str = "all"
    gate: str = "sigmoid"


@dataclass(frozen=True)
class SSDMixerSpec:
    """Mamba-2 state-space layer: one projection gives gate z, input x, the
    grouped B and C and a step per head; x|B|C pass a short causal filter with
    bias and silu; per head S_t = exp(-exp(A_log) dt) S_(t-1) + dt B_t x_t^T
    ([state, vdim]), y_t = S_t^T C_t + D x_t; y * silu(z) is RMS-normed in
    `norm_groups` equal parts."""

    heads: int
    vdim: int
    state: int
    groups: int
    conv: int
    norm_groups: int = 1


MixerSpec = Union[AttnMixerSpec, DeltaMixerSpec, ParallelMixerSpec,
                  TiedAttnMixerSpec, LatentAttnMixerSpec, MLSTMMixerSpec,
                  DecayAttnMixerSpec, SSDMixerSpec]


@dataclass(frozen=True)
class RoutedExpertsSpec:
    """Mixture-of-experts feed-forward: `experts` small two-matrix
    feed-forwards of inner width `ff`, of which a token uses `top`.

    ``router``: "sigmoid" scores every expert by the sigmoid of its logit and
    weights the chosen ones by score / (sum of chosen scores + 1e-20), or by
    the score itself (``renorm`` off). ``weigh_input``: the weight multiplies
    the input of an expert instead of its result.
    ``groups`` / ``keep``: the experts form `groups` equal runs of neighbours;
    a run is worth the sum of its `group_rank` largest scores and only experts
    of the `keep` best runs can be chosen (groups = keep = 1: no restriction).
    ``act``: "relu2" = the square of relu between the two matrices.

    ``router`` "softmax": scores are the softmax over all router outputs;
    the choice (and the worth of a group, with `group_rank` 1 its largest
    member) looks at score + `correction` (a learned vector), experts outside
    the kept groups cannot be chosen whatever their sign, and the weights are
    the plain scores times `route_scale`, not renormalised. The last
    `identity` router outputs are identity experts (result = the input) that
    have no matrices; they belong to the groups like the others.
    ``act`` "clamped_glu": three-matrix experts, g = min(gate h, limit),
    u = clamp(up h, -limit, limit), down(g sigmoid(1.702 g) (u + 1)).
    ``act`` "silu_glu": three-matrix experts, down(silu(gate h) (up h)).
    ``router`` "table": no router; row `token id` of an integer table names
    the token's experts, each with weight 1 / top.
    ``shared_ff``: inner width of a shared expert of the same form (own
    `shared_limit`) that every token uses, weighted by the sigmoid of a
    one-row projection of the input (``shared_gate``) or simply added; 0 =
    none. ``vocab``: rows of the table."""

    ff: int
    experts: int
    top: int
    groups: int = 1
    keep: int = 1
    group_rank: int = 2
    router: str = "sigmoid"
    act: str = "relu2"
    identity: int = 0
    route_scale: float = 1.0
    correction: bool = False
    limit: float = 0.0
    shared_ff: int = 0
    shared_limit: float = 0.0
    shared_gate: bool = True
    vocab: int = 0
    renorm: bool = True
    weigh_input: bool = False


@dataclass(frozen=True)
class HybridLayerSpec:
    kind: str                # the config's layer type
    mixer: MixerSpec
    ff: int = 0              # 0 = the layer has no (dense) feed-forward
    # how a dense feed-forward looks where designs differ: "swiglu" =
    # down(silu(gate h) (up h)), "relu2" = down(max(up h, 0)^2)
    ff_kind: str = "dense"
    moe: Optional[RoutedExpertsSpec] = None
    # index of the layer whose parameters this layer uses (its cache is its
    # own); None = the layer has parameters of its own
    weights_of: Optional[int] = None


@dataclass(frozen=True)
class HybridSpec:
    """Engine-facing spec of a layer-list decoder (the counterpart of
    ``registry.ModelSpec`` for the uniform Qwen3 family)."""

    name: str
    arch: str
    hidden_size: int
    vocab_size: int
    layers: Tuple[HybridLayerSpec, ...]
    norm_eps: float = 1e-6
    residual_mult: float = 1.0
    max_context: int = 32768
    checkpoint_dir: Optional[str] = None
    # hashed bigram table added to the token embedding: (buckets, multiplier
    # of the previous token, multiplier of the current token); None = none
    bigram: Optional[Tuple[int, int, int]] = None
    pos_base: float = 0.0        # base of the additive sinusoid (0 = none)
    logit_scale: float = 1.0
    embed_scale: float = 1.0     # multiplies the token row
    logit_softcap: float = 0.0   # c * tanh(logits / c); 0 = none
    # (start, stop, times): the layers of range(start, stop) are gone through
    # `times` times, sharing weights but not cache or state; with
    # `loop_reenter` the embedding output re-enters the stream whenever a
    # further pass begins
    loop: Optional[Tuple[int, int, int]] = None
    loop_reenter: bool = True
    # hyper-connections: that many residual streams, mixed and read through
    # learned weights around every sublayer; 0 = one plain residual
    streams: int = 0
    # what is added to a stored norm weight of the pre-norm layers (1.0 where
    # checkpoints keep the gain's distance from one)
    norm_offset: float = 0.0
    # behavior flags shared with ModelSpec
    reasoning: bool = False
    embedding: bool = False
    tie_embeddings: bool = False
    recommended_tp: int = 1
    num_experts: int = 0

    @property
    def num_layers(self) -> int:
        return len(self.layers)

    @property
    def runs(self) -> Tuple[Tuple[int, int], ...]:
        """(layer index, pass) in the order the layers run."""
        n = len(self.layers)
        if self.loop is None:
            return tuple((i, 0) for i in range(n))
        a, b, times = self.loop
        return (tuple((i, 0) for i in range(a))
                + tuple((i, r) for r in range(times) for i in range(a, b))
                + tuple((i, 0) for i in range(b, n)))

    def param_count(self) -> int:
        h = self.hidden_size
        n = 2 * self.vocab_size * h

        def delta(m: DeltaMixerSpec) -> int:
            qk = 2 * m.kv_heads * m.dim
            v = m.heads * m.vdim
            return (h * (qk + v + m.heads + m.decay_rank + m.gate_rank)
                    + m.decay_rank * m.heads * m.dim + m.gate_rank * v
                    + v * h + (qk + v) * m.conv)

        def attn(m: AttnMixerSpec) -> int:
            return h * (m.heads * m.dim + m.kv_heads * (m.dim + m.vdim)
                        + m.heads) + m.heads * m.vdim * h

        if self.arch == "ruludra":
            return self._sandwich_param_count()
        if self.arch == "vukotar":
            return self._parallel_param_count(active=False)
        if self.arch in ("nosalorn", "vanulorn", "tubepel"):
            return self._prenorm_param_count(active=False)
        for layer in self.layers:
            m = layer.mixer
            if isinstance(m, ParallelMixerSpec):
                n += attn(m.left) + delta(m.right)
            elif isinstance(m, AttnMixerSpec):
                n += attn(m)
            else:
                n += delta(m)
            n += h * h                      # residual gate of the mixer
            if layer.ff:
                n += 3 * h * layer.ff + h * h
        return n

    def _sandwich_param_count(self) -> int:
        h = self.hidden_size
        n = 2 * self.vocab_size * h + h
        if self.bigram:
            n += (self.bigram[0] + 1) * h
        for i, layer in enumerate(self.layers):
            m = layer.mixer
            if isinstance(m, TiedAttnMixerSpec):
                qd, kd = m.heads * m.dim, m.kv_heads * m.dim
                n += h * (qd + kd) + qd + kd + 2 * m.heads + qd * h
            elif isinstance(m, LatentAttnMixerSpec):
                hv = m.heads * m.vdim
                n += h * m.q_rank + m.q_rank + m.heads * m.dim * m.q_rank
                if m.kv_from is None:
                    n += h * m.kv_rank + m.kv_rank
                n += (m.heads * m.dim + hv) * m.kv_rank + 2 * hv * h
            elif isinstance(m, MLSTMMixerSpec):
                hv = m.heads * m.vdim
                n += h * (2 * m.heads * m.dim + 2 * hv + 2 * m.heads)
                n += 2 * m.heads + hv + hv * h
            n += 2 * h + (i + 2)
            if layer.ff:
                n += 2 * h * layer.ff + 4 + 2 * h
        return n

    def _parallel_param_count(self, active: bool) -> int:
        """Tied embedding, Dynamic-Tanh norms, layer scales; layers that
        borrow another layer's parameters add none. `active`: count only the
        experts a token uses."""
        h = self.hidden_size
        n = self.vocab_size * h + 2 * h + 1
        for layer in self.layers:
            if layer.weights_of is not None and not active:
                continue
            m = layer.mixer
            n += 2 * h + 1 + h
            n += h * (m.heads * m.dim + m.kv_heads * (m.dim + m.vdim))
            n += m.heads * m.vdim * h
            if layer.moe:
                e = layer.moe
                n += h + e.experts * h
                n += (e.top if active else e.experts) * 2 * h * e.ff
        return n

    def _prenorm_param_count(self, active: bool) -> int:
        """Pre-norm layers with attention, latent attention, decay attention,
        delta-rule or state-space mixers and SwiGLU or routed feed-forwards.
        `active`: count only the experts a token uses, and a looped layer
        once per pass."""
        h = self.hidden_size
        n = (1 if self.tie_embeddings else 2) * self.vocab_size * h + h
        if self.bigram:
            n += (self.bigram[0] + 1) * h
        for i in ([i for i, _ in self.runs] if active
                  else range(self.num_layers)):
            layer = self.layers[i]
            m = layer.mixer
            n += h
            if self.streams:
                n += (2 if layer.ff or layer.moe else 1) \
                    * self.streams * (self.streams + 2)
            if isinstance(m, AttnMixerSpec):
                cols = m.heads * m.dim + m.kv_heads * (m.dim + m.vdim)
                n += (h + int(m.bias)) * cols + m.heads * m.vdim * h
                n += int(m.v_mix) + (m.heads if m.sink_learned else 0)
                if m.out_gate:
                    n += h * m.heads * (m.vdim if m.gate_elements else 1)
            elif isinstance(m, LatentAttnMixerSpec):
                H, R, qc = m.heads, m.kv_rank, m.heads * (m.dim + m.rot_dim)
                n += m.q_rank * (h + 1 + qc) if m.q_rank else h * qc
                n += h * (R + m.rot_dim) + R
                n += H * (m.dim + m.vdim) * R + H * m.vdim * h
                n += h * H * m.vdim if m.out_gate else 0
            elif isinstance(m, DecayAttnMixerSpec):
                hv = m.heads * m.vdim
                n += h * (2 * m.heads * m.dim + 2 * hv) + hv * h
                n += hv if m.norm == "all" else 0
            elif isinstance(m, DeltaMixerSpec):
                qk, hv = 2 * m.kv_heads * m.dim, m.heads * m.vdim
                n += h * (qk + 2 * hv + 2 * m.heads) + (qk + hv) * m.conv
                n += 2 * m.heads + m.vdim + hv * h
            elif isinstance(m, SSDMixerSpec):
                inner, bc = m.heads * m.vdim, 2 * m.groups * m.state
                n += h * (2 * inner + bc + m.heads)
                n += (inner + bc) * (m.conv + 1) + 3 * m.heads + inner
                n += inner * h
            if layer.ff:
                n += h + (2 if layer.ff_kind == "relu2" else 3) * h * layer.ff
            if layer.moe:
                e = layer.moe
                n += h
                if e.router != "table":
                    n += (e.experts + e.identity) * (h + int(e.correction))
                n += (min(e.top, e.experts) if active else e.experts) \
                    * 3 * h * e.ff
                if e.shared_ff:
                    n += 3 * h * e.shared_ff + (h if e.shared_gate else 0)
        return n

    def active_param_count(self) -> int:
        if self.arch == "vukotar":
            return self._parallel_param_count(active=True)
        if self.arch in ("nosalorn", "vanulorn", "tubepel"):
            return self._prenorm_param_count(active=True)
        return self.param_count()


def _rot_scaling(rot: dict) -> Optional[Tuple[float, float, float, float]]:
    sc = rot.get("scaling")
    if not sc:
        return None
    return (float(sc["factor"]), float(sc["original"]), float(sc["fast"]),
            float(sc["slow"]))


def _loop(config: dict, n_layers: int) -> Optional[Tuple[int, int, int]]:
    """(start, stop, times) of a config's loop; None where nothing repeats."""
    lp = config.get("loop")
    if not lp or int(lp["times"]) == 1 or int(lp["start"]) == int(lp["stop"]):
        return None
    loop = (int(lp["start"]), int(lp["stop"]), int(lp["times"]))
    if not 0 <= loop[0] < loop[1] <= n_layers or loop[2] < 1:
        raise ValueError("loop must name a run of layers and be passed at "
                         "least once")
    return loop


def _delta_from_config(m: dict, ranks: Tuple[int, int]) -> DeltaMixerSpec:
    return DeltaMixerSpec(heads=int(m["heads"]), kv_heads=int(m["kv_heads"]),
                          dim=int(m["dim"]), vdim=int(m["vdim"]),
                          conv=int(m["conv"]), decay_rank=ranks[0],
                          gate_rank=ranks[1])


def _attn_from_config(m: dict) -> AttnMixerSpec:
    rot = m.get("rot") or {}
    mask = m.get("mask") or {}
    return AttnMixerSpec(heads=int(m["heads"]), kv_heads=int(m["kv_heads"]),
                         dim=int(m["dim"]), vdim=int(m["vdim"]),
                         scale=float(m["scale"]),
                         rot_dims=int(rot.get("dims", 0)),
                         rot_base=float(rot.get("base", 10000.0)),
                         chunk=int(mask.get("size", 0)))


def vodinex_spec(config: dict, name: str = "vodinex",
                 checkpoint_dir: Optional[str] = None,
                 tensor_shapes: Optional[dict] = None) -> HybridSpec:
    """Build the spec of a Vodinex checkpoint from its ``config.json``.

    The inner sizes of the low-rank decay and gate projections are not in the
    config; they are the row counts of ``<mixer>.a1`` / ``<mixer>.g1`` and are
    taken from ``tensor_shapes`` (tensor name -> shape). Callers that build a
    model in code pass them in the layer's mixer dict as ``decay_rank`` /
    ``gate_rank`` instead."""
    shapes = tensor_shapes or {}

    def ranks(prefix: str, m: dict) -> Tuple[int, int]:
        a = shapes.get(prefix + ".a1")
        g = shapes.get(prefix + ".g1")
        return (int(a[0]) if a else int(m.get("decay_rank", 16)),
                int(g[0]) if g else int(m.get("gate_rank", 16)))

    layers = []
    for i, lc in enumerate(config["layers"]):
        kind = lc["type"]
        m = lc["mixer"]
        if kind == "channel_delta":
            mixer: MixerSpec = _delta_from_config(m, ranks(f"l{i}.mix", m))
        elif kind == "parallel":
            mixer = ParallelMixerSpec(
                left=_attn_from_config(m["left"]),
                right=_delta_from_config(
                    m["right"], ranks(f"l{i}.mix.right", m["right"])),
                left_scale=float(m["left_scale"]),
                right_scale=float(m["right_scale"]))
        else:
            raise ValueError(f"unknown layer type {kind!r} in layer {i}")
        mlp = lc.get("mlp")
        if mlp is not None and mlp.get("kind", "dense") != "dense":
            raise ValueError(f"unknown feed-forward kind {mlp['kind']!r}")
        layers.append(HybridLayerSpec(kind=kind, mixer=mixer,
                                      ff=int(mlp["ff"]) if mlp else 0))
    return HybridSpec(name=name, arch="vodinex",
                      hidden_size=int(config["width"]),
                      vocab_size=int(config["vocab"]),
                      layers=tuple(layers),
                      norm_eps=float(config["norm"]["eps"]),
                      residual_mult=float(config["residual_mult"]),
                      max_context=int(config.get("max_context", 1 << 20)),
                      checkpoint_dir=checkpoint_dir)


def ruludra_spec(config: dict, name: str = "ruludra",
                 checkpoint_dir: Optional[str] = None,
                 tensor_shapes: Optional[dict] = None) -> HybridSpec:
    """Build the spec of a Ruludra checkpoint from its ``config.json``: a
    list of layers, each with a tied-value windowed attention, a latent
    attention or an mLSTM mixer and an optional PolyNorm feed-forward; token +
    hashed-bigram + sinusoid embedding; every layer's input is a learned
    weighted sum of the embedding output and all earlier layer results.
    A latent's query rank is `q_rank` of the mixer dict, or else the row count
    of ``<mixer>.dq`` in ``tensor_shapes``."""
    shapes = tensor_shapes or {}
    layers = []
    for i, lc in enumerate(config["layers"]):
        kind = lc["type"]
        m = lc["mixer"]
        mask = m.get("mask") or {}
        if kind == "attention":
            if int(m.get("vdim", m["dim"])) != int(m["dim"]):
                raise ValueError(f"layer {i}: values are the keys, so vdim "
                                 f"must equal dim")
            qt = m.get("q_temp") or {}
            mixer: MixerSpec = TiedAttnMixerSpec(
                heads=int(m["heads"]), kv_heads=int(m["kv_heads"]),
                dim=int(m["dim"]), scale=float(m["scale"]),
                window=int(mask.get("size", 0)),
                temp_coef=float(qt.get("coef", 0.0)),
                temp_every=int(qt.get("every", 0)))
        elif kind == "latent_attention":
            src = m.get("kv_from")
            dq = shapes.get(f"l{i}.mix.dq")
            if src is not None:
                src = int(src)
                other = config["layers"][src] if 0 <= src < i else None
                if (other is None or other["type"] != "latent_attention"
                        or other["mixer"].get("kv_from") is not None
                        or int(other["mixer"]["kv_rank"]) != int(m["kv_rank"])):
                    raise ValueError(
                        f"layer {i}: kv_from must name an earlier latent "
                        f"layer of equal kv_rank that owns its latent")
            mixer = LatentAttnMixerSpec(
                heads=int(m["heads"]), dim=int(m["dim"]), vdim=int(m["vdim"]),
                q_rank=int(m["q_rank"]) if "q_rank" in m else int(dq[0]),
                kv_rank=int(m["kv_rank"]), scale=float(m["scale"]),
                window=int(mask.get("size", 0)), kv_from=src)
        elif kind == "mlstm":
            mixer = MLSTMMixerSpec(heads=int(m["heads"]), dim=int(m["dim"]),
                                   vdim=int(m["vdim"]),
                                   gate_cap=float(m["gate_cap"]))
        else:
            raise ValueError(f"unknown layer type {kind!r} in layer {i}")
        mlp = lc.get("mlp")
        if mlp is not None and mlp.get("kind", "dense") != "dense":
            raise ValueError(f"unknown feed-forward kind {mlp['kind']!r}")
        layers.append(HybridLayerSpec(kind=kind, mixer=mixer,
                                      ff=int(mlp["ff"]) if mlp else 0,
                                      ff_kind="poly_norm"))
    big = (config.get("embedding") or {}).get("bigram")
    return HybridSpec(
        name=name, arch="ruludra", hidden_size=int(config["width"]),
        vocab_size=int(config["vocab"]), layers=tuple(layers),
        norm_eps=float(config["norm"]["eps"]),
        max_context=int(config.get("max_context", 1 << 20)),
        checkpoint_dir=checkpoint_dir,
        bigram=(int(big["buckets"]), int(big["mul_prev"]),
                int(big["mul_cur"])) if big else None,
        pos_base=10000.0, logit_scale=float(config.get("logit_scale", 1.0)))


def vukotar_spec(config: dict, name: str = "vukotar",
                 checkpoint_dir: Optional[str] = None,
                 tensor_shapes: Optional[dict] = None) -> HybridSpec:
    """Build the spec of a Vukotar checkpoint from its ``config.json``: a
    list of parallel layers (one Dynamic-Tanh norm feeding a sink-softmax
    attention and a routed-experts feed-forward, each under a layer scale),
    layers that borrow an earlier or later layer's tensors (``weights_of``),
    scaled token embedding + sinusoid, tied and soft-capped logits."""
    raw = config["layers"]

    def owner(i: int) -> int:
        seen = set()
        while raw[i].get("weights_of") is not None:
            if i in seen:
                raise ValueError(f"layer {i}: weights_of runs in a circle")
            seen.add(i)
            i = int(raw[i]["weights_of"])
            if not 0 <= i < len(raw):
                raise ValueError("weights_of names no layer")
        return i

    layers = []
    for i, lc in enumerate(raw):
        kind = lc["type"]
        if kind != "attention":
            raise ValueError(f"unknown layer type {kind!r} in layer {i}")
        m = lc["mixer"]
        mixer = AttnMixerSpec(
            heads=int(m["heads"]), kv_heads=int(m["kv_heads"]),
            dim=int(m["dim"]), vdim=int(m["vdim"]), scale=float(m["scale"]),
            qk_norm=False, bias=False, out_gate=False, sink=True)
        mlp = lc.get("mlp")
        moe = None
        if mlp is not None:
            if mlp.get("kind") != "moe":
                raise ValueError(f"unknown feed-forward kind {mlp.get('kind')!r}")
            r = mlp["router"]
            g = r.get("groups") or {"count": 1, "keep": 1}
            moe = RoutedExpertsSpec(
                ff=int(mlp["expert"]["ff"]), experts=int(r["experts"]),
                top=int(r["top"]), groups=int(g["count"]), keep=int(g["keep"]))
            if moe.experts % moe.groups or not 1 <= moe.keep <= moe.groups:
                raise ValueError(f"layer {i}: experts must split into equal "
                                 f"groups, of which 1..groups are kept")
            if moe.top > moe.keep * (moe.experts // moe.groups):
                raise ValueError(f"layer {i}: the kept groups hold fewer "
                                 f"experts than a token uses")
        own = owner(i)
        layers.append(HybridLayerSpec(kind=kind, mixer=mixer, moe=moe,
                                      weights_of=None if own == i else own))
    for i, layer in enumerate(layers):
        if layer.weights_of is not None:
            src = layers[layer.weights_of]
            if (src.mixer, src.moe) != (layer.mixer, layer.moe):
                raise ValueError(f"layer {i} borrows the tensors of layer "
                                 f"{layer.weights_of} but differs in shape")
    return HybridSpec(
        name=name, arch="vukotar", hidden_size=int(config["width"]),
        vocab_size=int(config["vocab"]), layers=tuple(layers),
        norm_eps=float(config["norm"]["eps"]),
        max_context=int(config.get("max_context", 1 << 20)),
        checkpoint_dir=checkpoint_dir, pos_base=10000.0,
        embed_scale=float((config.get("embedding") or {}).get("scale", 1.0)),
        logit_softcap=float(config.get("logit_softcap", 0.0) or 0.0),
        tie_embeddings=True,
        num_experts=max((l.moe.experts if l.moe else 0) for l in layers))


def nosalorn_spec(config: dict, name: str = "nosalorn",
                  checkpoint_dir: Optional[str] = None,
                  tensor_shapes: Optional[dict] = None) -> HybridSpec:
    """Build the spec of a Nosalorn checkpoint from its ``config.json``: a
    list of pre-norm layers (weighted RMS norms), each with a windowed
    rotary attention (biased projections, YaRN frequencies, kept first
    tokens, values blended with the first blending layer's), a fixed-decay
    linear attention or a Mamba-2 mixer, and an optional SwiGLU or
    routed-experts feed-forward; scaled token embedding, untied head, scaled
    logits."""
    layers = []
    first_mix = None
    for i, lc in enumerate(config["layers"]):
        kind = lc["type"]
        m = lc["mixer"]
        if kind == "attention":
            rot = m.get("rot") or {}
            mask = m.get("mask") or {}
            mixer: MixerSpec = AttnMixerSpec(
                heads=int(m["heads"]), kv_heads=int(m["kv_heads"]),
                dim=int(m["dim"]), vdim=int(m["vdim"]),
                scale=float(m["scale"]), rot_dims=int(rot.get("dims", 0)),
                rot_base=float(rot.get("base", 10000.0)),
                window=int(mask.get("size", 0) or 0),
                keep_first=int(mask.get("keep_first", 0) or 0),
                rot_scaling=_rot_scaling(rot),
                qk_norm=False, bias=True, out_bias=False, out_gate=False,
                v_mix=bool(m.get("v_mix", False)))
            if mixer.v_mix:
                cols = mixer.kv_heads * mixer.vdim
                if first_mix is None:
                    first_mix = cols
                elif cols != first_mix:
                    raise ValueError(
                        f"layer {i}: blended values must be as wide as the "
                        f"first blending layer's ({first_mix})")
        elif kind == "lightning":
            mixer = DecayAttnMixerSpec(
                heads=int(m["heads"]), dim=int(m["dim"]), vdim=int(m["vdim"]),
                decay=tuple(float(d) for d in m["decay"]))
            if len(mixer.decay) != mixer.heads:
                raise ValueError(f"layer {i}: one decay per head is needed")
        elif kind == "mamba2":
            mixer = SSDMixerSpec(
                heads=int(m["heads"]), vdim=int(m["vdim"]),
                state=int(m["state"]), groups=int(m.get("groups", 1)),
                conv=int(m["conv"]), norm_groups=int(m.get("norm_groups", 1)))
            if mixer.heads % mixer.groups or \
                    (mixer.heads * mixer.vdim) % mixer.norm_groups:
                raise ValueError(f"layer {i}: heads must split into the "
                                 f"groups and the width into the norm groups")
        else:
            raise ValueError(f"unknown layer type {kind!r} in layer {i}")
        mlp = lc.get("mlp")
        ff, moe = 0, None
        if mlp is not None:
            fk = mlp.get("kind", "dense")
            if fk == "dense":
                ff = int(mlp["ff"])
            elif fk == "moe":
                r = mlp["router"]
                g = r.get("groups") or {"count": 1, "keep": 1}
                sh = mlp.get("shared") or {}
                moe = RoutedExpertsSpec(
                    ff=int(mlp["expert"]["ff"]), experts=int(r["experts"]),
                    top=int(r["top"]), groups=int(g["count"]),
                    keep=int(g["keep"]), group_rank=1, router="softmax",
                    act="clamped_glu", identity=int(r.get("identity", 0) or 0),
                    route_scale=float(r.get("scale", 1.0)), correction=True,
                    limit=float(mlp["expert"]["limit"]),
                    shared_ff=int(sh.get("ff", 0) or 0),
                    shared_limit=float(sh.get("limit", 0.0) or 0.0))
                n = moe.experts + moe.identity
                if n % moe.groups or not 1 <= moe.keep <= moe.groups:
                    raise ValueError(
                        f"layer {i}: experts and identity experts must split "
                        f"into equal groups, of which 1..groups are kept")
                if moe.top > moe.keep * (n // moe.groups):
                    raise ValueError(f"layer {i}: the kept groups hold fewer "
                                     f"experts than a token uses")
            else:
                raise ValueError(f"unknown feed-forward kind {fk!r}")
        layers.append(HybridLayerSpec(kind=kind, mixer=mixer, ff=ff,
                                      ff_kind="swiglu", moe=moe))
    return HybridSpec(
        name=name, arch="nosalorn", hidden_size=int(config["width"]),
        vocab_size=int(config["vocab"]), layers=tuple(layers),
        norm_eps=float(config["norm"]["eps"]),
        max_context=int(config.get("max_context", 1 << 20)),
        checkpoint_dir=checkpoint_dir,
        embed_scale=float((config.get("embedding") or {}).get("scale", 1.0)),
        logit_scale=float(config.get("logit_scale", 1.0)),
        num_experts=max([(l.moe.experts if l.moe else 0) for l in layers]
                        + [0]))


def vanulorn_spec(config: dict, name: str = "vanulorn",
                  checkpoint_dir: Optional[str] = None,
                  tensor_shapes: Optional[dict] = None) -> HybridSpec:
    """Build the spec of a Vanulorn checkpoint from its ``config.json``: a
    list of pre-norm layers (RMS norms with gain 1 + weight), each with a
    retention, a rotary latent attention or a gated-delta-rule mixer (one
    decay per head) and an optional SwiGLU or token-table experts
    feed-forward; a run of layers that is passed several times; scaled token +
    hashed-bigram embedding, tied head."""
    layers = []
    vocab = int(config["vocab"])
    for i, lc in enumerate(config["layers"]):
        kind = lc["type"]
        m = lc["mixer"]
        rot = m.get("rot") or {}
        if kind == "retention":
            mixer: MixerSpec = DecayAttnMixerSpec(
                heads=int(m["heads"]), dim=int(m["dim"]), vdim=int(m["vdim"]),
                decay=tuple(float(d) for d in m["decay"]), act="none",
                rot_dims=int(rot.get("dims", 0) or 0),
                rot_base=float(rot.get("base", 10000.0)),
                rot_scaling=_rot_scaling(rot), k_scale=float(m["dim"]) ** -0.5,
                norm="head", gate="silu")
            if len(mixer.decay) != mixer.heads:
                raise ValueError(f"layer {i}: one decay per head is needed")
        elif kind == "latent_attention":
            mixer = LatentAttnMixerSpec(
                heads=int(m["heads"]), dim=int(m["dim"]), vdim=int(m["vdim"]),
                q_rank=0, kv_rank=int(m["kv_rank"]), scale=float(m["scale"]),
                rot_dim=int(m.get("rot_dim", 0) or 0),
                rot_base=float(rot.get("base", 10000.0)),
                rot_scaling=_rot_scaling(rot), out_gate=False)
            if int(rot.get("dims", mixer.rot_dim)) != mixer.rot_dim:
                raise ValueError(f"layer {i}: the whole rotated part turns, so "
                                 f"rot.dims must equal rot_dim")
        elif kind == "delta":
            mixer = DeltaMixerSpec(
                heads=int(m["heads"]), kv_heads=int(m["kv_heads"]),
                dim=int(m["dim"]), vdim=int(m["vdim"]), conv=int(m["conv"]),
                decay="head", gate="silu")
        else:
            raise ValueError(f"unknown layer type {kind!r} in layer {i}")
        mlp = lc.get("mlp")
        ff, moe = 0, None
        if mlp is not None:
            fk = mlp.get("kind", "dense")
            if fk == "dense":
                ff = int(mlp["ff"])
            elif fk == "moe":
                r = mlp["router"]
                moe = RoutedExpertsSpec(
                    ff=int(mlp["expert"]["ff"]), experts=int(r["experts"]),
                    top=int(r["top"]), router="table", act="silu_glu",
                    shared_ff=int((mlp.get("shared") or {}).get("ff", 0) or 0),
                    shared_gate=False, vocab=vocab)
                if not 1 <= moe.top <= moe.experts:
                    raise ValueError(f"layer {i}: a token uses 1..experts "
                                     f"experts")
            else:
                raise ValueError(f"unknown feed-forward kind {fk!r}")
        layers.append(HybridLayerSpec(kind=kind, mixer=mixer, ff=ff,
                                      ff_kind="swiglu", moe=moe))
    emb = config.get("embedding") or {}
    big = emb.get("bigram")
    return HybridSpec(
        name=name, arch="vanulorn", hidden_size=int(config["width"]),
        vocab_size=vocab, layers=tuple(layers),
        norm_eps=float(config["norm"]["eps"]),
        max_context=int(config.get("max_context", 1 << 20)),
        checkpoint_dir=checkpoint_dir,
        bigram=(int(big["buckets"]), int(big["mul_prev"]),
                int(big["mul_cur"])) if big else None,
        embed_scale=float(emb.get("scale", 1.0)),
        loop=_loop(config, len(layers)), norm_offset=1.0,
        tie_embeddings=True,
        num_experts=max([(l.moe.experts if l.moe else 0) for l in layers]
                        + [0]))


def tubepel_spec(config: dict, name: str = "tubepel",
                 checkpoint_dir: Optional[str] = None,
                 tensor_shapes: Optional[dict] = None) -> HybridSpec:
    """Build the spec of a Tubepel checkpoint from its ``config.json``: a list
    of pre-norm layers (weighted RMS norms) over several residual streams
    (hyper-connections), each with a rotary latent attention with a query
    latent (two kinds, which differ in the pairing of the rotated dimensions)
    or a windowed attention with kept first tokens, learned sinks and an
    elementwise output gate, and an optional squared-ReLU or routed-experts
    feed-forward (sigmoid scores that weigh the experts' input); a run of
    layers that is passed several times; untied head. A latent's query rank is
    `q_rank` of the mixer dict, or else the row count of ``<mixer>.dq`` in
    ``tensor_shapes``."""
    shapes = tensor_shapes or {}
    layers = []
    for i, lc in enumerate(config["layers"]):
        kind = lc["type"]
        m = lc["mixer"]
        rot = m.get("rot") or {}
        if kind in ("latent_attention", "latent_attention_2"):
            q_rank = m.get("q_rank")
            if q_rank is None:
                q_rank = shapes[f"l{i}.mix.dq"][0]
            mixer: MixerSpec = LatentAttnMixerSpec(
                heads=int(m["heads"]), dim=int(m["dim"]), vdim=int(m["vdim"]),
                q_rank=int(q_rank), kv_rank=int(m["kv_rank"]),
                scale=float(m["scale"]), rot_dim=int(m.get("rot_dim", 0) or 0),
                rot_base=float(rot.get("base", 10000.0)), out_gate=False,
                rot_adjacent=kind == "latent_attention")
            if int(rot.get("dims", mixer.rot_dim)) != mixer.rot_dim:
                raise ValueError(f"layer {i}: the whole rotated part turns, so "
                                 f"rot.dims must equal rot_dim")
        elif kind == "attention":
            mask = m.get("mask") or {}
            mixer = AttnMixerSpec(
                heads=int(m["heads"]), kv_heads=int(m["kv_heads"]),
                dim=int(m["dim"]), vdim=int(m["vdim"]),
                scale=float(m["scale"]), rot_dims=int(rot.get("dims", 0) or 0),
                rot_base=float(rot.get("base", 10000.0)),
                window=int(mask.get("size", 0) or 0),
                keep_first=int(mask.get("keep_first", 0) or 0),
                qk_norm=False, bias=False, out_gate=True, gate_elements=True,
                sink=True, sink_learned=True)
        else:
            raise ValueError(f"unknown layer type {kind!r} in layer {i}")
        mlp = lc.get("mlp")
        ff, moe = 0, None
        if mlp is not None:
            fk = mlp.get("kind", "dense")
            if fk == "dense":
                ff = int(mlp["ff"])
            elif fk == "moe":
                r = mlp["router"]
                moe = RoutedExpertsSpec(
                    ff=int(mlp["expert"]["ff"]), experts=int(r["experts"]),
                    top=int(r["top"]), router="sigmoid", act="silu_glu",
                    shared_ff=int((mlp.get("shared") or {}).get("ff", 0) or 0),
                    shared_gate=False, renorm=False, weigh_input=True)
                if not 1 <= moe.top <= moe.experts:
                    raise ValueError(f"layer {i}: a token uses 1..experts "
                                     f"experts")
            else:
                raise ValueError(f"unknown feed-forward kind {fk!r}")
        layers.append(HybridLayerSpec(kind=kind, mixer=mixer, ff=ff,
                                      ff_kind="relu2", moe=moe))
    streams = int(config["streams"])
    if streams < 1:
        raise ValueError("streams must be at least 1")
    return HybridSpec(
        name=name, arch="tubepel", hidden_size=int(config["width"]),
        vocab_size=int(config["vocab"]), layers=tuple(layers),
        norm_eps=float(config["norm"]["eps"]),
        max_context=int(config.get("max_context", 1 << 20)),
        checkpoint_dir=checkpoint_dir, loop=_loop(config, len(layers)),
        loop_reenter=False, streams=streams,
        num_experts=max([(l.moe.experts if l.moe else 0) for l in layers]
                        + [0]))
