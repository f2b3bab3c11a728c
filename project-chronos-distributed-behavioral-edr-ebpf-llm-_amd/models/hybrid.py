"""Hybrid decoders: a list of layers, each with a token mixer of some kind (recurrent matrix memory, latent
attention, windowed or chunked attention, gated delta rule, gated linear attention, state-space duality, real-gated
linear recurrence, retention, two mixers side by side) and an optional feed-forward (dense, gated, mixture of
experts), on a float32 residual stream.
The stream's rule is a parameter of the configuration: the norm on the sublayer's OUTPUT (``out_norm``:
x <- x + layer_norm(sublayer(x))), AFTER the sum (``post_norm``: x <- rms_norm(alpha x + sublayer(x))), on the
sublayer's INPUT (``pre_norm``: x <- x + sublayer(rms_norm(x))), on both sides (``sandwich``:
x <- x + norm_b(sublayer(norm_a(x))), RMS norms over ``norm_groups`` equal parts of the row), or one norm that both
sublayers of a layer read (``parallel``: x <- x + mixer(h) + ff(h), h = layer_norm(x)).  A pre-norm stream may
use Dynamic Tanh in place of the RMS norm, scale what it adds, gate every sublayer's result by a projection of what
the sublayer read, and hand on weighted sums of all earlier layers' results.  A range of layers may repeat, back to
back, on shared weights (``loop``), or single layers may name another layer whose weights they use
(``share``); every run has its own pages and state.

This module is the design-independent part: the mixer and feed-forward kinds with their sizes and constants as
parameters, the cache that holds pages for the attention layers and state slots for the recurrent ones, and the
forward over the engine's flattened step batch (:class:`chronos.models.llama.StepBatch`: prefill chunks, decode rows
or both in one step).  A design (``zokunex.py``) reads its configuration file and tensor names into these.

New mixer / feed-forward kinds register in ``MIXERS`` / ``FEED_FORWARDS``.
"""
from __future__ import annotations

from dataclasses import dataclass, field
from typing import Optional

import torch

from ..ops import hybrid as hops
from ..parallel.tp import TPContext
from .llama import StepBatch, h2d


# -----------------------------------------------------------------------------------------------------------------
# configuration
# -----------------------------------------------------------------------------------------------------------------


@dataclass
class MLSTMSpec:
    """Matrix-memory recurrent mixer: per head a D x Dv state, exponential input gate and sigmoid forget gate in
    log space, both soft-capped (cap * tanh(z / cap)) and stabilised by a running maximum."""
    heads: int
    dim: int
    vdim: int
    gate_cap: float
    kind: str = "mlstm"


@dataclass
class LatentAttentionSpec:
    """Attention whose keys and values are up-projections of one cached low-rank latent per token, plus a rotated key
    part shared by all heads; through a sliding window or over the whole prefix; a sigmoid output gate (one number per
    head, or with ``gate_wide`` one per output column; none with ``gate`` off).  ``rope_interleaved``: neighbouring
    columns form the rotated pairs (else column i pairs with i + rope_dims / 2).  ``two_term``: on the matrix cores
    the softmax weights enter the weighted sum as two bfloat16 terms each.  ``q_rank`` > 0: the queries are
    up-projections of an RMS-normed latent of that size.  ``sink``: a learned softmax sink per head.  ``kv_from``: the
    layer writes no latents, it reads the pages of that earlier layer (same kv_rank, rot_dim and rotation)."""
    heads: int
    dim: int        # unrotated query / key columns per head
    rot_dim: int    # rotated columns per head (the shared rotated key has as many)
    vdim: int
    kv_rank: int
    scale: float
    rope_base: float
    rope_dims: int  # leading columns of the rotated part that are actually rotated
    window: int = 0            # > 0: only the last ``window`` positions (the query's own included) are visible
    rope_interleaved: bool = False
    gate_wide: bool = False
    two_term: bool = False
    gate: bool = True
    q_rank: int = 0
    sink: bool = False
    kv_from: Optional[int] = None
    rope_scaling: Optional[tuple] = None   # see rope_cos_sin
    kind: str = "latent_attention"

    def params(self, d: int) -> int:
        nq = self.heads * (self.dim + self.rot_dim)
        n = self.q_rank * (d + 1 + nq) if self.q_rank else d * nq
        n += d * self.heads * (self.vdim if self.gate_wide else 1) * self.gate + self.heads * self.sink
        if self.kv_from is None:
            n += d * (self.kv_rank + self.rot_dim) + self.kv_rank
        return n + self.kv_rank * self.heads * (self.dim + self.vdim) + self.heads * self.vdim * d


@dataclass
class DenseFFSpec:
    ff: int
    act: int = hops.ACT_RELU2
    kind: str = "dense"


@dataclass
class PolyFFSpec:
    """Dense feed-forward with the PolyNorm activation a N(z) + b N(z^2) + c N(z^3) + e, N = division by the row's root
    mean square over the ``ff`` values."""
    ff: int
    kind: str = "poly"


@dataclass
class MoEFFSpec:
    experts: int     # experts with weights
    identity: int    # further router outputs whose expert returns its input
    top: int
    ff: int
    act: int = hops.ACT_GELU
    shared_ff: int = 0   # > 0: a shared expert of this size (same form, no router weight) runs for every token
    correction: bool = True   # the checkpoint holds a per-output term that steers the router's choice
    kind: str = "moe"


@dataclass
class WindowAttentionSpec:
    """Grouped-query softmax attention through a sliding window that also keeps each sequence's first tokens, with
    per-head RMS norm of queries and keys, rotation of the leading ``rope_dims`` columns (``rope_scaling``: see
    :func:`rope_cos_sin`), a learned softmax sink per head, an optional mix of every token's values with those of the
    first such layer, and a sigmoid output gate (one number per head, or with ``gate_wide`` one per output column).
    ``pool`` > 0 (with a window): beside the window's tokens a query sees one key and value per block of ``pool``
    positions that lies wholly before its window — the means of the block's cached keys and values.  ``v_from_k``:
    there is no value projection, the values are the keys before norm and rotation.  ``v_rot``: values
    are cached rotated by their position over all ``vdim`` columns (frequencies rope_base^(-2m/vdim), unscaled) and
    every head's output is turned back by the query's position.  ``conv`` > 0: queries, keys and values pass a short
    causal convolution of that many taps right after the projection.  ``q_temp`` = (coef, every): queries are multiplied
    by 1 + coef ln(floor((p + 1) / every) + 1) at position p.

    Where keys are values divided by their root mean square (``v_from_k``, a norm without weights, no rotation) only
    the values are cached, and one float32 number per token and head: ``unit_keys``."""
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    scale: float
    window: int = 0          # 0: every earlier token is visible
    keep_first: int = 0      # tokens at positions below this stay visible past the window
    rope_base: float = 10000.0
    rope_dims: int = 0       # 0: no rotation
    rope_scaling: Optional[tuple] = None
    v_mix: bool = False
    v_mix_first: bool = False  # this layer is the source of the mixed-in values (and does not mix itself)
    chunk: int = 0           # > 0: a query sees only the keys of its own chunk of this many positions
    qk_norm: bool = True     # per-head RMS norm of queries and keys
    sink: bool = True        # a learned softmax sink per head
    gate: bool = True        # a sigmoid output gate per head
    bias: bool = False       # the q, k, v projections add a bias
    pool: int = 0            # > 0: pooled blocks of this many positions stay visible before the window
    v_from_k: bool = False   # values = the keys as projected
    v_rot: bool = False      # values rotated by their position, outputs turned back
    gate_wide: bool = False  # the sigmoid output gate has heads * vdim rows instead of heads
    sink_fixed: Optional[float] = None  # with ``sink``: every head's sink score is this constant (no weights)
    bias_o: bool = False     # the output projection adds a bias
    conv: int = 0            # > 0: taps of a causal convolution over time on the projected columns
    qk_norm_weight: bool = True   # with ``qk_norm``: the norms of queries and keys have weights
    q_temp: Optional[tuple] = None  # (coef, every): the queries' temperature by position
    kind: str = "window_attention"

    @property
    def unit_keys(self) -> bool:
        return self.v_from_k and self.qk_norm and not self.qk_norm_weight and not self.rope_dims and not self.v_rot \
            and not self.v_mix and not self.pool and self.dim == self.vdim

    def params(self, d: int) -> int:
        qkv = self.heads * self.dim + self.kv_heads * (self.dim + (0 if self.v_from_k else self.vdim))
        gate = self.heads * (self.vdim if self.gate_wide else 1) * self.gate
        return d * (qkv + gate) + qkv * self.conv + 2 * self.dim * (self.qk_norm and self.qk_norm_weight) + \
            (self.heads if self.sink and self.sink_fixed is None else 0) + self.bias_o * d + \
            (1 if self.v_mix and not self.v_mix_first else 0) + \
            self.heads * self.vdim * d + qkv * self.bias


@dataclass
class RetentionSpec:
    """Linear attention with one fixed decay per head and no softmax or denominator: per head a dim x vdim state
    S <- decay_h S + k v^T, o = S^T q, with q and k rotated (``rope_dims`` leading columns) and k times dim^(-1/2);
    each head's read-out is scaled to unit RMS and multiplied by silu of a gate projection."""
    heads: int
    dim: int
    vdim: int
    decay: tuple
    rope_base: float = 10000.0
    rope_dims: int = 0
    rope_scaling: Optional[tuple] = None
    kind: str = "retention"

    def params(self, d: int) -> int:
        return d * (2 * self.heads * self.dim + 2 * self.heads * self.vdim) + self.heads * self.vdim * d


@dataclass
class ParallelSpec:
    """Two mixers side by side on the same input; the result is half the sum of their outputs, each first scaled to
    unit RMS over the model width and multiplied by a weight of its own."""
    left: object
    right: object
    kind: str = "parallel"

    def params(self, d: int) -> int:
        return self.left.params(d) + self.right.params(d) + 2 * d


@dataclass
class DeltaRuleSpec:
    """Gated delta rule: per value head a dim x vdim state that decays, is corrected towards the current value along
    the current (unit) key, and is read by the (unit) query; q, k, v pass a short causal convolution and SiLU."""
    heads: int
    kv_heads: int   # query / key heads (value head h reads head h // (heads / kv_heads))
    dim: int
    vdim: int
    conv: int
    kind: str = "delta_rule"

    def params(self, d: int) -> int:
        c = 2 * self.kv_heads * self.dim + self.heads * self.vdim
        return c * (d + self.conv) + self.heads * (2 * d + 2) + self.vdim + 2 * self.heads * self.vdim * d


@dataclass
class GLASpec:
    """Gated linear attention: per head a dim x vdim state whose rows decay by sigmoid(z)^(1/tau), z a low-rank
    projection of the input with a bias."""
    heads: int
    dim: int
    vdim: int
    tau: float
    rank: int
    kind: str = "gla"

    def params(self, d: int) -> int:
        hd, hv = self.heads * self.dim, self.heads * self.vdim
        return d * (2 * hd + 2 * hv) + self.rank * (d + hd) + hd + self.vdim + hv * d


@dataclass
class Mamba2Spec:
    """State-space duality: per head a state x vdim matrix S <- exp(-exp(A) dt) S + dt B x^T, read by C, with B and C
    shared by the heads of a group; x, B and C pass a short causal convolution (with bias) and SiLU; the read-out
    plus D x is gated by silu(z) first and RMS-normed afterwards, over ``norm_groups`` column ranges of equal size."""
    heads: int
    vdim: int
    state: int
    groups: int
    conv: int
    norm_groups: int = 1
    kind: str = "mamba2"

    @property
    def inner(self) -> int:
        return self.heads * self.vdim

    @property
    def conv_channels(self) -> int:
        return self.inner + 2 * self.groups * self.state

    def params(self, d: int) -> int:
        n_in = 2 * self.inner + 2 * self.groups * self.state + self.heads
        return d * n_in + self.conv_channels * (self.conv + 1) + 3 * self.heads + self.inner + self.inner * d


@dataclass
class RGLRUSpec:
    """Real-gated linear recurrent unit: per channel S <- a S + sqrt(1 - a^2) i u with a = exp(-c r softplus(lam)),
    the gates r and i sigmoids of block-diagonal projections of u, u a short causal convolution (with bias) of one
    input branch; the other branch, through gelu, multiplies the state on the way out."""
    width: int
    blocks: int
    conv: int
    c: float = 8.0
    kind: str = "rglru"

    def params(self, d: int) -> int:
        bw = self.width // self.blocks
        gates = 2 * self.blocks * bw * (bw + 1)
        return 2 * self.width * (d + 1) + self.width * (self.conv + 1) + gates + self.width + self.width * d


@dataclass
class GluFFSpec:
    """Gated feed-forward: y = g sigmoid(slope g) (u + shift) with g = min(W_gate h, limit) and
    u = clamp(W_up h, -limit, limit)."""
    ff: int
    limit: float
    slope: float = 1.702
    shift: float = 1.0
    kind: str = "glu"


@dataclass
class MoEGluSpec:
    """Mixture of gated experts; the router adds a bias to its logits, takes the ``top`` largest and weighs them by
    the softmax over the chosen logits only."""
    experts: int
    top: int
    ff: int
    limit: float
    slope: float = 1.702
    shift: float = 1.0
    kind: str = "moe_glu"


@dataclass
class MoEGroupGluSpec:
    """Mixture of gated experts behind a sigmoid router whose choice is limited to the best groups of neighbouring
    experts (a group scores its top two scores added up); weights = chosen scores / their sum * scale.  With
    ``shared_ff`` > 0 a shared gated expert of that size runs for every token, times sigmoid of one more projection."""
    experts: int
    top: int
    ff: int
    groups: int = 1
    keep: int = 1
    scale: float = 1.0
    shared_ff: int = 0
    limit: float = float("inf")   # the gated unit without clamp: silu(g) u
    slope: float = 1.0
    shift: float = 0.0
    kind: str = "moe_group_glu"


@dataclass
class LayerSpec:
    mixer: object
    ff: Optional[object]


@dataclass
class HybridConfig:
    name: str
    vocab_size: int
    hidden_size: int
    layers: list
    norm_eps: float
    logit_scale: float = 1.0
    max_position: int = 8192
    architecture: str = "hybrid"
    residual: str = "out_norm"     # "out_norm": x <- x + layer_norm(y);  "post_norm": x <- rms_norm(alpha x + y);
    #                                "pre_norm": x <- x + sublayer(rms_norm(x));
    #                                "sandwich": x <- x + norm_b(sublayer(norm_a(x)));
    #                                "parallel": x <- x + mixer(h) + ff(h), h = norm(x)
    norm_groups: int = 1           # sandwich: the stream's RMS norms work on this many equal parts of a row
    embed_scale: float = 1.0       # the embedding rows are multiplied by this
    share: Optional[list] = None   # share[i] = j: layer i runs on layer j's weights (j itself has its own)
    residual_alpha: float = 1.0
    tied_head: bool = False        # the logits come from the embedding table
    loop: Optional[tuple] = None   # (start, stop, times): layers [start, stop) run ``times`` times, back to back
    norm: str = "rms"              # pre_norm: the stream's norms, "rms" or "tanh" (Dynamic Tanh: tanh(alpha x) w + b);
    #                                parallel: "layer" (layer norm with weight and bias)
    residual_mult: float = 1.0     # pre_norm: x <- x + residual_mult * sublayer(norm(x))
    residual_gate: bool = False    # pre_norm: a sublayer's result times sigmoid(W h + b), h what the sublayer read
    depth_average: bool = False    # pre_norm: after layer i the stream is sum_j dwa_i[j] X_j over the embedding output
    #                                X_0 and the layers' own results X_1 .. X_(i+1)
    token_side: int = 0            # > 0: after every layer's feed-forward a gated, RMS-normed projection of this many
    #                                columns of a second embedding table (layer i owns columns [i dim, (i+1) dim))

    @property
    def num_layers(self) -> int:
        return len(self.runs)

    @property
    def runs(self) -> list:
        """Layer index of every layer run, in order (the looped range repeated); pages and state are per run."""
        n = len(self.layers)
        if self.share is not None:
            return [int(j) for j in self.share]
        if not self.loop or self.loop[2] <= 1:
            return list(range(n))
        a, b, t = self.loop
        return list(range(a)) + list(range(a, b)) * t + list(range(b, n))

    def param_count(self) -> int:
        d = self.hidden_size
        extra = {"tanh": d + 1, "layer": d}.get(self.norm, 0)     # what a norm carries beside its weight
        n = (1 if self.tied_head else 2) * self.vocab_size * d + d + extra
        own = set(self.runs)
        for i, l in enumerate(self.layers):
            if i not in own:
                continue
            m = l.mixer
            if hasattr(m, "params"):
                n += m.params(d)
            elif m.kind == "mlstm":
                n += d * (2 * m.heads * m.dim + 2 * m.heads * m.vdim) + 2 * m.heads * (d + 1) + m.heads * m.vdim * (d + 1)
            sub = d * (2 if self.residual == "sandwich" else 1)    # what every sublayer carries beside its own weights
            sub += extra
            if self.residual_gate:
                sub += d * (d + 1)
            n += sub + (i + 2 if self.depth_average else 0)
            if l.ff is not None:
                f = l.ff
                n += sub if self.residual != "parallel" else 0     # (one norm for both sublayers)
                n += {"dense": lambda: 2 * d * f.ff, "poly": lambda: 2 * d * f.ff + 4, "glu": lambda: 3 * d * f.ff,
                      "moe": lambda: (f.experts * f.ff + f.shared_ff) * 2 * d + (f.experts + f.identity) * (d + f.correction),
                      "moe_glu": lambda: f.experts * (3 * d * f.ff + d + 1),
                      "moe_group_glu": lambda: f.experts * (3 * d * f.ff + d) + (
                          3 * d * f.shared_ff + d if f.shared_ff else 0)}[f.kind]()
            if self.token_side:
                n += self.token_side * (2 * d + self.vocab_size) + d
        return n


# -----------------------------------------------------------------------------------------------------------------
# cache: pages for the attention layers, state slots for the recurrent layers
# -----------------------------------------------------------------------------------------------------------------


def _conv_channels(mx: WindowAttentionSpec) -> int:
    """Columns that pass an attention layer's short convolution: q | k (| v)."""
    return (mx.heads + mx.kv_heads) * mx.dim + (0 if mx.v_from_k else mx.kv_heads * mx.vdim)


class HybridCache:
    """Per latent-attention layer run a paged latent cache [NB, BS, kv_rank + rot_dim] (a run that reads another layer's
    latents names the same tensor), per windowed-attention run
    paged keys [NB, BS, G, D] and values [NB, BS, G, Dv] (with pooled blocks also their means, ``kp`` / ``vp``
    [NB, ceil(BS / pool), G, .]: block e of a sequence sits in row e % EP of the sequence's page e // EP; where keys are
    scaled values no keys but their factors, ``ks`` float32 [NB, BS, G]), all else in the
    activation dtype (block 0 is the engine's scratch block); per recurrent run float32 state rows S [NS, H, D, Dv]
    (the matrix-memory layers also n [NS, H, D] and m [NS, H]; the gated linear recurrence keeps S [NS, width];
    layers with a short convolution also its last conv - 1 inputs, ``hist`` [NS, conv - 1, C] in the activation
    dtype), one row per engine slot plus a scratch row (``scratch_slot``) for the decode rows of slots that hold no
    running sequence.  Tensors are keyed by the index of the layer RUN: a layer inside a loop has one set per pass;
    the two halves of a parallel mixer are keyed (run, 0) and (run, 1).

    A sequence's state needs no reset: a step whose first token sits at position 0 starts from zero."""

    def __init__(self, cfg: HybridConfig, num_blocks: int, block_size: int, device, act_dtype, slots: int):
        self.num_blocks, self.block_size = num_blocks, block_size
        self.slots = slots
        self.scratch_slot = slots
        self.lat: dict = {}
        self.S: dict = {}
        self.n: dict = {}
        self.m: dict = {}
        self.kc: dict = {}
        self.vc: dict = {}
        self.kp: dict = {}
        self.vp: dict = {}
        self.ks: dict = {}
        self.hist: dict = {}
        self._dev, self._at = device, act_dtype
        for li, l in enumerate(cfg.layers[i] for i in cfg.runs):
            self._alloc(li, l.mixer)

    def _alloc(self, li, mx) -> None:
        num_blocks, block_size, slots, device, act_dtype = self.num_blocks, self.block_size, self.slots, self._dev, self._at
        if mx.kind == "parallel":
            self._alloc((li, 0), mx.left)
            self._alloc((li, 1), mx.right)
        elif mx.kind == "latent_attention" and mx.kv_from is not None:
            self.lat[li] = self.lat[mx.kv_from]
        elif mx.kind == "latent_attention":
            self.lat[li] = torch.zeros(num_blocks, block_size, mx.kv_rank + mx.rot_dim, device=device, dtype=act_dtype)
        elif mx.kind == "mlstm":
            f32 = dict(device=device, dtype=torch.float32)
            self.S[li] = torch.zeros(slots + 1, mx.heads, mx.dim, mx.vdim, **f32)
            self.n[li] = torch.zeros(slots + 1, mx.heads, mx.dim, **f32)
            self.m[li] = torch.zeros(slots + 1, mx.heads, **f32)
        elif mx.kind == "window_attention":
            pg = dict(device=device, dtype=act_dtype)
            if mx.unit_keys:
                self.ks[li] = torch.zeros(num_blocks, block_size, mx.kv_heads, device=device, dtype=torch.float32)
            else:
                self.kc[li] = torch.zeros(num_blocks, block_size, mx.kv_heads, mx.dim, **pg)
            if mx.conv:
                self.hist[li] = torch.zeros(slots + 1, mx.conv - 1, _conv_channels(mx), **pg)
            self.vc[li] = torch.zeros(num_blocks, block_size, mx.kv_heads, mx.vdim, **pg)
            if mx.pool:
                ep = (block_size + mx.pool - 1) // mx.pool
                self.kp[li] = torch.zeros(num_blocks, ep, mx.kv_heads, mx.dim, **pg)
                self.vp[li] = torch.zeros(num_blocks, ep, mx.kv_heads, mx.vdim, **pg)
        elif mx.kind in ("delta_rule", "gla", "retention"):
            self.S[li] = torch.zeros(slots + 1, mx.heads, mx.dim, mx.vdim, device=device, dtype=torch.float32)
            if mx.kind == "delta_rule":
                ch = 2 * mx.kv_heads * mx.dim + mx.heads * mx.vdim
                self.hist[li] = torch.zeros(slots + 1, max(0, mx.conv - 1), ch, device=device, dtype=act_dtype)
        elif mx.kind == "mamba2":
            self.S[li] = torch.zeros(slots + 1, mx.heads, mx.state, mx.vdim, device=device, dtype=torch.float32)
            self.hist[li] = torch.zeros(slots + 1, max(0, mx.conv - 1), mx.conv_channels, device=device, dtype=act_dtype)
        elif mx.kind == "rglru":
            self.S[li] = torch.zeros(slots + 1, mx.width, device=device, dtype=torch.float32)
            self.hist[li] = torch.zeros(slots + 1, max(0, mx.conv - 1), mx.width, device=device, dtype=act_dtype)

    @staticmethod
    def bytes_per_block(cfg: HybridConfig, block_size: int, act_dtype) -> int:
        eb = 4 if act_dtype == torch.float32 else 2

        def per_page(m) -> int:   # bytes one page of this mixer holds
            if m.kind == "parallel":
                return per_page(m.left) + per_page(m.right)
            if m.kind == "latent_attention":
                return block_size * (m.kv_rank + m.rot_dim) * eb if m.kv_from is None else 0
            if m.kind == "window_attention" and m.unit_keys:
                return block_size * m.kv_heads * (m.vdim * eb + 4)
            if m.kind == "window_attention":
                rows = block_size + ((block_size + m.pool - 1) // m.pool if m.pool else 0)
                return rows * m.kv_heads * (m.dim + m.vdim) * eb
            return 0

        return max(1, sum(per_page(cfg.layers[i].mixer) for i in cfg.runs))

    def move_slots(self, src: torch.Tensor, dst: torch.Tensor) -> None:
        """Slot compaction: the recurrent state rows follow their sequences."""
        for t in (*self.S.values(), *self.n.values(), *self.m.values(), *self.hist.values()):
            t.index_copy_(0, dst, t.index_select(0, src))


# -----------------------------------------------------------------------------------------------------------------
# weights
# -----------------------------------------------------------------------------------------------------------------


@dataclass
class HybridLayerWeights:
    norm1: torch.Tensor
    mix: dict
    norm2: Optional[torch.Tensor] = None
    ff: dict = field(default_factory=dict)
    side: dict = field(default_factory=dict)   # the per-layer token input: w_gate, w_proj, norm, col0
    norm1b: Optional[torch.Tensor] = None      # sandwich stream: the norms on the sublayers' outputs
    norm2b: Optional[torch.Tensor] = None
    gate1: dict = field(default_factory=dict)  # residual gates: b (float32 bias) and, when the sublayer's own first
    gate2: dict = field(default_factory=dict)  # projection does not carry the gate's rows, w
    dwa: Optional[torch.Tensor] = None         # depth average: float32 [layer + 2]


@dataclass
class HybridWeights:
    embed: torch.Tensor
    layers: list
    final_norm: torch.Tensor
    head: torch.Tensor
    side_embed: Optional[torch.Tensor] = None

    def nbytes(self) -> int:
        n = 0
        for t in (self.embed, self.final_norm, self.head, self.side_embed):
            if t is not None:
                n += t.numel() * t.element_size()
        for l in {id(l): l for l in self.layers}.values():   # a layer that runs on another's weights counts once
            for t in (l.norm1, l.norm2, l.norm1b, l.norm2b, l.dwa, *l.mix.values(), *l.ff.values(), *l.side.values(),
                      *l.gate1.values(), *l.gate2.values()):
                if isinstance(t, torch.Tensor):
                    n += t.numel() * t.element_size()
                elif isinstance(t, dict):
                    n += sum(v.numel() * v.element_size() for v in t.values() if isinstance(v, torch.Tensor))
        return n


def _in_proj(rows: list, t: dict, out: dict, key: str, cast, gate: bool = False) -> None:
    """out[key] = the sublayer's first projection: ``rows`` stacked and behind them what else reads the same input, each
    from a column of its own on: with t["rg"] a residual gate's rows (out["rg_off"]); with t["ff"] = (spec, gate and up
    rows, down) the first projection of a gated feed-forward that runs beside the mixer (out["ff"] = its column and
    its spec) and, with ``gate``, the per-head gate's rows t["g"] (out["g_off"]).  The latter start on multiples of 8
    columns and end on one of 16 (rows of zeros between)."""
    if "rg" in t:
        out["rg_off"] = sum(r.shape[0] for r in rows)
        rows = rows + [t["rg"]]
    if "ff" in t:
        n, stack = 0, []

        def put(r, unit):
            nonlocal n
            stack.append(r)
            n += r.shape[0]
            pad = -n % unit
            if pad:
                stack.append(torch.zeros(pad, r.shape[1], dtype=r.dtype, device=r.device))
                n += pad

        for i, r in enumerate(rows):
            put(r, 8 if i == len(rows) - 1 else 1)
        spec, gu, _ = t["ff"]
        out["ff"] = (n, spec)
        put(gu, 8 if gate else 16)
        if gate:
            out["g_off"] = n
            put(t["g"], 16)
        rows = stack
    out[key] = cast(rows[0] if len(rows) == 1 else torch.cat(rows, 0))


def _out_proj(t: dict, out: dict, cast) -> None:
    """out["w_o"] = the mixer's output projection; with a feed-forward beside it (t["ff"]) the down projection's columns
    follow: one product over [mixer output | feed-forward activation] is the sum of the two sublayers."""
    out["w_o"] = cast(torch.cat([t["o"], t["ff"][2]], 1) if "ff" in t else t["o"])


def ff_rides_along(mixer, ff) -> bool:
    """Can a layer's feed-forward, on a parallel stream, share the mixer's first and last products?  A gated one beside
    an attention mixer, with both parts of the last product on 16-byte columns."""
    return ff is not None and ff.kind == "glu" and mixer.kind in ("latent_attention", "window_attention") and \
        ff.ff % 8 == 0 and mixer.heads * mixer.vdim % 8 == 0


def pack_mlstm(spec: MLSTMSpec, t: dict, device, act_dtype) -> dict:
    """t: q, k, v, g, o, norm, i, i.b, f, f.b (checkpoint layout, [out, in]).  q | k | v | g become one projection,
    the two gate rows one few-row float32-output projection."""
    a = lambda x: x.to(device=device, dtype=act_dtype).contiguous()  # noqa: E731
    f = lambda x: x.to(device=device, dtype=torch.float32).contiguous()  # noqa: E731
    return dict(w_proj=a(torch.cat([t["q"], t["k"], t["v"], t["g"]], 0)), w_if=a(torch.cat([t["i"], t["f"]], 0)),
                b_if=f(torch.cat([t["i.b"], t["f.b"]], 0)), norm=f(t["norm"]), w_o=a(t["o"]))


def pack_latent(spec: LatentAttentionSpec, t: dict, device, act_dtype) -> dict:
    """t: q (or dq, dq.norm, uq), dkv, dkv.norm (not with kv_from), uk, uv, g, sink, o.  q | dkv (| g with a gate per
    output column) are one projection, with a query latent dq | dkv are; per-head
    gate rows are a few-row float32-output projection.  The per-head up-projections are kept as [H, rank, D] and
    [H, Dv, rank]: keys are never materialised (the query is carried into the latent space instead) and the value
    up-projection is applied to the attention's latent-space output."""
    a = lambda x: x.to(device=device, dtype=act_dtype).contiguous()  # noqa: E731
    f = lambda x: x.to(device=device, dtype=torch.float32).contiguous()  # noqa: E731
    out = dict(w_uk=a(t["uk"].view(spec.heads, spec.dim, spec.kv_rank).transpose(1, 2)),
               w_uv=a(t["uv"].view(spec.heads, spec.vdim, spec.kv_rank)))
    rows = [t["dq"] if spec.q_rank else t["q"]]
    if spec.q_rank:
        out.update(dq_norm=f(t["dq.norm"]), w_uq=a(t["uq"]))
    if spec.kv_from is None:
        out["dkv_norm"] = f(t["dkv.norm"])
        rows.append(t["dkv"])
    _in_proj(rows + ([t["g"]] if spec.gate and spec.gate_wide else []), t, out, "w_in", a)
    _out_proj(t, out, a)
    if spec.sink:
        out["sink"] = f(t["sink"])
    if spec.gate and not spec.gate_wide:
        out["w_g"] = a(t["g"])
    return out


def pack_dense(spec: DenseFFSpec, t: dict, device, act_dtype) -> dict:
    a = lambda x: x.to(device=device, dtype=act_dtype).contiguous()  # noqa: E731
    return dict(w_up=a(t["up"]), w_down=a(t["down"]))


def pack_poly(spec: PolyFFSpec, t: dict, device, act_dtype) -> dict:
    """t: up, down, act (a, b, c, e)."""
    a = lambda x: x.to(device=device, dtype=act_dtype).contiguous()  # noqa: E731
    out = dict(w_down=a(t["down"]), act=t["act"].to(device=device, dtype=torch.float32).contiguous())
    _in_proj([t["up"]], t, out, "w_up", a)
    return out


def pack_moe(spec: MoEFFSpec, t: dict, device, act_dtype) -> dict:
    """t: router, correction (zeros when the design has none), e<k>.up, e<k>.down and, with a shared expert, shared.up, shared.down.
    Expert weights are stacked [E, ...] for the grouped kernels."""
    a = lambda x: x.to(device=device, dtype=act_dtype).contiguous()  # noqa: E731
    corr = t["correction"] if spec.correction else torch.zeros(spec.experts + spec.identity)
    out = dict(w_router=a(t["router"]), correction=corr.to(device=device, dtype=torch.float32).contiguous(),
               w_up=a(torch.stack([t[f"e{e}.up"] for e in range(spec.experts)])),
               w_down=a(torch.stack([t[f"e{e}.down"] for e in range(spec.experts)])))
    if spec.shared_ff:
        out.update(ws_up=a(t["shared.up"]), ws_down=a(t["shared.down"]))
    return out


def pack_window_attention(spec: WindowAttentionSpec, t: dict, device, act_dtype) -> dict:
    """t: q, k, v, q.norm, k.norm, sink, g, o, the convolution's taps q.conv, k.conv, v.conv and, in value-mixing
    layers, vmix.  q | k | v become one projection
    (q | k when the values are the keys; q | k | v | g with a gate per output column); per-head gate rows are a
    few-row float32-output projection (with a feed-forward beside the mixer they end the one projection)."""
    a = lambda x: x.to(device=device, dtype=act_dtype).contiguous()  # noqa: E731
    f = lambda x: x.to(device=device, dtype=torch.float32).contiguous()  # noqa: E731
    rows = [t["q"], t["k"]] + ([] if spec.v_from_k else [t["v"]]) + ([t["g"]] if spec.gate and spec.gate_wide else [])
    out = {}
    few = spec.gate and not spec.gate_wide
    _in_proj(rows, t, out, "w_qkv", a, few)
    _out_proj(t, out, a)
    if spec.conv:
        out["taps"] = f(torch.cat([t["q.conv"], t["k.conv"]] + ([] if spec.v_from_k else [t["v.conv"]]), 0))
    if spec.qk_norm and not spec.unit_keys:
        one = torch.ones(spec.dim)
        out.update(q_norm=f(t["q.norm"] if spec.qk_norm_weight else one), k_norm=f(t["k.norm"] if spec.qk_norm_weight else one))
    if spec.sink:
        out["sink"] = f(t["sink"] if spec.sink_fixed is None else torch.full((spec.heads,), float(spec.sink_fixed)))
    if few and "g_off" not in out:
        out["w_g"] = a(t["g"])
    if spec.bias:
        rest = out["w_qkv"].shape[0] - spec.heads * spec.dim - spec.kv_heads * (spec.dim + spec.vdim)  # gate rows: none
        out["b_qkv"] = a(torch.cat([t["q.b"], t["k.b"], t["v.b"], torch.zeros(rest, dtype=t["q.b"].dtype)], 0))
    if spec.bias_o:
        out["b_o"] = a(t["o.b"])
    if spec.v_mix and not spec.v_mix_first:
        out["vmix"] = f(t["vmix"]).reshape(1)
    return out


def pack_mamba2(spec: Mamba2Spec, t: dict, device, act_dtype) -> dict:
    """t: in ([z | x | B | C | dt] rows), conv, conv.b, dt_bias, A_log, D, norm, o.  The dt rows leave the big
    projection for a few-row float32-output projection whose bias is dt_bias."""
    a = lambda x: x.to(device=device, dtype=act_dtype).contiguous()  # noqa: E731
    f = lambda x: x.to(device=device, dtype=torch.float32).contiguous()  # noqa: E731
    n = 2 * spec.inner + 2 * spec.groups * spec.state
    return dict(w_in=a(t["in"][:n]), w_dt=a(t["in"][n:]), b_dt=f(t["dt_bias"]), taps=f(t["conv"]),
                b_conv=f(t["conv.b"]), a_log=f(t["A_log"]), skip=f(t["D"]), norm=f(t["norm"]), w_o=a(t["o"]))


def pack_rglru(spec: RGLRUSpec, t: dict, device, act_dtype) -> dict:
    """t: y, y.b, x, x.b, conv, conv.b, ra, ra.b, ri, ri.b, lam, o.  y | x are one biased projection; the two gate
    matrices of a block become one [blocks, in, 2 out] operand (its product accumulates and lands in float32);
    softplus(lam) is formed once, in float32."""
    a = lambda x: x.to(device=device, dtype=act_dtype).contiguous()  # noqa: E731
    f = lambda x: x.to(device=device, dtype=torch.float32).contiguous()  # noqa: E731
    wg = torch.cat([t["ra"].float().transpose(1, 2), t["ri"].float().transpose(1, 2)], 2)
    bg = torch.cat([t["ra.b"].float(), t["ri.b"].float()], 1)[:, None, :]
    return dict(w_yx=a(torch.cat([t["y"], t["x"]], 0)), b_yx=a(torch.cat([t["y.b"], t["x.b"]], 0)), taps=f(t["conv"]),
                b_conv=f(t["conv.b"]), w_gates=a(wg), b_gates=f(bg),
                sp=f(torch.nn.functional.softplus(t["lam"].float(), threshold=30.0)), w_o=a(t["o"]))


def pack_delta_rule(spec: DeltaRuleSpec, t: dict, device, act_dtype) -> dict:
    """t: q, k, v (+ .conv each), b, a, dt_bias, A_log, g, norm, o.  q | k | v | g are one projection, the
    convolution taps of q | k | v one [C, conv] float32 table, decay and write-strength rows one few-row
    float32-output projection (bias: dt_bias for the decay rows, zero for the others)."""
    a = lambda x: x.to(device=device, dtype=act_dtype).contiguous()  # noqa: E731
    f = lambda x: x.to(device=device, dtype=torch.float32).contiguous()  # noqa: E731
    return dict(w_proj=a(torch.cat([t["q"], t["k"], t["v"], t["g"]], 0)),
                taps=f(torch.cat([t["q.conv"], t["k.conv"], t["v.conv"]], 0)),
                w_ab=a(torch.cat([t["a"], t["b"]], 0)),
                b_ab=f(torch.cat([t["dt_bias"].float(), torch.zeros(spec.heads)], 0)), a_log=f(t["A_log"]),
                norm=f(t["norm"].float().repeat(spec.heads)), w_o=a(t["o"]))


def pack_gla(spec: GLASpec, t: dict, device, act_dtype) -> dict:
    """t: q, k, v, g, a1, a2, a2.b, norm, o.  q | k | v | g are one projection; the decay's low-rank projection keeps
    float32 outputs (a1 through the few-row projection, a2 as a float32 matrix)."""
    a = lambda x: x.to(device=device, dtype=act_dtype).contiguous()  # noqa: E731
    f = lambda x: x.to(device=device, dtype=torch.float32).contiguous()  # noqa: E731
    out = dict(w_a1=a(t["a1"]), w_a2t=f(t["a2"].float().t()), b_a2=f(t["a2.b"]),
               norm=f(t["norm"].float().repeat(spec.heads)), w_o=a(t["o"]))
    _in_proj([t["q"], t["k"], t["v"], t["g"]], t, out, "w_proj", a)
    return out


def pack_retention(spec: RetentionSpec, t: dict, device, act_dtype) -> dict:
    """t: q, k, v, g, o.  q | k | v | g are one projection; the decays are a float32 row, one number per head."""
    a = lambda x: x.to(device=device, dtype=act_dtype).contiguous()  # noqa: E731
    return dict(w_proj=a(torch.cat([t["q"], t["k"], t["v"], t["g"]], 0)), w_o=a(t["o"]),
                decay=torch.tensor(list(spec.decay), dtype=torch.float64).to(device=device, dtype=torch.float32),
                ones=torch.ones(spec.heads * spec.vdim, device=device, dtype=torch.float32))


def pack_parallel(spec: ParallelSpec, t: dict, device, act_dtype) -> dict:
    """t: left.* and right.* (each side's own tensors) plus left.out and right.out, the weights of the two outputs'
    norms over the model width."""
    f = lambda x: x.to(device=device, dtype=torch.float32).contiguous()  # noqa: E731
    side = lambda p: {k[len(p):]: v for k, v in t.items() if k.startswith(p) and k != p + "out"}  # noqa: E731
    return dict(left=MIXERS[spec.left.kind][1](spec.left, side("left."), device, act_dtype),
                right=MIXERS[spec.right.kind][1](spec.right, side("right."), device, act_dtype),
                out_l=f(t["left.out"]), out_r=f(t["right.out"]))


def pack_glu(spec: GluFFSpec, t: dict, device, act_dtype) -> dict:
    a = lambda x: x.to(device=device, dtype=act_dtype).contiguous()  # noqa: E731
    return dict(w_gu=a(torch.cat([t["gate"], t["up"]], 0)), w_down=a(t["down"]))


def pack_moe_glu(spec: MoEGluSpec, t: dict, device, act_dtype) -> dict:
    """t: router, router.b, e<k>.gate, e<k>.up, e<k>.down.  Per expert gate rows then up rows, stacked [E, 2F, d]."""
    a = lambda x: x.to(device=device, dtype=act_dtype).contiguous()  # noqa: E731
    out = dict(w_router=a(t["router"]), b_router=t["router.b"].to(device=device, dtype=torch.float32).contiguous(),
               w_gu=a(torch.stack([torch.cat([t[f"e{e}.gate"], t[f"e{e}.up"]], 0) for e in range(spec.experts)])),
               w_down=a(torch.stack([t[f"e{e}.down"] for e in range(spec.experts)])))
    d = out["w_gu"].shape[2]
    if act_dtype == torch.bfloat16 and torch.device(device).type == "cuda" and d % 128 == 0 and spec.ff % 128 == 0:
        # prompt portions take the grouped matrix-core path, which wants gate and up rows interleaved per tile
        out["w_gu"] = out["w_gu"][:, hops.moe_glu_row_order(spec.ff).to(out["w_gu"].device)].contiguous()
        out["gu_tiled"] = True
    return out


def pack_moe_group_glu(spec: MoEGroupGluSpec, t: dict, device, act_dtype) -> dict:
    """t: router, e<k>.gate / .up / .down and, with a shared expert, shared.gate / .up / .down / .sg."""
    a = lambda x: x.to(device=device, dtype=act_dtype).contiguous()  # noqa: E731
    out = pack_moe_glu(spec, {**t, "router.b": torch.zeros(spec.experts)}, device, act_dtype)
    del out["b_router"]
    if spec.shared_ff:
        out.update(ws_gu=a(torch.cat([t["shared.gate"], t["shared.up"]], 0)), ws_down=a(t["shared.down"]),
                   ws_gate=a(t["shared.sg"].reshape(1, -1)))
    return out


def rope_cos_sin(base: float, dims: int, max_pos: int, device, scaling: Optional[tuple] = None) -> torch.Tensor:
    """[max_pos, dims] float32: cos(p f_i) for i < dims/2, then sin(p f_i), f_i = base^(-2i/dims); angles in float64
    before the rounding to float32.  ``scaling``:

    (factor, low, high, original): frequencies whose wavelength is shorter than original/high stay, those longer than
        original/low are divided by factor, and between the two the frequency is interpolated linearly in
        original/wavelength;
    ("linear", factor): every frequency is divided by factor;
    ("ramp", factor, original, fast, slow): with n(t) = dims ln(original / (2 pi t)) / (2 ln base) the pair index at
        which ``original`` positions make t turns, lo = max(floor(n(fast)), 0), hi = min(ceil(n(slow)), dims - 1) and
        r_i = clamp((i - lo) / max(hi - lo, 0.001), 0, 1), the frequency is f_i / factor r_i + f_i (1 - r_i), and
        cos and sin are multiplied by 0.1 ln(factor) + 1."""
    import math

    inv = base ** (-torch.arange(0, dims, 2, dtype=torch.float64) / dims)
    mag = 1.0
    if scaling is not None and scaling[0] == "linear":
        inv = inv / float(scaling[1])
    elif scaling is not None and scaling[0] == "ramp":
        factor, orig, fast, slow = (float(v) for v in scaling[1:])
        where = lambda t: dims * math.log(orig / (2 * math.pi * t)) / (2 * math.log(base))  # noqa: E731
        lo, hi = max(math.floor(where(fast)), 0), min(math.ceil(where(slow)), dims - 1)
        r = ((torch.arange(dims // 2, dtype=torch.float64) - lo) / max(hi - lo, 0.001)).clamp(0.0, 1.0)
        inv = inv / factor * r + inv * (1 - r)
        mag = 0.1 * math.log(factor) + 1.0
    elif scaling is not None:
        factor, low, high, orig = (float(v) for v in scaling)
        wl = 2 * math.pi / inv
        s = ((orig / wl - low) / (high - low)).clamp(0.0, 1.0) if high != low else torch.ones_like(inv)
        mid = (1 - s) * inv / factor + s * inv
        inv = torch.where(wl < orig / high, inv, torch.where(wl > orig / low, inv / factor, mid))
    fr = torch.outer(torch.arange(max_pos, dtype=torch.float64), inv)
    return (torch.cat([fr.cos(), fr.sin()], 1) * mag).float().to(device)


def query_temperature(coef: float, every: float, max_pos: int, device) -> torch.Tensor:
    """[max_pos] float32: 1 + coef ln(floor((p + 1) / every) + 1), in float64 before the rounding."""
    p = torch.arange(1, max_pos + 1, dtype=torch.float64)
    return (1.0 + coef * torch.log(torch.floor(p / every) + 1.0)).float().to(device)


# -----------------------------------------------------------------------------------------------------------------
# mixers and feed-forwards (one function per kind: h [T, d] in the activation dtype -> [T, d])
# -----------------------------------------------------------------------------------------------------------------


@dataclass
class StepMeta:
    """One step's flattened token stream, prefill chunks and decode rows alike: sequence b owns tokens
    q_start[b]:q_start[b+1], the first of them at position pos0[b], its pages in block_table[b], its state in row
    slots[b] of the recurrent-state tensors."""
    ids: torch.Tensor
    pos: torch.Tensor
    tok_seq: torch.Tensor
    block_table: torch.Tensor
    q_start: torch.Tensor
    pos0: torch.Tensor
    slots: torch.Tensor
    last_idx: torch.Tensor
    max_q: int
    shared: dict = field(default_factory=dict)  # what one layer of a step leaves for later layers of the same step


def mix_mlstm(model, li: int, spec: MLSTMSpec, w: dict, h, meta: StepMeta, cache: HybridCache):
    H, D, Dv = spec.heads, spec.dim, spec.vdim
    proj = hops.matmul(h, w["w_proj"])
    gate_pre = hops.rowdot(h, w["w_if"], w["b_if"])
    o = hops.mlstm_scan(proj, gate_pre, meta.q_start, meta.pos0, meta.slots, cache.S[li], cache.n[li], cache.m[li],
                        H, D, Dv, spec.gate_cap, meta.max_q)
    y = hops.mlstm_out(o, proj, 2 * H * D + H * Dv, w["norm"], model.cfg.norm_eps, model.act_dtype)
    return hops.matmul(y, w["w_o"])


@dataclass
class GatedOut:
    """A sublayer's output together with the pre-activations of its residual gate, which its first projection carried:
    columns off .. off + d of src."""
    y: torch.Tensor
    src: torch.Tensor
    off: int


def _with_gate(y, proj, w: dict):
    return GatedOut(y, proj, w["rg_off"]) if "rg_off" in w else y


def _wide_out(w: dict, proj, n: int):
    """Rows for a mixer's output of n columns.  With a feed-forward beside the mixer they are the first n columns of
    wider ones, whose other columns receive the feed-forward's activation here; the caller's last product takes the
    wide rows.  Returns (wide rows or None, the mixer's columns or None: the op makes its own)."""
    if "ff" not in w:
        return None, None
    off, ff = w["ff"]
    wide = torch.empty(proj.shape[0], n + ff.ff, device=proj.device, dtype=proj.dtype)
    hops.glu_cols(proj, off, ff.ff, ff.limit, ff.slope, ff.shift, wide[:, n:])
    return wide, wide[:, :n]


def mix_latent_attention(model, li: int, spec: LatentAttentionSpec, w: dict, h, meta: StepMeta, cache: HybridCache):
    T = h.shape[0]
    H, D, R, rank = spec.heads, spec.dim, spec.rot_dim, spec.kv_rank
    eps = model.cfg.norm_eps
    nq, nkv = spec.q_rank or H * (D + R), rank + R
    proj = hops.matmul(h, w["w_in"])    # q or its latent | dkv (| one gate per output column)
    q = proj[:, :nq]
    if spec.q_rank:
        q = hops.matmul(hops.norm_cols(proj, 0, nq, w["dq_norm"], eps), w["w_uq"])
    q = q.view(T, H, D + R)
    gate = hops.rowdot(h, w["w_g"]) if spec.gate and not spec.gate_wide else None
    own = spec.kv_from is None
    # the query goes into the latent space (q_u W_uk per head), so a key is the cached row itself; the output
    # comes back through W_uv per head
    qa = torch.empty(T, H, rank + R, device=h.device, dtype=h.dtype)
    hops.latent_prep(q, proj[:, nq:nq + nkv] if own else None, meta.pos, meta.tok_seq, meta.block_table, w.get("dkv_norm"),
                     eps, model.rope.get(li), spec.rope_dims, rank, cache.lat[li], qa, spec.rope_interleaved)
    hops.head_matmul(q[:, :, :D], w["w_uk"], qa[:, :, :rank])
    oa = hops.latent_attention(qa, cache.lat[li], meta.block_table, meta.q_start, meta.pos, gate, spec.scale, rank,
                               model.act_dtype, meta.max_q, spec.window, spec.two_term, w.get("sink"))
    wide, ov = _wide_out(w, proj, H * spec.vdim)
    ov = hops.head_matmul(oa, w["w_uv"], None if ov is None else ov.view(T, H, spec.vdim),
                          proj if spec.gate and spec.gate_wide else None, nq + nkv if own else nq)
    return _with_gate(hops.matmul(ov.view(T, H * spec.vdim) if wide is None else wide, w["w_o"]), proj, w)


def mix_window_attention(model, li, spec: WindowAttentionSpec, w: dict, h, meta: StepMeta, cache: HybridCache):
    H, G, D, Dv = spec.heads, spec.kv_heads, spec.dim, spec.vdim
    proj = qkv = hops.matmul(h, w["w_qkv"], w.get("b_qkv"))
    gate = hops.rowdot(h, w["w_g"]) if "w_g" in w else None
    temp = model.q_temp.get(li)
    if spec.conv and spec.unit_keys:
        # convolution, norms, temperature, cache write and the gate's float32 copy in one pass over the projection
        qkv, gate_cols = hops.conv_prep(proj, w["taps"], meta.tok_seq, meta.q_start, meta.pos0, meta.slots, cache.hist[li],
                                        meta.pos, meta.block_table, H, G, D, model.cfg.norm_eps, temp, cache.ks[li],
                                        cache.vc[li], w.get("g_off", -1), meta.max_q)
        gate = gate if gate_cols is None else gate_cols
    else:
        if spec.conv:
            qkv = hops.short_conv(proj, w["taps"], meta.tok_seq, meta.q_start, meta.pos0, meta.slots, cache.hist[li], False)
        if "g_off" in w:
            gate = proj[:, w["g_off"]:w["g_off"] + H].float()
        mixes = spec.v_mix and not spec.v_mix_first
        v = hops.window_prep(qkv, H, G, D, Dv, meta.shared["v_first"] if mixes else None, w.get("vmix"), meta.pos,
                             meta.tok_seq, meta.block_table, w.get("q_norm"), w.get("k_norm"), model.cfg.norm_eps,
                             model.rope.get(li), spec.rope_dims, cache.kc.get(li), cache.vc[li], spec.v_mix_first,
                             H * D if spec.v_from_k else -1, model.rope_v.get(li), temp, cache.ks.get(li))
        if spec.v_mix_first:
            meta.shared["v_first"] = v
    pooled = spec.pool > 0 and spec.window > 0
    if pooled:   # the blocks this step's tokens complete get their means before any query of the step looks
        hops.pool_blocks(cache.kc[li], cache.vc[li], cache.kp[li], cache.vp[li], meta.block_table, meta.q_start,
                         meta.pos0, spec.pool, meta.max_q)
    wide, out = _wide_out(w, proj, H * Dv)
    o = hops.window_attention(qkv, cache.kc.get(li), cache.vc[li], meta.block_table, meta.q_start, meta.pos, w.get("sink"),
                              gate, spec.scale, spec.window, spec.keep_first, H, model.act_dtype, meta.max_q,
                              spec.chunk, spec.pool if pooled else 0, cache.kp.get(li), cache.vp.get(li),
                              model.rope_v.get(li), (H + G) * D + G * Dv if spec.gate and spec.gate_wide else -1,
                              cache.ks.get(li), out)
    return _with_gate(hops.matmul(o if wide is None else wide, w["w_o"], w.get("b_o")), proj, w)


def mix_retention(model, li, spec: RetentionSpec, w: dict, h, meta: StepMeta, cache: HybridCache):
    H, D, Dv = spec.heads, spec.dim, spec.vdim
    proj = hops.matmul(h, w["w_proj"])          # q | k | v | g
    hops.rotate_qk(proj, 0, H * D, H, H, D, spec.rope_dims, model.rope.get(li), meta.pos, 1.0, D ** -0.5)
    o = hops.linear_scan(proj, 0, H * D, 2 * H * D, None, None, 1.0, w["decay"], None, meta.q_start, meta.pos0,
                         meta.slots, cache.S[li], H, H, D, Dv)
    return hops.matmul(hops.head_norm_gate(o, proj, 2 * H * D + H * Dv, w["ones"], model.cfg.norm_eps, True,
                                           model.act_dtype), w["w_o"])


@dataclass
class PairOut:
    """What a parallel mixer hands to the stream's join: the two outputs and the weights of their norms."""
    y: torch.Tensor
    y2: torch.Tensor
    w: torch.Tensor
    w2: torch.Tensor


def mix_parallel(model, li, spec: ParallelSpec, w: dict, h, meta: StepMeta, cache: HybridCache):
    yl = MIXERS[spec.left.kind][0](model, (li, 0), spec.left, w["left"], h, meta, cache)
    yr = MIXERS[spec.right.kind][0](model, (li, 1), spec.right, w["right"], h, meta, cache)
    return PairOut(yl, yr, w["out_l"], w["out_r"])


def mix_mamba2(model, li: int, spec: Mamba2Spec, w: dict, h, meta: StepMeta, cache: HybridCache):
    H, P, N, G = spec.heads, spec.vdim, spec.state, spec.groups
    inner, GN = spec.inner, spec.groups * spec.state
    proj = hops.matmul(h, w["w_in"])                 # z | x | B | C
    dt_pre = hops.rowdot(h, w["w_dt"], w["b_dt"])    # float32 step pre-activations, bias included
    xbc = hops.short_conv(proj, w["taps"], meta.tok_seq, meta.q_start, meta.pos0, meta.slots, cache.hist[li], True,
                          w["b_conv"], inner)        # x | B | C after convolution and SiLU
    decay, dt = hops.ssm_prep(dt_pre, w["a_log"])
    # state rows = B, read by C, written with dt x: S <- decay S + B (dt x)^T, o = S^T C
    o = hops.linear_scan(xbc, inner + GN, inner, 0, None, None, 1.0, decay, None, meta.q_start, meta.pos0, meta.slots,
                         cache.S[li], G, H, N, P, dt)
    y = hops.gated_group_norm(o, xbc, 0, w["skip"], proj, 0, w["norm"], spec.norm_groups, model.cfg.norm_eps,
                              model.act_dtype)
    return hops.matmul(y, w["w_o"])


def mix_rglru(model, li: int, spec: RGLRUSpec, w: dict, h, meta: StepMeta, cache: HybridCache):
    W = spec.width
    proj = hops.matmul(h, w["w_yx"], w["b_yx"])      # y branch | x branch
    u = hops.short_conv(proj, w["taps"], meta.tok_seq, meta.q_start, meta.pos0, meta.slots, cache.hist[li], False,
                        w["b_conv"], W)
    gates = hops.block_gates(u, w["w_gates"], w["b_gates"])   # float32 [blocks, T, 2 W / blocks]
    o = hops.rglru_scan(u, gates, w["sp"], spec.c, proj, 0, meta.q_start, meta.pos0, meta.slots, cache.S[li],
                        model.act_dtype, meta.max_q)
    return hops.matmul(o, w["w_o"])


def mix_delta_rule(model, li: int, spec: DeltaRuleSpec, w: dict, h, meta: StepMeta, cache: HybridCache):
    H, HK, D, Dv = spec.heads, spec.kv_heads, spec.dim, spec.vdim
    C = 2 * HK * D + H * Dv
    proj = hops.matmul(h, w["w_proj"])          # q | k | v | g
    ab = hops.rowdot(h, w["w_ab"], w["b_ab"])   # decay and write-strength pre-activations, float32
    y = hops.short_conv(proj, w["taps"], meta.tok_seq, meta.q_start, meta.pos0, meta.slots, cache.hist[li], True)
    qscale, kscale, decay, beta = hops.delta_prep(y, ab, w["a_log"], HK, H, D, D ** -0.5)
    o = hops.linear_scan(y, 0, HK * D, 2 * HK * D, qscale, kscale, 1.0, decay, beta, meta.q_start, meta.pos0,
                         meta.slots, cache.S[li], HK, H, D, Dv)
    return hops.matmul(hops.head_norm_gate(o, proj, C, w["norm"], model.cfg.norm_eps, True, model.act_dtype), w["w_o"])


def mix_gla(model, li: int, spec: GLASpec, w: dict, h, meta: StepMeta, cache: HybridCache):
    H, D, Dv = spec.heads, spec.dim, spec.vdim
    proj = hops.matmul(h, w["w_proj"])          # q | k | v | g
    z = torch.addmm(w["b_a2"], hops.rowdot(h, w["w_a1"]), w["w_a2t"])  # float32 decay logits [T, H D]
    decay = hops.decay_pow(z, 1.0 / spec.tau)
    o = hops.linear_scan(proj, 0, H * D, 2 * H * D, None, None, D ** -0.5, decay, None, meta.q_start, meta.pos0,
                         meta.slots, cache.S[li], H, H, D, Dv)
    o = hops.head_norm_gate(o, proj, 2 * H * D + H * Dv, w["norm"], model.cfg.norm_eps, True, model.act_dtype)
    return _with_gate(hops.matmul(o, w["w_o"]), proj, w)


def ff_glu(model, spec: GluFFSpec, w: dict, h):
    return hops.matmul(hops.glu(hops.matmul(h, w["w_gu"]), spec.limit, spec.slope, spec.shift, model.act_dtype),
                       w["w_down"])


def ff_moe_glu(model, spec: MoEGluSpec, w: dict, h):
    idx, wt = hops.moe_route_topk(h, w["w_router"], w["b_router"], spec.top)
    return hops.moe_glu_ffn(h, idx, wt, w["w_gu"], w["w_down"], spec.limit, spec.slope, spec.shift, model.act_dtype,
                            bool(w.get("gu_tiled", False)))


def ff_moe_group_glu(model, spec: MoEGroupGluSpec, w: dict, h):
    """Returns the routed experts' sum and, with a shared expert, (sum, shared output, float32 gate logits [T, 1]):
    the stream's join adds sigmoid(gate) * shared."""
    idx, wt = hops.moe_route_group(h, w["w_router"], spec.top, spec.groups, spec.keep, spec.scale)
    y = hops.moe_glu_ffn(h, idx, wt, w["w_gu"], w["w_down"], spec.limit, spec.slope, spec.shift, model.act_dtype,
                         bool(w.get("gu_tiled", False)))
    if not spec.shared_ff:
        return y
    ys = hops.matmul(hops.glu(hops.matmul(h, w["ws_gu"]), spec.limit, spec.slope, spec.shift, model.act_dtype),
                     w["ws_down"])
    return y, ys, hops.rowdot(h, w["ws_gate"])


def ff_dense(model, spec: DenseFFSpec, w: dict, h):
    return hops.matmul(hops.act_inplace(hops.matmul(h, w["w_up"]), spec.act), w["w_down"])


def ff_poly(model, spec: PolyFFSpec, w: dict, h):
    z = hops.matmul(h, w["w_up"])
    return _with_gate(hops.matmul(hops.poly_norm(z, spec.ff, w["act"], model.cfg.norm_eps, model.act_dtype), w["w_down"]),
                      z, w)


def ff_moe(model, spec: MoEFFSpec, w: dict, h):
    """Returns the routed experts' sum and, with a shared expert, (sum, shared output): the stream's join adds both."""
    idx, wt = hops.moe_route(h, w["w_router"], w["correction"], spec.top)
    y = hops.moe_ffn(h, idx, wt, w["w_up"], w["w_down"], spec.act, model.act_dtype)
    if not spec.shared_ff:
        return y
    return y, hops.matmul(hops.act_inplace(hops.matmul(h, w["ws_up"]), spec.act), w["ws_down"])


MIXERS = {"mlstm": (mix_mlstm, pack_mlstm), "latent_attention": (mix_latent_attention, pack_latent),
          "window_attention": (mix_window_attention, pack_window_attention),
          "delta_rule": (mix_delta_rule, pack_delta_rule), "gla": (mix_gla, pack_gla),
          "mamba2": (mix_mamba2, pack_mamba2), "rglru": (mix_rglru, pack_rglru),
          "retention": (mix_retention, pack_retention), "parallel": (mix_parallel, pack_parallel)}
FEED_FORWARDS = {"dense": (ff_dense, pack_dense), "poly": (ff_poly, pack_poly), "moe": (ff_moe, pack_moe), "glu": (ff_glu, pack_glu),
                 "moe_glu": (ff_moe_glu, pack_moe_glu), "moe_group_glu": (ff_moe_group_glu, pack_moe_group_glu)}
RECURRENT_MIXERS = ("mlstm", "delta_rule", "gla", "mamba2", "rglru", "retention")


def _is_recurrent(mx) -> bool:
    """Does a sequence hold something beyond the tokens of its own pages?  A recurrent state, the last inputs of a short
    convolution; or pooled blocks, whose
    pair sits in the page e // EP while its tokens may lie on later pages (blocks off the page grid), so that a page
    shared between sequences as a common prefix could be written with one sequence's continuation."""
    if mx.kind == "parallel":
        return _is_recurrent(mx.left) or _is_recurrent(mx.right)
    return mx.kind in RECURRENT_MIXERS or (mx.kind == "window_attention" and (mx.conv > 1 or (mx.pool > 0 and mx.window > 0)))


# -----------------------------------------------------------------------------------------------------------------
# model
# -----------------------------------------------------------------------------------------------------------------


class HybridDecoder:
    """Serves through the same engine as the Llama models (same step batches, block manager, sampler).  What the
    engine needs from a model: ``cfg.vocab_size``, ``make_cache``, ``cache_bytes_per_block``, ``prefill_batch``,
    ``forward``, ``recurrent`` (state slots: no prefix sharing between sequences) and ``hq`` / ``hkv`` for its
    decode-split heuristics."""
    recurrent = True
    hq = hkv = 1

    def __init__(self, cfg: HybridConfig, weights: HybridWeights, device="cpu", max_position: int | None = None,
                 act_dtype=torch.bfloat16, tp: TPContext | None = None):
        self.cfg, self.w = cfg, weights
        self.tp = tp or TPContext.single()
        if self.tp.world > 1:
            raise NotImplementedError("the hybrid decoders run on full-weight ranks (data-parallel replicas only)")
        self.device = torch.device(device)
        self.act_dtype = act_dtype
        self.sequence_parallel = False
        self.decode_overlap_rows = 0
        P = max_position or cfg.max_position
        # rotation tables by run (the halves of a parallel mixer: (run, 0) and (run, 1)); equal tables are one tensor
        self.rope, self.rope_v, self.q_temp, made = {}, {}, {}, {}

        def table(base, dims, scaling):
            key = (float(base), int(dims), tuple(scaling) if scaling else None)
            if key not in made:
                made[key] = rope_cos_sin(base, dims, P, self.device, scaling)
            return made[key]

        def tables(key, mx):
            if mx.kind == "parallel":
                tables((key, 0), mx.left)
                tables((key, 1), mx.right)
            elif mx.kind in ("latent_attention", "window_attention", "retention"):
                if mx.rope_dims:
                    self.rope[key] = table(mx.rope_base, mx.rope_dims, getattr(mx, "rope_scaling", None))
                if getattr(mx, "v_rot", False):
                    self.rope_v[key] = table(mx.rope_base, mx.vdim, None)
                if getattr(mx, "q_temp", None):
                    tk = tuple(float(v) for v in mx.q_temp)
                    if tk not in made:
                        made[tk] = query_temperature(*tk, P, self.device)
                    self.q_temp[key] = made[tk]

        for ri, l in enumerate(cfg.layers[i] for i in cfg.runs):
            tables(ri, l.mixer)
        self.recurrent = any(_is_recurrent(l.mixer) for l in cfg.layers)
        if cfg.residual not in ("out_norm", "post_norm", "pre_norm", "sandwich", "parallel"):
            raise ValueError(f"unknown residual rule {cfg.residual!r}")
        if (cfg.residual == "parallel") != (cfg.norm == "layer"):
            raise ValueError("the parallel stream has layer norms with weight and bias, the others do not")
        for i, l in enumerate(cfg.layers):
            src = getattr(l.mixer, "kv_from", None)
            if src is None:
                continue
            m, o = l.mixer, cfg.layers[src].mixer if 0 <= src < i else None
            if cfg.loop or cfg.share is not None or getattr(o, "kind", "") != "latent_attention" or o.kv_from is not None:
                raise ValueError(f"layer {i}: kv_from names an earlier latent-attention layer with latents of its own, in "
                                 "a model whose layers run once")
            same = lambda a: (a.kv_rank, a.rot_dim, a.rope_base, a.rope_dims, a.rope_scaling, a.rope_interleaved)  # noqa: E731
            if same(m) != same(o):
                raise ValueError(f"layer {i}: kv_rank, rot_dim and rotation must be those of layer {src}")
        if cfg.token_side and cfg.residual != "pre_norm":
            raise ValueError("the per-layer token input is part of the pre-norm stream's join")
        if cfg.norm not in ("rms", "tanh", "layer"):
            raise ValueError(f"unknown norm {cfg.norm!r}")
        self.gated_stream = cfg.norm == "tanh" or cfg.residual_gate or cfg.depth_average or cfg.residual_mult != 1.0
        if self.gated_stream and (cfg.residual != "pre_norm" or cfg.token_side):
            raise ValueError("Dynamic Tanh norms, a residual multiplier, residual gates and depth averages belong to the "
                             "pre-norm stream, without a per-layer token input")
        if cfg.depth_average and (cfg.loop or cfg.share is not None):
            raise ValueError("a depth average weighs the layers' results one by one: layers may not repeat")

    # ---- what the engine calls --------------------------------------------------------------------------------
    def make_cache(self, num_blocks: int, block_size: int, slots: int, kv_dtype: str = "bf16", k_scale: float = 1.0,
                   v_scale: float = 1.0) -> HybridCache:
        if kv_dtype != "bf16":
            raise ValueError("the hybrid decoders cache in their activation dtype (kv_dtype must stay 'bf16')")
        return HybridCache(self.cfg, num_blocks, block_size, self.device, self.act_dtype, slots)

    def cache_bytes_per_block(self, block_size: int, kv_dtype: str = "bf16") -> int:
        return HybridCache.bytes_per_block(self.cfg, block_size, self.act_dtype)

    def prefill_batch(self, chunks, starts, block_tables, slots, max_blocks=None, nqt: int = 2, split: int = 1,
                      want=None) -> StepBatch:
        """Host builder of a prefill step: chunks[b] are sequence b's next tokens, the first at position starts[b];
        slots[b] its state slot.  ``want``: token indices (into the flattened stream) whose logits are asked for
        (default: every sequence's last token)."""
        ids, pos, tok_seq, qs = [], [], [], [0]
        for b, (toks, s0) in enumerate(zip(chunks, starts)):
            ids += toks
            pos += list(range(s0, s0 + len(toks)))
            tok_seq += [b] * len(toks)
            qs.append(qs[-1] + len(toks))
        mb = max_blocks or max(len(x) for x in block_tables)
        bt = torch.zeros(len(chunks), mb, dtype=torch.int32)
        for b, blks in enumerate(block_tables):
            bt[b, :len(blks)] = torch.tensor(blks, dtype=torch.int32)
        it = lambda x: torch.tensor(x, dtype=torch.int32)  # noqa: E731
        last = torch.tensor([q - 1 for q in qs[1:]] if want is None else list(want), dtype=torch.int64)
        dv = lambda t: h2d(t, self.device)  # noqa: E731
        mq = max((len(c) for c in chunks), default=0)
        return StepBatch(dv(it(ids)), dv(it(pos)), dv(it(tok_seq)), dv(bt), dv(it(qs)),
                         dv(it([s0 + len(t) for t, s0 in zip(chunks, starts)])), dv(last),
                         dv(torch.zeros(max(1, len(chunks)), 2, dtype=torch.int32)), len(chunks), nqt, 1,
                         slots=dv(it(list(slots))), max_q=mq)

    def _meta(self, sb: StepBatch) -> StepMeta:
        def one(p: StepBatch) -> StepMeta:
            if p.slots is None:
                raise ValueError("a hybrid decoder's step batch needs the sequences' state slots")
            if p.tiles is None:  # decode rows: token i is sequence i
                return StepMeta(p.ids, p.pos, p.tok_seq, p.block_table, p.q_start, p.pos, p.slots, p.last_idx, 1)
            pos0 = p.pos.index_select(0, p.q_start[:-1].long().clamp(max=max(0, p.pos.numel() - 1)))
            return StepMeta(p.ids, p.pos, p.tok_seq, p.block_table, p.q_start, pos0, p.slots, p.last_idx,
                            p.max_q or p.ids.numel())

        m = one(sb)
        if sb.dec is None:
            return m
        d = one(sb.dec)
        T, B = m.ids.numel(), m.block_table.shape[0]
        return StepMeta(torch.cat([m.ids, d.ids]), torch.cat([m.pos, d.pos]), torch.cat([m.tok_seq, d.tok_seq + B]),
                        torch.cat([m.block_table, d.block_table]), torch.cat([m.q_start, d.q_start[1:] + T]),
                        torch.cat([m.pos0, d.pos0]), torch.cat([m.slots, d.slots]), sb.last_idx, max(m.max_q, 1))

    def forward(self, sb: StepBatch, cache: HybridCache, logits_dtype=torch.float32) -> torch.Tensor:
        """Logits [len(sb.last_idx), V] of the tokens at sb.last_idx (with ``sb.dec``: indices into prefill tokens
        followed by decode rows)."""
        cfg, w, at = self.cfg, self.w, self.act_dtype
        meta = self._meta(sb)
        x, h = hops.embed_rows(meta.ids, w.embed, at, cfg.embed_scale, cfg.residual not in ("pre_norm", "sandwich", "parallel"))
        if self.gated_stream:
            self._forward_gated(x, meta, cache)
        elif cfg.residual == "pre_norm":
            self._forward_pre_norm(x, meta, cache)
        elif cfg.residual == "sandwich":
            self._forward_sandwich(x, meta, cache)
        elif cfg.residual == "parallel":
            self._forward_parallel(x, meta, cache)
        else:
            for ri, li in enumerate(cfg.runs):   # the cache is keyed by run, the weights by layer
                spec, lw = cfg.layers[li], w.layers[li]
                y = MIXERS[spec.mixer.kind][0](self, ri, spec.mixer, lw.mix, h, meta, cache)
                h = self._join(y, x, lw.norm1)
                if spec.ff is not None:
                    y = FEED_FORWARDS[spec.ff.kind][0](self, spec.ff, lw.ff, h)
                    h = self._join(y, x, lw.norm2)
                if self.layer_tap is not None:
                    self.layer_tap(ri, x)
        xs = x.index_select(0, meta.last_idx)
        if cfg.residual == "out_norm":
            xn = hops.layer_norm(xs, w.final_norm, cfg.norm_eps, at)
        elif cfg.norm == "tanh":
            xn = hops.dyn_tanh(xs, w.final_norm, at)
        elif cfg.norm == "layer":
            xn = hops.layer_norm_join(None, xs, w.final_norm, cfg.norm_eps, at)
        else:
            xn = hops.rms_norm(xs, w.final_norm, cfg.norm_eps, at, cfg.norm_groups if cfg.residual == "sandwich" else 1)
        logits = hops.matmul(xn, w.head).float()
        if cfg.logit_scale != 1.0:
            logits = logits * cfg.logit_scale
        return logits if logits.dtype == logits_dtype else logits.to(logits_dtype)

    def _forward_pre_norm(self, x, meta: StepMeta, cache: HybridCache) -> None:
        """x <- x + mixer(norm1(x)); x <- x + ff(norm2(x)); with a per-layer token input
        x <- x + rms_unit(W_proj (gelu(W_gate x) * e)) * w, e the layer's columns of each token's row of a second
        embedding table.  Every join kernel adds to the float32 stream in place and emits what the next sublayer
        reads: the next norm's output, or the stream's copy in the activation dtype for the token input's gate."""
        cfg, w, at, eps = self.cfg, self.w, self.act_dtype, self.cfg.norm_eps
        runs = cfg.runs
        h = hops.rms_norm(x, w.layers[runs[0]].norm1, eps, at) if runs else None
        for ri, li in enumerate(runs):
            spec, lw = cfg.layers[li], w.layers[li]
            nxt = w.layers[runs[ri + 1]].norm1 if ri + 1 < len(runs) else None   # the last run emits nothing:
            last = ri + 1 == len(runs)                                           # the final norm reads chosen rows
            y = MIXERS[spec.mixer.kind][0](self, ri, spec.mixer, lw.mix, h, meta, cache)
            y2 = g2 = None
            if spec.ff is not None:
                h = hops.add_rms_norm(y, x, lw.norm2, eps, at)
                y = FEED_FORWARDS[spec.ff.kind][0](self, spec.ff, lw.ff, h)
                if isinstance(y, tuple):
                    y, y2, g2 = y
            if cfg.token_side:
                xa = hops.add_rms_norm(y, x, None, eps, at, y2, g2)
                g = hops.token_gate(hops.matmul(xa, lw.side["w_gate"]), meta.ids, w.side_embed, lw.side["col0"], at)
                h = hops.add_rms_norm(hops.matmul(g, lw.side["w_proj"]), x, nxt, eps, at, w_y=lw.side["norm"],
                                      emit=not last)
            else:
                h = hops.add_rms_norm(y, x, nxt, eps, at, y2, g2, emit=not last)
            if self.layer_tap is not None:
                self.layer_tap(ri, x)

    def _forward_gated(self, x, meta: StepMeta, cache: HybridCache) -> None:
        """x <- x + m g1 * mixer(h), h = norm1(x); x <- x + m g2 * ff(h), h = norm2(x); then, with a depth average,
        x <- sum_j dwa[j] X_j over the embedding output and the layers' own results so far.  g1, g2: sigmoid of a
        projection of h (its rows ride in the sublayer's own first projection).  One join kernel per sublayer gates,
        scales and adds the sublayer's output, averages at a layer's end and emits the next norm."""
        cfg, w, at = self.cfg, self.w, self.act_dtype
        runs, hist = cfg.runs, None
        if cfg.depth_average and runs:   # X_0 .. X_(last - 1): the last layer's own result is needed by nobody else
            hist = torch.empty(len(runs), *x.shape, device=x.device, dtype=torch.float32)
            hist[0].copy_(x)
        tanh = cfg.norm == "tanh"
        norm = lambda wn: hops.dyn_tanh(x, wn, at) if tanh else hops.rms_norm(x, wn, cfg.norm_eps, at)  # noqa: E731

        def join(out, h, gate, wn, ri, dwa):
            if isinstance(out, (tuple, PairOut)):
                raise NotImplementedError("a sublayer with a separate part on a gated pre-norm stream")
            y, src, off = (out.y, out.src, out.off) if isinstance(out, GatedOut) else (out, None, -1)
            if cfg.residual_gate and src is None:
                src, off = hops.matmul(h, gate["w"]), 0
            hn = hops.gated_join(y, x, src, off, gate.get("b"), cfg.residual_mult, wn if tanh else None, at, hist, ri, dwa,
                                 tanh and wn is not None)
            return hn if tanh or wn is None else norm(wn)

        h = norm(w.layers[runs[0]].norm1) if runs else None
        for ri, li in enumerate(runs):
            spec, lw = cfg.layers[li], w.layers[li]
            nxt = w.layers[runs[ri + 1]].norm1 if ri + 1 < len(runs) else None   # the last run emits nothing
            y = MIXERS[spec.mixer.kind][0](self, ri, spec.mixer, lw.mix, h, meta, cache)
            if spec.ff is not None:
                h = join(y, h, lw.gate1, lw.norm2, ri, None)
                y = FEED_FORWARDS[spec.ff.kind][0](self, spec.ff, lw.ff, h)
                h = join(y, h, lw.gate2, nxt, ri, lw.dwa)
            else:
                h = join(y, h, lw.gate1, nxt, ri, lw.dwa)
            if self.layer_tap is not None:
                self.layer_tap(ri, x)

    def _forward_sandwich(self, x, meta: StepMeta, cache: HybridCache) -> None:
        """x <- x + norm1b(mixer(norm1(x))); x <- x + norm2b(ff(norm2(x))), every norm an RMS norm over
        ``norm_groups`` equal parts of the row.  One join kernel per sublayer: it norms the sublayer's output (a
        parallel mixer's two outputs are normed over the width and averaged first, a shared expert's output is added
        first), adds it to the float32 stream in place and emits the norm the next sublayer reads."""
        cfg, w, at, eps, ng = self.cfg, self.w, self.act_dtype, self.cfg.norm_eps, self.cfg.norm_groups
        runs = cfg.runs
        h = hops.rms_norm(x, w.layers[runs[0]].norm1, eps, at, ng) if runs else None
        for ri, li in enumerate(runs):
            spec, lw = cfg.layers[li], w.layers[li]
            last = ri + 1 == len(runs)    # the last run emits nothing: the final norm reads the wanted rows only
            nxt = None if last else w.layers[runs[ri + 1]].norm1
            y = MIXERS[spec.mixer.kind][0](self, ri, spec.mixer, lw.mix, h, meta, cache)
            y2 = pair = None
            if isinstance(y, PairOut):
                y, y2, pair = y.y, y.y2, (y.w, y.w2)
            if spec.ff is None:
                h = hops.sandwich_join(y, x, lw.norm1b, nxt, ng, eps, at, y2, pair, emit=not last)
            else:
                h = hops.sandwich_join(y, x, lw.norm1b, lw.norm2, ng, eps, at, y2, pair)
                y = FEED_FORWARDS[spec.ff.kind][0](self, spec.ff, lw.ff, h)
                y, y2 = y if isinstance(y, tuple) else (y, None)
                h = hops.sandwich_join(y, x, lw.norm2b, nxt, ng, eps, at, y2, None, emit=not last)
            if self.layer_tap is not None:
                self.layer_tap(ri, x)

    def _forward_parallel(self, x, meta: StepMeta, cache: HybridCache) -> None:
        """x <- x + mixer(h) + ff(h), h = layer_norm(x): both sublayers of a layer read one norm.  A feed-forward that
        rides along in the mixer's first and last products leaves one output to add, any other its own.  One join
        kernel per layer adds to the float32 stream in place and emits the next layer's norm."""
        cfg, w, at, eps = self.cfg, self.w, self.act_dtype, self.cfg.norm_eps
        runs = cfg.runs
        h = hops.layer_norm_join(None, x, w.layers[runs[0]].norm1, eps, at) if runs else None
        for ri, li in enumerate(runs):
            spec, lw = cfg.layers[li], w.layers[li]
            last = ri + 1 == len(runs)    # the last run emits nothing: the final norm reads the wanted rows only
            y = MIXERS[spec.mixer.kind][0](self, ri, spec.mixer, lw.mix, h, meta, cache)
            y2 = None
            if spec.ff is not None and "ff" not in lw.mix:
                y2 = FEED_FORWARDS[spec.ff.kind][0](self, spec.ff, lw.ff, h)
            if isinstance(y, PairOut) or isinstance(y2, tuple):
                raise NotImplementedError("a sublayer with a separate part on the parallel stream")
            h = hops.layer_norm_join(y, x, None if last else w.layers[runs[ri + 1]].norm1, eps, at, y2, emit=not last)
            if self.layer_tap is not None:
                self.layer_tap(ri, x)

    def _join(self, y, x, w):
        """The residual rule: folds the sublayer output y into the float32 stream x (in place) and returns the
        stream in the activation dtype for the next sublayer."""
        cfg = self.cfg
        if isinstance(y, (tuple, PairOut)):
            raise NotImplementedError("a feed-forward with a separate part needs the pre-norm or the sandwich stream, "
                                      "a parallel mixer the sandwich stream")
        if cfg.residual == "post_norm":
            return hops.scale_add_rms_norm(y, x, w, cfg.residual_alpha, cfg.norm_eps, self.act_dtype)
        return hops.add_layer_norm(y, x, w, cfg.norm_eps, self.act_dtype)

    layer_tap = None  # debugging hook: called with (layer index, residual stream) after every layer
