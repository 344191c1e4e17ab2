"""Architecture-neutral description of a decoder: parts, blocks, run order.

A ``ModelSpec`` is what an architecture's configuration is turned into before
anything is built.  It names every size and constant of every part, layer by
layer, so that no part needs to know which model it belongs to, and the order
in which layers run is a list of its own (``schedule``).  The reference fixes
all of this in one struct for one architecture (rocml/src/config.rs:32-54) and
keeps its constants in code (docs/multiarch-audit.md lists them as gaps 1-8);
here they are fields.

A part's spec is any object with a ``kind`` attribute; ``kind`` selects the
builder in ``rocml_amd.parts.registry``.  The dataclasses below are the specs of
the parts this library ships.
"""
from __future__ import annotations

from dataclasses import dataclass
from typing import Any, Optional, Tuple


@dataclass(frozen=True)
class NormSpec:
    """Root-mean-square norm over the last ``size`` values with a gain vector.  ``unit_offset``:
    the stored weight lies around zero and the gain is one plus it.  ``learned`` false: the norm
    has no weight, the values are only divided by their root mean square."""
    size: int
    eps: float
    kind: str = "rmsnorm"
    unit_offset: bool = False
    learned: bool = True


@dataclass(frozen=True)
class LayerNormSpec:
    """Norm with a weight and a bias: ``(x - mean) / sqrt(var + eps) * weight + bias``, ``var`` the
    mean of the squared deviations from the mean."""
    size: int
    eps: float
    kind: str = "layernorm"


@dataclass(frozen=True)
class RopeStretch:
    """Frequencies slowed down for contexts longer than ``original`` positions (YaRN): with
    ``d(t) = rot_dim ln(original / (2 pi t)) / (2 ln theta)``, ``lo = max(floor(d(fast)), 0)``,
    ``hi = min(ceil(d(slow)), rot_dim - 1)`` and ``r_i = clamp((i - lo) / max(hi - lo, 0.001), 0, 1)``,
    frequency ``i`` becomes ``f_i / factor * r_i + f_i (1 - r_i)``, and cosines and sines are
    multiplied by ``0.1 ln(factor) + 1``."""
    factor: float
    original: float
    fast: float
    slow: float


@dataclass(frozen=True)
class RopeSpec:
    """Rotary position encoding with NEOX pairing ``(i, i + rot_dim/2)`` over the
    first ``rot_dim`` values of a head; ``theta`` is the frequency base.  ``stretch``: the
    frequencies are slowed down as ``RopeStretch`` says.  ``pairing`` ``"neighbours"``: the pairs are
    ``(2 i, 2 i + 1)`` instead."""
    head_dim: int
    rot_dim: int
    theta: float
    kind: str = "rope_neox"
    stretch: Optional[RopeStretch] = None
    pairing: str = "halves"


@dataclass(frozen=True)
class AttentionSpec:
    """Softmax attention with grouped key/value heads over a cache.

    ``window`` is ``None`` for full causal attention, else the number of most
    recent positions (the query's own included) a query may see.  ``qk_norm`` is
    the per-head norm of queries and keys before rotation, or ``None``.

    ``v_head_dim``: the size of a value head when it is not ``head_dim``.  ``bias``: the four
    projections add a bias vector.  ``chunk``: instead of a window, positions are cut into blocks
    of so many, counted from position 0, and a query sees the keys of its own block up to itself.
    ``distance_slopes``: one number per query head; ``slope * (i - j)`` is taken off the score of
    query ``i`` and key ``j``.  ``sink``: the softmax's denominator has one more term, ``exp(0)``,
    which has no value.  ``q_temp``: ``(coef, every)``; the query at position ``p`` is multiplied by
    ``1 + coef * ln(floor((p + 1) / every) + 1)`` after its norm.  ``gate``: the concatenated heads
    are multiplied by ``sigmoid(W_g h)`` of the mixer's input before the output projection; with
    ``gate_per_head`` the gate is one number per query head instead of one per value.
    ``o_bias``: whether the output projection has a bias when it is not what ``bias`` says (None: as
    ``bias``).  ``qk_norm_span``: ``"head"``, every head of q and of k is normed by itself with a gain
    of the head's size, or ``"projection"``, a token's whole q row (all heads side by side) is
    normed at once with a gain of that size, and its k row likewise.  ``sink_learned`` (with ``sink``):
    the extra term is ``exp(sink_h)`` with a learned number per query head instead of ``exp(0)``.
    ``softcap``: the scaled score ``s`` becomes ``softcap * tanh(s / softcap)`` before the mask.
    ``conv``: q, k and v pass a causal convolution of so many taps per channel (no bias, no
    activation) right after their projection; the last ``conv - 1`` projected rows of a sequence
    are part of its state.  ``keep_first`` (with a window): the first so many positions stay visible
    whatever their distance.  ``values_are_keys``: there is no value projection, the values are the keys
    as projected (with their bias), before norm and rotation."""
    hidden: int
    n_heads: int
    n_kv_heads: int
    head_dim: int
    scale: float
    window: Optional[int] = None
    qk_norm: Optional[NormSpec] = None
    position: Optional[RopeSpec] = None
    kind: str = "attention"
    v_head_dim: Optional[int] = None
    bias: bool = False
    chunk: Optional[int] = None
    distance_slopes: Optional[Tuple[float, ...]] = None
    sink: bool = False
    q_temp: Optional[Tuple[float, int]] = None
    gate: bool = False
    gate_per_head: bool = False
    o_bias: Optional[bool] = None
    qk_norm_span: str = "head"
    sink_learned: bool = False
    softcap: Optional[float] = None
    conv: Optional[int] = None
    keep_first: int = 0
    values_are_keys: bool = False


@dataclass(frozen=True)
class LatentAttentionSpec:
    """Softmax attention whose keys and values are expanded from one small latent vector per
    position, which is all the cache holds besides one rotated key part that the heads share.

    Queries: ``c_q = norm(W_dq h)`` (``q_rank`` wide), ``q = W_uq c_q``, per head ``head_dim``
    values that are not rotated followed by ``rot_dim`` that are.  Keys and values:
    ``W_dkv h`` gives ``kv_rank`` values, normed into the latent ``c``, and ``rot_dim`` more, the
    shared rotated key part; per head the unrotated key is ``W_uk c`` and the value ``W_uv c``
    (``v_head_dim`` wide).  ``gate``: the concatenated heads are multiplied by
    ``sigmoid(W_g h)`` before the output projection; with ``gate_per_head`` the gate is one number per
    head.  ``own_rows`` false: the layer has no ``W_dkv`` and runs on the rows another layer keeps (an entry
    of the schedule with ``reads_cache_of``), with expansions of its own."""
    hidden: int
    n_heads: int
    head_dim: int
    rot_dim: int
    v_head_dim: int
    q_rank: int
    kv_rank: int
    scale: float
    q_norm: NormSpec
    kv_norm: NormSpec
    position: RopeSpec
    window: Optional[int] = None
    gate: bool = False
    kind: str = "latent_attention"
    gate_per_head: bool = False
    own_rows: bool = True


@dataclass(frozen=True)
class DifferentialAttentionSpec:
    """Softmax attention with two maps per head over the same values.  ``q`` has ``n_heads * 2 * head_dim`` rows and ``k``
    ``n_kv_heads * 2 * head_dim``, head by head ``[map 1, map 2]``; ``v`` has ``n_kv_heads * v_head_dim``.  Each map is an attention of its
    own (rotated as ``position`` says, scaled by ``scale``, under ``window``); with ``a1``, ``a2`` their outputs and
    ``lam = exp(sum(lq1 lk1)) - exp(sum(lq2 lk2)) + diff`` (one number for the layer, from four learned vectors of ``head_dim``), the
    head's output is ``o = a1 - lam a2`` divided by its root mean square (``eps`` inside the root), times ``1 - diff``."""
    hidden: int
    n_heads: int
    n_kv_heads: int
    head_dim: int
    v_head_dim: int
    scale: float
    diff: float
    eps: float
    window: Optional[int] = None
    position: Optional[RopeSpec] = None
    kind: str = "differential_attention"


@dataclass(frozen=True)
class GatedMlpSpec:
    """Dense gated feed-forward: ``down(act(g) * (u + up_offset))`` with ``g = gate(x)``,
    ``u = up(x)``.  ``limit``: ``g`` is cut off above at ``limit`` and ``u`` is held inside
    ``[-limit, limit]`` before anything else."""
    hidden: int
    intermediate: int
    activation: str = "silu"
    kind: str = "gated_mlp"
    limit: Optional[float] = None
    up_offset: float = 0.0


@dataclass(frozen=True)
class MlpSpec:
    """Dense feed-forward without a gate: ``down(act(up(x)))``; ``relu2`` is ``max(z, 0)^2``."""
    hidden: int
    intermediate: int
    activation: str = "relu2"
    kind: str = "mlp"


@dataclass(frozen=True)
class RoutedExpertsSpec:
    """A feed-forward of ``n_experts`` small gated feed-forwards (``down(act(gate x) * up x)``,
    no biases) of which each token uses ``top``.  The router's logits ``W_router h`` and their
    softmax over all experts are 32-bit.  ``groups``: ``(count, keep)``; the experts form ``count``
    equal groups of neighbours, a group's score is its largest expert score, and only experts of
    the ``keep`` best groups can be chosen.  The chosen experts' scores, divided by their sum plus
    ``sum_eps``, weight their outputs.  ``weighting`` ``"softmax_chosen"`` instead: the experts with
    the largest logits are chosen and the weights are the softmax over the chosen logits alone (no
    groups).  ``router_bias``: a bias vector is added to the router's logits.  ``weighting`` ``"sigmoid"``:
    an expert's score is ``sigmoid(logit)`` by itself.  ``correction``: a learned number per expert is added to the
    scores for the choice (of groups and of experts) only; the weights use the scores without it.
    ``group_score`` ``"top2_sum"``: a group's score is the sum of its two largest (corrected) scores instead of
    its largest.  ``shared_intermediate``: one more expert of that size runs for every token and is added, with
    ``shared_gate`` times ``sigmoid(W_sg h)`` (one number per token).  ``activation``, ``limit``, ``up_offset``: as in ``GatedMlpSpec``, for the
    experts and (with ``shared_limit`` as its limit) the shared one.  ``identity``: behind the ``n_experts`` the router knows so many
    more, whose output is their input and which have no matrices; scores, choice and weights do not tell them apart.
    ``weight_scale``: the weights are multiplied by it in the end."""
    hidden: int
    n_experts: int
    top: int
    intermediate: int
    activation: str = "silu"
    groups: Optional[Tuple[int, int]] = None
    sum_eps: float = 1e-20
    kind: str = "routed_experts"
    weighting: str = "softmax_all"
    router_bias: bool = False
    correction: bool = False
    group_score: str = "max"
    shared_intermediate: Optional[int] = None
    shared_gate: bool = False
    limit: Optional[float] = None
    up_offset: float = 0.0
    shared_limit: Optional[float] = None
    identity: int = 0
    weight_scale: float = 1.0


@dataclass(frozen=True)
class StateSpaceSpec:
    """A recurrence with one scalar decay per head (state-space duality): the input projection gives
    ``[z: inner | x: inner | B: groups * state | C: groups * state | dt: n_heads]`` with
    ``inner = n_heads * head_dim``; x, B and C pass a causal convolution of ``conv`` taps per channel
    (with bias) and silu; ``dt <- softplus(dt + dt_bias)``; per head (head ``a`` uses group
    ``a // (n_heads / groups)``) ``S <- exp(-exp(A_log) dt) S + dt B x^T``, ``y = S^T C + D x``;
    ``y * silu(z)`` is normed in ``norm_groups`` equal parts and projected back.  The state
    (``state x head_dim`` per head) and the convolution's last ``conv - 1`` inputs are 32-bit and
    live per sequence."""
    hidden: int
    n_heads: int
    head_dim: int
    state: int
    groups: int
    conv: int
    norm_groups: int
    eps: float
    kind: str = "state_space"


@dataclass(frozen=True)
class MatrixMemorySpec:
    """A recurrence whose state per head is a matrix ``S`` (``head_dim x v_head_dim``), a vector
    ``n`` (``head_dim``) and a running maximum ``m``, all zero when a sequence starts (the mLSTM of
    xLSTM).  ``q = W_q h / sqrt(head_dim)``, ``k = W_k h``, ``v = W_v h``; per head a log input gate
    ``i = cap tanh((W_i h + b_i) / cap)`` and a log forget gate
    ``f = logsigmoid(cap tanh((W_f h + b_f) / cap))``; ``m' = max(f + m, i)``,
    ``S' = exp(f + m - m') S + exp(i - m') k v^T``, ``n'`` the same with ``k`` alone, and the head's
    output is ``S'^T q / (max(|n' . q|, exp(-m')) + floor)``.  Every head's output is divided by its
    root mean square, the heads side by side are multiplied by a gain and by ``sigmoid(W_g h)`` and
    projected back.  State and gates are 32-bit."""
    hidden: int
    n_heads: int
    head_dim: int
    v_head_dim: int
    gate_cap: float
    eps: float
    floor: float = 1e-6
    kind: str = "matrix_memory"


@dataclass(frozen=True)
class RetentionSpec:
    """Linear attention with one fixed decay per head and neither softmax nor denominator:
    ``q = W_q h``, ``k = W_k h`` (rotated as ``position`` says, k then times ``head_dim^(-1/2)``),
    ``v = W_v h``; per head ``S <- decay_h S + k v^T`` and ``o = S^T q`` with the new ``S``.  Every head's
    output is divided by its root mean square, the heads side by side are multiplied by
    ``silu(W_g h)`` and projected back.  The state (``head_dim x v_head_dim`` per head) is 32-bit."""
    hidden: int
    n_heads: int
    head_dim: int
    v_head_dim: int
    decay: Tuple[float, ...]
    eps: float
    position: Optional[RopeSpec] = None
    kind: str = "retention"


@dataclass(frozen=True)
class TimeMixSpec:
    """A recurrence whose decay depends on the token, per head and key channel (the time mixing of
    RWKV-6).  With ``h'`` the previous token's input (zeros before the first), each of r, k, v, g, w
    reads its own mix ``h + (h' - h) mu``; ``r``, ``k``, ``v`` are ``n_heads x head_dim`` wide;
    ``w = exp(-exp(W_w2 tanh(W_w1 mix_w) + w0))`` with an inner width of ``decay_rank``; per head
    ``o = (S + diag(u) k v^T)^T r``, then ``S <- diag(w) S + k v^T``.  Every head's output is divided by
    its root mean square, the heads side by side are multiplied by a gain and by ``silu(W_g mix_g)``
    and projected back.  The state and the previous token's input live per sequence."""
    hidden: int
    n_heads: int
    head_dim: int
    decay_rank: int
    eps: float
    kind: str = "time_mix"


@dataclass(frozen=True)
class Hgrn2Spec:
    """Linear attention in which the forget gate also decides what is written (HGRN2): ``q = silu(W_q h)``,
    ``v = W_v h`` and per head and key channel ``f = l + (1 - l) sigmoid(W_f h + b)`` with a learned lower bound
    ``l``; per head ``S <- diag(f) S + (1 - f) v^T``, ``o = S^T q`` with the new ``S``.  Every head's output is
    normed over ``v_head_dim`` with one gain for all heads, the heads side by side are projected back.  The
    state (``head_dim x v_head_dim`` per head) is 32-bit."""
    hidden: int
    n_heads: int
    head_dim: int
    v_head_dim: int
    eps: float
    kind: str = "hgrn2"


@dataclass(frozen=True)
class GatedLinearAttentionSpec:
    """Linear attention with a decay per token and key channel (gated linear attention): ``q = W_q h``, ``k = W_k h``, ``v = W_v h``;
    ``alpha = sigmoid(W_a2 (W_a1 h) + b)^(1 / tau)`` with an inner width of ``decay_rank``; per head
    ``S <- diag(alpha) S + k v^T``, ``o = S^T q head_dim^(-1/2)`` with the new ``S``.  Every head's output is normed over ``v_head_dim`` with
    one gain for all heads, the heads side by side are multiplied by ``silu(W_g h)`` and projected back.  The state
    (``head_dim x v_head_dim`` per head) is 32-bit."""
    hidden: int
    n_heads: int
    head_dim: int
    v_head_dim: int
    decay_rank: int
    tau: float
    eps: float
    kind: str = "gated_linear_attention"


@dataclass(frozen=True)
class TokenSideSpec:
    """A per-token input that depends on the token's id: with ``e`` the columns ``column0 ..
    column0 + dim - 1`` of the token's row of the model's table ``table``, the result is
    ``W_proj (act(W_gate x) * e)``."""
    hidden: int
    dim: int
    table: str
    column0: int
    activation: str = "gelu_tanh"
    kind: str = "token_side"


@dataclass(frozen=True)
class TableSpec:
    """A matrix ``[rows, cols]`` of the model that several layers read (each its own columns)."""
    name: str
    rows: int
    cols: int


@dataclass(frozen=True)
class ParallelMixerSpec:
    """A set of mixers that all run on one input.  The result is
    ``weight * sum_b norm_b(out_b)``: each branch's output is normed over the model width with a
    gain of its own.  ``branches`` are ``(name, mixer spec)`` pairs; a branch's parameters and
    its output norm carry its name.  ``normed`` false: the branches' outputs are taken as they
    are.  ``branch_weights``: one factor per branch, ``sum_b branch_weights[b] * f_b(out_b)`` (then
    ``weight`` is not used)."""
    hidden: int
    branches: Tuple[Tuple[str, Any], ...]
    weight: float
    eps: float
    kind: str = "parallel"
    normed: bool = True
    branch_weights: Optional[Tuple[float, ...]] = None


@dataclass(frozen=True)
class TokenTableSpec:
    """The model's input: a row of a ``[vocab, hidden]`` table per token, times ``scale``."""
    vocab: int
    hidden: int
    scale: float = 1.0
    kind: str = "token_table"


@dataclass(frozen=True)
class TokenPositionTableSpec:
    """The model's input: a token's row of a ``[vocab, hidden]`` table times ``scale`` plus the
    row of its position in a learned ``[max_positions, hidden]`` table (not scaled)."""
    vocab: int
    hidden: int
    max_positions: int
    scale: float = 1.0
    kind: str = "token_position_table"


@dataclass(frozen=True)
class NormLinearHeadSpec:
    """The model's output: a norm of the wanted rows of the residual stream, then their
    product with a ``[vocab, hidden]`` matrix; ``tied``: that matrix is the input's table.
    ``scale``: the logits are multiplied by it.  ``softcap``: the logits ``z`` become ``softcap * tanh(z / softcap)`` (behind the
    scale)."""
    vocab: int
    hidden: int
    norm: NormSpec
    tied: bool
    kind: str = "norm_linear"
    softcap: Optional[float] = None
    scale: float = 1.0


@dataclass(frozen=True)
class BlockSpec:
    """One layer: a mixer and a feed-forward with their norms.

    ``arrangement`` names how they are wired; ``pre_norm`` is
    ``x += mixer(norm(x)); x += ffn(norm(x))``.  ``ffn`` (and then ``ffn_norm``) may be None:
    the layer is its mixer alone.  ``post_norm`` is
    ``x <- norm(residual_scale * x + mixer(x)); x <- norm(residual_scale * x + ffn(x))``: the
    sublayers read the stream itself and the norms come after the sums.  ``sublayer_norm`` is
    ``x += norm(mixer(x)); x += norm(ffn(x))``: the sublayers read the stream itself and a norm
    is applied to a sublayer's output alone.  ``side`` (with ``side_norm``): one more sublayer
    that runs last in the same way (only in ``sublayer_norm``).  ``sandwich_norm`` is
    ``x += mixer_out_norm(mixer(mixer_norm(x))); x += ffn_out_norm(ffn(ffn_norm(x)))``: a norm before
    and one after every sublayer.  ``input_conv``: what the mixer reads, ``h``, is first replaced by ``h`` plus
    a causal convolution of so many taps over it per channel (no bias); the last ``input_conv - 1`` rows of
    ``h`` are part of a sequence's state (only in ``pre_norm`` and ``sandwich_norm``).

    ``linked_streams`` keeps ``streams`` copies ``x_1 .. x_s`` of the stream (hyper-connections): a sublayer reads
    ``norm(sum_s in[s] x_s)``, and with ``y`` its output every copy becomes ``sum_s mix[s, t] x_s + branch_scale * out[t] * y``; ``in``,
    ``out`` and ``mix`` are learned numbers of the layer, for each of its sublayers.  A run of such layers starts with copies equal to
    the stream and leaves their sum as the stream."""
    mixer: Any
    ffn: Any
    mixer_norm: Any
    ffn_norm: Optional[Any]
    arrangement: str = "pre_norm"
    residual_scale: float = 1.0
    side: Any = None
    side_norm: Optional[Any] = None
    mixer_out_norm: Optional[Any] = None
    ffn_out_norm: Optional[Any] = None
    input_conv: Optional[int] = None
    streams: int = 1
    branch_scale: float = 1.0


@dataclass(frozen=True)
class ScheduleEntry:
    """One execution of a layer.  ``layer`` indexes ``ModelSpec.layers`` (a layer
    may appear in several entries and then runs its weights again with a cache
    line of its own).  ``reads_cache_of`` names an earlier entry of the schedule
    whose cache line this execution reads instead of writing its own.  ``offset_row``: row of
    the model's table of pass offsets (``ModelSpec.pass_offsets`` rows of ``hidden`` values) that
    is added to the residual stream of every token right before this execution.  ``add_embedding``:
    the embedding's output for the step's tokens (the stream as it was before the first entry) is
    added to the stream right before this execution."""
    layer: int
    reads_cache_of: Optional[int] = None
    offset_row: Optional[int] = None
    add_embedding: bool = False


@dataclass(frozen=True)
class ModelSpec:
    architecture: str
    vocab: int
    hidden: int
    layers: Tuple[BlockSpec, ...]
    schedule: Tuple[ScheduleEntry, ...]
    final_norm: Any
    tie_lm_head: bool
    max_positions: int
    embed_scale: float = 1.0
    eos_token_ids: Tuple[int, ...] = ()     # generation stops at any of these unless told otherwise
    # The parts at the model's two ends, chosen by ``kind`` like every other part.  None: the token
    # table and the norm-then-matrix head that the fields above describe.
    embedding: Any = None
    head: Any = None
    pass_offsets: int = 0                   # rows of the table that schedule entries add to the stream
    tables: Tuple[Any, ...] = ()            # matrices that parts of several layers read (``TableSpec``)
    logit_softcap: Optional[float] = None   # the default head's soft cap on the logits
    logit_scale: float = 1.0                # the default head's factor on the logits

    def embedding_spec(self) -> Any:
        return self.embedding if self.embedding is not None else \
            TokenTableSpec(self.vocab, self.hidden, self.embed_scale)

    def head_spec(self) -> Any:
        return self.head if self.head is not None else \
            NormLinearHeadSpec(self.vocab, self.hidden, self.final_norm, self.tie_lm_head, softcap=self.logit_softcap,
                               scale=self.logit_scale)

    def validate(self) -> None:
        from ..errors import ConfigError
        if not self.layers:
            raise ConfigError("a model needs at least one layer")
        for i, entry in enumerate(self.schedule):
            if not 0 <= entry.layer < len(self.layers):
                raise ConfigError(f"schedule entry {i} names layer {entry.layer}, "
                                  f"the model has {len(self.layers)}")
            if entry.offset_row is not None and not 0 <= entry.offset_row < self.pass_offsets:
                raise ConfigError(f"schedule entry {i} adds row {entry.offset_row} of the pass offsets, "
                                  f"the model has {self.pass_offsets}")
            src = entry.reads_cache_of
            if src is not None:
                if not 0 <= src < i:
                    raise ConfigError(f"schedule entry {i} reads the cache of entry {src}, "
                                      "which does not run before it")
                if self.schedule[src].reads_cache_of is not None:
                    raise ConfigError(f"schedule entry {i} reads the cache of entry {src}, "
                                      "which has no cache line of its own")


def default_schedule(n_layers: int) -> Tuple[ScheduleEntry, ...]:
    """Every layer once, in order, each with its own cache line."""
    return tuple(ScheduleEntry(layer=i) for i in range(n_layers))
