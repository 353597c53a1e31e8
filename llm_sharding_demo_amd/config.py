"""Configuration: model presets, engine settings, env-var compatibility.

The reference configures itself only through six environment variables
(`/root/reference/server.py:20-25`): MODEL_ID, SHARD_ROLE, SPLIT_AT,
SHARD_A_SERVICE, SHARD_B_SERVICE, SHARD_PORT.  Those names are kept here with
the same defaults; everything else the MI355X engine needs (stage count,
microbatching, KV budget, sampling defaults) is a dataclass field that can be
set from CLI > env > defaults.

Sampling defaults match the reference's hard-coded sampler
(`server.py:187-188`: temperature 0.6, top-k 40, multinomial).
"""
from __future__ import annotations

import dataclasses
import math
import os
from dataclasses import dataclass, field
from typing import Optional, Sequence, Tuple, Union


# ---------------------------------------------------------------------------
# Model presets
# ---------------------------------------------------------------------------

@dataclass(frozen=True)
class RopeScaling:
    """Wavelengths above original / low are stretched by `factor`, those below
    original / high stay, a linear ramp lies between."""

    factor: float
    low: float
    high: float
    original: float


@dataclass(frozen=True)
class RopeSpec:
    """Rotation of the first `dims` dimensions of a head, pairs (i, i + dims / 2)
    or, interleaved, (2i, 2i + 1)."""

    dims: int
    base: float
    scaling: Optional[RopeScaling] = None
    interleaved: bool = False

    def frequencies(self) -> list:
        out = []
        for i in range(self.dims // 2):
            f = self.base ** (-2.0 * i / self.dims)
            s = self.scaling
            if s is not None:
                turns = s.original * f / (2.0 * math.pi)  # original context in wavelengths
                if turns < s.low:
                    f /= s.factor
                elif turns <= s.high:
                    keep = (turns - s.low) / (s.high - s.low)
                    f = (1.0 - keep) * f / s.factor + keep * f
            out.append(f)
        return out


@dataclass(frozen=True)
class LatentAttentionSpec:
    """Attention whose keys and values are linear images of one cached latent
    row per token; every size is the layer's own.  With `rope`, a head's queries
    have rope.dims further dimensions that turn with the position, and all heads
    share one turned key part, cached behind the latent.  q_rank: queries come
    from a normed latent of their own.  sink: a learned score per head that
    takes part in the softmax without a value.  gate: a sigmoid gate per output
    channel."""

    heads: int
    dim: int                       # query / key dimensions per head (without positions)
    vdim: int                      # value dimensions per head
    kv_rank: int                   # latent dimensions: what the cache holds
    scale: float                   # score = (q . k) * scale
    window: Optional[int] = None   # keys per query, itself included (None: all)
    kv_from: Optional[int] = None  # use this earlier layer's cached latents
    rope: Optional[RopeSpec] = None
    q_rank: Optional[int] = None
    sink: bool = False
    gate: bool = False

    @property
    def rot_dim(self) -> int:
        return self.rope.dims if self.rope is not None else 0

    @property
    def q_dim(self) -> int:
        """Query dimensions per head."""
        return self.dim + self.rot_dim

    @property
    def cached_per_token(self) -> int:
        return self.kv_rank + self.rot_dim if self.kv_from is None else 0

    @property
    def in_columns(self) -> int:
        """Rows of the projections that read the layer's input."""
        q = self.heads * self.q_dim if self.q_rank is None else self.q_rank
        return q + self.cached_per_token + (self.heads * self.vdim if self.gate else 0)

    def params(self, hidden: int) -> int:
        n = hidden * (self.in_columns + self.heads * self.vdim) + self.heads * (self.dim + self.vdim) * self.kv_rank
        n += (self.kv_rank if self.kv_from is None else 0) + (self.heads if self.sink else 0)
        return n + (self.q_rank * (1 + self.heads * self.q_dim) if self.q_rank is not None else 0)

    def check(self) -> None:
        if min(self.heads, self.dim, self.vdim, self.kv_rank) < 1 or (self.window is not None and self.window < 1):
            raise ValueError("attention sizes must be positive")
        if self.rot_dim % 2 or (self.q_rank is not None and self.q_rank < 1):
            raise ValueError(f"cannot rotate {self.rot_dim} dimensions, or no query latent of {self.q_rank}")


@dataclass(frozen=True)
class AttentionSpec:
    """Grouped-query attention over a paged K/V cache.  In front of the scores:
    projection biases, a short convolution of q, k and v over time, unit RMS
    norms of q and k per head, partial rotation, and values mixed with those of
    an earlier layer.  Scores: capped (softcap tanh(s / softcap)), less a
    distance bias of the head's slope, a sliding window beside the first
    `keep_first` tokens.  `talking`: a learned [heads, heads] matrix mixes the
    scores over the heads before the softmax, or (talk_weights) the weights
    behind it.  head_gate: a sigmoid gate per head on its output."""

    heads: int
    kv_heads: int
    dim: int
    vdim: int
    scale: float
    window: Optional[int] = None
    rope: Optional[RopeSpec] = None
    softcap: Optional[float] = None
    talking: bool = True
    talk_weights: bool = False
    keep_first: int = 0
    distance_bias: bool = False
    conv: int = 0                   # taps (0: none)
    qk_norm: bool = False
    bias: bool = False              # of the projections in and out
    head_gate: bool = False
    mix_values: Optional[int] = None  # v <- (1 - l) v + l v of this layer (its own index: the values others mix in)
    kv_from: None = None

    @property
    def cached_per_token(self) -> int:
        return self.kv_heads * (self.dim + self.vdim)

    @property
    def conv_channels(self) -> int:
        return self.heads * self.dim + self.cached_per_token

    def slopes(self) -> list:
        """Distance bias per head: slope (i - j) is taken off the score."""
        return [2.0 ** (-8.0 * (h + 1) / self.heads) for h in range(self.heads)]

    def params(self, hidden: int) -> int:
        n = hidden * (self.conv_channels + self.heads * self.vdim) + self.conv_channels * self.conv
        n += (self.conv_channels + hidden if self.bias else 0) + (self.heads * hidden if self.head_gate else 0)
        return n + (self.heads ** 2 if self.talking else 0) + (self.mix_values is not None)

    def check(self) -> None:
        if min(self.heads, self.kv_heads, self.dim, self.vdim) < 1 or (self.window is not None and self.window < 1):
            raise ValueError("attention sizes must be positive")
        if self.conv < 0 or self.keep_first < 0:
            raise ValueError("convolution taps and kept tokens must not be negative")
        if self.heads % self.kv_heads:
            raise ValueError(f"{self.heads} heads cannot share {self.kv_heads} key / value heads evenly")
        if self.rope is not None and (self.rope.dims % 2 or not 0 <= self.rope.dims <= self.dim):
            raise ValueError(f"cannot rotate {self.rope.dims} of {self.dim} dimensions")
        if self.softcap is not None and self.softcap <= 0:
            raise ValueError("softcap must be positive")


@dataclass(frozen=True)
class ChannelDeltaSpec:
    """Gated delta rule with one decay per head and key channel: a state
    [dim, vdim] per head, a short convolution in front of q, k and v."""

    heads: int
    kv_heads: int                  # q / k heads; head h uses h // (heads / kv_heads)
    dim: int
    vdim: int
    conv: int                      # taps
    decay_rank: int                # inner width of the decay projection
    gate_rank: int                 # ... and of the output gate's
    kv_from: None = None
    cached_per_token = 0

    @property
    def conv_channels(self) -> int:
        return 2 * self.kv_heads * self.dim + self.heads * self.vdim

    def params(self, hidden: int) -> int:
        o, hd = self.heads * self.vdim, self.heads * self.dim
        n = hidden * (self.conv_channels + self.heads + self.decay_rank + self.gate_rank + o)
        return n + self.conv_channels * self.conv + self.decay_rank * hd + self.gate_rank * o + hd + self.heads + self.vdim

    def check(self) -> None:
        if min(self.heads, self.kv_heads, self.dim, self.vdim, self.conv, self.decay_rank, self.gate_rank) < 1:
            raise ValueError("delta rule sizes must be positive")
        if self.heads % self.kv_heads:
            raise ValueError(f"{self.heads} heads cannot share {self.kv_heads} key heads evenly")


@dataclass(frozen=True)
class SSMSpec:
    """Mamba-2: a state [state, vdim] per head with one decay per head and
    token; B and C shared by heads / groups heads, gated norm in norm_groups parts."""

    heads: int
    vdim: int
    state: int
    groups: int
    norm_groups: int
    conv: int
    kv_from: None = None
    cached_per_token = 0

    @property
    def inner(self) -> int:
        return self.heads * self.vdim

    @property
    def conv_channels(self) -> int:
        return self.inner + 2 * self.groups * self.state

    def params(self, hidden: int) -> int:
        n = hidden * (2 * self.inner + 2 * self.groups * self.state + self.heads + self.inner)
        return n + self.conv_channels * (self.conv + 1) + 3 * self.heads + self.inner

    def check(self) -> None:
        if min(self.heads, self.vdim, self.state, self.groups, self.norm_groups, self.conv) < 1:
            raise ValueError("state-space sizes must be positive")
        if self.heads % self.groups or self.inner % self.norm_groups:
            raise ValueError(f"{self.heads} heads in {self.groups} groups, width {self.inner} in "
                             f"{self.norm_groups} norm groups: must divide evenly")


@dataclass(frozen=True)
class ForgetSpec:
    """Linear attention whose forget gate, per head and channel, also decides
    what is written (HGRN2): a state [dim, vdim] per head, no keys."""

    heads: int
    dim: int
    vdim: int
    kv_from: None = None
    cached_per_token = 0

    def params(self, hidden: int) -> int:
        n, v = self.heads * self.dim, self.heads * self.vdim
        return hidden * 2 * (n + v) + 2 * n + self.vdim

    def check(self) -> None:
        if min(self.heads, self.dim, self.vdim) < 1:
            raise ValueError("recurrence sizes must be positive")


@dataclass(frozen=True)
class DenseSpec:
    """Gated feed-forward W_down(gelu_tanh(W_gate h) * W_up h), or with a
    `limit` the clamped gate of the experts."""

    ff: int
    limit: Optional[float] = None

    def params(self, hidden: int) -> int:
        return 3 * hidden * self.ff


@dataclass(frozen=True)
class ExpertSpec:
    """Gated feed-forward, SiLU or with clamped gate / up (`limit`)."""

    ff: int
    limit: Optional[float] = None


@dataclass(frozen=True)
class MoESpec:
    """Experts chosen by corrected sigmoid scores, which weigh them too, or
    (softmax) by their logits, with the softmax over the chosen ones as weights.
    shared_gate: a sigmoid per token weighs the shared expert."""

    experts: int
    top: int
    expert: ExpertSpec
    shared: Optional[ExpertSpec] = None  # runs for every token
    softmax: bool = False
    shared_gate: bool = False

    def params(self, hidden: int) -> int:
        n = self.experts * (hidden + (not self.softmax) + 3 * hidden * self.expert.ff)
        return n + (3 * hidden * self.shared.ff + hidden * self.shared_gate if self.shared is not None else 0)


MixerSpec = Union[LatentAttentionSpec, AttentionSpec, ChannelDeltaSpec, SSMSpec, ForgetSpec]


@dataclass(frozen=True)
class LayerSpec:
    """One layer as it runs.  A loop over layers is written out: every pass has
    entries of its own (and so its own cache or state), `weights` names the
    layer whose tensors they share (None: its own), and `enter` is the pass
    that begins in front of this entry with a step of its own (None: no such
    step)."""

    mixer: MixerSpec
    mlp: Union[MoESpec, DenseSpec, None] = None
    weights: Optional[int] = None
    enter: Optional[int] = None


# digits (base 256, exact in bf16) of a token id on the wire between stages
ID_DIGITS = 3


@dataclass(frozen=True)
class ModelConfig:
    """Architecture description of one model.

    GPT-2 and Llama have uniform layers: the scalar fields say everything.
    Models whose layers differ list them in `layers` (arch "timisun": parallel
    blocks of latent attention and experts; "vizalix": parallel blocks of
    attention, delta rule or Mamba-2 and a dense feed-forward, some of them
    looped; "kedasun": attention and a dense feed-forward one after the other,
    each between two norms; "fagunex": latent attention or a recurrence, and
    experts, each between two norms, behind a token shift and in front of rows of
    the tokens' own, some of them looped); the scalar head / ffn fields then only
    describe the first layer."""

    name: str
    arch: str  # "gpt2" | "llama" | "timisun" | "vizalix" | "kedasun" | "fagunex"
    vocab_size: int
    hidden: int
    n_layers: int
    n_heads: int
    n_kv_heads: int
    ffn: int
    max_positions: int
    norm_eps: float
    tie_embeddings: bool
    rope_theta: float = 0.0
    bos_token_id: int = 50256
    eos_token_id: int = 50256
    embed_scale: float = 1.0
    layers: Tuple[LayerSpec, ...] = ()
    norm_groups: int = 1  # equal parts of a row, each normed by itself
    token_shift: bool = False  # mixers read rows mixed with those of the previous token
    token_side: int = 0  # width of the rows that tokens bring to every layer (0: none)

    @property
    def whole_layers(self) -> bool:
        """A stage starts at a layer, never between its mixer and feed-forward."""
        return bool(self.layers)

    @property
    def paged_cache(self) -> bool:
        """The cache is a pool of token pages shared by the sequences
        (runtime/kv_cache.py PagedCache) instead of a region per slot."""
        return bool(self.layers)

    @property
    def shared_weights(self) -> bool:
        """Several layer runs may use the tensors of one layer."""
        return any(l.weights is not None for l in self.layers)

    @property
    def shift_width(self) -> int:
        """Columns of the previous token's row that every layer keeps of a sequence."""
        return self.hidden if self.token_shift else 0

    @property
    def loop_times(self) -> int:
        """Passes of the looped layers that begin with a step of their own (0: none)."""
        return max((l.enter + 1 for l in self.layers if l.enter is not None), default=0)

    @property
    def mixed_values(self) -> Optional[AttentionSpec]:
        """The layer whose values later layers mix in (None: no layer does)."""
        first = next((l.mixer.mix_values for l in self.layers if getattr(l.mixer, "mix_values", None) is not None), None)
        return None if first is None else self.layers[first].mixer

    @property
    def boundary(self) -> int:
        """Columns a stage hands to the next: the residual, the embedding
        output where a loop's passes read it again, the values that later
        layers mix in, and the token ids where every layer looks them up."""
        m = self.mixed_values
        n = self.hidden * (2 if self.loop_times else 1) + (m.kv_heads * m.vdim if m is not None else 0)
        return n + (ID_DIGITS if self.token_side else 0)

    def weight_layer(self, i: int) -> int:
        """The layer whose tensors layer i uses."""
        return i if not self.layers or self.layers[i].weights is None else self.layers[i].weights

    def stage_params(self, layers: Sequence[int]) -> int:
        """Parameters a stage with these layers holds (shared ones once)."""
        n = sum(self.layer_params(i) for i in {self.weight_layer(i): i for i in layers}.values())
        if any(self.layers and self.layers[i].enter is not None for i in layers):
            n += 2 * self.hidden * self.hidden + self.loop_times * self.hidden
        return n

    def cache_layers(self, layers: Sequence[int]) -> list:
        """Those of `layers` that own a cache (others share an earlier one)."""
        if not self.layers:
            return list(layers)
        return [i for i in layers if self.layers[i].mixer.kv_from is None]

    @property
    def head_dim(self) -> int:
        return self.hidden // self.n_heads

    @property
    def q_size(self) -> int:
        return self.n_heads * self.head_dim

    @property
    def kv_size(self) -> int:
        return self.n_kv_heads * self.head_dim

    @property
    def qkv_size(self) -> int:
        return self.q_size + 2 * self.kv_size

    @property
    def vocab_padded(self) -> int:
        """Vocab rounded up to a multiple of 64 so lm_head tiles evenly."""
        return (self.vocab_size + 63) // 64 * 64

    def layer_params(self, i: int) -> int:
        """Parameters of layer i."""
        if not self.layers:
            return self.block_params()
        h, m, f = self.hidden, self.layers[i].mixer, self.layers[i].mlp
        subs = 1 + (f is not None)
        norms = {"timisun": h, "kedasun": 2 * h * subs, "fagunex": 2 * (2 * h + 1) * subs}.get(self.arch, subs)
        side = (2 * h + self.vocab_size) * self.token_side + h if self.token_side else 0
        return norms + self.shift_width + side + m.params(h) + (f.params(h) if f is not None else 0)

    def block_params(self) -> int:
        """Parameters of a layer (of the mean layer when they differ)."""
        if self.layers:
            return sum(self.layer_params(i) for i in range(self.n_layers)) // self.n_layers
        h, f = self.hidden, self.ffn
        if self.arch == "gpt2":
            return 12 * h * h + 13 * h  # qkv+proj+fc+proj weights/biases + 2 LN
        return h * self.qkv_size + self.q_size * h + 3 * h * f + 2 * h

    def embed_params(self) -> int:
        n = self.vocab_size * self.hidden
        if self.arch == "gpt2":
            n += self.max_positions * self.hidden
        return n

    def lm_head_params(self) -> int:
        return self.vocab_size * self.hidden

    def kv_bytes_per_token_per_layer(self, dtype_bytes: int = 2) -> int:
        if self.layers:
            return sum(l.mixer.cached_per_token for l in self.layers) * dtype_bytes // self.n_layers
        return 2 * self.kv_size * dtype_bytes


def _gpt2(name: str, h: int, l: int, nh: int, vocab: int = 50257) -> ModelConfig:
    return ModelConfig(
        name=name, arch="gpt2", vocab_size=vocab, hidden=h, n_layers=l,
        n_heads=nh, n_kv_heads=nh, ffn=4 * h, max_positions=1024,
        norm_eps=1e-5, tie_embeddings=True)


# Dims from [tf5.15] models/gpt2/configuration_gpt2.py and SURVEY.md §2.5.
MODEL_PRESETS = {
    # sshleifer/tiny-gpt2: the reference default MODEL_ID (server.py:20)
    "tiny-gpt2": _gpt2("tiny-gpt2", 2, 2, 2),
    "gpt2": _gpt2("gpt2", 768, 12, 12),
    "gpt2-medium": _gpt2("gpt2-medium", 1024, 24, 16),
    "gpt2-large": _gpt2("gpt2-large", 1280, 36, 20),
    "gpt2-xl": _gpt2("gpt2-xl", 1600, 48, 25),
    # Small GPT-2 shapes used by kernel / pipeline tests (hd = 64 like real GPT-2).
    "gpt2-test": _gpt2("gpt2-test", 128, 4, 2, vocab=1000),
    "llama-3-8b": ModelConfig(
        name="llama-3-8b", arch="llama", vocab_size=128256, hidden=4096,
        n_layers=32, n_heads=32, n_kv_heads=8, ffn=14336, max_positions=8192,
        norm_eps=1e-5, tie_embeddings=False, rope_theta=500000.0,
        bos_token_id=128000, eos_token_id=128001),
    "llama-test": ModelConfig(
        name="llama-test", arch="llama", vocab_size=1000, hidden=256,
        n_layers=4, n_heads=4, n_kv_heads=2, ffn=512, max_positions=2048,
        norm_eps=1e-5, tie_embeddings=False, rope_theta=10000.0,
        bos_token_id=1, eos_token_id=2),
}


def _timisun(name: str, vocab: int, width: int, layers: Sequence[LayerSpec], eps: float = 1e-5,
             embed_scale: Optional[float] = None) -> ModelConfig:
    layers = tuple(layers)
    check_layers(layers)
    first = layers[0]
    ffn = first.mlp.expert.ff if first.mlp else 0
    return ModelConfig(
        name=name, arch="timisun", vocab_size=vocab, hidden=width, n_layers=len(layers),
        n_heads=first.mixer.heads, n_kv_heads=1, ffn=ffn,
        max_positions=1 << 30,  # no positions anywhere: only the cache bounds a sequence
        norm_eps=eps, tie_embeddings=True, bos_token_id=0, eos_token_id=-1,
        embed_scale=width ** 0.5 if embed_scale is None else embed_scale, layers=layers)


def check_layers(layers: Sequence[LayerSpec]) -> None:
    """Sizes are positive and every shared cache comes from an earlier layer
    that owns one of the same rank."""
    if not layers:
        raise ValueError("a model needs at least one layer")
    for i, l in enumerate(layers):
        m, f = l.mixer, l.mlp
        try:
            m.check()
        except ValueError as e:
            raise ValueError(f"layer {i}: {e}") from None
        if m.kv_from is not None:
            j = m.kv_from
            if not 0 <= j < i or layers[j].mixer.kv_from is not None or layers[j].mixer.kv_rank != m.kv_rank:
                raise ValueError(f"layer {i}: kv_from {j} must name an earlier layer with its own latents of "
                                 f"rank {m.kv_rank}")
        if isinstance(f, MoESpec) and not 1 <= f.top <= f.experts:
            raise ValueError(f"layer {i}: top must be in [1, experts]")
        if isinstance(f, DenseSpec) and f.ff < 1:
            raise ValueError(f"layer {i}: feed-forward width must be positive")
        j = getattr(m, "mix_values", None)
        if j is not None and not (0 <= j <= i and (layers[j].mixer.mix_values, layers[j].mixer.kv_heads, layers[j].mixer.vdim)
                                  == (j, m.kv_heads, m.vdim)):
            raise ValueError(f"layer {i}: cannot mix in the values of layer {j}")


def _timisun_layers(n: int, share: int = 2, experts: int = 16, **kw) -> list:
    """n layers; each group of `share` uses the latents of its first layer."""
    moe = MoESpec(experts, kw.pop("top"), ExpertSpec(kw.pop("ff"), kw.pop("limit", 7.0)),
                  ExpertSpec(kw.pop("shared_ff"), kw.pop("shared_limit", 7.0)))
    return [LayerSpec(LatentAttentionSpec(kv_from=None if i % share == 0 else i - i % share, **kw), moe)
            for i in range(n)]


MODEL_PRESETS.update({
    # Timisun: small test sizes (none a multiple of the GEMM tiles), and two
    # sizes that resemble the layers of models that are served today
    "timisun-test": _timisun("timisun-test", 300, 104, _timisun_layers(
        4, heads=3, dim=24, vdim=40, kv_rank=56, scale=0.25, window=90, experts=6, top=2, ff=48, shared_ff=72,
        limit=1.25, shared_limit=1.75)),
    "timisun-2b": _timisun("timisun-2b", 32000, 2048, _timisun_layers(
        8, heads=16, dim=128, vdim=128, kv_rank=512, scale=128 ** -0.5, window=1024, experts=32, top=4, ff=1024,
        shared_ff=2048)),
    "timisun-8b": _timisun("timisun-8b", 32000, 4096, _timisun_layers(
        6, heads=32, dim=128, vdim=128, kv_rank=256, scale=128 ** -0.5, window=1024, experts=32, top=4, ff=2048,
        shared_ff=4096)),
})

def unroll(layers: Sequence[LayerSpec], start: int, stop: int, times: int, steps: bool = True) -> list:
    """Layers start .. stop - 1 run `times` times in a row, written out; steps:
    every pass begins with a step of its own."""
    if not (0 <= start < stop <= len(layers) and times >= 1):
        raise ValueError(f"loop over layers {start} .. {stop - 1}, {times} times: outside the {len(layers)} layers")
    rep = dataclasses.replace
    out = [rep(l, weights=i) for i, l in enumerate(layers[:start])]
    for t in range(times):
        out += [rep(layers[i], weights=i, enter=t if steps and i == start else None) for i in range(start, stop)]
    return out + [rep(layers[i], weights=i) for i in range(stop, len(layers))]


def _vizalix(name: str, vocab: int, width: int, layers: Sequence[LayerSpec], loop: Optional[Tuple[int, int, int]] = None,
             eps: float = 1e-6) -> ModelConfig:
    check_layers(layers)
    runs = tuple(unroll(layers, *loop) if loop else layers)
    first = layers[0]
    return ModelConfig(
        name=name, arch="vizalix", vocab_size=vocab, hidden=width, n_layers=len(runs), n_heads=first.mixer.heads,
        n_kv_heads=getattr(first.mixer, "kv_heads", 1), ffn=first.mlp.ff if first.mlp else 0,
        max_positions=1 << 20,  # rows of the rotation tables
        norm_eps=eps, tie_embeddings=False, bos_token_id=0, eos_token_id=-1, layers=runs)


def _vizalix_layers(ff: int, delta: dict, attention: dict, ssm: dict, repeat: int = 1) -> list:
    """delta rule, attention, Mamba-2, `repeat` times."""
    mixers = (ChannelDeltaSpec(**delta), AttentionSpec(**attention), SSMSpec(**ssm))
    return [LayerSpec(m, DenseSpec(ff)) for m in mixers * repeat]


_VIZALIX_ROPE = RopeSpec(64, 500000.0, RopeScaling(8.0, 1.0, 4.0, 8192))
MODEL_PRESETS.update({
    # Vizalix: small test sizes (none a multiple of the GEMM tiles), and two
    # sizes that resemble the layers of models that are served today
    "vizalix-test": _vizalix("vizalix-test", 300, 104, _vizalix_layers(
        72, dict(heads=4, kv_heads=2, dim=24, vdim=20, conv=3, decay_rank=10, gate_rank=6),
        dict(heads=6, kv_heads=3, dim=40, vdim=24, scale=0.2, window=90, softcap=20.0,
             rope=RopeSpec(24, 10000.0, RopeScaling(4.0, 1.0, 4.0, 256))),
        dict(heads=6, vdim=20, state=24, groups=2, norm_groups=2, conv=4)), loop=(0, 2, 2)),
    "vizalix-2b": _vizalix("vizalix-2b", 32000, 2048, _vizalix_layers(
        5632, dict(heads=16, kv_heads=16, dim=128, vdim=128, conv=4, decay_rank=128, gate_rank=128),
        dict(heads=16, kv_heads=4, dim=128, vdim=128, scale=128 ** -0.5, window=1024, softcap=50.0, rope=_VIZALIX_ROPE),
        dict(heads=64, vdim=64, state=128, groups=1, norm_groups=1, conv=4), repeat=2), loop=(0, 3, 2)),
    "vizalix-8b": _vizalix("vizalix-8b", 32000, 4096, _vizalix_layers(
        14336, dict(heads=32, kv_heads=32, dim=128, vdim=128, conv=4, decay_rank=128, gate_rank=128),
        dict(heads=32, kv_heads=8, dim=128, vdim=128, scale=128 ** -0.5, window=1024, softcap=50.0, rope=_VIZALIX_ROPE),
        dict(heads=128, vdim=64, state=128, groups=8, norm_groups=8, conv=4)), loop=(0, 3, 2)),
})


def _kedasun(name: str, vocab: int, width: int, layers: Sequence[LayerSpec], groups: int, eps: float = 1e-6,
             embed_scale: float = 1.0) -> ModelConfig:
    """The first attention layer with mix_values set is the one whose values the others mix in."""
    rep = dataclasses.replace
    first = next((i for i, l in enumerate(layers) if l.mixer.mix_values is not None), None)
    layers = tuple(l if l.mixer.mix_values is None else rep(l, mixer=rep(l.mixer, mix_values=first)) for l in layers)
    check_layers(layers)
    if groups < 1 or width % groups:
        raise ValueError(f"width {width} does not divide into {groups} norm groups")
    m, f = layers[0].mixer, layers[0].mlp
    return ModelConfig(
        name=name, arch="kedasun", vocab_size=vocab, hidden=width, n_layers=len(layers), n_heads=m.heads,
        n_kv_heads=m.kv_heads, ffn=f.ff if f else 0, max_positions=1 << 20,  # rows of the rotation tables
        norm_eps=eps, tie_embeddings=False, bos_token_id=0, eos_token_id=-1, embed_scale=embed_scale, layers=layers,
        norm_groups=groups)


def _kedasun_full(rot: Tuple[int, float], v_mix: bool = True, **sizes) -> AttentionSpec:
    return AttentionSpec(rope=RopeSpec(*rot, interleaved=True) if rot[0] else None, talking=False,
                         mix_values=0 if v_mix else None, **sizes)


def _kedasun_window(v_mix: bool = True, **sizes) -> AttentionSpec:
    return AttentionSpec(talk_weights=True, distance_bias=True, qk_norm=True, bias=True, head_gate=True,
                         mix_values=0 if v_mix else None, **sizes)


def _kedasun_layers(ff: int, limit: float, rot: Tuple[int, float], window: dict, repeat: int, **sizes) -> list:
    """A windowed layer and two full ones, `repeat` times."""
    f = DenseSpec(ff, limit)
    return [LayerSpec(m, f) for m in [_kedasun_window(**window, **sizes)] + [_kedasun_full(rot, **sizes)] * 2] * repeat


MODEL_PRESETS.update({
    # Kedasun: small test sizes (none a multiple of the GEMM tiles), and two
    # sizes that resemble the layers of models that are served today
    "kedasun-test": _kedasun("kedasun-test", 300, 104, _kedasun_layers(
        72, 1.5, (24, 10000.0), dict(window=90, keep_first=3, conv=3), 1, heads=6, kv_heads=3, dim=40, vdim=24,
        scale=0.2), groups=2, embed_scale=0.6),
    "kedasun-2b": _kedasun("kedasun-2b", 32000, 2048, _kedasun_layers(
        5632, 7.0, (64, 500000.0), dict(window=1024, keep_first=4, conv=4), 4, heads=16, kv_heads=4, dim=128, vdim=128,
        scale=128 ** -0.5), groups=4),
    "kedasun-8b": _kedasun("kedasun-8b", 32000, 4096, _kedasun_layers(
        14336, 7.0, (64, 500000.0), dict(window=1024, keep_first=4, conv=4), 2, heads=32, kv_heads=8, dim=128, vdim=128,
        scale=128 ** -0.5), groups=4),
})


def _fagunex(name: str, vocab: int, width: int, layers: Sequence[LayerSpec], loop: Optional[Tuple[int, int, int]] = None,
             side: int = 0, eps: float = 1e-6) -> ModelConfig:
    check_layers(layers)
    if side < 0:
        raise ValueError("the token-side rows need a positive width")
    layers = tuple(unroll(layers, *loop, steps=False) if loop else layers)
    m, f = layers[0].mixer, layers[0].mlp
    return ModelConfig(
        name=name, arch="fagunex", vocab_size=vocab, hidden=width, n_layers=len(layers), n_heads=m.heads, n_kv_heads=1,
        ffn=f.expert.ff if f else 0, max_positions=1 << 20,  # rows of the rotation tables
        norm_eps=eps, tie_embeddings=False, bos_token_id=0, eos_token_id=-1, layers=layers, token_shift=True,
        token_side=side)


def _fagunex_moe(experts: int, top: int, ff: int, shared_ff: Optional[int]) -> MoESpec:
    return MoESpec(experts, top, ExpertSpec(ff), ExpertSpec(shared_ff) if shared_ff else None, softmax=True,
                   shared_gate=bool(shared_ff))


def _fagunex_windowed(rot: Tuple[int, float], **sizes) -> LatentAttentionSpec:
    """The kind with a query latent, a sliding window, a sink and an output gate."""
    return LatentAttentionSpec(rope=RopeSpec(*rot, interleaved=True), sink=True, gate=True, **sizes)


def _fagunex_full(rot: Tuple[int, float], **sizes) -> LatentAttentionSpec:
    return LatentAttentionSpec(rope=RopeSpec(*rot), **sizes)


def _fagunex_layers(moe: MoESpec, attention: dict, windowed: dict, forget: dict) -> list:
    """Full attention, recurrence, windowed attention, recurrence."""
    r = ForgetSpec(**forget)
    mixers = (_fagunex_full(**attention), r, _fagunex_windowed(**attention, **windowed), r)
    return [LayerSpec(m, moe) for m in mixers]


MODEL_PRESETS.update({
    # Fagunex: small test sizes (none a multiple of the GEMM tiles), and two
    # sizes that resemble the layers of models that are served today
    "fagunex-test": _fagunex("fagunex-test", 300, 104, _fagunex_layers(
        _fagunex_moe(6, 2, 48, 72), dict(heads=3, dim=24, vdim=40, kv_rank=56, scale=0.2, rot=(12, 10000.0)),
        dict(q_rank=44, window=90), dict(heads=4, dim=20, vdim=28)), loop=(0, 2, 2), side=20),
    "fagunex-2b": _fagunex("fagunex-2b", 32000, 2048, _fagunex_layers(
        _fagunex_moe(32, 4, 1024, 2048), dict(heads=16, dim=128, vdim=128, kv_rank=512, scale=192 ** -0.5, rot=(64, 500000.0)),
        dict(q_rank=1024, window=1024), dict(heads=16, dim=128, vdim=128)), loop=(0, 4, 2), side=256),
    "fagunex-8b": _fagunex("fagunex-8b", 32000, 4096, _fagunex_layers(
        _fagunex_moe(32, 4, 2048, 4096), dict(heads=32, dim=128, vdim=128, kv_rank=256, scale=192 ** -0.5, rot=(64, 500000.0)),
        dict(q_rank=1536, window=1024), dict(heads=32, dim=128, vdim=128)), loop=(1, 3, 2), side=256),
})

_ALIASES = {
    "sshleifer/tiny-gpt2": "tiny-gpt2",
    "openai-community/gpt2": "gpt2",
    "gpt2-small": "gpt2",
    "openai-community/gpt2-medium": "gpt2-medium",
    "openai-community/gpt2-large": "gpt2-large",
    "openai-community/gpt2-xl": "gpt2-xl",
    "meta-llama/Meta-Llama-3-8B": "llama-3-8b",
    "meta-llama/Llama-3.1-8B": "llama-3-8b",
    "llama3-8b": "llama-3-8b",
}


def get_model_config(model_id: str) -> ModelConfig:
    """Resolve a preset name or HF-style id to a ModelConfig."""
    key = _ALIASES.get(model_id, model_id)
    if key in MODEL_PRESETS:
        return MODEL_PRESETS[key]
    # A local HF directory with a config.json: read the dims from it.
    cfg_path = os.path.join(model_id, "config.json")
    if os.path.isfile(cfg_path):
        return model_config_from_hf_json(cfg_path)
    raise KeyError(f"unknown model {model_id!r}; presets: {sorted(MODEL_PRESETS)}")


def _timisun_from_json(c: dict, name: str) -> ModelConfig:
    """The design's own config.json: every size and constant per layer."""
    layers = []
    for i, l in enumerate(c["layers"]):
        if l["type"] != "latent_attention":
            raise ValueError(f"layer {i}: unknown mixer {l['type']!r}")
        m, f = l["mixer"], l.get("mlp")
        mask = m.get("mask") or {}
        moe = None
        if f:
            if f.get("kind", "moe") != "moe":
                raise ValueError(f"layer {i}: unknown feed-forward {f['kind']!r}")
            sh = f.get("shared")
            moe = MoESpec(f["router"]["experts"], f["router"]["top"],
                          ExpertSpec(f["expert"]["ff"], float(f["expert"]["limit"])),
                          ExpertSpec(sh["ff"], float(sh["limit"])) if sh else None)
        layers.append(LayerSpec(LatentAttentionSpec(
            heads=m["heads"], dim=m["dim"], vdim=m["vdim"], kv_rank=m["kv_rank"], scale=float(m["scale"]),
            window=mask.get("size"), kv_from=m.get("kv_from")), moe))
    return _timisun(name, c["vocab"], c["width"], layers, eps=float(c["norm"]["eps"]),
                    embed_scale=float(c["embedding"]["scale"]))


def _vizalix_from_json(c: dict, name: str, shape) -> ModelConfig:
    """The design's own config.json; `shape(tensor name)` gives the two sizes
    that only the checkpoint's tensors have (ranks of the delta rule's decay
    and gate projections)."""
    layers = []
    for i, l in enumerate(c["layers"]):
        m, f = l["mixer"], l.get("mlp")
        if l["type"] == "channel_delta":
            mix = ChannelDeltaSpec(
                heads=m["heads"], kv_heads=m["kv_heads"], dim=m["dim"], vdim=m["vdim"], conv=m["conv"],
                decay_rank=shape(f"l{i}.mix.a1")[0], gate_rank=shape(f"l{i}.mix.g1")[0])
        elif l["type"] == "attention":
            r = m.get("rot") or {}
            s = r.get("scaling")
            rope = RopeSpec(r["dims"], float(r["base"]), RopeScaling(
                float(s["factor"]), float(s["low"]), float(s["high"]), float(s["original"])) if s else None) if r else None
            cap = m.get("softcap")
            mix = AttentionSpec(
                heads=m["heads"], kv_heads=m["kv_heads"], dim=m["dim"], vdim=m["vdim"], scale=float(m["scale"]),
                window=(m.get("mask") or {}).get("size"), rope=rope, softcap=float(cap) if cap else None)
        elif l["type"] == "mamba2":
            mix = SSMSpec(heads=m["heads"], vdim=m["vdim"], state=m["state"], groups=m["groups"],
                          norm_groups=m["norm_groups"], conv=m["conv"])
        else:
            raise ValueError(f"layer {i}: unknown mixer {l['type']!r}")
        if f and f.get("kind", "dense") != "dense":
            raise ValueError(f"layer {i}: unknown feed-forward {f['kind']!r}")
        layers.append(LayerSpec(mix, DenseSpec(f["ff"]) if f else None))
    lp = c.get("loop")
    return _vizalix(name, c["vocab"], c["width"], layers, loop=(lp["start"], lp["stop"], lp["times"]) if lp else None,
                    eps=float(c["norm"]["eps"]))


def _kedasun_from_json(c: dict, name: str) -> ModelConfig:
    """The design's own config.json."""
    layers = []
    for i, l in enumerate(c["layers"]):
        m, f = l["mixer"], l.get("mlp")
        sizes = dict(heads=m["heads"], kv_heads=m["kv_heads"], dim=m["dim"], vdim=m["vdim"], scale=float(m["scale"]),
                     v_mix=bool(m.get("v_mix")))
        if l["type"] == "attention":
            r = m.get("rot") or {"dims": 0, "base": 1.0}
            mix = _kedasun_full((r["dims"], float(r["base"])), **sizes)
        elif l["type"] == "attention_2":
            mask = m.get("mask") or {}
            mix = _kedasun_window(window=mask.get("size"), keep_first=mask.get("keep_first") or 0, conv=m.get("conv") or 0,
                                  **sizes)
        else:
            raise ValueError(f"layer {i}: unknown mixer {l['type']!r}")
        if f and f.get("kind", "dense") != "dense":
            raise ValueError(f"layer {i}: unknown feed-forward {f['kind']!r}")
        layers.append(LayerSpec(mix, DenseSpec(f["ff"], float(f["limit"])) if f else None))
    return _kedasun(name, c["vocab"], c["width"], layers, groups=c["norm"]["groups"], eps=float(c["norm"]["eps"]),
                    embed_scale=float(c["embedding"]["scale"]))


def _fagunex_from_json(c: dict, name: str) -> ModelConfig:
    """The design's own config.json."""
    layers = []
    for i, l in enumerate(c["layers"]):
        m, f = l["mixer"], l.get("mlp")
        if l["type"] == "hgrn2":
            mix: MixerSpec = ForgetSpec(heads=m["heads"], dim=m["dim"], vdim=m["vdim"])
        elif l["type"] in ("latent_attention", "latent_attention_2"):
            sizes = dict(heads=m["heads"], dim=m["dim"], vdim=m["vdim"], kv_rank=m["kv_rank"], scale=float(m["scale"]),
                         rot=(m["rot_dim"], float(m["rot"]["base"])))
            if m["rot"].get("dims", m["rot_dim"]) != m["rot_dim"]:
                raise ValueError(f"layer {i}: the whole rotated part turns")
            mix = (_fagunex_full(**sizes) if l["type"] == "latent_attention_2" else
                   _fagunex_windowed(q_rank=m["q_rank"], window=(m.get("mask") or {}).get("size"), **sizes))
        else:
            raise ValueError(f"layer {i}: unknown mixer {l['type']!r}")
        moe = None
        if f:
            if f.get("kind", "moe") != "moe":
                raise ValueError(f"layer {i}: unknown feed-forward {f['kind']!r}")
            moe = _fagunex_moe(f["router"]["experts"], f["router"]["top"], f["expert"]["ff"],
                               (f.get("shared") or {}).get("ff"))
        layers.append(LayerSpec(mix, moe))
    lp = c.get("loop")
    return _fagunex(name, c["vocab"], c["width"], layers, loop=(lp["start"], lp["stop"], lp["times"]) if lp else None,
                    side=(c.get("token_side") or {}).get("dim") or 0, eps=float(c["norm"]["eps"]))


def _checkpoint_shapes(folder: str):
    """name -> shape of the tensors in a folder's safetensors files (headers only)."""
    import json

    shapes = {}
    for fn in sorted(os.listdir(folder)):
        if fn.endswith(".safetensors"):
            with open(os.path.join(folder, fn), "rb") as f:
                n = int.from_bytes(f.read(8), "little")
                shapes.update((k, tuple(v["shape"])) for k, v in json.loads(f.read(n)).items() if "shape" in v)

    def shape(name: str) -> tuple:
        if name not in shapes:
            raise ValueError(f"{folder}: no tensor {name!r} beside config.json to read a size from")
        return shapes[name]
    return shape


def model_config_from_hf_json(path: str) -> ModelConfig:
    import json

    with open(path) as f:
        c = json.load(f)
    if c.get("architecture") == "Vizalix":
        folder = os.path.dirname(os.path.abspath(path))
        return _vizalix_from_json(c, os.path.basename(folder) or "vizalix", _checkpoint_shapes(folder))
    own = {"Timisun": _timisun_from_json, "Kedasun": _kedasun_from_json, "Fagunex": _fagunex_from_json}.get(
        c.get("architecture"))
    if own is not None:
        return own(c, os.path.basename(os.path.dirname(os.path.abspath(path))) or c["architecture"].lower())
    mt = c.get("model_type", "gpt2")
    if mt == "gpt2":
        h = c["n_embd"]
        return ModelConfig(
            name=os.path.basename(os.path.dirname(path)) or "gpt2", arch="gpt2",
            vocab_size=c["vocab_size"], hidden=h, n_layers=c["n_layer"],
            n_heads=c["n_head"], n_kv_heads=c["n_head"],
            ffn=c.get("n_inner") or 4 * h, max_positions=c["n_positions"],
            norm_eps=c.get("layer_norm_epsilon", 1e-5), tie_embeddings=True,
            bos_token_id=c.get("bos_token_id", 50256),
            eos_token_id=c.get("eos_token_id", 50256))
    if mt == "llama":
        eos = c.get("eos_token_id", 2)
        if isinstance(eos, list):
            eos = eos[0]
        return ModelConfig(
            name=os.path.basename(os.path.dirname(path)) or "llama", arch="llama",
            vocab_size=c["vocab_size"], hidden=c["hidden_size"],
            n_layers=c["num_hidden_layers"], n_heads=c["num_attention_heads"],
            n_kv_heads=c.get("num_key_value_heads", c["num_attention_heads"]),
            ffn=c["intermediate_size"], max_positions=c.get("max_position_embeddings", 8192),
            norm_eps=c.get("rms_norm_eps", 1e-5),
            tie_embeddings=c.get("tie_word_embeddings", False),
            rope_theta=c.get("rope_theta", 10000.0),
            bos_token_id=c.get("bos_token_id", 1), eos_token_id=eos)
    raise ValueError(f"unsupported model_type {mt!r} in {path}")


# ---------------------------------------------------------------------------
# Sampling
# ---------------------------------------------------------------------------

@dataclass
class SamplingParams:
    """Per-request sampling.  Defaults reproduce `server.py:187-205`."""

    temperature: float = 0.6
    top_k: int = 40
    greedy: bool = False
    seed: Optional[int] = None
    max_new_tokens: int = 20
    stop_at_eos: bool = False  # reference never stops early (quirk Q10)

    def validate(self) -> None:
        if self.max_new_tokens < 0:
            raise ValueError("max_new_tokens must be >= 0")
        if not self.greedy:
            if self.temperature <= 0:
                raise ValueError("temperature must be > 0 (use greedy=True for argmax)")
            if not (1 <= self.top_k <= 1024):
                raise ValueError("top_k must be in [1, 1024]")


# ---------------------------------------------------------------------------
# Engine config
# ---------------------------------------------------------------------------

def _env(name: str, default: str) -> str:
    return os.environ.get(name, default)


@dataclass
class EngineConfig:
    model_id: str = "sshleifer/tiny-gpt2"
    # Pipeline: number of stages (= GPUs, one rank per GPU) and the layer split.
    num_stages: int = 1
    # Data parallelism over whole pipelines: world = num_stages x dp_replicas
    # ranks; replica r owns ranks [r*P, (r+1)*P).  Requests are spread over
    # the replicas (SURVEY.md §2.2 "DP -- request-level replicas").
    dp_replicas: int = 1
    # Explicit split points (len num_stages-1), e.g. SPLIT_AT=2 -> [2].  None = cost model.
    split_points: Optional[Sequence[int]] = None
    # Explicit split points in half-layer units: a stage starts at unit u, where
    # u = 2i is layer i's attention half and u = 2i + 1 its MLP half, e.g.
    # [13] cuts layer 6 between attention and MLP.
    split_units: Optional[Sequence[int]] = None
    # Auto partition may cut between a layer's attention and MLP halves
    # (finer balance of the last stage's lm_head + sampler).
    half_layer_split: bool = True
    dtype: str = "bf16"  # compute / storage dtype on GPU; CPU golden runs in fp32
    device: str = "auto"  # "auto" -> cuda if available else cpu
    max_batch: int = 64  # max concurrent sequences (KV slots)
    max_seq_len: int = 1024
    num_microbatches: int = 0  # 0 -> num_stages (1 when single stage)
    use_graphs: bool = True  # hipGraph-capture decode steps
    seed: int = 0
    weights: Optional[str] = None  # safetensors / HF dir; None -> random init
    sampling: SamplingParams = field(default_factory=SamplingParams)
    # Compat roles (reference server.py:21): "coordinator" | "a" | "b" | "engine".
    role: str = "coordinator"
    shard_a_service: str = "llm-shard-a"
    shard_b_service: str = "llm-shard-b"
    shard_port: int = 5000
    # auto | nccl | rccl | gloo | local | http | loopback (P stage threads on
    # one GPU, device-async event hand-off) | devloop (P stage threads on one
    # GPU joined by device loopback channels with graph-captured transfers:
    # the single-GPU rehearsal of the rccl data plane) | strict (host queues
    # per (edge, lane) with receive-size checks: CPU protocol tests)
    transport: str = "auto"
    # Boundary hidden states on the wire: "fp32" (the residual stream as is:
    # bit-identical to one stage) or "bf16" (half the bytes per hop; the
    # stream is rounded to bf16 at each stage boundary).  The reference ships
    # them as JSON floats (server.py:140,148).
    wire_dtype: str = "fp32"
    # Serving (runtime/scheduler.py): concurrent /generate requests arriving
    # within batch_window_ms share one pipeline round; a round running longer
    # than round_timeout_s marks the engine unhealthy; an HTTP request waits at
    # most request_timeout_s.
    batch_window_ms: float = 2.0
    # Chunked prefill: prompts are prefilled in steps of at most this many
    # tokens per sequence (0 = whole prompt in one step).  Bounds prefill
    # activation memory for long contexts and lets chunks of different
    # microbatches pipeline across stages.
    prefill_chunk: int = 0
    round_timeout_s: float = 600.0
    request_timeout_s: float = 900.0
    # Prefill tokens per microbatch group per step when requests join a
    # running batch (0 = unlimited: every waiting prompt joins at once).
    prefill_budget: int = 0
    # Join policy (runtime/sched_core.h set_join_policy): a running group
    # admits waiting requests only when it has room for all of them or for
    # join_min of them, when idle, or after deferring join_max_wait steps --
    # larger, rarer prefill items (1: admit whatever fits at every step).  Closed-loop serving, 512
    # in flight (profiles/r6_join_policy.log), 1 -> 32 / 4: GPT-2 XL 37.4-38.2k
    # -> 41.4k tok/s, GPT-2 small 156-164k -> 209k, Llama-3 8B 20.1k -> 21.6k,
    # TTFT p50 lower, p90 unchanged.
    join_min: int = 32
    join_max_wait: int = 4
    # One stage: a step's prefill items of groups that all only join
    # sequences run as one forward (parallel/pipeline.py _merged_prefill).
    # Off for references that must match a multi-stage pipeline bit for bit
    # (other GEMM row counts round differently).
    merge_prefill: bool = True
    # Paged caches (ModelConfig.paged_cache): tokens the page pool holds over
    # all live sequences (0: max_batch x max_seq_len, capped by the HBM budget)
    kv_tokens: int = 0
    # Fraction of the HBM left after the weights that the KV cache may use.
    kv_fraction: float = 0.85
    # Serving: record per-stage busy / bubble timing on one pipeline session
    # in this many (0 = never) -- it costs a control-plane gather per session.
    metrics_every: int = 16

    @property
    def model(self) -> ModelConfig:
        return get_model_config(self.model_id)

    @classmethod
    def from_env(cls, **overrides) -> "EngineConfig":
        """Build from the reference's env vars (server.py:20-25) plus extras."""
        split = _env("SPLIT_AT", "")
        cfg = cls(
            model_id=_env("MODEL_ID", "sshleifer/tiny-gpt2"),
            role=_env("SHARD_ROLE", "coordinator").lower(),
            split_points=[int(s) for s in split.split(",") if s.strip()] or None,
            shard_a_service=_env("SHARD_A_SERVICE", "llm-shard-a"),
            shard_b_service=_env("SHARD_B_SERVICE", "llm-shard-b"),
            shard_port=int(_env("SHARD_PORT", "5000")),
            num_stages=int(_env("NUM_STAGES", "0") or 0) or 1,
            max_batch=int(_env("MAX_BATCH", "64")),
            max_seq_len=int(_env("MAX_SEQ_LEN", "1024")),
            dtype=_env("DTYPE", "bf16"),
            weights=os.environ.get("WEIGHTS") or None,
            transport=_env("TRANSPORT", "auto"),
            wire_dtype=_env("WIRE_DTYPE", "fp32"),
            dp_replicas=int(_env("DP_REPLICAS", "1") or 1),
            batch_window_ms=float(_env("BATCH_WINDOW_MS", "2.0")),
            prefill_chunk=int(_env("PREFILL_CHUNK", "0")),
            round_timeout_s=float(_env("ROUND_TIMEOUT_S", "600")),
            request_timeout_s=float(_env("REQUEST_TIMEOUT_S", "900")),
            prefill_budget=int(_env("PREFILL_BUDGET", "0")),
            join_min=int(_env("JOIN_MIN", "32")),
            join_max_wait=int(_env("JOIN_MAX_WAIT", "4")),
            kv_tokens=int(_env("KV_TOKENS", "0")),
            kv_fraction=float(_env("KV_FRACTION", "0.85")),
            metrics_every=int(_env("METRICS_EVERY", "16")),
        )
        if cfg.split_points and cfg.num_stages == 1:
            cfg.num_stages = len(cfg.split_points) + 1
        for k, v in overrides.items():
            if not hasattr(cfg, k):
                raise AttributeError(f"EngineConfig has no field {k!r}")
            setattr(cfg, k, v)
        return cfg

    def replace(self, **kw) -> "EngineConfig":
        return dataclasses.replace(self, **kw)

    @property
    def microbatches(self) -> int:
        return self.num_microbatches or self.num_stages
