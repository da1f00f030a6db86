"""Per-layer descriptions for models whose layers are not all alike.

A ``HybridSpec`` is a ``ModelSpec`` with an explicit list of layers, each one
mixer (windowed differential attention, windowed latent attention, windowed
softmax attention with kept first tokens, chunked sigmoid attention, gated
linear attention, matrix LSTM, lightning attention) and an optional
feed-forward (dense, or a mixture of experts).  Every size and constant of a
layer part is a field here; the layer classes in ``hyperspot.models.mixers``
read nothing else.

``cache_layout`` tells the cache manager what a layer keeps per sequence:
pages that grow with the tokens (``PagedKV``, ``LatentPages``), a fixed-size
recurrent state (``StateSlots``), the last inputs of a convolution
(``ConvTail``), or nothing of its own (``SharedCache``), all already divided
over the tensor-parallel ranks.
"""

from __future__ import annotations

from dataclasses import dataclass, field, replace
from typing import List, Optional, Tuple, Union

from .config import ModelSpec
from .rotary import Stretch, Yarn

# a window that holds every position
UNBOUNDED = 1 << 30


# ------------------------------------------------------------- cache layout

@dataclass(frozen=True)
class PagedKV:
    """Paged keys [NB, G, BS, k_dim] and values [NB, G, BS, v_dim]
    (or [NB, G, v_dim, BS] when the kernels want V pages transposed)."""

    kv_heads: int
    k_dim: int
    v_dim: int
    v_transposed: bool = False

    def bytes_per_token(self, elem: int) -> int:
        return self.kv_heads * (self.k_dim + self.v_dim) * elem


@dataclass(frozen=True)
class LatentPages:
    """Pages [NB, BS, width] of one row per token that all heads share (every
    tensor-parallel rank keeps the whole row)."""

    width: int

    def bytes_per_token(self, elem: int) -> int:
        return self.width * elem


@dataclass(frozen=True)
class SharedCache:
    """The layer reads the cache of an earlier layer and keeps nothing."""

    layer: int

    def bytes_per_token(self, elem: int) -> int:
        return 0


@dataclass(frozen=True)
class StateSlots:
    """One float matrix [heads, dim, vdim] per sequence; `normalizer` adds a
    [heads, dim] vector and a [heads] running maximum."""

    heads: int
    dim: int
    vdim: int
    normalizer: bool = False

    def bytes_per_slot(self, elem: int = 4) -> int:
        n = self.heads * self.dim * self.vdim
        if self.normalizer:
            n += self.heads * (self.dim + 1)
        return 4 * n


@dataclass(frozen=True)
class ConvTail:
    """The last `rows` inputs of a convolution over time per sequence, in the
    model's element type (every tensor-parallel rank keeps all channels)."""

    rows: int
    width: int

    def bytes_per_slot(self, elem: int) -> int:
        return elem * self.rows * self.width


@dataclass(frozen=True)
class MixerAndTails:
    """What a layer with input convolutions keeps: its mixer's part and one
    tail per sublayer."""

    mixer: Union[PagedKV, LatentPages, SharedCache, StateSlots]
    tails: Tuple[ConvTail, ...]


def cache_parts(layout: list) -> list:
    """The single parts of a layout."""
    out = []
    for c in layout:
        out += [c.mixer, *c.tails] if isinstance(c, MixerAndTails) else [c]
    return out


# ------------------------------------------------------------------- mixers

@dataclass(frozen=True)
class DiffAttention:
    """Sliding-window differential attention: two softmax maps per head."""

    heads: int
    kv_heads: int
    dim: int            # per map
    vdim: int
    scale: float
    window: int
    rot_dims: int
    rot_base: float
    diff: float

    def cache(self, tp: int) -> PagedKV:
        return PagedKV(self.kv_heads // tp, 2 * self.dim, self.vdim,
                       v_transposed=True)

    def params(self, width: int) -> int:
        return (width * self.dim * 2 * (self.heads + self.kv_heads)
                + width * self.vdim * (self.heads + self.kv_heads)
                + 4 * self.dim)

    def check(self) -> None:
        if self.heads % self.kv_heads:
            raise ValueError("attention: heads must be a multiple of kv_heads")
        if self.rot_dims % 2 or not 0 <= self.rot_dims <= self.dim:
            raise ValueError("attention: rotary dims must be even and <= dim")
        if self.window < 1:
            raise ValueError("attention: window must be at least 1")


@dataclass(frozen=True)
class GatedLinear:
    """Gated linear attention with a low-rank decay per key channel."""

    heads: int
    dim: int
    vdim: int
    tau: float
    rank: int           # inner size of the decay projection

    def cache(self, tp: int) -> StateSlots:
        return StateSlots(self.heads // tp, self.dim, self.vdim)

    def params(self, width: int) -> int:
        d, e = self.heads * self.dim, self.heads * self.vdim
        return (width * (2 * d + 3 * e + self.rank)
                + d * (self.rank + 1) + self.vdim)

    def check(self) -> None:
        if self.tau == 0:
            raise ValueError("gla: tau must not be zero")


@dataclass(frozen=True)
class MatrixLSTM:
    """Matrix-memory LSTM with capped exponential gates."""

    heads: int
    dim: int
    vdim: int
    gate_cap: float

    def cache(self, tp: int) -> StateSlots:
        return StateSlots(self.heads // tp, self.dim, self.vdim,
                          normalizer=True)

    def params(self, width: int) -> int:
        d, e = self.heads * self.dim, self.heads * self.vdim
        return width * (2 * d + 3 * e) + 2 * self.heads * (width + 1) + e

    def check(self) -> None:
        if self.gate_cap == 0:
            raise ValueError("mlstm: gate_cap must not be zero")


@dataclass(frozen=True)
class LatentAttention:
    """Sliding-window attention whose keys and values are expanded per head
    from one latent per token; a rotated key part is shared by all heads.
    With `kv_from` the latents are those of an earlier layer.  `halves`: a
    checkpoint's rotated pairs lie half the rotated size apart; `sink`: every
    head's softmax has a learned score without a value in its denominator;
    `gate`: a sigmoid of the input scales every head's output."""

    heads: int
    dim: int            # unrotated query/key size per head
    rot_dim: int        # rotated query/key size
    vdim: int
    kv_rank: int
    scale: float
    window: int
    rot_base: float
    kv_from: Optional[int] = None
    stretch: Stretch = 1.0
    halves: bool = False
    sink: bool = False
    gate: bool = False

    def cache(self, tp: int) -> Union[LatentPages, SharedCache]:
        if self.kv_from is not None:
            return SharedCache(self.kv_from)
        return LatentPages(self.kv_rank + self.rot_dim)

    def params(self, width: int) -> int:
        n = (width * self.heads * (self.dim + self.rot_dim + self.vdim)
             + self.kv_rank * self.heads * (self.dim + self.vdim))
        if self.kv_from is None:
            n += width * (self.kv_rank + self.rot_dim) + self.kv_rank
        return n + self.heads * (self.sink + width * self.gate)

    def check(self) -> None:
        if self.rot_dim % 2:
            raise ValueError("latent attention: rotary size must be even")
        if self.window < 1:
            raise ValueError("latent attention: window must be at least 1")
        check_rotation(self.rot_base, self.stretch)


@dataclass(frozen=True)
class Lightning:
    """Linear attention with a constant decay per head, SiLU on queries, keys
    and values, one norm over all heads together and a sigmoid gate."""

    heads: int
    dim: int
    vdim: int
    decay: Tuple[float, ...]

    def cache(self, tp: int) -> StateSlots:
        return StateSlots(self.heads // tp, self.dim, self.vdim)

    def params(self, width: int) -> int:
        d, e = self.heads * self.dim, self.heads * self.vdim
        return width * (2 * d + 3 * e) + e

    def check(self) -> None:
        if len(self.decay) != self.heads:
            raise ValueError("lightning: one decay per head")
        if not all(0.0 <= x <= 1.0 for x in self.decay):
            raise ValueError("lightning: decays must be within [0, 1]")


@dataclass(frozen=True)
class SigmoidAttention:
    """Attention within chunks of `chunk` positions: a key weighs the sigmoid
    of its capped score plus a bias per head, without normalization over keys.
    Queries and keys are normed per head; positions do not enter."""

    heads: int
    kv_heads: int
    dim: int
    vdim: int
    scale: float
    cap: float          # scores are cap * tanh(score / cap)
    chunk: int

    def cache(self, tp: int) -> PagedKV:
        return PagedKV(self.kv_heads // tp, self.dim, self.vdim,
                       v_transposed=True)

    def params(self, width: int) -> int:
        return (width * (self.heads + self.kv_heads) * (self.dim + self.vdim)
                + 2 * self.dim + self.heads)

    def check(self) -> None:
        if self.heads % self.kv_heads:
            raise ValueError("attention: heads must be a multiple of kv_heads")
        if self.chunk < 1:
            raise ValueError("attention: chunks must be at least 1 long")
        if not self.cap > 0:
            raise ValueError("attention: the score cap must be positive")


@dataclass(frozen=True)
class WindowAttention:
    """Grouped-query softmax attention over a sliding window and the first
    `keep_first` tokens of the sequence.

    The first `rot_dims` dimensions of queries and keys are rotated, in pairs
    half that size apart with `halves`; with `qk_norm` every head of both is
    then divided by its root mean square.  With `turn_values` the value of
    position j is turned by j over all its dimensions before it is kept, and
    position i's output back by i.  `sink` is a fixed score without a value in
    the softmax denominator (None: there is none)."""

    heads: int
    kv_heads: int
    dim: int
    vdim: int
    scale: float
    window: int
    rot_dims: int
    rot_base: float
    keep_first: int = 0
    stretch: Stretch = 1.0
    halves: bool = False
    qk_norm: bool = False
    turn_values: bool = False
    sink: Optional[float] = None

    def cache(self, tp: int) -> PagedKV:
        return PagedKV(self.kv_heads // tp, self.dim, self.vdim,
                       v_transposed=True)

    def params(self, width: int) -> int:
        return width * (self.heads + self.kv_heads) * (self.dim + self.vdim)

    def check(self) -> None:
        if self.heads % self.kv_heads:
            raise ValueError("attention: heads must be a multiple of kv_heads")
        if self.rot_dims % 2 or not 0 <= self.rot_dims <= self.dim:
            raise ValueError("attention: rotary dims must be even and <= dim")
        if self.turn_values and self.vdim % 2:
            raise ValueError("attention: turned values must have an even size")
        if self.window < 1 or self.keep_first < 0:
            raise ValueError("attention: window must be at least 1, kept "
                             "tokens at least 0")
        check_rotation(self.rot_base, self.stretch)


def check_rotation(base: float, stretch: Stretch) -> None:
    if base <= 0 or isinstance(stretch, Yarn) and base == 1:
        raise ValueError("rotation: the base must be positive, with YaRN "
                         "other than 1")
    if isinstance(stretch, Yarn):
        stretch.check()
    elif not stretch > 0:
        raise ValueError("rotation: the factor must be positive")


Mixer = Union[DiffAttention, GatedLinear, MatrixLSTM, LatentAttention,
              Lightning, SigmoidAttention, WindowAttention]


# ------------------------------------------------------------- feed-forward

@dataclass(frozen=True)
class SquaredRelu:
    """Dense feed-forward without a gate: down(relu(up x)^2)."""

    ff: int

    def params(self, width: int) -> int:
        return 2 * width * self.ff

    def check(self) -> None:
        pass


@dataclass(frozen=True)
class Experts:
    """Mixture of gated experts.

    `shared` is the size of an expert that every token also passes, weighted
    by a sigmoid gate (None: there is none).  `identity` further outputs of
    the router stand for experts that return their input.  With `limit` an
    expert computes g sigmoid(1.702 g) (u + 1) from g = min(gate, limit) and
    u = up clamped to +-limit; without, silu(gate) * up.  `over_all`: weights
    are the softmax over all router outputs, and a correction is added to it
    for the choice only; otherwise the softmax over the chosen."""

    experts: int
    top: int
    ff: int
    shared: Optional[int] = None
    identity: int = 0
    over_all: bool = False
    limit: Optional[float] = None

    def params(self, width: int) -> int:
        n = width * (self.experts * (1 + 3 * self.ff) + self.identity)
        if self.over_all:
            n += self.experts + self.identity
        if self.shared is not None:
            n += width * (1 + 3 * self.shared)
        return n

    def check(self) -> None:
        if not 1 <= self.top <= self.experts + self.identity:
            raise ValueError("experts: top must be between 1 and the number "
                             "of experts")


@dataclass(frozen=True)
class LayerSpec:
    mixer: Mixer
    # size of a dense gated feed-forward, a description of another kind, or
    # None for no feed-forward
    ff: Union[None, int, SquaredRelu, Experts] = None
    # the layer whose tensors this one uses, with a cache of its own
    weights_of: Optional[int] = None


@dataclass
class HybridSpec(ModelSpec):
    """A decoder made of explicit layers.  ``architecture`` names the design
    in the model registry."""

    architecture: str = ""
    layers: Tuple[LayerSpec, ...] = field(default_factory=tuple)
    norm_params: int = 0          # parameters of one norm
    norms: int = 2                # norms per sublayer
    # mixer and feed-forward read one normed input; both are added at once
    parallel: bool = False
    embed_scale: float = 1.0
    # size of a token's own input to every layer (0: there is none)
    side_dim: int = 0
    # taps of the convolution over time on every sublayer's input (0: none)
    conv_taps: int = 0

    def param_count(self) -> int:
        h = self.hidden_size
        n = self.vocab_size * h * (1 if self.tie_embeddings else 2)
        n += self.norm_params
        sublayer = self.norms * self.norm_params + h * self.conv_taps
        for layer in self.layers:
            if layer.weights_of is not None:
                continue
            n += layer.mixer.params(h) + sublayer
            if layer.ff is not None:
                n += 3 * h * layer.ff if isinstance(layer.ff, int) \
                    else layer.ff.params(h)
                n += 0 if self.parallel else sublayer
            if self.side_dim:
                n += (self.vocab_size + 2 * h) * self.side_dim + h
        return n

    def cache_layout(self, tp: int) -> list:
        if not self.conv_taps:
            return [layer.mixer.cache(tp) for layer in self.layers]
        tail = ConvTail(self.conv_taps - 1, self.hidden_size)
        return [MixerAndTails(layer.mixer.cache(tp),
                              (tail,) * (1 if layer.ff is None else 2))
                for layer in self.layers]

    @property
    def is_hybrid(self) -> bool:
        return True

    @property
    def has_state(self) -> bool:
        return any(isinstance(c, StateSlots)
                   or isinstance(c, ConvTail) and c.rows > 0
                   for c in cache_parts(self.cache_layout(1)))

    @property
    def latent_windows(self) -> List[int]:
        """Distinct windows of the latent-attention layers."""
        return sorted({layer.mixer.window for layer in self.layers
                       if isinstance(layer.mixer, LatentAttention)})


def hybrid_spec(name: str, architecture: str, width: int, vocab: int,
                eps: float, layers, max_position: int = 1 << 20,
                tie_embeddings: bool = True, **kw) -> HybridSpec:
    """Build a checked HybridSpec; `kw` are its own fields.  The per-model
    fields of ModelSpec that only make sense for uniform layers are zero."""
    layers = tuple(layers)
    for i, layer in enumerate(layers):
        layer.mixer.check()
        if layer.ff is not None and not isinstance(layer.ff, int):
            layer.ff.check()
        _check_shared_cache(layers, i)
        _check_shared_weights(layers, i)
    return HybridSpec(
        name=name, hidden_size=width, num_layers=len(layers), num_heads=0,
        num_kv_heads=0, head_dim=0, intermediate_size=0, vocab_size=vocab,
        rms_eps=eps, max_position=max_position,
        tie_embeddings=tie_embeddings, architecture=architecture,
        layers=layers, **kw)


def looped(layers, start: int, stop: int, times: int) -> List[LayerSpec]:
    """Layer runs in which layers start ... stop - 1 come `times` times in a
    row, later passes with the tensors of the first and caches of their
    own."""
    if not 0 <= start <= stop <= len(layers) or times < 1:
        raise ValueError(f"loop: layers {start} ... {stop - 1}, {times} times, "
                         f"of {len(layers)}")
    again = [replace(layers[i], weights_of=i) for i in range(start, stop)]
    return [*layers[:stop], *again * (times - 1), *layers[stop:]]


def _check_shared_cache(layers, i: int) -> None:
    m = layers[i].mixer
    j = getattr(m, "kv_from", None)
    if j is None:
        return
    o = layers[j].mixer if 0 <= j < i else None
    if not isinstance(o, LatentAttention) or o.kv_from is not None:
        raise ValueError(f"layer {i}: kv_from must name an earlier "
                         "latent-attention layer with latents of its own")
    rotated = lambda x: (x.kv_rank, x.rot_dim, x.rot_base, x.stretch, x.halves)
    if rotated(o) != rotated(m):
        raise ValueError(f"layer {i}: latent sizes and rotation differ from "
                         f"layer {j}'s")


def _check_shared_weights(layers, i: int) -> None:
    j = layers[i].weights_of
    if j is None:
        return
    o = layers[j] if 0 <= j < len(layers) else None
    if o is None or o.weights_of is not None:
        raise ValueError(f"layer {i}: weights_of must name a layer with "
                         "tensors of its own")
    if (o.mixer, o.ff) != (layers[i].mixer, layers[i].ff):
        raise ValueError(f"layer {i}: sizes differ from those of layer {j}, "
                         "whose tensors it uses")
