"""Interfaces of the parts a layer is put together from, and their registries.

A part is built from its specification (plain sizes and constants), declares the
tensors it wants by relative name, receives them, and runs on the tokens of one
step.  No part sees a configuration, a layer index or the model it is in.

Five kinds of parts, each with a registry from the specification's ``kind`` to a class:

===================  =====================================================================
``Norm``             ``forward(stream) -> h``: folds the stream's pending branch output
                     into the 32-bit residual and returns the normalised activations.
``PositionEncoding`` ``apply(q, k, positions)``: in place on ``[T, heads, head_dim]`` views.
``Mixer``            ``forward(h, ctx, cache) -> [T, hidden]``: mixes tokens; declares the
                     cache it needs (pages per token and/or a fixed-size state per request).
``FeedForward``      ``forward(h, ctx) -> [T, hidden]``: stateless.
``Block``            ``forward(stream, ctx, cache) -> stream``: arranges the four above.
===================  =====================================================================
"""
from __future__ import annotations

from dataclasses import dataclass
from typing import Callable

import torch

from ..config.base import ConfigError, PartSpec


# ------------------------------------------------------------------ weights of a part

# How a tensor is kept on the GPU, whatever its shape: a dtype policy.
KEEP_COMPUTE = "compute"     # the engine's compute dtype (matrix-product operands)
KEEP_STORED = "stored"       # as stored: bfloat16 stays bfloat16, 32-bit stays 32-bit; a 32-bit engine widens
KEEP_FLOAT32 = "float32"     # always 32-bit, also under a bfloat16 engine (a router, a gate, a decay)
KEEP_INT32 = "int32"         # integer tables
DTYPE_POLICIES = (KEEP_COMPUTE, KEEP_STORED, KEEP_FLOAT32, KEEP_INT32)

# The laws of the random-weights mode: name -> f(shape, generator, device, std) -> float32 (or int32) tensor.
# A part that needs another law (a log-decay, a positive-only scale) adds it here by name and declares it.
INIT_LAWS: dict[str, Callable] = {}


def register_init_law(name: str) -> Callable[[Callable], Callable]:
    def add(fn: Callable) -> Callable:
        INIT_LAWS[name] = fn
        return fn
    return add


@register_init_law("normal")
def _init_normal(shape, gen, device, std):
    return torch.randn(shape, generator=gen, device=device, dtype=torch.float32) * std


@register_init_law("one_plus_normal")
def _init_one_plus_normal(shape, gen, device, std):
    return torch.randn(shape, generator=gen, device=device, dtype=torch.float32) * std + 1.0


@register_init_law("near_identity")
def _init_near_identity(shape, gen, device, std):
    """A square matrix: the identity plus N(0, std)."""
    return torch.eye(shape[0], shape[1], device=device, dtype=torch.float32) + torch.randn(shape, generator=gen, device=device, dtype=torch.float32) * std


@register_init_law("random_table")
def _init_random_table(shape, gen, device, std):
    return torch.randint(0, 2 ** 15, shape, generator=gen, device=device, dtype=torch.int32)


@dataclass(frozen=True)
class WeightSpec:
    """One tensor a part wants from the checkpoint.

    ``keep``: the dtype policy, one of :data:`DTYPE_POLICIES`, independent of the tensor's shape:
    ``compute`` tensors take the engine's compute dtype (matrix-product operands), ``stored``
    tensors keep the dtype they are stored in (bfloat16 stays bfloat16, 32-bit stays 32-bit; a 32-bit
    engine widens them: norm weights, biases), ``float32`` tensors are 32-bit under every engine,
    ``int32`` tensors are integer tables.
    ``init``: the name of a law in :data:`INIT_LAWS` for the random-weights mode (``normal`` =
    N(0, std), ``one_plus_normal`` = 1 + N(0, std), ``random_table`` = integers).
    ``optional``: the checkpoint may leave it out (a tied head).
    ``free_axes``: axes whose size the checkpoint's tensor decides; ``shape`` holds the random-weights mode's size there.
    """
    shape: tuple[int, ...]
    keep: str = KEEP_COMPUTE
    init: str = "normal"
    optional: bool = False
    free_axes: tuple[int, ...] = ()

    def __post_init__(self):
        if self.keep not in DTYPE_POLICIES:
            raise ConfigError(f"a tensor's dtype policy is one of {', '.join(DTYPE_POLICIES)}, not {self.keep!r}")
        if self.init not in INIT_LAWS:
            raise ConfigError(f"no initialisation law {self.init!r}; known: {', '.join(sorted(INIT_LAWS))}")

    @property
    def integer(self) -> bool:
        return self.keep == KEEP_INT32

    def fits(self, shape: tuple[int, ...]) -> bool:
        """Whether a stored tensor of this shape is one the part takes."""
        return len(shape) == len(self.shape) and all(g == w or (i in self.free_axes and g > 0) for i, (g, w) in enumerate(zip(shape, self.shape)))


def join_name(prefix: str, name: str) -> str:
    """``prefix.name``; a part whose one tensor bears the part's own name declares it as ``""``."""
    return f"{prefix}.{name}" if name else prefix


def under(tensors, prefix: str) -> dict:
    """The tensors of the part called ``prefix``, by the names the part declared them with (``""`` for ``prefix`` itself)."""
    out = {k[len(prefix) + 1:]: tensors[k] for k in list(tensors) if k.startswith(prefix + ".")}
    if prefix in tensors:
        out[""] = tensors[prefix]
    return out


def place(t: torch.Tensor, keep: str, dtype: torch.dtype, device) -> torch.Tensor:
    """``t`` on ``device`` in the dtype that the policy ``keep`` gives it under an engine of ``dtype``."""
    if keep not in DTYPE_POLICIES:
        raise ConfigError(f"a tensor's dtype policy is one of {', '.join(DTYPE_POLICIES)}, not {keep!r}")
    if keep == KEEP_COMPUTE:
        return t.to(device=device, dtype=dtype).contiguous()
    if keep == KEEP_INT32:
        return t.to(device=device, dtype=torch.int32).contiguous()
    if keep == KEEP_FLOAT32 or dtype == torch.float32 or t.dtype not in (torch.bfloat16, torch.float32):
        t = t.to(torch.float32)
    return t.to(device).contiguous()


class Part:
    """Common protocol: declare tensors, receive them, say whether a step may be recorded.

    ``graph_safe``: nothing in the part's ``forward`` depends on host-side values of the step (no
    ``.item()``, ``.nonzero()``, shapes that follow the tokens), so a decode step through it can be
    captured once as a HIP graph and replayed.  ``False`` unless a part says otherwise; a model runs
    under graphs only if every part of every block says ``True``.  A subclass that overrides a stage or
    adds a hook that reads host values must set it back to ``False``."""

    graph_safe = False

    def __init__(self, spec: PartSpec, dtype: torch.dtype, device: torch.device):
        self.spec = spec
        self.dtype = dtype
        self.device = device

    def weight_specs(self) -> dict[str, WeightSpec]:
        return {}

    def load_weights(self, tensors: dict[str, torch.Tensor]) -> None:
        """``tensors``: the declared names (those present) -> CPU tensors as stored."""

    def parts(self):
        """This part and every part inside it (a block's four, a mixer's position encoding)."""
        yield self

    # helpers ---------------------------------------------------------------------
    def _place(self, t: torch.Tensor, keep: str) -> torch.Tensor:
        return place(t, keep, self.dtype, self.device)


# ------------------------------------------------------------------------ cache needs

@dataclass(frozen=True)
class PagedNeed:
    """Per-token cache: some planes of ``[heads, width]`` per token, kept for all tokens
    (``window=None``) or for the last ``window`` tokens.  ``planes`` is a count of planes of
    ``[num_heads, head_dim]`` each (keys and values are two), or a tuple of ``(heads, width)``, one per
    plane, for planes that differ (a compressed latent beside a small rotated part).  ``dtype``: the
    planes' element type; ``None`` is the model's.  Layers with equal needs share a group of pages.  ``chunk``: a query reads only
    keys of its own chunk of ``chunk`` positions (counted from position 0), so pages that lie wholly before the chunk of the next
    position are kept no longer.  ``stride``: the planes hold one row for every ``stride`` positions (row ``p // stride``: a summary of a
    block of tokens), so a page of them spans ``stride`` times as many positions.  A mixer that keeps rows at two rates (tokens inside
    a window, summaries of what lies before it) declares two needs, each a group of its own.  ``keep_first``: beside a window, the first
    ``keep_first`` positions of a sequence are read by every later query, so the pages that hold them stay with the request."""
    num_heads: int
    head_dim: int
    window: int | None = None
    planes: int | tuple[tuple[int, int], ...] = 2
    dtype: torch.dtype | None = None
    chunk: int | None = None
    stride: int = 1
    keep_first: int = 0

    @property
    def bounded(self) -> bool:
        """Whether a request keeps only a bounded stretch of its tokens (a window or a chunk)."""
        return self.window is not None or self.chunk is not None

    @property
    def reach(self) -> int | None:
        """Most positions back from a query that it can read, itself included (the smaller of window and chunk)."""
        spans = [s for s in (self.window, self.chunk) if s is not None]
        return min(spans) if spans else None

    @property
    def plane_shapes(self) -> tuple[tuple[int, int], ...]:
        """``(heads, width)`` of every plane."""
        if isinstance(self.planes, int):
            return ((self.num_heads, self.head_dim),) * self.planes
        return tuple((int(h), int(w)) for h, w in self.planes)


@dataclass(frozen=True)
class StateNeed:
    """Fixed-size per-request state: one tensor of ``shape`` per slot, zero when a
    request is admitted."""
    shape: tuple[int, ...]
    dtype: torch.dtype = torch.float32


# --------------------------------------------------------------------------- streams

class Stream:
    """The hidden state between parts: a 32-bit residual ``[T, hidden]`` and the output
    of the last branch that is still to be added to it (``pending``, or ``None``).
    The next norm adds ``pending`` in 32-bit while it normalises, which saves one pass
    over the residual per branch.  ``pending`` is ``[T, hidden]`` in the activation dtype, or
    float32 ``[P, T, hidden]``: P slabs of partial sums that the norm adds up as well.

    Blocks that keep several copies of the residual (hyper-connections) hold them as ``residual [S, T, hidden]``; ``fold`` then says
    how the pending output enters them: ``(mix [S, S], out [S])``, 32-bit tensors on the GPU, for ``x_t <- sum_s mix[s, t] x_s +
    out[t] * pending`` (``None``: ``pending`` is added to every stream as it is).

    Blocks that norm a branch's output before it is added leave that norm on the stream as well: ``post = (weight, eps)`` means that
    ``pending`` enters as ``pending / sqrt(mean(pending^2) + eps) * weight`` (32-bit; ``weight`` one number or ``hidden`` of them).
    ``extra``: a 32-bit ``[T, hidden]`` tensor that the next norm adds to the residual too (an embedding that enters the stream again).
    ``gain``: a factor with which ``pending`` enters.  Only norms that say ``folds_post_norm`` know the three.  A mixer that says ``reads_stream`` may be handed the stream itself: it reads the
    32-bit residual with what is pending on it and leaves the stream settled (nothing pending)."""

    __slots__ = ("residual", "pending", "normed", "fold", "post", "extra", "gain")

    def __init__(self, residual: torch.Tensor, pending: torch.Tensor | None = None):
        self.residual = residual
        self.pending = pending
        self.normed = None      # blocks whose norm follows the sum: the residual in the activation dtype, as the last norm left it
        self.fold = None
        self.post = None
        self.extra = None
        self.gain = 1.0


class LazyNorm:
    """A norm that has not run yet, handed to the part that reads its output: ``norm(residual + pending)`` of
    the stream.  It states which norm it is (``kind``, the norm's registry name) and carries that kind's
    constants (``rmsnorm``: ``weight`` and ``eps``), so that a consumer whose kernel can make a norm of that
    kind itself does so and calls :meth:`done` with the new residual it wrote; a consumer that does not know the
    kind, or whose shapes do not fit, calls :meth:`value`, which runs the norm the usual way (once).  The norm's
    own kernel is a launch and a trip to memory that a step of one token can do without."""

    def __init__(self, norm, stream: "Stream", kind: str, **constants):
        self.norm = norm
        self.stream = stream
        self.kind = kind
        self.constants = constants
        self._value = None

    def rmsnorm(self):
        """``(weight, eps)`` if this is a root-mean-square norm with one weight vector, else ``None``."""
        if self.kind != "rmsnorm":
            return None
        return self.constants["weight"], self.constants["eps"]

    @property
    def residual(self):
        return self.stream.residual

    @property
    def pending(self):
        return self.stream.pending

    def value(self) -> torch.Tensor:
        if self._value is None:
            self._value = self.norm.forward(self.stream)
        return self._value

    def done(self, residual_out: torch.Tensor) -> None:
        self.stream.residual = residual_out
        self.stream.pending = None


# ----------------------------------------------------------------------- part kinds

class Norm(Part):
    def forward(self, stream: Stream, rows: torch.Tensor | None = None, gain: float = 1.0, read: torch.Tensor | None = None) -> torch.Tensor:
        """Add ``stream.pending`` into ``stream.residual`` (both kept up to date) and
        return ``norm(residual) * gain`` in the activation dtype (the factor applied in 32-bit, before
        the one rounding of the result).  With ``rows`` (int32 indices) only those rows are read
        and returned, and the stream is left untouched.  Over several copies of the residual (``residual [S, T, hidden]``) the
        pending output enters through ``stream.fold`` and the norm reads ``sum_s read[s] x_s`` (``read``: 32-bit ``[S]`` on the GPU;
        ``None``: the sum of the streams)."""
        raise NotImplementedError

    def renorm(self, stream: Stream, alpha: float = 1.0) -> torch.Tensor:
        """The norm after the sum: ``stream.residual <- norm(alpha * residual + pending)`` in 32-bit (the pending branch is
        used up), returned in the activation dtype as well, for the next sublayer to read."""
        raise NotImplementedError

    def settle(self, stream: Stream) -> torch.Tensor:
        """Add what is pending (``pending`` with its ``post`` norm, ``extra``) into ``stream.residual`` and return the sum itself, without a norm, in
        the activation dtype.  Offered by norms that say ``folds_post_norm``."""
        raise NotImplementedError

    def lazy(self, stream: Stream) -> "LazyNorm | None":
        """A :class:`LazyNorm` of the stream where a consumer's kernel could make this norm itself (the
        norm says for which steps that is worth offering), else ``None``.  The :class:`LazyNorm` must name
        its kind and carry that kind's constants: consumers fuse only the kinds they know and run every
        other through :meth:`LazyNorm.value`."""
        return None


class PositionEncoding(Part):
    def apply(self, q: torch.Tensor, k: torch.Tensor | None, positions: torch.Tensor) -> None:
        """Encode ``positions [T]`` into ``q [T, heads, head_dim]`` and ``k`` in place
        (views with unit stride on the last axis)."""
        raise NotImplementedError

    def fused_inv_freq(self) -> torch.Tensor | None:
        """A declared capability: an encoding that is the split-half rotary form over the whole head,
        ``angle[j] = float32(position) * inv_freq[j]`` turning the pair ``(j, j + head_dim/2)``, returns its
        float32 ``inv_freq [head_dim/2]`` here, and a mixer may then fold the rotation into its own kernels
        (the projection's epilogue, the cache write) instead of calling :meth:`apply`.  ``None`` (the
        default): the encoding is applied through :meth:`apply` only."""
        return None


class Mixer(Part):
    def paged_need(self) -> "PagedNeed | tuple[PagedNeed, ...] | None":
        """One need, or several (each a group of pages with a block table of its own: ``cache.group`` / ``cache.planes`` are the first
        one's, ``cache.more[i]`` the others')."""
        return None

    def state_need(self) -> StateNeed | None:
        return None

    def forward(self, h: torch.Tensor, ctx, cache) -> torch.Tensor:
        """``h [T, hidden]`` -> ``[T, hidden]``.  ``cache`` is this run's
        :class:`torchlet_amd.cache.manager.LayerCache` (or ``None`` when the mixer
        declared no need)."""
        raise NotImplementedError


class StagedMixer(Mixer):
    """A mixer in three stages, so that it can also stand beside others on one input (``parallel``): an input projection
    ``w_in [in_width, hidden]`` whose result it reads in the activation dtype, ``mix``, which turns that result into ``mix_width``
    numbers per token, and an output projection ``w_o [hidden, mix_width]`` without bias.  A mixer of several such branches
    stacks the ``w_in`` into one product and the ``w_o`` into another."""
    in_width: int = 0
    mix_width: int = 0
    w_in: torch.Tensor | None = None
    w_o: torch.Tensor | None = None
    b_in: torch.Tensor | None = None      # biases of the two projections (a mixer that stands alone may have them; branches of a
    b_o: torch.Tensor | None = None       # mixer that stacks several projections into one may not)

    def mix(self, proj: torch.Tensor, h: torch.Tensor, ctx, cache, out: torch.Tensor, gain: float = 1.0) -> None:
        """``proj [T, in_width]`` (a row-strided view of ``h @ w_in.T``) and ``h`` itself (for what the mixer projects on its own,
        in 32-bit) -> ``out [T, mix_width]`` (a row-strided view), times ``gain``."""
        raise NotImplementedError

    def forward(self, h, ctx, cache):
        from ..kernels import ops
        T = h.shape[0]
        proj = torch.empty((T, self.in_width), dtype=self.dtype, device=h.device)
        ops.linear(h, self.w_in, self.b_in, proj)
        mixed = torch.empty((T, self.mix_width), dtype=self.dtype, device=h.device)
        self.mix(proj, h, ctx, cache, mixed)
        return project_out(mixed, self.w_o, self.dtype, self.b_o)


def project_out(mixed: torch.Tensor, w_o: torch.Tensor, dtype: torch.dtype, bias: torch.Tensor | None = None) -> torch.Tensor:
    """A mixer's output projection ``[T, hidden]``, or (few rows against a narrow matrix, bfloat16, no bias) float32 slabs of partial sums
    ``[P, T, hidden]`` that the next norm adds up."""
    from ..kernels import ops
    T, hidden = mixed.shape[0], w_o.shape[0]
    if bias is None and dtype == torch.bfloat16 and mixed.shape[1] % 64 == 0 and ops.linear_partials_pay(T, hidden, mixed.shape[1]):
        return ops.linear_partials(mixed, w_o)
    out = torch.empty((T, hidden), dtype=dtype, device=mixed.device)
    ops.linear(mixed, w_o, bias, out)
    return out


class FeedForward(Part):
    def forward(self, h: torch.Tensor, ctx) -> torch.Tensor:
        raise NotImplementedError


class Block(Part):
    mixer: Mixer

    def forward(self, stream: Stream, ctx, cache) -> Stream:
        raise NotImplementedError


# ------------------------------------------------------------------------ registries

class Registry:
    """``kind`` -> class, with a decorator to add to it and a clear error on a miss."""

    def __init__(self, what: str):
        self.what = what
        self._classes: dict[str, type] = {}

    def register(self, kind: str) -> Callable[[type], type]:
        def add(cls: type) -> type:
            self._classes[kind] = cls
            return cls
        return add

    def unregister(self, kind: str) -> None:
        self._classes.pop(kind, None)

    def names(self) -> list[str]:
        return sorted(self._classes)

    def build(self, spec: PartSpec, dtype: torch.dtype, device: torch.device):
        cls = self._classes.get(spec.kind)
        if cls is None:
            raise ConfigError(f"no {self.what} of kind {spec.kind!r}; known: {', '.join(self.names())}")
        return cls(spec, dtype, device)


NORMS = Registry("norm")
POSITION_ENCODINGS = Registry("position encoding")
MIXERS = Registry("mixer")
FEED_FORWARDS = Registry("feed-forward")
BLOCKS = Registry("block")
