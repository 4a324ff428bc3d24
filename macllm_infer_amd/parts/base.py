"""What every part of a layer looks like from outside, and the registry of part kinds.

A part is built from its spec (sizes and constants as fields), the path of its
tensors, the tensors themselves and a ``BuildContext``; it never learns which model it
is in.  ``register_part(kind)`` maps the ``kind`` string of a spec dataclass to the class
that runs it, so a new mixer, feed-forward, norm or position encoding is added by
registering a class, without a change to this package.

Interfaces
----------
every part      ``expected_tensors(spec, prefix, hidden_size) -> [Expect]`` (classmethod),
                ``kernel_modules`` (names of the HIP modules it launches),
                ``__init__(spec, prefix, tensors, build)``
mixer           ``cache_needs(spec) -> [KVNeed | StateNeed]`` (classmethod);
                ``forward(x [T, d], step, cache: EntryCache) -> [T, d]``;
                optional ``step_tables() -> [StepTable]``: index tables of its own in every step;
                optional ``projections()`` + ``mix(...)``: see ``Mixer.projections``;
                ``takes_tail = True``: ``forward`` (a feed-forward's too) takes ``tail``, see ``StreamTail``
feed-forward    ``forward(x [T, d]) -> [T, d]``; optional ``gated_projections()``
norm            ``forward(residual, rows=None) -> normed activations``; optional ``rms_prologue() ->
                (weight, eps)``: the norm is y = x / sqrt(mean(x^2) + eps) * weight, which the skinny
                kernels compute in their prologue, or take over altogether (``Residual.scaled``)
position        ``rotate_and_store(qkv, heads, kv_heads, head_dim, step, cache)``; optional
                ``fused_rotation() -> (inv_freq or None, rotary_dim) | None``: what the fused decode kernel
                applies in its place
every part      ``graph_safe = True`` if its forward may be captured in a HIP graph;
                ``limits(spec, hidden_size) -> [Limit]`` (classmethod): sizes its kernels refuse
"""
from __future__ import annotations

from dataclasses import dataclass
from typing import Dict, List, Optional

import torch

_PARTS: Dict[str, type] = {}


def register_part(kind: str):
    def decorate(cls):
        _PARTS[kind] = cls
        cls.kind = kind
        return cls
    return decorate


def part_class(spec) -> type:
    kind = getattr(spec, "kind", None)
    if kind not in _PARTS:
        raise KeyError(f"no part is registered for kind {kind!r}; registered: {sorted(_PARTS)}")
    return _PARTS[kind]


@dataclass
class BuildContext:
    hidden_size: int
    dtype: torch.dtype            # activation dtype: torch.float32 or torch.bfloat16
    device: torch.device
    max_context: int
    # Where two kernels can serve a product, a fast path may time both when the model is built and take the
    # faster one; False: fixed rules only, so that which kernel runs (and with it the last bits of bfloat16
    # results) is the same in every process.
    measure_paths: bool = True


@dataclass
class ScaledRows:
    """The residual stream's rows as the product behind a norm wants them, but for the division by the root mean
    square: ``rows`` bfloat16 [T, d] = h * weight, with the partial sums of squares of h (``ssq``, float32
    [workgroups, rows rounded up to 16]) that give it.  ``weight`` is the norm's weight they were made for."""
    rows: torch.Tensor
    ssq: torch.Tensor
    weight: torch.Tensor


@dataclass
class ScaledBranch:
    """A branch output [T, d] that is multiplied, feature by feature, by ``scale`` (float32 [d]) where it is added
    to the residual stream: an entry of ``Residual.pending`` in place of the plain tensor."""
    rows: torch.Tensor
    scale: torch.Tensor


@dataclass
class WeightedBranch:
    """A branch output [T, d] (float32 or the activation dtype) that is multiplied by one number, ``factor``, in
    float32 where it is added to the residual stream."""
    rows: torch.Tensor
    factor: float = 1.0


@dataclass
class RowVector:
    """One vector (float32 [d]) that is added to every row of the residual stream."""
    vector: torch.Tensor


@dataclass
class NormedBranches:
    """Branch outputs whose weighted sum goes through a norm of its own before it joins the residual stream:
    x <- x + ((s - mean) / sqrt(variance + eps) * weight + bias) with s = sum of factor * rows over ``branches``
    [(rows [T, d], factor)], everything in float32; with ``alpha`` the norm is the one without statistics,
    x <- x + (tanh(alpha s) * weight + bias); with no ``bias`` it is an RMS norm, x <- x + s / sqrt(mean(s^2) + eps) *
    weight."""
    branches: list
    weight: torch.Tensor
    bias: Optional[torch.Tensor] = None
    eps: float = 0.0
    alpha: Optional[float] = None


@dataclass
class NormedRows:
    """The residual stream's rows already through ``norm`` (the part): what that norm would return."""
    rows: torch.Tensor
    norm: object


class StreamTail:
    """What stands between a branch's last launch and the part behind it in a layer whose norms compute no statistics:
    the norm behind the branch, the add to the residual stream and the next norm are element by element, so the launch
    that makes the branch's output can do them on its way out.  A part that ``takes_tail`` may end its forward with
    ``project`` or ``stream_arguments`` and return None; ``done`` then says so and ``rows`` holds the next norm's rows."""

    def __init__(self, h: torch.Tensor, post, following, dtype: torch.dtype):
        self.h, self.post, self.following, self.dtype = h, post, following, dtype
        self.done, self.rows = False, None

    def stream_arguments(self) -> tuple:
        """(h, post norm, next norm or None, next rows or None) for a launch that does the rest; counts as done."""
        numbers = lambda norm: (norm.weight, norm.bias, norm.alpha)
        if self.following is not None:
            self.rows = torch.empty(self.h.shape, dtype=self.dtype, device=self.h.device)
        self.done = True
        return (self.h, numbers(self.post), None if self.following is None else numbers(self.following), self.rows)

    def project(self, linear, x: torch.Tensor) -> bool:
        """The branch's output projection with the rest in its epilogue, where the step is small enough for it."""
        from ..kernels import ops
        rows, width = x.shape
        if (x.dtype != torch.bfloat16 or linear.weight.dtype != torch.bfloat16 or rows > TAIL_PROJECT_ROWS or width % 32 != 0
                or x.stride(1) != 1 or x.stride(0) % 8 != 0 or x.data_ptr() % 16 != 0
                or not ops.fused_gemm_supported(False, rows, width)):
            return False
        ops.fused_gemm_tanh(linear.weight, linear.bias, x, self.stream_arguments(), row_tiles=-(-rows // 16))
        return True


TAIL_PROJECT_ROWS = 64        # rows of a step up to which a projection takes the way into the stream into its epilogue


class Residual:
    """The float32 residual stream [T, d] plus the branch outputs not yet added to it (tensors,
    ``ScaledBranch``es, ``WeightedBranch``es, ``NormedBranches`` or ``RowVector``s).  The next norm adds them and normalizes in one kernel.

    ``next_norm``: (weight, eps) of the norm that the layer after the one running starts with (the final norm
    after the last), if that norm is a root-mean-square norm, set by whoever runs the layers; a layer whose last
    projection adds to the stream itself may then leave ``scaled`` rows for it.  ``following``: the norm part that
    the layer after the one running starts with (the final norm after the last; None where something joins the stream
    before it); a layer may leave the stream's rows through that norm in ``normed``.  ``scaled`` and ``normed`` are
    dropped whenever ``h`` or ``pending`` is assigned: whoever changes the stream without knowing of them makes them
    stale."""

    def __init__(self, h: torch.Tensor):
        self._h = h
        self._pending: List[torch.Tensor] = []
        self.scaled: Optional[ScaledRows] = None
        self.next_norm: Optional[tuple] = None
        self.normed: Optional[NormedRows] = None
        self.following = None

    @property
    def h(self) -> torch.Tensor:
        return self._h

    @h.setter
    def h(self, value: torch.Tensor) -> None:
        self._h, self.scaled, self.normed = value, None, None

    @property
    def pending(self) -> List[torch.Tensor]:
        return self._pending

    @pending.setter
    def pending(self, value: List[torch.Tensor]) -> None:
        self._pending, self.scaled, self.normed = value, None, None


class Part:
    kernel_modules = ()
    # True when ``forward`` only enqueues work on the current stream (no host read-back, no
    # data-dependent launch shapes), so that a decode step containing the part can be captured
    # as a HIP graph.  Parts that do not say so run eagerly.
    graph_safe = False

    @classmethod
    def modules_of(cls, spec) -> tuple:
        """The HIP modules that a part of this spec launches: all of the class's, unless some are for forms it has not."""
        return tuple(cls.kernel_modules)

    @classmethod
    def expected_tensors(cls, spec, prefix: str, hidden_size: int):
        return []

    @classmethod
    def limits(cls, spec, hidden_size: int):
        """The sizes of ``spec`` that no kernel of this part takes, as ``kernels.limits.Limit``s: asked when a
        model is built, before its weights are read.  A part whose kernels take every size reports none."""
        return []


class Mixer(Part):
    # rows of one lane that one workgroup of the mixer's prompt kernel takes: the step's table of such runs
    # is cut to the largest tile any mixer of the model names (0: the mixer reads no such table)
    query_tile = 0
    # tokens of a chunk: the step then carries every lane cut from its first token into chunks of that many
    # (``step.chunk_tables[chunk_tokens]``); 0: the mixer reads no such table
    chunk_tokens = 0

    @classmethod
    def cache_needs(cls, spec):
        return []

    def step_tables(self):
        """Index tables of its own that the mixer wants in every step, as ``engine.context.StepTable``s: each is
        written on the host from the step's lanes by the function the mixer gives, uploaded with the step's
        other arrays, and found in ``step.tables[name]`` (int32, on the device); in a step that a captured graph
        reads it has the size of the step's capacity and a fixed address.  Mixers that declare the same name
        share one table."""
        return ()

    def forward(self, x: torch.Tensor, step, cache) -> torch.Tensor:
        raise NotImplementedError

    def projections(self):
        """A mixer that is "input projection of the normed rows, something in between, output projection"
        may hand out the three pieces: ``(in Linear, out Linear, width of what lies between)``, with
        ``mix(projected [T, in.out_features], step, cache, out [T, width])`` doing the part in between on
        column views of wider matrices.  A layer can then run the projections of all its mixers as one
        product each (and, for steps of single tokens, through the skinny kernels).  None: the mixer is
        only ever run through ``forward``."""
        return None


class FeedForward(Part):
    def forward(self, x: torch.Tensor) -> torch.Tensor:
        raise NotImplementedError

    def gated_projections(self):
        """A feed-forward that is down(SiLU(gate(x)) * up(x)) may hand out ``(gate_up Linear, down Linear,
        tile)``: gate and up rows of the first interleaved in tiles of ``tile`` rows.  None: it is only
        ever run through ``forward``."""
        return None
