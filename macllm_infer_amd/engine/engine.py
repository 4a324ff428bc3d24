"""The engine: a loaded model, its cache manager and the one step function.

``step`` takes a batch of lanes (request, its next tokens, the places whose logits are
wanted): portions of prompts beside single decoded tokens, cut anywhere.  It runs only
the tokens it is given, as one batch, from the cache earlier steps left, and returns the
logits at the wanted places.  Everything is validated and all pages are reserved before
anything is launched, so a refused step (``StepError``, ``CacheExhausted``) changes nothing.
Sizes that a kernel would refuse are found when the engine is built, before a weight is
read (``ConfigError``).  A step that fails after its reservation, in a launch or anywhere
else, leaves nothing half done behind: the kernels write keys, values and state in place, so
the requests of that step cannot go on; they are ended, their pages and slots given back,
and ``StepFailed`` names them
(reference: src/architecture.rs:1187-1227 contract, src/decoder.rs:3878-3968 checks,
:4125-4201 transactional execute, which restores a checkpoint where this ends the requests;
src/architecture.rs:367-667 validation before load).
"""
from __future__ import annotations

from typing import Hashable, Optional, Sequence

import numpy as np
import torch

from ..cache.manager import CacheManager
from ..config.registry import config_from_dict, load_config
from ..config.spec import ConfigError
from ..kernels import build as kernel_build
from ..kernels import ops
from ..parts.base import BuildContext
from ..weights.loader import WeightSource, bind
from .context import Lane, LoweredLanes, apply_feeds, build_step_context, lower_lanes
from .model import DecoderModel

_DTYPES = {"bfloat16": torch.bfloat16, "bf16": torch.bfloat16, "float32": torch.float32, "fp32": torch.float32,
           "f32": torch.float32}


class StepError(ValueError):
    """A step was refused before anything ran; the engine's state is unchanged."""


class StepFailed(RuntimeError):
    """A step failed after its pages were reserved.  ``requests``: the requests of its lanes, which have
    been ended (their pages and state slots are free again, their tokens so far are lost); every other
    request is as it was.  ``__cause__`` is the error that stopped the step."""

    def __init__(self, requests, cause: BaseException):
        self.requests = list(requests)
        super().__init__(f"the step failed and its requests {self.requests!r} were ended: "
                         f"{type(cause).__name__}: {cause}")


def resolve_dtype(dtype) -> torch.dtype:
    if isinstance(dtype, torch.dtype):
        if dtype not in (torch.bfloat16, torch.float32):
            raise ValueError(f"dtype must be bfloat16 or float32, got {dtype}")
        return dtype
    if dtype not in _DTYPES:
        raise ValueError(f"dtype must be one of {sorted(_DTYPES)}, got {dtype!r}")
    return _DTYPES[dtype]


# A step with portions of prompts beside several single decoded tokens runs as two batches (see
# ``Engine._run_in_two``) when the single tokens cost more as part of the portions' batch than as a batch of their
# own.  As part of it every one of them is a prompt of one token to the prompt kernels (beside 2,048 prompt tokens
# of the 0.5B shape, 8 decoded tokens cost 2.7 ms and 63 cost 13); a batch of their own reads every weight once
# more and pays its dependent kernels.  Both depend on the model and on the GPU, so the clock decides when the
# first step that could be split comes (``DecodeGraphs.measure_split``): from so many single tokens on that they
# cost, beside the portions, what a batch of their own costs (the 0.5B shape: 17 beside a portion of 256 tokens, 9
# beside one of 2,048; eight layers of the 7B shape: 20 and 7; a third of a second for the three graphs).  Without a clock (no graphs, or ``measured_paths=False``) a step
# is split from SPLIT_FROM_LANES single tokens on, which is also the fewest the clock can say.
SPLIT_FROM_LANES = 4
SPLIT_NEVER = 1 << 30
# A step of more single decoded tokens than the skinny kernels take rows runs as two halves at once, each a
# captured graph of its own on a stream of its own (``Engine._run_in_halves``): a half's products go through the
# skinny kernels instead of the library, and while one half's mixer kernel streams states, keys and values the
# other half's products, which wait on latency rather than on bandwidth, run beside it.  The 0.5B shape at
# 2,048-token contexts: 96 single tokens in 3.97 ms instead of 4.53 as one graph, 128 in 4.41 instead of 5.03
# (two halves of 32 gain nothing on one graph of 64: 3.14 ms against 3.04).  The halves read every weight twice: a
# model whose steps wait for their weights loses (the 7B shape: 96 single tokens in 20.8 ms instead of 15.6), so the
# clock decides when the first such step comes (``DecodeGraphs.measure_halves``; the halves have to win by
# HALVES_MARGIN); without a clock such a step stays one graph.
HALVES_FROM_LANES = 65
HALVES_MOST_LANES = 128        # beyond, a half would leave the skinny kernels too: one graph, as measured for no such size
HALVES_MARGIN = 0.95


def split_from_lanes(lane_share: Optional[float]) -> int:
    """From how many single decoded tokens beside portions of prompts on a step runs as two batches.
    ``lane_share``: what one of them costs beside the portions, as a share of what a batch of them costs alone
    (None: not measured)."""
    if lane_share is None:
        return SPLIT_FROM_LANES
    if lane_share <= 0:
        return SPLIT_NEVER
    return max(SPLIT_FROM_LANES, int(1.0 / lane_share + 0.5))


class Engine:
    def __init__(self, model_dir: Optional[str] = None, *, config=None, tensors=None, dtype="bfloat16",
                 device="cuda:0", kv_cache_block_tokens: int = 16,
                 kv_cache_capacity_tokens: Optional[int] = None, max_active_sequences: int = 8,
                 check_device: bool = True, decode_graphs: bool = True, measured_paths: bool = True):
        """Load from ``model_dir`` (config.json + safetensors), or from a config object (or raw
        dict) plus a name -> tensor mapping.  ``kv_cache_capacity_tokens`` defaults to one
        model context shared by all requests (reference: src/runtime.rs:175-201).  With
        ``decode_graphs`` steps run as captured HIP graphs.  ``measured_paths``: where two kernels can
        serve a projection, the layers time both when the model is built and take the faster
        (``path_choices()`` says which); False: fixed rules only, so that the same kernels run in every
        process and bfloat16 results are the same bits from run to run."""
        self.dtype = resolve_dtype(dtype)
        self.device = ops.require_gpu(device) if check_device else torch.device(device)
        if model_dir is not None:
            self.config = load_config(model_dir)
        else:
            self.config = config_from_dict(config) if isinstance(config, dict) else config
        self.spec = self.config.to_model_spec()
        self.spec.validate()
        beyond = DecoderModel.limits(self.spec)
        if beyond:                                  # before any weight is read
            raise ConfigError("config.json: " + "; ".join(limit.text(self.spec.field_names) for limit in beyond))
        source = WeightSource.from_dir(model_dir) if model_dir is not None else WeightSource.from_tensors(tensors)
        if check_device:
            # (bfloat16 products of few rows go through the skinny kernels)
            skinny = ["decode"] if self.dtype == torch.bfloat16 else []
            kernel_build.ensure_modules(DecoderModel.kernel_modules(self.spec) + skinny + list(kernel_build.HOST_MODULES))
        source.apply_aliases(self.spec.tensor_aliases, root_prefix=self.spec.root_namespace)
        expected = DecoderModel.expected_tensors(self.spec)
        if self.spec.stored_name_rules:
            source.apply_stored_names(self.spec.stored_name, [expect.name for expect in expected])
        bound = bind(source, expected, DecoderModel.tensor_copies(self.spec))
        source.close()
        build = BuildContext(hidden_size=self.spec.hidden_size, dtype=self.dtype, device=self.device,
                             max_context=self.spec.max_context, measure_paths=measured_paths)
        self.model = DecoderModel(self.spec, bound, build)
        self.lane_share: Optional[float] = None
        self._split_from_lanes: Optional[int] = None
        self._measure_split = measured_paths
        needs, shared = DecoderModel.cache_layout(self.spec)
        capacity = kv_cache_capacity_tokens or self.spec.max_context
        self.cache = CacheManager(needs, shared, kv_cache_block_tokens, capacity, max_active_sequences,
                                  self.dtype, self.device)
        self.vocab_size = self.spec.vocab_size
        self.max_context = self.spec.max_context
        self.graphs = None
        self.graphs_beside = None                    # the graphs of the second half of a step that runs as two halves at once
        self._beside = None                          # and the stream they are replayed on
        self._in_halves: Optional[bool] = None
        self.halves_share: Optional[float] = None
        if decode_graphs and check_device and self.model.graph_safe:
            from .graphs import DecodeGraphs
            # the pool bounds a request's length only where some layer keeps every key: a model whose attention
            # layers all have windows or chunks (or that has none) gives passed pages back, and a request outgrows the pool
            bound = any(group.need.keeps_every_key for group in self.cache.groups)
            self.graphs = DecodeGraphs(self.model, self.cache, self.device,
                                       min(self.max_context, capacity) if bound else self.max_context)

    @property
    def split_from_lanes(self) -> int:
        """From how many single decoded tokens beside portions of prompts on a step runs as two batches: asked of
        the clock when it is first needed (or by ``warm_up``), where there is one."""
        if self._split_from_lanes is None:
            if self._measure_split and self.graphs is not None:
                self.lane_share = self.graphs.measure_split()
                self._split_from_lanes = split_from_lanes(self.lane_share) if self.lane_share is not None else SPLIT_NEVER
            else:
                self._split_from_lanes = split_from_lanes(None)
        return self._split_from_lanes

    @split_from_lanes.setter
    def split_from_lanes(self, value: int) -> None:
        self._split_from_lanes = int(value)

    @property
    def in_halves(self) -> bool:
        """Whether a step of HALVES_FROM_LANES single tokens or more runs as two halves at once: asked of the clock
        when it is first needed (or by ``warm_up``), where there is one."""
        if self._in_halves is None:
            self._in_halves = False
            if self._measure_split and self.graphs is not None:
                self.halves_share = self.graphs.measure_halves()
                self._in_halves = self.halves_share is not None and self.halves_share < HALVES_MARGIN
        return self._in_halves

    @in_halves.setter
    def in_halves(self, value: bool) -> None:
        self._in_halves = bool(value)

    def path_choices(self) -> dict:
        """What the first layer's fast path chose at build (empty when the layer has none): to be recorded
        beside a result, since a close call of the clock can fall either way from one process to the next."""
        fusion = getattr(self.model.blocks[0], "fusion", None) if self.model.blocks else None
        choices = getattr(fusion, "path_choices", None)
        return choices() if choices is not None else {}

    def warm_up(self, steps, context: int = 2048) -> list:
        """Capture the graphs of steps of (lanes, tokens) before the first request comes (a serving process
        does this once: no step of such a size is then ever launched kernel by kernel).  ``context``: the
        longest context the steps' requests will hold.  Returns what was captured; nothing without graphs."""
        self.split_from_lanes                        # the clock's say on mixed steps, before the first of them
        if self.graphs is None:
            return []
        whole, halves = [], []
        for lanes, tokens in steps:
            if tokens == lanes and HALVES_FROM_LANES <= lanes <= HALVES_MOST_LANES and self.in_halves:      # runs as two halves: a graph for each
                halves.append(((lanes + 1) // 2, lanes - (lanes + 1) // 2))
            else:
                whole.append((lanes, tokens))
        done = self.graphs.warm_up(whole + [(first, first) for first, _ in halves], context)
        if halves:
            from .graphs import DecodeGraphs
            if self.graphs_beside is None:
                self.graphs_beside = DecodeGraphs(self.model, self.cache, self.device, self.graphs.max_seq_len)
                self._beside = torch.cuda.Stream(device=self.device)
            done += self.graphs_beside.warm_up([(second, second) for _, second in halves], context)
        return done

    def step_token_target(self, lanes: int, tokens: int) -> int:
        """How many tokens (at most ``tokens``) a step of ``lanes`` lanes should hold if whoever makes it is free
        to cut a prompt portion shorter: the size at which the step fills the capacity of a captured graph
        instead of padding the next larger one."""
        return self.graphs.token_target(lanes, tokens) if self.graphs is not None else tokens

    # ------------------------------------------------------------------ requests
    def add_request(self, request: Hashable) -> None:
        """Make ``request`` live: a zeroed state slot and empty block tables."""
        self.cache.add_request(request)

    def finish(self, request: Hashable) -> None:
        """Give back everything ``request`` holds."""
        self.cache.finish(request)

    def has_request(self, request: Hashable) -> bool:
        return request in self.cache.requests

    def length(self, request: Hashable) -> int:
        return self.cache.requests[request].length

    # ------------------------------------------------------------------ the step function
    def validate(self, lanes: Sequence[Lane]) -> LoweredLanes:
        """StepError for a step that cannot run; otherwise its lanes as arrays."""
        if not lanes:
            raise StepError("a step needs at least one lane")
        try:
            lowered = lower_lanes(lanes, self.cache)
        except KeyError as error:
            raise StepError(str(error.args[0])) from None
        except (OverflowError, TypeError, ValueError) as error:
            raise StepError(f"tokens and wanted places must be integers: {error}") from None
        names = [lane.request for lane in lanes]
        if len(set(lowered.slots.tolist())) != len(lanes):
            twice = next(name for index, name in enumerate(names) if name in names[:index])
            raise StepError(f"request {twice!r} appears twice in one step")
        lengths, tokens = lowered.lengths, lowered.tokens
        if int(lengths.min()) == 0:
            raise StepError(f"request {names[int(np.argmin(lengths))]!r}: a lane cannot be empty")
        lane_of_token = np.repeat(np.arange(len(lanes)), lengths)
        outside = (tokens < 0) | (tokens >= self.vocab_size)
        if outside.any():
            where = int(np.argmax(outside))
            raise StepError(f"request {names[int(lane_of_token[where])]!r}: token {int(tokens[where])} is outside "
                            f"the vocabulary of {self.vocab_size}")
        starts = self.cache.lengths_of(lowered.slots)
        beyond = starts.astype(np.int64) + lengths > self.max_context
        if beyond.any():
            where = int(np.argmax(beyond))
            raise StepError(f"request {names[where]!r}: {int(starts[where])} + {int(lengths[where])} "
                            f"tokens exceed the context limit {self.max_context}")
        if any(lane.feed is not None for lane in lanes):
            first_rows = np.concatenate(([0], np.cumsum(lengths)[:-1]))
            feeds = []
            for index, lane in enumerate(lanes):
                if lane.feed is None:
                    continue
                source, row = lane.feed
                if int(lengths[index]) != 1:
                    raise StepError(f"request {names[index]!r}: a lane fed from the device holds one token")
                if not (isinstance(source, torch.Tensor) and source.dtype == torch.int32 and source.dim() == 1
                        and 0 <= int(row) < source.numel()):
                    raise StepError(f"request {names[index]!r}: the feed must be (an int32 vector, a row of it)")
                feeds.append((int(first_rows[index]), source, int(row)))
            lowered.feeds = tuple(feeds)
        if lowered.wants.size:
            lane_of_want = np.repeat(np.arange(len(lanes)), lowered.want_counts)
            outside = (lowered.wants < 0) | (lowered.wants >= lengths[lane_of_want])
            if outside.any():
                where = int(np.argmax(outside))
                lane = int(lane_of_want[where])
                raise StepError(f"request {names[lane]!r}: wanted place {int(lowered.wants[where])} is outside "
                                f"its {int(lengths[lane])} tokens")
        return lowered

    feeds_tokens = True          # a lane's token may come from the device (``Lane.feed``)

    def step(self, lanes: Sequence[Lane]) -> torch.Tensor:
        """Run one batch; returns float32 logits [wanted, vocab] in the order of the lanes and
        of each lane's ``want``.  Raises StepError or CacheExhausted with nothing changed, or
        StepFailed with the lanes' requests ended and everything they held given back.  The work is
        queued on the GPU; nothing here waits for it (a lane with ``feed`` takes its token from the device,
        so a caller may queue the next step before it has read this one's tokens)."""
        lowered = self.validate(lanes)
        single = lowered.lengths == 1
        singles = int(single.sum())
        # (the clock is asked, once, only by a step that may need its answer, and before anything is reserved)
        in_two = SPLIT_FROM_LANES <= singles < len(lanes) and self.split_from_lanes <= singles
        in_halves = (singles == len(lanes) and HALVES_FROM_LANES <= singles <= HALVES_MOST_LANES
                     and self.graphs is not None and self.in_halves)
        self.cache.reserve_slots(lowered.slots, lowered.lengths)
        try:
            if in_two:
                logits = self._run_in_two(lanes, lowered, single)
            elif in_halves:
                logits = self._run_in_halves(lanes)
            else:
                logits = self._run(lanes, lowered)
        except Exception as error:
            # earlier layers have written keys, values and state in place: these requests cannot go on
            names = [lane.request for lane in lanes]
            for name in names:
                self.cache.finish(name)
            raise StepFailed(names, error) from error
        self.cache.commit_slots(lowered.slots, lowered.lengths)
        return logits

    def _run(self, lanes: Sequence[Lane], lowered: LoweredLanes, graphs=None) -> torch.Tensor:
        """Queue the lanes' tokens as one batch: a captured graph where one fits, else launch by launch."""
        logits = None
        graphs = graphs if graphs is not None else self.graphs
        if graphs is not None:
            if int(lowered.lengths.max()) == 1:
                logits = graphs.run(lanes, lowered)                   # decode-only batch: a captured graph
            else:
                logits = graphs.run_bucket(lanes, lowered)            # prompt portions: a graph of their capacity
        if logits is None:
            context = build_step_context(lanes, self.cache, self.device, lowered, **self.model.step_layout)
            apply_feeds(context.token_ids, lowered.feeds)
            logits = self.model.forward(context, self.cache)
        return logits

    def _run_in_halves(self, lanes: Sequence[Lane]) -> torch.Tensor:
        """A step of many single decoded tokens as two halves at once: the second half's graph is replayed on a
        stream of its own, which starts behind everything queued so far (the tokens that lanes are fed from
        among it) and which the caller's stream waits for before it reads the rows.  The halves belong to
        different requests, so they share no page and no slot but the scratch ones of their padding lanes, whose
        contents nobody reads; their graphs have memory pools of their own."""
        main = torch.cuda.current_stream(self.device)
        if self.graphs_beside is None:
            from .graphs import DecodeGraphs
            self.graphs_beside = DecodeGraphs(self.model, self.cache, self.device, self.graphs.max_seq_len)
            self._beside = torch.cuda.Stream(device=self.device)
        half = (len(lanes) + 1) // 2
        first, second = list(lanes[:half]), list(lanes[half:])
        lowered_second = self.validate(second)
        self._beside.wait_stream(main)
        try:
            with torch.cuda.stream(self._beside):
                rows_second = self._run(second, lowered_second, self.graphs_beside)
            rows_first = self._run(first, self.validate(first))
        finally:
            # whatever happens, nothing queued behind this step (pages given back and used again among it) may
            # overtake what the second stream still has to do
            main.wait_stream(self._beside)
        rows_second.record_stream(main)
        return torch.cat([rows_first, rows_second])

    def _run_in_two(self, lanes: Sequence[Lane], lowered: LoweredLanes, single: np.ndarray) -> torch.Tensor:
        """A step that holds portions of prompts beside several single decoded tokens, as two batches one after
        the other: the portions through the prompt kernels, the single tokens through the decode kernels.  (As
        one batch the prompt kernels take every single token as a prompt of its own, a tile of the attention
        kernel and a chunk of the scan each: 2,048 prompt tokens beside 63 decoded ones took 19.4 ms on the
        0.5B shape, where the two batches take 6.3 and 3.1.)  The logits come back in the order of the lanes."""
        parts = []
        for chosen in (~single, single):
            members = [lane for lane, mine in zip(lanes, chosen) if mine]
            parts.append(self._run(members, self.validate(members)))
        # the rows of the two batches, back in the order of the lanes: runs of lanes of one kind are slices of that
        # kind's rows (no index travels to the device: that copy would wait for everything queued before it)
        pieces, cursor = [], [0, 0]
        run_kind, run_from = None, 0
        for kind, count in zip(single.astype(np.int64).tolist(), lowered.want_counts.tolist()):
            if kind != run_kind:
                if run_kind is not None and cursor[run_kind] > run_from:
                    pieces.append(parts[run_kind][run_from:cursor[run_kind]])
                run_kind, run_from = kind, cursor[kind]
            cursor[kind] += count
        if run_kind is not None and cursor[run_kind] > run_from:
            pieces.append(parts[run_kind][run_from:cursor[run_kind]])
        if not pieces:
            return parts[1]
        return pieces[0] if len(pieces) == 1 else torch.cat(pieces)
