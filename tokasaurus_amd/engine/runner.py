"""The step function: one batch of (request, its next tokens) through the model.

``ModelRunner`` owns the model, the cache manager and the cache tensors.  A step
runs only the tokens it is given, as one batch, reading everything earlier from
the cache, and returns the logits at the wanted places in 32-bit.  It is the
counterpart of the reference's preprocess/run_model pair
(tokasaurus/model/basic_worker.py:57-139) without the sampling, which sits on
top (the reference's forward never returns logits, tokasaurus/model/types.py:403-425).
"""

from __future__ import annotations

import gc
import time
from collections import OrderedDict
from dataclasses import dataclass
from pathlib import Path

import numpy as np
import torch

from tokasaurus_amd.cache.manager import CacheManager, plan_groups
from tokasaurus_amd.cache.storage import CacheStorage
from tokasaurus_amd.engine.batch import PlannedEntry, StepEntry, layout, to_device
from tokasaurus_amd.kernels import ops
from tokasaurus_amd.kernels.upload import upload
from tokasaurus_amd.models.causal_lm import CausalLM
from tokasaurus_amd.models.registry import build_model, config_from_folder
from tokasaurus_amd.parts.base import CacheView, StepContext
from tokasaurus_amd.weights.loader import read_tensors

DTYPES = {"bfloat16": torch.bfloat16, "float32": torch.float32}


def require_gpu() -> torch.device:
    if not torch.cuda.is_available():
        raise RuntimeError("no GPU is visible: this engine has no CPU path")
    return torch.device("cuda", torch.cuda.current_device())


@dataclass
class Sampling:
    """One temperature and one uniform number for every wanted row of a step."""

    temperatures: list[float]
    uniforms: list[float]


@dataclass
class StepOutput:
    logits: torch.Tensor  # [wanted, vocab] float32
    ids: torch.Tensor | None = None  # [wanted] int32, when the step sampled
    logprobs: torch.Tensor | None = None
    topk_ids: torch.Tensor | None = None  # [wanted, k] int32, when the runner ranks the most probable tokens
    topk_logprobs: torch.Tensor | None = None  # [wanted, k] float32
    # a sampled step also leaves ids and log-probabilities in pinned host memory (copied in
    # stream order right behind the step, or written there by a kernel of a recorded step): they
    # can be read while later steps already run.  ``ready.synchronize()`` waits for them.
    host: "HostResults | PublishedResults | None" = None
    ready: "torch.cuda.Event | PublishedResults | None" = None

    def sampled(self) -> tuple[list[int], list[float]]:
        """Token ids and their log-probabilities on the host; waits for this step only."""
        if self.ids is None:
            return [], []
        n = self.ids.shape[0]
        if self.host is None:
            return self.ids.tolist(), (self.logprobs.tolist() if self.logprobs is not None else [])
        self.ready.synchronize()
        ids, logprobs = self.host.ids[:n].tolist(), self.host.logprobs[:n].tolist()
        self._check_not_overwritten()
        return ids, logprobs

    def _check_not_overwritten(self) -> None:
        """A recorded step's results live in a ring of a few slots: whoever reads them after as
        many later runs of the same recording as the ring has slots finds another run's."""
        if isinstance(self.host, PublishedResults) and self.host.overwritten():
            raise RuntimeError("these results were read too late: later runs of the same recorded step have reused their "
                               f"slot (a step's results must be read before {RecordedDecodeStep.RING} more runs are launched)")

    def topk(self) -> tuple[list[list[int]], list[list[float]]] | None:
        """For every sampled row the most probable tokens and their log-probabilities, most
        probable first; None when the runner ranks none."""
        if self.topk_ids is None:
            return None
        n, k = self.topk_ids.shape
        if self.host is None:
            return self.topk_ids.tolist(), self.topk_logprobs.tolist()
        self.ready.synchronize()
        ranked = (self.host.topk_ids[: n * k].view(n, k).tolist(), self.host.topk_logprobs[: n * k].view(n, k).tolist())
        self._check_not_overwritten()
        return ranked


class HostResults:
    """Pinned host memory for one step's sampled ids, log-probabilities and ranked tokens:
    one allocation, viewed by kind."""

    def __init__(self, width: int, k: int):
        self.width, self.k = width, k
        self.buffer = torch.zeros((width * (2 + 2 * k),), dtype=torch.int32, pin_memory=True)
        self.ids = self.buffer[:width]
        self.logprobs = self.buffer[width : 2 * width].view(torch.float32)
        self.topk_ids = self.buffer[2 * width : (2 + k) * width]
        self.topk_logprobs = self.buffer[(2 + k) * width : (2 + 2 * k) * width].view(torch.float32)
        self.event = torch.cuda.Event()


class PublishedResults:
    """One slot of a recorded step's ring of results in pinned host memory, as the step's last
    kernel writes it: [run number + 1][ids][log-probabilities][ranked ids][their log-probabilities].
    The first word is written last; ``synchronize`` waits until it names the run."""

    WAIT_SECONDS = 60.0  # a step takes milliseconds: longer than this and the device is taken for lost

    def __init__(self, slot: torch.Tensor, slot_np: np.ndarray, run: int, width: int, k: int):
        self._seq, self.run = slot_np[:1], run
        self.ids = slot[1 : 1 + width]
        self.logprobs = slot[1 + width : 1 + 2 * width].view(torch.float32)
        self.topk_ids = slot[1 + 2 * width : 1 + (2 + k) * width]
        self.topk_logprobs = slot[1 + (2 + k) * width : 1 + (2 + 2 * k) * width].view(torch.float32)

    def _ahead(self) -> int:
        """How far the slot's number is past this run's own (0: this run's results are there); the
        device counts runs in 32 bits, so the difference is taken modulo 2^32."""
        return (int(self._seq[0]) - (self.run + 1)) & 0xFFFFFFFF

    def done(self) -> bool:
        return self._ahead() < 0x80000000

    def overwritten(self) -> bool:
        """A later run has published into this slot (checked after reading: a slot's number is written last)."""
        return self._ahead() != 0

    def synchronize(self) -> None:
        if self.done():
            return
        deadline = time.monotonic() + self.WAIT_SECONDS
        spins = 0
        while not self.done():
            spins += 1
            if spins % 4096 == 0 and time.monotonic() > deadline:
                torch.cuda.synchronize()  # a fault of the device is reported here
                if not self.done():
                    raise RuntimeError(f"run {self.run} of a recorded step never published its results")


def graph_buckets(max_size: int, step: int) -> list[int]:
    """Batch sizes decode steps are recorded at: 1, 2, 4, ... up to ``step``, then multiples of
    ``step`` up to 8 times ``step`` (the reference pads to multiples of 16 up to 128,
    tokasaurus/common_types.py:117-121), beyond that multiples of 2 times ``step`` up to 16 times
    ``step``, of 4 times ``step`` up to 32 times ``step`` and of 8 times ``step`` from there, up
    to ``max_size``: a batch of more than 128 rows is padded by fewer than 32 rows or a quarter
    (measured at 2,048 tokens of context: 129 rows padded to 192 took 3.65 ms, 128 rows 3.11),
    and a thousand rows take two dozen recordings, not sixty."""
    sizes = []
    b = 1
    while b < step and b <= max_size:
        sizes.append(b)
        b *= 2
    b = step
    while b <= max_size:
        sizes.append(b)
        b += step if b < 8 * step else (2 * step if b < 16 * step else (4 * step if b < 32 * step else 8 * step))
    return sizes


class RecordedDecodeStep:
    """A decode step of fixed size (one token per request, padded to ``size`` rows)
    recorded into a HIP graph: embedding, every block, the head and the sampler.

    All of the step's integers and the sampler's numbers live in one device buffer.  The host
    writes them into a slot of a ring in pinned memory; the step's first kernel fetches the slot
    that the step's run number names, and its last kernel writes what was sampled into a second
    such ring (``kernels.ops.stage_step``, ``publish_step``): a replay is one launch, with no copy
    commands between two steps.  The logits go to a buffer that all recordings of a runner share.
    Padding rows belong to no request: they read and write the null page and the
    extra slot.  The step is planned for contexts up to ``kv_bound`` (a power of two,
    at most the longest context a request may have), so one recording serves every
    length up to there; an eager step plans for the same bound and so gives the same bits.
    """

    def __init__(self, runner: "ModelRunner", size: int, kv_bound: int):
        # no reference to the runner is kept: a runner and its recorded steps must not form a
        # cycle, or they would be freed by the cyclic collector at a time of its choosing,
        # possibly while another step is being recorded, when memory must not be released
        self.size = size
        self.captured = runner.capture_graphs
        self.num_ranked = runner.topk_logprobs
        model, storage, manager = runner.model, runner.storage, runner.manager
        self.model, self.storage, self.manager = model, storage, manager
        device = model.device
        B = size
        # a table row as wide as the bound's pages, not as the longest request the engine allows
        pages_in_bound = -(-kv_bound // runner.page_size)
        widths = [min(t.shape[1], pages_in_bound) for t in manager.slot_tables]
        self.widths = widths
        fields = [("token_ids", B), ("positions", B), ("token_req", B), ("q_start", B + 1), ("kv_len", B),
                  ("slots", B), ("token_slots", B), ("want_rows", B), ("temperature", B), ("uniform", B)]
        fields += [(f"table{g}", B * w) for g, w in enumerate(widths)]
        self.spans, at = {}, 0
        for name, n in fields:
            self.spans[name] = (at, n)
            at += n
        at = -(-at // 4) * 4  # the staging kernel moves 16 bytes a thread
        self.in_ring = torch.zeros((self.RING, at), dtype=torch.int32, pin_memory=True)
        self.in_ring_np = self.in_ring.numpy()
        self.in_ring_f32 = self.in_ring.view(torch.float32).numpy()
        self.dev = torch.zeros((at,), dtype=torch.int32, device=device)
        k = self.num_ranked
        self.out_ring = torch.zeros((self.RING, ops.publish_words(B, k)), dtype=torch.int32, pin_memory=True)
        self.out_ring_np = self.out_ring.numpy()
        self.counter = torch.zeros((1,), dtype=torch.int32, device=device)  # runs of this step so far, on the device
        self.runs = 0  # the same count on the host
        self.null_slot = manager.slots.num_slots
        for slot in range(self.RING):
            self._fill(slot, [], [], [], [], [], [])
        self.logits_out = runner.shared_logits(B)

        def view(name: str) -> torch.Tensor:
            a, n = self.spans[name]
            return self.dev[a : a + n]

        self.ctx = StepContext(
            num_tokens=B, num_requests=B, dtype=model.dtype, device=device,
            token_ids=view("token_ids"), positions=view("positions"), token_req=view("token_req"),
            q_start=view("q_start"), kv_len=view("kv_len"), slots=view("slots"),
            host_q_start=list(range(B + 1)), host_kv_len=[kv_bound] * B, host_slots=[self.null_slot] * B,
            last_token=storage.last_token, embedding_state=storage.embedding_state, max_q_len=1, max_kv_len=kv_bound,
        )
        self.ctx.extras["static"] = True  # parts keep what they plan: the step is replayed
        self.ctx.extras["kv_bound"] = kv_bound
        self.ctx.extras["num_portions"] = 0
        tables = [view(f"table{g}").view(B, w) for g, w in enumerate(widths)]
        self.caches = runner.cache_views(tables)
        self.want_rows = view("want_rows")
        self.token_slots = view("token_slots")  # where the sampler leaves each row's token
        self.temperature = view("temperature").view(torch.float32)
        self.uniform = view("uniform").view(torch.float32)

        # once outside the graph (parts plan and allocate what they keep), then recorded;
        # the collector stays off meanwhile: nothing may be freed while a graph is recorded
        gc.collect()
        was_enabled = gc.isenabled()
        gc.disable()
        try:
            stream = torch.cuda.Stream()
            stream.wait_stream(torch.cuda.current_stream())
            with torch.cuda.stream(stream):
                self._forward()
            torch.cuda.current_stream().wait_stream(stream)
            torch.cuda.synchronize()
            if self.captured:
                self.graph = torch.cuda.CUDAGraph()
                # recorded steps run one at a time and their results are read before the next step:
                # they share one pool of memory
                with torch.cuda.graph(self.graph, pool=runner.graph_pool):
                    self.logits, self.ids, self.logprobs, self.topk = self._forward()
                torch.cuda.synchronize()
            self.runs = int(self.counter.item())  # the runs made while setting up
        finally:
            if was_enabled:
                gc.enable()

    RING = 4  # slots of the two rings: runs that may be under way or unread at a time

    def _forward(self):
        ops.stage_step(self.in_ring, self.counter, self.dev)
        # every row of a recorded step is wanted, in order: nothing to pick out
        logits = self.model.forward(self.ctx, self.caches, self.storage.states, None, logits_out=self.logits_out)
        ids, logprobs = ops.sample(logits, self.temperature, self.uniform, self.token_slots, self.storage.last_token)
        topk = ops.topk_logprobs(logits, self.temperature, self.num_ranked) if self.num_ranked else None
        ops.publish_step(self.out_ring, self.counter, ids, logprobs, *(topk or (None, None)))
        return logits, ids, logprobs, topk

    def output_bytes(self) -> int:
        """Device memory this recording keeps for its results beside the shared logits."""
        tensors = [self.ids, self.logprobs, *(self.topk or ())]
        return sum(t.numel() * t.element_size() for t in tensors if t is not None) + self.dev.numel() * 4

    def _fill(self, ring_slot, token_ids, positions, slots, write_slots, temperatures, uniforms) -> None:
        B, n = self.size, len(token_ids)
        a = self.in_ring_np[ring_slot]
        pad = B - n

        def put(name, values, fill):
            at, m = self.spans[name]
            a[at : at + n] = values
            a[at + n : at + m] = fill

        put("token_ids", token_ids, 0)
        put("positions", positions, 0)
        put("kv_len", [p + 1 for p in positions], 1)
        put("slots", slots, self.null_slot)
        put("token_slots", write_slots, self.null_slot)
        at, m = self.spans["token_req"]
        a[at : at + m] = np.arange(m, dtype=np.int32)
        at, m = self.spans["q_start"]
        a[at : at + m] = np.arange(m, dtype=np.int32)
        at, m = self.spans["want_rows"]
        a[at : at + m] = np.arange(m, dtype=np.int32)
        f = self.in_ring_f32[ring_slot]
        at, m = self.spans["temperature"]
        f[at : at + n] = temperatures
        f[at + n : at + m] = 0.0
        at, m = self.spans["uniform"]
        f[at : at + n] = uniforms
        f[at + n : at + m] = 0.0
        rows = np.asarray(list(slots) + [self.null_slot] * pad, dtype=np.int64)
        for g, table in enumerate(self.manager.slot_tables):
            at, m = self.spans[f"table{g}"]
            a[at : at + m].reshape(B, self.widths[g])[:] = table[rows, : self.widths[g]]

    def run(self, planned: list[PlannedEntry], sampling: Sampling | None, write_slots: bool) -> StepOutput:
        n = len(planned)
        token_ids = [(-(e.slot + 1) if e.tokens is None else e.tokens[0]) for e in planned]
        positions = [e.start for e in planned]
        # a step that only wants logits must not disturb the requests' last tokens
        slots = [e.slot for e in planned]
        out_slots = slots if write_slots else [self.null_slot] * n
        temps = sampling.temperatures if sampling is not None else [0.0] * n
        us = sampling.uniforms if sampling is not None else [0.0] * n
        run = self.runs
        ring_slot = run % self.RING
        if run >= self.RING:
            # the run that used these two slots last has read its input and published its results
            PublishedResults(self.out_ring[ring_slot], self.out_ring_np[ring_slot], run - self.RING, self.size,
                             self.num_ranked).synchronize()
        self._fill(ring_slot, token_ids, positions, slots, out_slots, temps, us)
        self.runs += 1
        if self.captured:
            self.graph.replay()
        else:
            # the same padded step launched kernel by kernel: what a replay must reproduce bit for bit
            self.logits, self.ids, self.logprobs, self.topk = self._forward()
        out = StepOutput(self.logits[:n], self.ids[:n], self.logprobs[:n] if self.logprobs is not None else None)
        if self.topk is not None:
            out.topk_ids, out.topk_logprobs = self.topk[0][:n], self.topk[1][:n]
        out.host = out.ready = PublishedResults(self.out_ring[ring_slot], self.out_ring_np[ring_slot], run, self.size,
                                                self.num_ranked)
        return out


class ModelRunner:
    def __init__(
        self,
        model: CausalLM,
        page_size: int,
        num_pages: int | list[int],
        max_slots: int,
        max_tokens_per_request: int | None = None,
        use_graphs: bool = True,
        graph_max_size: int | None = 128,
        graph_step: int = 16,
        topk_logprobs: int | None = None,
        first_kv_bound: int = 1024,
        kv_bound_factor: int = 2,
        max_recordings: int = 64,
    ):
        """``num_pages``: pages of every cache group's pool, or one number for each group (a group
        that keeps a window of keys needs fewer).  ``graph_max_size``: the most rows a recorded
        decode step has (None: as many as there are slots).  ``first_kv_bound`` and
        ``kv_bound_factor``: the context lengths that steps are planned (and recorded) for, see
        ``kv_bound``.  ``max_recordings``: recorded steps kept; the one unused longest goes first."""
        assert model.device is not None, "load the model's weights first"
        self.model = model
        # every sampled row also gets its most probable tokens ranked, this many of them
        # (tokasaurus/model/llama.py:407-416 ranks for every row what the engine was set up for)
        self.topk_logprobs = int(topk_logprobs) if topk_logprobs else 0
        self.page_size = page_size
        self.max_positions = model.spec.max_positions
        for block in model.blocks:  # a shape no attention kernel takes is refused here, not at the first step
            block.check_cache(page_size, model.dtype)
        needs = model.cache_needs()
        cache_of = [e.cache_of for e in model.spec.run_order]
        self.groups, self.where = plan_groups(needs, cache_of)
        pages = list(num_pages) if isinstance(num_pages, (list, tuple)) else [num_pages] * len(self.groups)
        if len(pages) != len(self.groups):
            raise ValueError(f"{len(pages)} page counts for {len(self.groups)} cache groups")
        # a request's length is bounded by the pools that keep every key; a windowed group recycles its pages
        whole = [n for n, g in zip(pages, self.groups) if g.need.keeps_all] or pages
        limit = min([self.max_positions] + [n * page_size for n in whole])
        if max_tokens_per_request is not None:
            limit = min(limit, max_tokens_per_request)
        self.max_tokens_per_request = limit
        self.manager = CacheManager(
            self.groups, pages, page_size, max_slots, max_blocks_per_request=-(-limit // page_size)
        )
        if first_kv_bound < 1 or kv_bound_factor < 2:
            raise ValueError("context bounds start at a positive length and grow by a factor of 2 or more")
        self.first_kv_bound, self.kv_bound_factor = int(first_kv_bound), int(kv_bound_factor)
        self.use_graphs = use_graphs
        # False (set by tests before the first decode step): recorded steps keep their padded
        # shapes and buffers but launch their kernels one by one instead of replaying a graph
        self.capture_graphs = True
        # Steps of more rows than the weight-streaming product takes on hold library products.
        # They are recorded too: at short contexts an eager step of 40 to 128 rows is bound by the
        # host's launches and takes up to twice as long (measured: 3.2 against 1.6 ms at 40 rows
        # and 1,024 tokens of context).  The tests replay every recorded size several times with
        # eager steps between and compare each replay's tokens with an eager run's.
        largest = max(max_slots, 1) if graph_max_size is None else min(graph_max_size, max(max_slots, 1))
        self.graph_sizes = [b for b in graph_buckets(largest, graph_step) if b <= largest] if use_graphs else []
        if use_graphs and largest not in self.graph_sizes:
            self.graph_sizes.append(largest)
            self.graph_sizes.sort()
        # by (rows, context bound), the one used last at the end
        self.recorded: "OrderedDict[tuple[int, int], RecordedDecodeStep]" = OrderedDict()
        self.max_recordings = max(1, int(max_recordings))
        self._shared_logits: torch.Tensor | None = None  # [largest recorded size, vocab], see shared_logits
        self.graph_pool = torch.cuda.graph_pool_handle() if use_graphs else None
        if model.dtype == torch.bfloat16:
            ops.library_workspace()  # made now, so that no recording of a step allocates it
        self._host_ring: list[HostResults] = []  # pinned buffers for what steps sampled
        self._host_at = 0
        self.storage = CacheStorage(
            self.groups,
            pages,
            page_size,
            model.state_needs(),
            max_slots,
            model.dtype,
            model.device,
            embedding_state_need=model.embedding_state_need(),
        )

    # ---- construction from a model folder
    @classmethod
    def from_folder(
        cls,
        model_dir: str | Path,
        dtype: str,
        page_size: int,
        num_pages: int,
        max_slots: int,
        rope_scaling_override: tuple[bool, dict | None] = (False, None),
        **options,
    ) -> "ModelRunner":
        device = require_gpu()
        if dtype not in DTYPES:
            raise ValueError(f"dtype {dtype!r}: this engine runs {sorted(DTYPES)}")
        arch, cfg = config_from_folder(model_dir, rope_scaling_override)
        model = build_model(arch, cfg)
        specs = model.tensor_specs()
        # a checkpoint that ties its head may still carry the head's tensor: read_tensors warns and goes on
        tensors = read_tensors(model_dir, specs, allow_unexpected=model.spec.ignorable_tensors)
        model.load(tensors, DTYPES[dtype], device)
        return cls(model, page_size, num_pages, max_slots, **options)

    @classmethod
    def from_random(
        cls,
        config: dict,
        seed: int,
        dtype: str,
        page_size: int,
        num_pages: int,
        max_slots: int,
        **options,
    ) -> "ModelRunner":
        """A runner on seeded random weights drawn on the device, for models too large to be
        worth a folder (benchmarks): ``config`` is what config.json would hold; the values are
        those of ``weights.draw_tensors`` with the device's generator."""
        from tokasaurus_amd.models.registry import architecture_of
        from tokasaurus_amd.weights.random_init import draw_tensors

        device = require_gpu()
        if dtype not in DTYPES:
            raise ValueError(f"dtype {dtype!r}: this engine runs {sorted(DTYPES)}")
        arch = architecture_of(config)
        model = build_model(arch, arch.config_from_dict(config))
        tensors = draw_tensors(model.tensor_specs(), seed=seed, device=device)
        model.load(tensors, DTYPES[dtype], device)
        del tensors
        torch.cuda.empty_cache()
        return cls(model, page_size, num_pages, max_slots, **options)

    # ---- requests
    def admit(self, request_id: str) -> None:
        self.manager.admit(request_id)

    def release(self, request_id: str) -> None:
        self.manager.release(request_id)

    # ---- the step
    def plan(self, entries: list[StepEntry]) -> list[PlannedEntry]:
        """Reserve pages for every entry (NoSpaceException leaves the cache usable)."""
        planned = []
        for e in entries:
            if e.request_id not in self.manager.requests:
                self.manager.admit(e.request_id)
            rc = self.manager.requests[e.request_id]
            q_len = 1 if e.tokens is None else len(e.tokens)
            new_len = rc.num_tokens + q_len
            if new_len > self.max_tokens_per_request:
                raise ValueError(
                    f"request {e.request_id!r} would reach {new_len} tokens, a request may hold "
                    f"{self.max_tokens_per_request} (the model's positions end at {self.max_positions})"
                )
            self.manager.reserve(e.request_id, new_len)
            planned.append(PlannedEntry(e.request_id, e.tokens, list(e.want), rc.slot, rc.num_tokens, rc.tables))
        return planned

    def cache_views(self, tables: list[torch.Tensor]) -> list[CacheView | None]:
        """For every run entry the pages it uses and its group's block table of this step."""
        caches: list = []
        for i, w in enumerate(self.where):
            writable = self.model.spec.run_order[i].cache_of is None

            def view(place: tuple[int, int]) -> CacheView:
                g, k = place
                return CacheView(keys=self.storage.keys[g][k], values=self.storage.values[g][k], block_table=tables[g],
                                 page_size=self.page_size, writable=writable)

            # a block that named several caches gets them as a list, in its order
            caches.append(None if w is None else ([view(p) for p in w] if isinstance(w, list) else view(w)))
        return caches

    def _recorded_for(self, planned: list[PlannedEntry]) -> RecordedDecodeStep | None:
        """The recorded step that takes this batch: every request brings one
        token and wants its logits, and a recorded size holds them."""
        if not self.graph_sizes or not planned or len(planned) > self.graph_sizes[-1]:
            return None
        if any(e.q_len != 1 or e.want != [0] for e in planned):
            return None
        size = next(b for b in self.graph_sizes if b >= len(planned))
        return self._recording((size, self.kv_bound(max(e.start + e.q_len for e in planned))))

    def _recording(self, key: tuple[int, int]) -> RecordedDecodeStep:
        """The recorded step of (rows, context bound), made now if it is not there; when more
        than ``max_recordings`` are kept, the one unused longest is dropped first (its graph
        and its buffers go back to the pool that the recordings share)."""
        step = self.recorded.get(key)
        if step is not None:
            self.recorded.move_to_end(key)
            return step
        while len(self.recorded) >= self.max_recordings:
            _, old = self.recorded.popitem(last=False)
            torch.cuda.synchronize()  # its last run is over before its memory may be used again
            del old
        self.recorded[key] = RecordedDecodeStep(self, *key)
        return self.recorded[key]

    def shared_logits(self, rows: int) -> torch.Tensor:
        """The first ``rows`` rows of the one 32-bit buffer [largest recorded size, vocabulary]
        that every recorded step writes its logits to: recorded steps run one at a time and a
        step's logits are read (by the sampler, or by whoever asked for them) before the next
        starts, so one buffer serves all sizes and context bounds.  Made at the first call,
        outside any recording."""
        if self._shared_logits is None:
            if torch.cuda.is_current_stream_capturing():
                raise RuntimeError("the shared logits buffer must exist before a step is recorded")
            self._shared_logits = torch.empty((self.graph_sizes[-1], self.model.spec.vocab_size), dtype=torch.float32,
                                              device=self.model.device)
        return self._shared_logits[:rows]

    def record_decode_steps(self, max_rows: int | None = None, bounds: list[int] | None = None) -> int:
        """Record the decode steps of every size up to ``max_rows`` (all sizes by default) for
        the given context bounds (by default the first, 1 024 tokens, where every request
        starts) now, instead of at their first use in the middle of a request's decoding: the
        reference records all its sizes and warms up before it serves
        (tokasaurus/model/utils.py:387-509,630-720).  Returns the number of recordings made;
        each holds its own [rows, vocab] logits (and ranked tokens) in the shared pool."""
        made = 0
        for bound in bounds or [self.kv_bound(1)]:
            for size in self.graph_sizes:
                if max_rows is not None and size > max(max_rows, self.graph_sizes[0]):
                    continue
                key = (size, self.kv_bound(bound))
                if key not in self.recorded:
                    self._recording(key)
                    made += 1
        return made

    def recorded_bytes(self) -> int:
        """Device memory that the recorded steps keep for what they take in and give out: the
        shared logits buffer and every recording's own small arrays.  It does not grow with the
        number of context bounds met (beyond a few KB a recording) and is bounded by
        ``max_recordings``; ``recorded_bytes_bound`` is that bound."""
        shared = self._shared_logits.numel() * 4 if self._shared_logits is not None else 0
        return shared + sum(step.output_bytes() for step in self.recorded.values())

    def recorded_bytes_bound(self) -> int:
        """What ``recorded_bytes`` can reach at most, known before any step is recorded: for the
        start-up account of device memory beside the cache."""
        if not self.graph_sizes:
            return 0
        rows, k = self.graph_sizes[-1], self.topk_logprobs
        widest = sum(t.shape[1] for t in self.manager.slot_tables) if self.manager.slot_tables else 0
        per_recording = rows * (2 + 2 * k) * 4 + (rows * (11 + widest) + 8) * 4
        return rows * self.model.spec.vocab_size * 4 + self.max_recordings * per_recording

    def kv_bound(self, max_kv_len: int) -> int:
        """The context length a step is planned for: the first of ``first_kv_bound`` times the
        powers of ``kv_bound_factor`` (1 024, 2 048, 4 096, ... by default) that holds the step's
        longest request, at most the longest a request may get.  Parts choose their launches
        from it and not from the batch's own lengths, so a recorded step and an eager one cut
        their work alike."""
        bound = self.first_kv_bound
        while bound < max_kv_len:
            bound *= self.kv_bound_factor
        return min(bound, self.max_tokens_per_request)

    def run(self, entries: list[StepEntry], sampling: Sampling | None = None, write_slots: bool | None = None) -> StepOutput:
        """Run one batch.  Logits [wanted, vocab] float32 come in the order of the
        entries and of their ``want`` lists; with ``sampling`` every wanted row is
        also sampled, and the token written to its request's slot."""
        planned = self.plan(entries)
        # requests admitted since the last step (here or by a scheduler) start from zeroed state;
        # in stream order before this step and after the last step of the slot's former holder
        self.storage.reset_slots(self.manager.take_fresh_slots())
        write_slots = (sampling is not None) if write_slots is None else write_slots
        recorded = self._recorded_for(planned)
        if recorded is not None:
            out = recorded.run(planned, sampling, write_slots)
        else:
            hb = layout(planned, self.model.spec.vocab_size, len(self.groups), self.manager.slot_tables)
            ctx, want_rows, tables = to_device(hb, self.model.dtype, self.model.device, self.storage.last_token)
            ctx.extras["kv_bound"] = self.kv_bound(ctx.max_kv_len)
            ctx.embedding_state = self.storage.embedding_state
            every_row = hb.want_rows == list(range(ctx.num_tokens))
            logits = self.model.forward(ctx, self.cache_views(tables), self.storage.states, None if every_row else want_rows)
            out = StepOutput(logits)
            if sampling is not None and logits.shape[0] > 0:
                # rows are in the order of the entries' wants; one slot a row
                slots = [e.slot for e in planned for _ in e.want]
                dev = self.model.device
                n_out = len(sampling.temperatures)
                params = upload(sampling.temperatures + sampling.uniforms, torch.float32, dev)
                slot_t = upload(slots, torch.int32, dev) if write_slots else None
                out.ids, out.logprobs = ops.sample(
                    logits, params[:n_out], params[n_out:], slot_t, self.storage.last_token if write_slots else None
                )
                if self.topk_logprobs:
                    out.topk_ids, out.topk_logprobs = ops.topk_logprobs(logits, params[:n_out], self.topk_logprobs)
        if out.host is None and out.ids is not None and out.ids.shape[0] > 0:
            self._copy_to_host(out)
        for e in planned:
            self.manager.advance(e.request_id, e.start + e.q_len)
        return out

    def warm_up(self, max_tokens: int, max_rows: int) -> list[tuple[int, int]]:
        """Run the largest steps once on requests of its own, before any real request is admitted:
        a prompt portion of ``max_tokens`` tokens, a step of ``max_rows`` single tokens, and both
        kinds together, each sampled from.  Memory that does not suffice for the engine's settings
        shows here and not in the middle of serving, and the library has chosen and loaded its
        kernels for the largest shapes (tokasaurus/model/utils.py:387-490 sends such batches "to
        check if it's gonna OOM").  Sizes are cut to what slots, pages and the longest request
        allow.  Returns the (prompt tokens, single-token rows) of the steps it ran."""
        if self.manager.requests:
            raise RuntimeError("warm_up runs before any request is admitted")
        P = self.page_size
        free_pages = min(self.manager.num_free_pages(), default=1 << 40)
        free_slots = self.manager.slots.num_free
        rows = max(0, min(max_rows, free_slots, free_pages, max_tokens)) if self.max_tokens_per_request >= 2 else 0
        ran: list[tuple[int, int]] = []

        def prompts(tokens: int, tag: str, slots: int, pages: int) -> list[StepEntry]:
            """Requests of this step alone that bring ``tokens`` prompt tokens between them."""
            entries: list[StepEntry] = []
            while tokens > 0 and slots > 0:
                n = min(tokens, self.max_tokens_per_request, pages * P)
                if n <= 0:
                    break
                entries.append(StepEntry(f"warm-up-{tag}-{len(entries)}", [0] * n, [n - 1]))
                tokens, slots, pages = tokens - n, slots - 1, pages - -(-n // P)
            return entries

        def run(portions: list[StepEntry], row_ids: list[str]) -> None:
            entries = portions + [StepEntry(rid, [0], [0]) for rid in row_ids]
            if entries:
                self.run(entries, Sampling([0.0] * len(entries), [0.0] * len(entries)))
                ran.append((sum(len(e.tokens) for e in portions), len(row_ids)))
            for e in portions:
                self.release(e.request_id)

        try:
            run(prompts(max_tokens, "prompt", free_slots, free_pages), [])
            if rows:
                ids = [f"warm-up-row-{i}" for i in range(rows)]
                run([], ids)  # every row's first token: a step of the shape of a decode step
                # their second tokens beside a prompt portion: a row holds one page
                run(prompts(max_tokens - rows, "mixed", free_slots - rows, free_pages - rows), ids)
        finally:
            for rid in list(self.manager.requests):
                self.release(rid)
        torch.cuda.synchronize()
        self.manager.check()
        return ran

    def _copy_to_host(self, out: StepOutput) -> None:
        n = out.ids.shape[0]
        k = self.topk_logprobs
        if not self._host_ring or self._host_ring[0].width < n:
            width = max(n, self.manager.slots.num_slots)
            self._host_ring = [HostResults(width, k) for _ in range(4)]
        host = self._host_ring[self._host_at % len(self._host_ring)]
        self._host_at += 1
        host.event.synchronize()  # whoever used this buffer four steps ago has long read it
        host.ids[:n].copy_(out.ids, non_blocking=True)
        if out.logprobs is not None:
            host.logprobs[:n].copy_(out.logprobs, non_blocking=True)
        if out.topk_ids is not None:
            host.topk_ids[: n * k].copy_(out.topk_ids.reshape(-1), non_blocking=True)
            host.topk_logprobs[: n * k].copy_(out.topk_logprobs.reshape(-1), non_blocking=True)
        host.event.record()
        out.host, out.ready = host, host.event

    def step(self, entries: list[StepEntry]) -> torch.Tensor:
        """Run one batch and return its logits only (nothing is sampled or written to slots)."""
        return self.run(entries).logits
