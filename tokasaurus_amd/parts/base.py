"""What a part is, what a step hands to it, and the registries parts are chosen from.

A model is put together from parts: a mixer (attention here), a feed-forward, norms,
a position encoding, and the arrangement of these in a block.  A part is built from
plain parameters (sizes, constants, the checkpoint names of its tensors); it does
not see a model configuration and does not know which model it is in.  The
reference hard-wires one class per role and swaps classes by subclassing
(tokasaurus/model/llama.py:342-359, tokasaurus/model/qwen.py:11-25); here the
roles are interfaces and the choice is data (``PartSpec``), layer by layer.
"""

from __future__ import annotations

from dataclasses import dataclass, field
from typing import Any, Callable

import torch


# --------------------------------------------------------------------------
# descriptions of tensors, caches and state that a part needs
# --------------------------------------------------------------------------

MATRIX = "matrix"  # a projection or table of floats: engine dtype, N(0, 0.02) when random
BIAS = "bias"  # a projection's bias vector: engine dtype, N(0, 0.02) when random
NORM_WEIGHT = "norm_weight"  # a norm's scale vector: 1 + N(0, 0.01) when random
NORM_OFFSET = "norm_offset"  # a norm's scale stored around zero (the norm multiplies by 1 + w): N(0, 0.01) when random
VECTOR = "vector"  # a learned vector of another role (a sink, a rate, a step's bias): N(0, 0.5) when random
CONV = "conv"  # the taps of short convolutions, [channels, taps]: N(0, 0.5) when random
SMALL_VECTOR = "small_vector"  # a learned vector that nudges (a router's correction): N(0, 0.01) when random
UNIT_INTERVAL = "unit_interval"  # a learned bound or rate between 0 and 1: uniform on (0.05, 0.95) when random
AVERAGE_WEIGHT = "average_weight"  # the weights of an average over n things, [n]: 1 / n + N(0, 0.1 / n) when random
INT_TABLE = "int_table"  # integer table: kept as int32


@dataclass(frozen=True)
class TensorSpec:
    """One tensor a part reads from the checkpoint, by its name there."""

    name: str
    shape: tuple[int, ...]
    kind: str = MATRIX
    below: int = 0  # integer tables: every row holds different numbers from 0 to below - 1 (0: any numbers)


@dataclass(frozen=True)
class CacheNeed:
    """Keys and values a mixer keeps per token.  Layers whose needs are equal
    share a cache group (one page pool, one block table per request)."""

    num_kv_heads: int
    head_dim: int
    window: int = 0  # 0: every key is kept; > 0: only the last `window` positions are read
    value_dim: int = 0  # size of a value head where it differs from a key head's (0: the same)
    section: int = 0  # > 0 (without a window): a query reads only keys of its own section of this many positions

    def __post_init__(self):
        if self.window and self.section:
            raise ValueError("keys are read within a window or within sections, not both")

    @property
    def value_size(self) -> int:
        return self.value_dim or self.head_dim

    @property
    def keeps_all(self) -> bool:
        """Whether a request's keys stay until it ends (else pages go back while it runs)."""
        return not self.window and not self.section

    def first_read(self, new_len: int) -> int:
        """The first position that a query at position ``new_len`` or later can read."""
        if self.section:
            return new_len // self.section * self.section
        return max(0, new_len - self.window + 1) if self.window else 0


@dataclass(frozen=True)
class StateNeed:
    """Per-request state of fixed size (for mixers that carry a recurrent state)."""

    shape: tuple[int, ...]
    dtype: torch.dtype = torch.float32


@dataclass(frozen=True)
class PartSpec:
    """The choice of a part: its registered kind and its constructor parameters."""

    kind: str
    params: dict[str, Any] = field(default_factory=dict)

    def __hash__(self) -> int:  # params may hold dicts; specs are compared by value
        return hash((self.kind, repr(sorted(self.params.items(), key=lambda kv: kv[0]))))


# --------------------------------------------------------------------------
# what a step hands to the parts
# --------------------------------------------------------------------------


@dataclass
class CacheView:
    """The pages of one cache-owning run entry, and its group's block table for this step."""

    keys: torch.Tensor  # [pages, nkv, d / 8, P, 8]
    values: torch.Tensor  # [pages, nkv, P / 4, d, 4]
    block_table: torch.Tensor  # [requests, width] int32, -1 where no page is held
    page_size: int
    writable: bool = True  # False when the entry reads another entry's cache


@dataclass
class StepContext:
    """One batch: tokens of several requests, laid out request by request.

    Request r owns tokens q_start[r] .. q_start[r+1]-1 at positions
    kv_len[r] - q_len[r] .. kv_len[r] - 1.  Host copies (lists) are kept beside
    the device arrays for parts that plan on the host.
    """

    num_tokens: int
    num_requests: int
    dtype: torch.dtype
    device: torch.device
    token_ids: torch.Tensor  # [N] int32; < 0: token is read from last_token[-id-1]
    positions: torch.Tensor  # [N] int32
    token_req: torch.Tensor  # [N] int32, index of each token's request in this batch
    q_start: torch.Tensor  # [R+1] int32
    kv_len: torch.Tensor  # [R] int32, keys of the request after this step's append
    slots: torch.Tensor  # [R] int32, the request's state slot
    host_q_start: list[int]
    host_kv_len: list[int]
    host_slots: list[int]
    last_token: torch.Tensor | None = None  # [slots] int32, written by the sampler
    embedding_state: torch.Tensor | None = None  # [slots + 1, ...]: what the embedding keeps per request, if anything
    max_q_len: int = 0
    max_kv_len: int = 0
    extras: dict[str, Any] = field(default_factory=dict)  # planning data of kernels, by name


# --------------------------------------------------------------------------
# a norm that has not been applied yet
# --------------------------------------------------------------------------


@dataclass
class Prepared:
    """What the product in front of a norm has already done for it, and the norm it did it
    for: either ``data``, the kernels' own record (``kernels.ops.Prenorm``: the rows times
    the norm's weight and partial sums of their squares, which the next product folds in),
    or ``normed``, the normed rows themselves (made in the pass that added the residual; for a
    block that begins with two norms of the same stream, ``norm`` is its pair of norms and
    ``normed`` the pair of their rows)."""

    data: Any
    norm: "Norm"
    normed: "torch.Tensor | tuple | None" = None


@dataclass
class Normed:
    """Rows that still have to pass ``norm``.  A part that says ``fuses_norm`` gets this
    instead of normed rows and may fold the norm into its first product (a product
    takes ``prepared`` when it is there and was made for this very norm); any part may
    call ``materialize()`` and go on with plain rows."""

    x: torch.Tensor
    norm: "Norm"
    prepared: Prepared | None = None

    def usable(self) -> Prepared | None:
        """The record a product can fold in, if it was made for this very norm."""
        p = self.prepared
        ok = p is not None and p.data is not None and p.norm is self.norm and getattr(self.norm, "fusable_rms", False)
        return p if ok else None

    def materialize(self) -> torch.Tensor:
        p = self.prepared
        if p is not None and p.normed is not None and p.norm is self.norm:
            return p.normed
        return self.norm.forward(self.x)


@dataclass
class NormedSum:
    """``mult * (rms_norm(a) * wa + rms_norm(b) * wb)`` of two 32-bit branches, not computed yet: whoever adds it to a stream
    norms, sums and adds in one pass.  ``rows()`` computes it alone."""

    a: torch.Tensor
    wa: torch.Tensor
    b: torch.Tensor
    wb: torch.Tensor
    eps: float
    mult: float

    def rows(self) -> torch.Tensor:
        from tokasaurus_amd.kernels import ops

        return ops.post_norm_residual(None, self.a, self.wa, self.eps, in_place=False, second=(self.b, self.wb), mult=self.mult)[0]


# --------------------------------------------------------------------------
# interfaces
# --------------------------------------------------------------------------


class Part:
    """Common to every part: which tensors it reads, and receiving them."""

    def tensor_specs(self) -> list[TensorSpec]:
        return []

    def load(self, tensors: dict[str, torch.Tensor], placer: Any) -> None:
        """Take this part's tensors (host tensors by checkpoint name, already
        checked against ``tensor_specs``) and put them on the device through
        ``placer`` (``parts.linear.Placer``: engine dtype, device, one buffer per
        tensor) in the layout the part's kernels want."""

    def children(self) -> list["Part"]:
        return []


class Norm(Part):
    def forward(self, x: torch.Tensor) -> torch.Tensor:
        raise NotImplementedError


class PositionEncoding(Part):
    """Prepared once (tables on the device), then handed to the mixers that use it."""

    def prepare(self, device: torch.device) -> None:
        raise NotImplementedError


class Mixer(Part):
    """Mixes information across the tokens of a request.

    ``forward`` gets the normed hidden states ``h`` [N, H], the residual stream
    ``residual`` ([N, H], or [len(rows), H] when ``rows`` is given) and returns
    the new residual stream ``residual + mix(h)``.  When ``rows`` (int32 indices)
    is given only those tokens' outputs are needed (the last block of a step
    keeps only the rows whose logits are wanted), but every token must still
    update the cache or state.

    A mixer (or feed-forward) with ``fuses_norm = True`` takes ``h`` as a ``Normed``
    and a keyword ``emit_norm`` (the norm that will be applied to its result, or
    None) and may return ``(stream, Prepared)`` instead of the stream alone.

    A mixer with ``gives_normed_sum = True`` also has ``normed_sum(h, ctx, cache, state, rows)``, which returns
    what ``mix`` returns as a ``NormedSum``: for a block that can add it to the stream in one pass.
    """

    fuses_norm = False
    gives_normed_sum = False

    def cache_need(self) -> CacheNeed | None:
        return None

    def state_need(self) -> StateNeed | None:
        return None

    def check_cache(self, page_size: int, dtype: torch.dtype) -> None:
        """Called before the cache is made for this mixer: raise if its kernels do not take
        pages of this size and storage type."""

    def forward(
        self,
        h: torch.Tensor,
        residual: torch.Tensor,
        ctx: StepContext,
        cache: CacheView | None,
        state: torch.Tensor | None,
        rows: torch.Tensor | None,
    ) -> torch.Tensor:
        raise NotImplementedError

    def mix(
        self,
        h: torch.Tensor,
        ctx: StepContext,
        cache: CacheView | None,
        state: torch.Tensor | None,
        rows: torch.Tensor | None,
        out_f32: bool = False,
    ) -> torch.Tensor:
        """The mixer's own output ``mix(h)`` with nothing added (for ``rows`` only when given;
        ``out_f32``: the last product's 32-bit sums leave unrounded): what a block needs that
        combines its branches itself.  A mixer need not have it; blocks that call it say so."""
        raise NotImplementedError(f"{type(self).__name__} gives its output only added to the stream")


class FeedForward(Part):
    """Token-wise transformation: returns ``residual + ff(h)`` (see ``Mixer`` for ``fuses_norm``).
    One that reads the tokens' ids beside their rows says ``reads_tokens = True`` and takes two more keywords,
    ``ctx`` (the step) and ``rows`` (the step's rows that ``h`` holds, None: all of them); blocks that hand
    them over say so."""

    fuses_norm = False
    reads_tokens = False

    def forward(self, h: torch.Tensor, residual: torch.Tensor) -> torch.Tensor:
        raise NotImplementedError


class Embedding(Part):
    """From the step's token ids to the first residual stream [N, H] in the engine dtype.
    ``ctx.token_ids`` holds ids, or -(slot + 1) for a token to be read from ``ctx.last_token``."""

    def state_need(self) -> "StateNeed | None":
        """Per-request state of fixed size that the embedding keeps in the request's slot (an
        embedding that reads the token before, say); it gets it as ``ctx.embedding_state``."""
        return None

    def forward(self, ctx: StepContext) -> torch.Tensor:
        """The stream, or (stream, ``Prepared``) when it has also made the rows of the first block's entry norm."""
        raise NotImplementedError


class Head(Part):
    """From the last residual stream (the wanted rows only) to logits [rows, vocab] in 32-bit.
    ``entry_norm()`` is the norm it applies to its input first (or None): the last block may
    prepare it, and hands what it prepared to ``forward`` as ``prepared``.  A head that says
    ``takes_out = True`` also takes a keyword ``out``: a contiguous 32-bit buffer [rows, vocab] to
    write the logits to and return (recorded steps share one such buffer); for any other head the
    model copies."""

    takes_out = False

    def entry_norm(self) -> "Norm | None":
        return None

    def forward(self, x: torch.Tensor, prepared: "Prepared | None" = None) -> torch.Tensor:
        raise NotImplementedError


class Connector(Part):
    """What a model does to its residual stream between two blocks, outside any block: it gets
    the stream ``x`` and the embedding's output ``x0`` of the same rows and returns the new
    stream (a new tensor: ``x0`` is read again later).  A run entry names the connector that
    runs before it (``models.spec.RunEntry.before``).  A connector that reads the stream alone says
    ``updates_stream = True`` and has ``update(x, pending, next_norm)`` instead: it changes ``x`` in place, adds
    the branch that the block in front has handed over unsummed (``parts.block.PendingSum`` or None) in the same pass,
    and may return (stream, ``Prepared``) for the norm that reads it.  One that does so and reads the embedding's output too
    says ``reads_embedding = True`` and gets it as the keyword ``x0``."""

    updates_stream = False
    reads_embedding = False

    def forward(self, x: torch.Tensor, x0: torch.Tensor) -> torch.Tensor:
        raise NotImplementedError


class Block(Part):
    """The arrangement of norms, a mixer and a feed-forward around the residual stream.

    A block with ``fuses_norm = True`` takes the keywords ``prepared`` (what the block
    before has done for this block's first norm) and ``next_norm`` (the norm the model
    applies to this block's result) and may return ``(stream, Prepared)``;
    ``entry_norm()`` is the norm it applies to its input first.

    The block, not its mixer, is asked what it keeps per request: ``cache_needs()`` and
    ``state_needs()`` list the caches and the states of everything inside it.  A block with one
    mixer (the default implementations below) has at most one of each and gets them as
    ``cache`` and ``state``; a block that lists several (two mixers side by side, say) gets
    lists in the order it named them."""

    mixer: Mixer
    fuses_norm = False

    def entry_norm(self) -> "Norm | None":
        return None

    def cache_needs(self) -> "list[CacheNeed]":
        need = self.mixer.cache_need()
        return [] if need is None else [need]

    def state_needs(self) -> "list[StateNeed]":
        need = self.mixer.state_need()
        return [] if need is None else [need]

    def check_cache(self, page_size: int, dtype: torch.dtype) -> None:
        """Called before the cache is made: raise if a kernel in here does not take pages of
        this size and storage type."""
        self.mixer.check_cache(page_size, dtype)

    def forward(
        self,
        x: torch.Tensor,
        ctx: StepContext,
        cache: CacheView | None,
        state: torch.Tensor | None,
        rows: torch.Tensor | None,
    ) -> torch.Tensor:
        raise NotImplementedError


# --------------------------------------------------------------------------
# registries
# --------------------------------------------------------------------------


class Registry:
    """Name -> constructor for one role.  Registering a name twice is an error
    unless ``replace=True`` (tests register toy parts)."""

    def __init__(self, role: str):
        self.role = role
        self._entries: dict[str, Callable[..., Any]] = {}

    def register(self, name: str, replace: bool = False):
        def deco(cls):
            if name in self._entries and not replace:
                raise KeyError(f"{self.role} {name!r} is already registered")
            self._entries[name] = cls
            return cls

        return deco

    def build(self, spec: PartSpec, **extra: Any):
        if spec.kind not in self._entries:
            raise KeyError(
                f"unknown {self.role} {spec.kind!r}; registered: {sorted(self._entries)}"
            )
        return self._entries[spec.kind](**spec.params, **extra)

    def names(self) -> list[str]:
        return sorted(self._entries)

    def __contains__(self, name: str) -> bool:
        return name in self._entries


NORMS = Registry("norm")
POSITION_ENCODINGS = Registry("position encoding")
MIXERS = Registry("mixer")
FEED_FORWARDS = Registry("feed-forward")
BLOCKS = Registry("block arrangement")
CONNECTORS = Registry("connector")
EMBEDDINGS = Registry("embedding")
HEADS = Registry("head")
