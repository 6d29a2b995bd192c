"""The cache manager: which pages and which slot each live request holds.

Layers (run entries) whose caches have equal needs form a *group*: one pool of
page ids and, per request, one block table that every layer of the group uses
(the reference has a single such group: one table per sequence shared by all
layers, tokasaurus/manager/types.py:46, tokasaurus/model/llama.py:675-691).
A group whose layers read only a window (or a section) of keys gives pages back as soon as
that has passed them; a full group gives pages back when the request ends.
Token ``pos`` of a request lives in page ``table[pos // P]`` at offset ``pos % P``
(tokasaurus/manager/input_building.py:138-148).

This class is host-side bookkeeping only; the tensors live in ``CacheStorage``.
"""

from __future__ import annotations

from dataclasses import dataclass, field

import numpy as np

from tokasaurus_amd.cache.pages import NoSpaceException, PagePool, SlotAllocator
from tokasaurus_amd.parts.base import CacheNeed

RELEASED = -1  # table entry of a page the window has passed


@dataclass(frozen=True)
class CacheGroup:
    need: CacheNeed
    entries: tuple[int, ...]  # run entries that own storage in this group, in run order


def plan_groups(needs: list, cache_of: list[int | None]) -> tuple[list[CacheGroup], list]:
    """Group the caches of the run entries by need.

    ``needs`` holds for every run entry None, one ``CacheNeed`` or a list of several (a block
    with more than one mixer that keeps keys).  Returns the groups and, for every run entry
    in the form it came, ``(group, index within the group's storage)`` of each cache it uses
    (its own, or the one it reads).  A group's ``entries`` name its caches' owners, one item a
    cache (an entry with two equal needs appears twice)."""
    as_list = [[] if n is None else (list(n) if isinstance(n, (list, tuple)) else [n]) for n in needs]
    groups: list[CacheGroup] = []
    members: dict[CacheNeed, list[int]] = {}
    index: dict[tuple[int, int], tuple[CacheNeed, int]] = {}  # (entry, which of its caches) -> (need, place in the group)
    for i, mine in enumerate(as_list):
        if cache_of[i] is None:
            for j, need in enumerate(mine):
                index[(i, j)] = (need, len(members.setdefault(need, [])))
                members[need].append(i)
    for need, entries in members.items():
        groups.append(CacheGroup(need, tuple(entries)))
    group_of = {grp.need: gi for gi, grp in enumerate(groups)}
    where: list = []
    for i, mine in enumerate(as_list):
        owner = i if cache_of[i] is None else cache_of[i]
        theirs = as_list[owner]
        if mine and len(theirs) != len(mine):
            raise ValueError(f"run entry {i} reads the cache of entry {owner}, which has "
                             + ("none" if not theirs else f"{len(theirs)} caches, not {len(mine)}"))
        places = []
        for j, need in enumerate(mine):
            owner_need = theirs[j]
            if (owner_need.num_kv_heads, owner_need.head_dim, owner_need.value_size) != (need.num_kv_heads, need.head_dim, need.value_size):
                raise ValueError(f"run entry {i} cannot read the cache of entry {owner}: head layout differs")
            if need.section != owner_need.section and not owner_need.keeps_all:
                raise ValueError(f"run entry {i} reads other keys than entry {owner} keeps")
            if owner_need.window and (not need.window or need.window > owner_need.window):
                raise ValueError(f"run entry {i} reads further back than entry {owner} keeps keys")
            places.append((group_of[owner_need], index[(owner, j)][1]))
        form = needs[i]
        where.append(None if form is None else (places if isinstance(form, (list, tuple)) else places[0]))
    return groups, where


@dataclass
class RequestCache:
    request_id: str
    slot: int
    tables: list[list[int]]  # per group: page of each logical block, RELEASED once passed
    num_tokens: int = 0  # tokens whose keys are in the cache
    reserved_tokens: int = 0  # tokens the tables have room for
    first_held: list[int] = field(default_factory=list)  # per group: first block not released


class CacheManager:
    def __init__(
        self,
        groups: list[CacheGroup],
        num_pages: int | list[int],
        page_size: int,
        max_slots: int,
        max_blocks_per_request: int | None = None,
    ):
        if page_size <= 0:
            raise ValueError("page_size must be positive")
        self.groups = groups
        self.page_size = page_size
        counts = num_pages if isinstance(num_pages, list) else [num_pages] * len(groups)
        self.pools = [PagePool(n) for n in counts]
        self.slots = SlotAllocator(max_slots)
        self.requests: dict[str, RequestCache] = {}
        # slots handed out since the owner of the state tensors last asked: a request must
        # not inherit the state that the slot's last holder left
        self.fresh_slots: list[int] = []
        # Per group, the block tables once more as one array indexed by slot, kept
        # up to date as pages come and go: a step whose shape is fixed (a recorded
        # decode step) gathers its rows from it instead of walking lists.  Row
        # `max_slots` belongs to no request: all its entries name the null page
        # (the page after the pool's last), where padding rows of a step write.
        self.max_blocks_per_request = max_blocks_per_request
        self.slot_tables: list[np.ndarray] | None = None
        if max_blocks_per_request is not None:
            self.slot_tables = [
                np.full((max_slots + 1, max_blocks_per_request), n, dtype=np.int32) for n in counts
            ]

    # ---- arithmetic
    def blocks_for(self, num_tokens: int) -> int:
        return -(-num_tokens // self.page_size)

    def pages_needed(self, request_id: str | None, new_len: int) -> list[int]:
        """Pages each group must still give for the request to hold ``new_len`` tokens."""
        have = self.requests[request_id].tables if request_id in self.requests else [[] for _ in self.groups]
        return [max(0, self.blocks_for(new_len) - len(t)) for t in have]

    def can_hold(self, request_id: str | None, new_len: int) -> bool:
        return all(n <= pool.num_free for n, pool in zip(self.pages_needed(request_id, new_len), self.pools))

    def num_free_pages(self) -> list[int]:
        return [p.num_free for p in self.pools]

    # ---- life of a request
    def admit(self, request_id: str) -> RequestCache:
        if request_id in self.requests:
            raise ValueError(f"request {request_id!r} is already live")
        slot = self.slots.allocate()
        self.fresh_slots.append(slot)
        rc = RequestCache(request_id, slot, [[] for _ in self.groups], first_held=[0] * len(self.groups))
        self.requests[request_id] = rc
        return rc

    def take_fresh_slots(self) -> list[int]:
        """The slots given to requests since the last call (each once): whoever owns
        per-slot state clears it for them before their first step."""
        out, self.fresh_slots = self.fresh_slots, []
        return out

    def reserve(self, request_id: str, new_len: int) -> None:
        """Make room for the request to hold ``new_len`` tokens in every group,
        or raise NoSpaceException with nothing taken."""
        rc = self.requests[request_id]
        if new_len <= rc.reserved_tokens:
            return
        need = self.pages_needed(request_id, new_len)
        for n, pool in zip(need, self.pools):
            if n > pool.num_free:
                raise NoSpaceException(
                    f"request {request_id!r} needs {need} more pages for {new_len} tokens, "
                    f"free: {self.num_free_pages()}"
                )
        if self.max_blocks_per_request is not None and self.blocks_for(new_len) > self.max_blocks_per_request:
            raise ValueError(
                f"request {request_id!r} would hold {new_len} tokens, more than the "
                f"{self.max_blocks_per_request * self.page_size} a request may hold"
            )
        for g, (table, n, pool) in enumerate(zip(rc.tables, need, self.pools)):
            new = pool.allocate(n)
            if self.slot_tables is not None and new:
                self.slot_tables[g][rc.slot, len(table) : len(table) + len(new)] = new
            table.extend(new)
        rc.reserved_tokens = self.blocks_for(new_len) * self.page_size

    def advance(self, request_id: str, new_len: int) -> None:
        """The request now holds ``new_len`` tokens: pages of windowed groups
        that no later token can read go back to their pool."""
        rc = self.requests[request_id]
        if new_len > rc.reserved_tokens:
            raise ValueError(f"request {request_id!r}: {new_len} tokens but room for {rc.reserved_tokens}")
        if new_len < rc.num_tokens:
            raise ValueError(f"request {request_id!r} cannot shrink")
        rc.num_tokens = new_len
        P = self.page_size
        for g, grp in enumerate(self.groups):
            if grp.need.keeps_all:
                continue
            # the next query sits at position >= new_len
            first_needed = grp.need.first_read(new_len) // P
            table = rc.tables[g]
            gone = []
            for b in range(rc.first_held[g], min(first_needed, len(table))):
                if table[b] != RELEASED:
                    gone.append(table[b])
                    table[b] = RELEASED
                    if self.slot_tables is not None:
                        self.slot_tables[g][rc.slot, b] = self.pools[g].num_pages
            if gone:
                self.pools[g].free(gone)
            rc.first_held[g] = max(rc.first_held[g], min(first_needed, len(table)))

    def release(self, request_id: str) -> None:
        """The request is over: every page and the slot go back."""
        rc = self.requests.pop(request_id)
        for table, pool in zip(rc.tables, self.pools):
            pool.free([p for p in table if p != RELEASED])
        if self.slot_tables is not None:
            for g, pool in enumerate(self.pools):
                self.slot_tables[g][rc.slot, :] = pool.num_pages
        self.slots.free(rc.slot)

    # ---- invariants (the reference's sanity_checks, allocator.py:158-194, without the tree)
    def check(self) -> None:
        for g, pool in enumerate(self.pools):
            pool.check()
            owned: list[int] = []
            for rc in self.requests.values():
                owned.extend(p for p in rc.tables[g] if p != RELEASED)
            assert len(owned) == len(set(owned)), f"group {g}: a page is held by two requests"
            assert set(owned) == pool.held_pages(), f"group {g}: tables and pool disagree"
        self.slots.check()
        slots = [rc.slot for rc in self.requests.values()]
        assert len(slots) == len(set(slots)), "a slot is held by two requests"
        for rc in self.requests.values():
            assert rc.num_tokens <= rc.reserved_tokens
            if self.slot_tables is not None:
                for g, table in enumerate(rc.tables):
                    null = self.pools[g].num_pages
                    row = self.slot_tables[g][rc.slot]
                    want = [null if p == RELEASED else p for p in table]
                    assert row[: len(table)].tolist() == want and (row[len(table) :] == null).all(), (
                        f"group {g}: the slot table of request {rc.request_id!r} differs from its block table"
                    )
