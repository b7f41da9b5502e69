"""Which cache each scheduled layer call has, and how calls with equal needs share a pool.

Calls whose mixers need the same pages (same KV heads, key and value widths, window, chunk and kept first keys) form a *group*:
one page pool, one block table per request, one device tensor holding every member's keys and
values.  A model whose layers differ (all keys in some, a window in others) has several
groups, each with pages of its own, so a windowed group can give pages back while the request
runs.  Calls that need fixed-size state get a state tensor indexed by the request's slot.
The reference has one pool with the same block ids for every layer
(src/turboserve/engine/core/kv_cache.py:372-400).
"""

from __future__ import annotations

import math
from collections.abc import Sequence
from dataclasses import dataclass

from turboserve_amd.parts.base import CacheNeed, FixedState, PagedKV, SharedKV, shares_pages


@dataclass(frozen=True)
class PageGroup:
    num_kv_heads: int
    head_dim: int
    window: int | None
    entries: tuple[int, ...]  # schedule entries that own a unit in this group (one per unit: an entry may own several)
    value_dim: int | None = None
    chunk: int | None = None  # a token reads no key below its own chunk of this many positions
    keep_first: int = 0  # the first keys of a request that are read behind a window too

    @property
    def value_width(self) -> int:
        return self.head_dim if self.value_dim is None else self.value_dim

    def elements_per_token(self) -> int:
        """Key and value elements one token takes over all members."""
        return len(self.entries) * self.num_kv_heads * (self.head_dim + self.value_width)


@dataclass(frozen=True)
class CacheLayout:
    groups: tuple[PageGroup, ...]
    state_entries: tuple[tuple[int, FixedState], ...]
    #: per schedule entry: ("pages", group, unit) | ("shared", group, unit) | ("state", index) | ("reads", entry) | None,
    #: or, for an entry whose mixer has several needs, a tuple of such units in the order of the needs
    entry_units: tuple[tuple | None, ...]

    @classmethod
    def from_needs(cls, needs: Sequence[CacheNeed], reads: Sequence[int | None]) -> "CacheLayout":
        """``needs[i]``: what schedule entry ``i`` owns (one need, or a tuple of needs);
        ``reads[i]``: the earlier entry whose cache it reads instead, or whose pages a ``SharedKV`` among
        its needs means."""
        keys: list[tuple] = []
        members: list[list[int]] = []
        states: list[tuple[int, FixedState]] = []
        units: list[tuple | None] = []

        def shared_pages(entry: int, need: SharedKV) -> tuple[int, int]:
            """The group and member of the pages that the entry named by ``reads`` owns, if they are what the reader takes them for."""
            source = reads[entry]
            if source is None:
                raise ValueError(f"schedule entry {entry} asks for another entry's pages and names none")
            owned = units[source] if units[source] is not None and units[source] and not isinstance(units[source][0], str) else (units[source],)
            pages = [unit for unit in owned if unit is not None and unit[0] == "pages"]
            if len(pages) != 1:
                raise ValueError(f"schedule entry {entry} asks for the pages of entry {source}, which owns {len(pages)} sets of them")
            _, group, member = pages[0]
            heads, dim, window, value_width, chunk, _ = keys[group]
            if (heads, dim, value_width) != (need.num_kv_heads, need.head_dim, need.value_width):
                raise ValueError(f"schedule entry {entry} reads {need.num_kv_heads} heads of {need.head_dim}/{need.value_width} where entry "
                                 f"{source} keeps {heads} of {dim}/{value_width}")
            if chunk is not None or (window is not None and (need.window is None or need.window > window)):
                raise ValueError(f"schedule entry {entry} reads keys that entry {source} does not keep")
            return group, member

        def unit_of(entry: int, need) -> tuple | None:
            if isinstance(need, PagedKV):
                key = (need.num_kv_heads, need.head_dim, need.window, need.value_width, need.chunk, need.keep_first if need.window is not None else 0)
                if key not in keys:
                    keys.append(key)
                    members.append([])
                group = keys.index(key)
                members[group].append(entry)
                return ("pages", group, len(members[group]) - 1)
            if isinstance(need, FixedState):
                states.append((entry, need))
                return ("state", len(states) - 1)
            if isinstance(need, SharedKV):
                return ("shared", *shared_pages(entry, need))
            if need is None:
                return None
            raise TypeError(f"schedule entry {entry} declares an unknown cache need {need!r}")

        for entry, need in enumerate(needs):
            if reads[entry] is not None and not shares_pages(need):
                units.append(("reads", reads[entry]))
            elif isinstance(need, (tuple, list)):
                units.append(tuple(unit_of(entry, one) for one in need))
            else:
                units.append(unit_of(entry, need))
        groups = tuple(PageGroup(k[0], k[1], k[2], tuple(m), None if k[3] == k[1] else k[3], k[4], k[5]) for k, m in zip(keys, members))
        return cls(groups, tuple(states), tuple(units))

    @classmethod
    def from_model(cls, model) -> "CacheLayout":
        needs = model.cache_needs()
        reads: list[int | None] = [call.cache_of for call in model.plan.schedule]
        return cls.from_needs(needs, reads + [None] * (len(needs) - len(reads)))  # (an embedding with state has an entry behind the calls)

    def windows(self) -> list[int | None]:
        return [group.window for group in self.groups]

    def chunks(self) -> list[int | None]:
        return [group.chunk for group in self.groups]

    def kept(self) -> list[int]:
        return [group.keep_first for group in self.groups]

    def bytes_per_page(self, page_size: int, itemsize: int) -> list[int]:
        """Bytes one page of each group takes (keys and values of all members); for one group
        of all layers this is the reference's ``bytes_per_block`` (kv_cache.py:481-494)."""
        return [group.elements_per_token() * page_size * itemsize for group in self.groups]

    def bytes_per_token(self, itemsize: int) -> int:
        return sum(group.elements_per_token() for group in self.groups) * itemsize

    def state_bytes_per_slot(self) -> int:
        """Bytes a request's slot takes in the state tensors of all entries."""
        return sum(math.prod(need.shape) * need.dtype.itemsize for _, need in self.state_entries)
