"""What a mixer asks of the cache, and how the layers' needs are grouped.

The reference keeps one uniform pool `[L, blocks, block_size, Hkv, D]` for all
layers (flow_engine/cache.py:21) and no per-request state. Here every cache
slot (one per layer run that writes a cache) declares its need; slots with the
same paged need share one GROUP: one page pool, one block table per request. A
slot may also (or instead) ask for a fixed-size state per request.
"""
from __future__ import annotations

from dataclasses import dataclass


@dataclass(frozen=True)
class PagedKV:
    """Keys and values of every token (window None) or of the last `window` tokens; with a window, `keep_first` says
    how many of a request's first tokens stay held whatever the window has passed. `chunks`, in place of a window: sizes of
    chunks of positions, counted from a request's start, whose queries see their own chunk only (several readers of one
    cache may have several sizes); tokens are held until every one of these chunks has ended."""
    kv_heads: int
    head_dim: int
    window: int | None = None
    value_dim: int | None = None      # size of a value if it differs from a key's (None: head_dim)
    keep_first: int = 0
    chunks: tuple = ()

    def __post_init__(self):
        object.__setattr__(self, "chunks", tuple(sorted({int(c) for c in self.chunks})))
        if any(c <= 0 for c in self.chunks) or (self.chunks and self.window is not None):
            raise ValueError("chunk sizes must be positive and take the place of a window")
        if self.value_dim == self.head_dim:
            object.__setattr__(self, "value_dim", None)
        if self.kv_heads <= 0 or self.head_dim <= 0 or (self.value_dim is not None and self.value_dim <= 0):
            raise ValueError("kv_heads, head_dim and value_dim must be positive")
        if self.window is not None and self.window <= 0:
            raise ValueError("a window must be positive (None means all keys)")
        if self.keep_first < 0:
            raise ValueError("keep_first cannot be negative")
        if self.window is None:
            object.__setattr__(self, "keep_first", 0)          # (without a window everything is kept anyway)

    @property
    def keeps_all(self):
        """Does a request hold every token's keys and values to its end?"""
        return self.window is None and not self.chunks

    @property
    def span(self):
        """Most positions a query sees, its own included (None: no bound)."""
        return self.window if self.window is not None else max(self.chunks, default=None)

    def first_position(self, position):
        """The first position that a query at POSITION or later can see (kept first tokens aside); POSITION may be an array."""
        if self.window is not None:
            return (position - self.window + 1) * (position >= self.window)
        if not self.chunks:
            return position * 0
        first = position // self.chunks[0] * self.chunks[0]
        for c in self.chunks[1:]:
            other = position // c * c
            first = first * (first <= other) + other * (other < first)
        return first


@dataclass(frozen=True)
class FixedState:
    """State of fixed size per request, e.g. a recurrent mixer's."""
    shape: tuple
    dtype: str = "float32"

    def __post_init__(self):
        object.__setattr__(self, "shape", tuple(int(s) for s in self.shape))
        if any(s <= 0 for s in self.shape):
            raise ValueError("state dimensions must be positive")
        if self.dtype not in ("float32", "bfloat16", "int32"):
            raise ValueError("state dtype must be float32, bfloat16 or int32")


@dataclass(frozen=True)
class CacheNeed:
    """What one cache slot holds: paged keys and values, one fixed-size state, and any number of further
    fixed-size states by name (a layer whose parts each carry something from token to token: a
    recurrence, the last inputs of a convolution)."""
    paged: PagedKV | None = None
    state: FixedState | None = None
    states: tuple = ()                # ((name, FixedState), ...)

    def __post_init__(self):
        object.__setattr__(self, "states", tuple((str(n), s) for n, s in self.states))
        names = [n for n, _ in self.states]
        if len(set(names)) != len(names):
            raise ValueError("two states of one cache slot share a name")

    def merged(self, other):
        """This need and OTHER's together (one cache slot for both); at most one of them may page or hold `state`."""
        if other is None:
            return self
        if (self.paged and other.paged) or (self.state and other.state):
            raise ValueError("two parts of one cache slot both ask for pages, or both for the unnamed state")
        return CacheNeed(self.paged or other.paged, self.state or other.state, self.states + other.states)


@dataclass(frozen=True)
class CacheGroup:
    spec: PagedKV
    slots: tuple          # cache slots stored in this group, in storage order


class CacheLayout:
    """Cache slots of a model, grouped by paged need."""

    def __init__(self, needs):
        self.needs = tuple(needs)
        groups: dict[PagedKV, list[int]] = {}
        for slot, need in enumerate(self.needs):
            if need is not None and need.paged is not None:
                groups.setdefault(need.paged, []).append(slot)
        self.groups = tuple(CacheGroup(spec, tuple(slots)) for spec, slots in groups.items())
        self.slot_group = {}
        for g, group in enumerate(self.groups):
            for i, slot in enumerate(group.slots):
                self.slot_group[slot] = (g, i)
        self.state_slots = tuple(slot for slot, need in enumerate(self.needs)
                                 if need is not None and need.state is not None)
        self.named_state_slots = tuple(slot for slot, need in enumerate(self.needs)
                                       if need is not None and need.states)

    @property
    def shares_prefixes(self):
        """Full pages of a prompt prefix can be reused only if they are all a request holds."""
        return (len(self.groups) == 1 and self.groups[0].spec.keeps_all
                and not self.state_slots and not self.named_state_slots)

    def bytes_per_token(self, element_bytes):
        return sum(len(g.slots) * g.spec.kv_heads * (g.spec.head_dim + (g.spec.value_dim or g.spec.head_dim)) * element_bytes
                   for g in self.groups)
