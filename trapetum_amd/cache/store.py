"""The cache's device storage.

Every run of a layer (a schedule entry) that keeps something between steps
declares what: tensors per token (of all tokens, or of a window of them), or a
state of fixed size.  Entries with the same needs form a group with storage of
its own:

  per token    one pool per named tensor; a tensor of shape (*lead, d) per token
               lives in a pool [entries, pages, *lead, page_size, d] (a page's rows
               stand before the last dimension, so that a row of d elements is
               contiguous); a sequence's rows are found through its page list.  A
               window group keeps a ring: position p lives in ring row p % rows_cap.
               (A window that keeps a sequence's first tokens as well has whole pages of
               `pinned` rows for them in front of the ring: positions below `pinned` stay
               in their rows, the others take the rows behind them in turn.)
               (Attention declares keys and values, each (kv_heads, head_dim); a
               mixer that keeps one tensor per token declares one.)
  state        [entries, slots, *shape], zeroed when a slot is taken.

Beyond what sequences can take, every pool has one spare page and every state one
spare slot (`ModelCache.spare_slot`): a row of a step that stands for no sequence
(padding of a captured decode graph to its batch size) writes and reads there.

The reference allocates cache_k / cache_v [max_seq, kv_heads * head_dim] per
layer for its one sequence, K stored after RoPE (runtime/src/lib.rs:4475,
:4488-4490), and models no window (:4455).
"""
import dataclasses
from typing import Optional

import numpy as np
import torch

from .slots import CacheError, GroupPages, SlotBook


@dataclasses.dataclass(frozen=True)
class TokenSpec:
    """What a mixer keeps of every token: named tensors, each of a fixed shape, in the engine's activation dtype."""
    tensors: tuple                      # ((name, shape), ...): hashable, in the mixer's order
    window: Optional[int] = None        # None: every token is kept
    every: int = 1                      # one row per `every` tokens: row b belongs to the positions b * every .. b * every + every - 1
                                        # and exists once the last of them does (a summary of a block of tokens)
    keep_first: int = 0                 # beside the window, the first `keep_first` tokens of a sequence are kept for good

    @staticmethod
    def of(window=None, every=1, keep_first=0, **tensors):
        """TokenSpec.of(window, k=(kv_heads, head_dim), v=(kv_heads, head_dim))"""
        for name, shape in tensors.items():
            if not shape or any(int(n) <= 0 for n in shape):
                raise CacheError(f"per-token tensor '{name}' needs a shape of positive sizes, found {shape!r}")
        if int(every) < 1 or (int(every) > 1 and window is not None):
            raise CacheError(f"a row per {every} tokens: the number must be positive, and such rows are kept of all tokens, not of a window")
        if int(keep_first) < 0 or (int(keep_first) > 0 and window is None):
            raise CacheError(f"{keep_first} first tokens are kept beside a window: the number must not be negative, and there must be a window")
        return TokenSpec(tuple((name, tuple(int(n) for n in shape)) for name, shape in tensors.items()), window, int(every), int(keep_first))

    def shape_of(self, name):
        for n, shape in self.tensors:
            if n == name:
                return shape
        raise CacheError(f"the cache keeps no per-token tensor '{name}' here (it keeps {[n for n, _ in self.tensors]})")


@dataclasses.dataclass(frozen=True)
class StateSpec:
    shape: tuple
    dtype: str = "float32"              # "float32" or "activation" (the engine's activation dtype)


class CacheSite:
    """What one schedule entry sees of the cache."""

    def __init__(self, spec, group_index, index_in_group, group):
        self.spec = spec
        self.group_index = group_index
        self.index_in_group = index_in_group
        self._group = group

    @property
    def per_token(self):
        return isinstance(self.spec, TokenSpec)

    def tensor(self, name):
        """The pool of one of the per-token tensors the entry declared: [pages, *lead, page_size, d]."""
        self.spec.shape_of(name)
        return self._group.pools[name][self.index_in_group]

    @property
    def rows_cap(self):
        return self._group.pages.rows_cap

    @property
    def pinned(self):
        """Rows in front of the ring that keep a sequence's first tokens (0 without a ring)."""
        return self._group.pages.pinned

    @property
    def state(self):
        return self._group.tensor[self.index_in_group]


class _TokenGroup:
    def __init__(self, spec, entries, n_pages, max_slots, page_size, max_context, dtype, device, name):
        self.spec = spec
        self.entries = entries
        rows_cap, pinned = None, 0
        if spec.window is not None and spec.window < max_context:
            pinned = -(-spec.keep_first // page_size) * page_size            # whole pages, so that a page is of one kind
            rows_cap = pinned + -(-spec.window // page_size) * page_size
            n_pages = min(n_pages, max_slots * (rows_cap // page_size))      # a ring never grows beyond its rows
        if spec.every > 1:                                                   # whole pages of rows, and a last page per sequence
            n_pages = min(n_pages, -(-n_pages // spec.every) + max_slots)
        self.pages = GroupPages(n_pages, page_size, rows_cap, name, every=spec.every, pinned=pinned)
        self.spare_page = n_pages                                          # the pool's last page, never handed out
        self.pools = {}
        for tname, shape in spec.tensors:
            self.pools[tname] = torch.zeros((len(entries), n_pages + 1) + shape[:-1] + (page_size, shape[-1]), dtype=dtype, device=device)
        self.max_pages_per_seq = self.pages.max_pages(max_context)


class _StateGroup:
    def __init__(self, spec, entries, max_slots, dtype, device):
        self.spec = spec
        self.entries = entries
        dt = torch.float32 if spec.dtype == "float32" else dtype
        self.tensor = torch.zeros((len(entries), max_slots + 1) + tuple(spec.shape), dtype=dt, device=device)


class ModelCache:
    """Slots, pages and storage for one model instance.

    entry_specs: for every schedule entry a TokenSpec, a StateSpec or None.
    max_tokens:  tokens that live sequences may hold together, each rounded up to a page.
    max_context: longest single sequence.
    """

    def __init__(self, entry_specs, max_tokens, max_context, max_slots, page_size, dtype, device, entry_states=None, entry_tokens=None):
        """entry_states: for every schedule entry, {name: StateSpec} of states it keeps beside its mixer's cache (what a
        block's own operations carry from step to step); a run that reads another run's cache still has its own.
        entry_tokens: for every schedule entry, {name: TokenSpec} of further paged tensors it keeps by name (rows at
        another rate than its mixer's cache: one per block of tokens)."""
        if page_size <= 0 or page_size % 16:
            raise CacheError(f"page size {page_size} must be a positive multiple of 16")
        self.page_size = page_size
        self.max_context = max_context
        self.max_tokens = max_tokens
        self.max_slots = max_slots
        self.spare_slot = max_slots           # a slot no sequence takes: see the module's text
        n_pages = max(1, -(-max_tokens // page_size))
        self.token_groups, self.state_groups = [], []
        self._site_of = {}
        keyed = {}
        for entry, spec in enumerate(entry_specs):
            if spec is not None:
                keyed.setdefault(spec, []).append(entry)
        def token_group(spec, entries):
            name = f"tokens{len(self.token_groups)}:" + ("all" if spec.window is None else f"window{spec.window}") + \
                (f"+{spec.keep_first}" if spec.keep_first else "") + \
                (f"/{spec.every}" if spec.every > 1 else "")
            g = _TokenGroup(spec, entries, n_pages, max_slots, page_size, max_context, dtype, device, name)
            self.token_groups.append(g)
            return g, len(self.token_groups) - 1
        for spec, entries in keyed.items():
            if isinstance(spec, TokenSpec):
                g, gi = token_group(spec, entries)
            elif isinstance(spec, StateSpec):
                g = _StateGroup(spec, entries, max_slots, dtype, device)
                gi = len(self.state_groups)
                self.state_groups.append(g)
            else:
                raise CacheError(f"schedule entry declares an unknown cache need: {spec!r}")
            for i, entry in enumerate(entries):
                self._site_of[entry] = CacheSite(spec, gi, i, g)
        self._named_sites = {}
        keyed = {}
        for entry, named in enumerate(entry_tokens or ()):
            for name, spec in (named or {}).items():
                if not isinstance(spec, TokenSpec):
                    raise CacheError(f"schedule entry {entry} declares paged tensors '{name}' as {spec!r}: not a TokenSpec")
                keyed.setdefault(spec, []).append((entry, name))
        for spec, owners in keyed.items():
            g, gi = token_group(spec, [e for e, _ in owners])
            for i, owner in enumerate(owners):
                self._named_sites[owner] = CacheSite(spec, gi, i, g)
        self._named_states = {}
        keyed = {}
        for entry, states in enumerate(entry_states or ()):
            for name, spec in (states or {}).items():
                if not isinstance(spec, StateSpec):
                    raise CacheError(f"schedule entry {entry} declares state '{name}' as {spec!r}: not a StateSpec")
                keyed.setdefault(spec, []).append((entry, name))
        for spec, owners in keyed.items():
            g = _StateGroup(spec, [e for e, _ in owners], max_slots, dtype, device)
            self.state_groups.append(g)
            for i, owner in enumerate(owners):
                self._named_states[owner] = g.tensor[i]
        self.book = SlotBook(max_slots, [g.pages for g in self.token_groups], max_context)

    # --- what parts use -------------------------------------------------------------
    def site(self, entry):
        return self._site_of.get(entry)

    def entry_state(self, entry, name):
        """A state the entry declared by name: [slots + 1, *shape], zero for a slot that was just taken."""
        if (entry, name) not in self._named_states:
            raise CacheError(f"schedule entry {entry} declared no state '{name}'")
        return self._named_states[(entry, name)]

    def entry_site(self, entry, name):
        """The paged tensors an entry declared by name, as a site like the one of its mixer's cache."""
        if (entry, name) not in self._named_sites:
            raise CacheError(f"schedule entry {entry} declared no paged tensors '{name}'")
        return self._named_sites[(entry, name)]

    # --- what the engine uses ---------------------------------------------------------
    def acquire(self):
        slot = self.book.acquire()
        for g in self.state_groups:
            g.tensor[:, slot].zero_()
        return slot

    def release(self, slot):
        self.book.release(slot)

    def grow(self, slot, count):
        return self.book.grow(slot, count)

    def check_grow(self, slots, counts):
        self.book.check_grow(slots, counts)

    def length(self, slot):
        return self.book.length[slot]

    def live_slots(self):
        return self.book.live()

    def tokens_held(self):
        return self.book.tokens_held(self.page_size)

    def page_table(self, group_index, slots, width=None):
        """int32 [len(slots), width]: page ids of each slot in a group, -1 where it has none; the spare slot's row
        names the spare page."""
        g = self.token_groups[group_index]
        width = width or max(1, max(len(g.pages.lists.get(s, ())) for s in slots))
        t = np.full((len(slots), width), -1, dtype=np.int32)
        for i, s in enumerate(slots):
            if s == self.spare_slot:
                t[i, 0] = g.spare_page
                continue
            p = g.pages.lists.get(s, ())
            t[i, :len(p)] = p
        return t

    def bytes(self):
        n = 0
        for g in self.token_groups:
            n += sum(p.numel() * p.element_size() for p in g.pools.values())
        for g in self.state_groups:
            n += g.tensor.numel() * g.tensor.element_size()
        return n
