"""The cache manager: page pools per group of layers, block tables per request,
slots for fixed-size per-request state, and the device storage behind them.

Needs come from the model (``CausalLM.cache_needs()``), one per schedule entry.
Entries with equal paged needs (``KVNeed``: kv heads, head size, window; or a ``PagedNeed`` with
tensors of the mixer's own) form a group with a page pool of its own; every group has its own block tables, so a windowed group
can give pages back while a full group keeps them.  Entries with equal state
needs form a state group.  Device layout of a KV group:
``k : [entries, pages, kv_heads, page_size, head_dim]`` and, transposed within a page so
that the value product's matrix-core operands load directly,
``v : [entries, pages, kv_heads, head_dim, page_size]``, in the model's dtype; a token's slot
number is ``page * page_size + position % page_size`` (qil/cache.py:79-82).  Storage is never cleared: kernels read only positions below a
request's computed length and inside its window (qil/cache.py:127-128,137;
tests fill the pool with NaN).

One page more than the pool hands out lies behind every page group's storage, and one state slot more than there
are requests behind every state group's (``spare_page``, ``spare_slot``): no request ever gets them.  Inert rows
that pad a captured step to its graph's size, and a new graph's warm-up run, write there.

Per request the manager keeps ``last_tokens``, the last token of its steps so far (an embedding of token pairs
needs the token before a step's first), and ``computed``: how many tokens every layer has
cached.  A step must start exactly there (qil/cache.py:84-95,113-116) and
``advance`` moves it after the step ran.
"""
from collections import deque
from dataclasses import dataclass

import torch

from ..parts.base import KVNeed, PagedNeed, StateNeed, CompoundNeed
from .pages import PagePool, CacheFull


@dataclass
class KVView:
    """What an attention-like mixer sees of its schedule entry's cache in one step."""
    k: torch.Tensor              # [pages, kv_heads, page_size, head_dim]
    v: torch.Tensor              # [pages, kv_heads, head_dim, page_size]
    page_size: int
    writes: bool                 # False for an entry that reads another entry's cache
    group: int
    block_tables: torch.Tensor = None    # int32 [n_seqs, stride], filled per step
    slots: torch.Tensor = None           # int32 [n_tokens], slot of each new token


@dataclass
class PagedView:
    """What a mixer with a ``PagedNeed`` sees of its schedule entry's cache in one step."""
    tensors: dict                # name -> [pages, page_size, *shape of a token's entry]
    page_size: int
    writes: bool
    group: int
    block_tables: torch.Tensor = None    # int32 [n_seqs, stride], filled per step
    slots: torch.Tensor = None           # int32 [n_tokens], slot of each new token


@dataclass
class StateView:
    """Fixed-size state of a schedule entry: ``state[slot]`` belongs to one live request."""
    state: torch.Tensor          # [slots, *shape]
    writes: bool
    group: int


class CacheManager:
    def __init__(self, needs, *, num_pages, page_size, max_requests, dtype=torch.float32, device='cpu',
                 max_step_tokens=None, allocate=True):
        self.page_size, self.max_requests, self.dtype, self.device = page_size, max_requests, dtype, torch.device(device)
        self.kv_groups, self.state_groups = [], []     # dicts: need, entries, pool / need, entries
        # per schedule entry: None | (kind, group, index, writes) | a list of those (an entry with a CompoundNeed)
        self.binding = []
        for position, need in enumerate(needs):
            if need is None:
                self.binding.append(None)
            elif isinstance(need, tuple) and need[0] == 'shared':
                owner = self.binding[need[1]]
                if isinstance(owner, list):
                    self.binding.append([(kind, group, index, False) for kind, group, index, _ in owner])
                else:
                    self.binding.append((owner[0], owner[1], owner[2], False))
            elif isinstance(need, CompoundNeed):
                self.binding.append([self._bind(position, one) for one in need.needs])
            else:
                self.binding.append(self._bind(position, need))
        pages = num_pages if isinstance(num_pages, (list, tuple)) else [num_pages] * len(self.kv_groups)
        if len(pages) != len(self.kv_groups):
            raise ValueError(f'{len(self.kv_groups)} page groups, {len(pages)} page counts')
        for group, count in zip(self.kv_groups, pages):
            group['pool'] = PagePool(num_pages=count, page_size=page_size, window=group['need'].window,
                                     max_step_tokens=max_step_tokens, keep_first=getattr(group['need'], 'keep_first', 0))
        self.free_slots = deque(range(max_requests))
        self.slots, self.computed, self.limits = {}, {}, {}
        self.last_tokens = {}            # request -> the last token its steps brought (None before the first)
        if allocate:
            self._allocate()

    def _bind(self, position, need):
        if isinstance(need, (KVNeed, PagedNeed)):
            group = self._group(self.kv_groups, need)
            self.kv_groups[group]['entries'].append(position)
            return ('kv', group, len(self.kv_groups[group]['entries']) - 1, True)
        if isinstance(need, StateNeed):
            group = self._group(self.state_groups, need)
            self.state_groups[group]['entries'].append(position)
            return ('state', group, len(self.state_groups[group]['entries']) - 1, True)
        raise TypeError(f'unknown cache need {need!r}')

    @staticmethod
    def _group(groups, need):
        for index, group in enumerate(groups):
            if group['need'] == need:
                return index
        groups.append(dict(need=need, entries=[]))
        return len(groups) - 1

    def _allocate(self):
        for group in self.kv_groups:
            need, pool = group['need'], group['pool']
            entries, pages = len(group['entries']), pool.capacity + 1          # + the spare page
            if isinstance(need, PagedNeed):
                group['tensors'] = {
                    name: torch.empty((entries, pages, self.page_size, *shape),
                                      dtype=torch.float32 if kind == 'float32' else self.dtype, device=self.device)
                    for name, shape, kind in need.tensors}
                continue
            group['k'] = torch.empty((entries, pages, need.kv_heads, self.page_size, need.head_dim),
                                     dtype=self.dtype, device=self.device)
            group['v'] = torch.empty((entries, pages, need.kv_heads, need.head_dim, self.page_size),
                                     dtype=self.dtype, device=self.device)
        for group in self.state_groups:
            need = group['need']
            dtype = torch.float32 if need.dtype == 'float32' else self.dtype
            group['state'] = torch.zeros((len(group['entries']), self.max_requests + 1, *need.shape),
                                         dtype=dtype, device=self.device)                   # + the spare slot

    @property
    def spare_slot(self):
        """The state slot that belongs to no request."""
        return self.max_requests

    def spare_page(self, group):
        """The page of page group ``group`` that belongs to no request."""
        return self.kv_groups[group]['pool'].capacity

    # ------------------------------------------------------------------ requests
    def pages_for(self, tokens):
        return (tokens + self.page_size - 1) // self.page_size

    def fits_at_all(self, tokens):
        """Could a request of ``tokens`` cached tokens ever be admitted (empty cache)?"""
        return all(g['pool'].reservation_for(tokens) <= g['pool'].capacity for g in self.kv_groups)

    def admit(self, request, max_cached_tokens=None):
        """Reserve credits in every group and a state slot; False if they do not fit now.

        ``max_cached_tokens`` None admits without reservation (trace replay, where a
        request's length is not known ahead): ``ensure`` may then raise CacheFull.
        """
        if request in self.slots:
            raise ValueError('duplicate cache owner')
        if max_cached_tokens is not None and (type(max_cached_tokens) is not int or max_cached_tokens < 1):
            raise ValueError('cache reservation must be a positive integer')
        if not self.free_slots or not all(g['pool'].can_admit(max_cached_tokens) for g in self.kv_groups):
            return False
        for group in self.kv_groups:
            group['pool'].admit(request, max_cached_tokens)
        self.slots[request] = self.free_slots.popleft()
        self.computed[request] = 0
        self.last_tokens[request] = None
        self.limits[request] = max_cached_tokens
        return True

    def ensure(self, request, end):
        """Physical pages for positions below ``end`` in every group (all or nothing)."""
        limit = self.limits[request]
        if end <= 0 or (limit is not None and end > limit):
            raise ValueError('write exceeds reserved context')
        for group in self.kv_groups:
            pool = group['pool']
            if pool.pages_for(end) > len(pool.tables[request]):
                break
        else:
            return                                      # every group holds the pages already (most decode steps)
        short = [g for g in self.kv_groups
                 if g['pool'].pages_for(end) - len(g['pool'].tables[request]) > len(g['pool'].free)]
        if short:
            if limit is not None:
                raise RuntimeError('cache reservation invariant violated')    # qil/cache.py:75-76
            raise CacheFull(f'out of pages for request {request!r} at {end} tokens')
        for group in self.kv_groups:
            group['pool'].ensure(request, end)

    def advance(self, request, end, last_token=None):
        """The step has cached tokens up to ``end``, of which ``last_token`` is the last; windows give passed pages
        back."""
        if end < self.computed[request]:
            raise ValueError('computed length cannot shrink')
        self.computed[request] = end
        self.last_tokens[request] = last_token
        for group in self.kv_groups:
            group['pool'].pass_window(request, end)

    def release(self, request):
        if request not in self.slots:
            raise ValueError('unknown cache owner')
        for group in self.kv_groups:
            group['pool'].release(request)
        self.free_slots.append(self.slots.pop(request))
        del self.computed[request], self.limits[request], self.last_tokens[request]

    def owns(self, request):
        return request in self.slots

    def table(self, group, request):
        return self.kv_groups[group]['pool'].tables[request]

    @property
    def free_pages(self):
        return [len(g['pool'].free) for g in self.kv_groups]

    def check(self):
        for group in self.kv_groups:
            group['pool'].check()
            if set(group['pool'].tables) != set(self.slots):
                raise AssertionError('pools and slots disagree about live requests')
        slots = sorted(list(self.free_slots) + list(self.slots.values()))
        if slots != list(range(self.max_requests)):
            raise AssertionError(f'state slots broken: {slots}')

    # ------------------------------------------------------------------ views
    def views(self):
        """One view per schedule entry (None where the entry keeps nothing; a tuple of views for an entry with a
        ``CompoundNeed``, in the order of its needs)."""
        def view(bound):
            kind, group, index, writes = bound
            if kind == 'kv':
                g = self.kv_groups[group]
                if isinstance(g['need'], PagedNeed):
                    return PagedView({name: t[index] for name, t in g['tensors'].items()}, self.page_size, writes, group)
                return KVView(g['k'][index], g['v'][index], self.page_size, writes, group)
            return StateView(self.state_groups[group]['state'][index], writes, group)
        return [None if bound is None else tuple(view(one) for one in bound) if isinstance(bound, list) else view(bound)
                for bound in self.binding]

    def bytes_per_token(self):
        size = torch.empty((), dtype=self.dtype).element_size()
        total = 0
        for g in self.kv_groups:
            need = g['need']
            if isinstance(need, PagedNeed):
                per_token = sum(_count(shape) * (4 if kind == 'float32' else size) for _, shape, kind in need.tensors)
            else:
                per_token = 2 * need.kv_heads * need.head_dim * size
            total += len(g['entries']) * per_token
        return total


def _count(shape):
    n = 1
    for extent in shape:
        n *= extent
    return n
