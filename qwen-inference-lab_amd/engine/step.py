"""The step function: one batch of (request, its next tokens) through the model.

A step may hold portions of prompts beside single decoded tokens, cut anywhere;
all of it runs as ONE batch over the packed rows (the reference runs each prompt
portion as a forward of its own and only decode rows together,
qil/engine.py:59-82).  It runs only the tokens it is given, reads everything
else from the cache that earlier steps left, and returns float32 logits at the
wanted places, in entry order.  With nothing wanted, neither the final norm nor
the head runs (qil/model.py:130-131).
"""
import numpy as np
import torch

from ..cache import CacheManager
from .batch import StepContext, StepEntry, StepPieces
from .graphs import DecodeGraphs


class ModelRunner:
    """Owns the cache of a loaded model and steps batches through it."""

    def __init__(self, model, *, num_pages, page_size=16, max_requests=64, max_step_tokens=None, graphs=True):
        if not model.loaded:
            raise ValueError('the model has no weights yet')
        self.model = model
        self.max_positions = getattr(model.config, 'max_position_embeddings', None)
        self.cache = CacheManager(model.cache_needs(), num_pages=num_pages, page_size=page_size,
                                  max_requests=max_requests, dtype=model.dtype, device=model.device,
                                  max_step_tokens=max_step_tokens)
        self.views = self.cache.views()
        self.previous_tokens = bool(getattr(model.embedding, 'needs_previous_tokens', False))
        self.steps = 0
        self.graphs = DecodeGraphs(self) if graphs and self.model.device.type == 'cuda' else None

    # -- request lifetime (thin: the cache manager decides)
    def admit(self, request, max_cached_tokens=None):
        return self.cache.admit(request, max_cached_tokens)

    def release(self, request):
        self.cache.release(request)

    def computed(self, request):
        return self.cache.computed[request]

    # -- the step
    def _validate(self, entries):
        if not entries:
            raise ValueError('a step needs at least one entry')
        seen = set()
        vocab = self.model.vocab
        for entry in entries:
            if entry.request in seen:
                raise ValueError(f'request {entry.request!r} appears twice in one step')
            seen.add(entry.request)
            if not self.cache.owns(entry.request):
                raise ValueError(f'request {entry.request!r} was not admitted')
            tokens, want = entry.tokens, entry.want
            if not tokens:
                raise ValueError(f'request {entry.request!r} brings no tokens')
            if len(tokens) == 1:                          # a decoded token: no generator for one element
                bad = type(tokens[0]) is not int or not 0 <= tokens[0] < vocab
            else:
                bad = any(type(t) is not int or not 0 <= t < vocab for t in tokens)
            if bad:                                                                       # qil/model.py:145-146
                raise ValueError(f'request {entry.request!r}: token ids must be integers in [0, {vocab})')
            end = self.cache.computed[entry.request] + len(tokens)
            if self.max_positions is not None and end > self.max_positions:               # qil/model.py:120
                raise ValueError(f'request {entry.request!r} would exceed {self.max_positions} positions')
            plain_first = len(want) == 1 and type(want[0]) is int and want[0] == 0       # a decoded token's logits
            if not plain_first and any(type(w) is not int or not 0 <= w < len(tokens) for w in want):
                raise ValueError(f'request {entry.request!r}: wanted places must index its tokens')

    def _describe(self, entries, table_width=None, validate=True, pad_rows=0):
        """Pages, then the batch description as host arrays: (entries, pieces, facts); pieces: a ``StepPieces``.

        ``pad_rows``: so many inert rows follow the entries' (a captured decode step is padded to its graph's size):
        sequences of one token at position 0 whose page is the spare page and whose state slot is the spare slot,
        with their logits wanted like the others'; what they compute is dropped."""
        entries = [e if isinstance(e, StepEntry) else StepEntry(e[0], tuple(e[1]), tuple(e[2]) if len(e) > 2 else ())
                   for e in entries]
        if validate:
            self._validate(entries)
        # Requests that bring several tokens come first (the caller's order among them and among the others): the
        # kernel for sequences of several rows then gets blocks for those sequences only.  The wanted places keep
        # the caller's order.
        given = entries
        entries = sorted(given, key=lambda e: len(e.tokens) < 2)
        cache, ps = self.cache, self.cache.page_size
        starts = [cache.computed[e.request] for e in entries]
        for entry, start in zip(entries, starts):
            cache.ensure(entry.request, start + len(entry.tokens))

        real = len(entries)
        starts = starts + [0] * pad_rows
        counts = [len(e.tokens) for e in entries] + [1] * pad_rows
        n, s = sum(counts), len(counts)
        cu = np.zeros(s + 1, dtype=np.int64)
        cu[1:] = np.cumsum(counts)
        tokens = np.fromiter([t for e in entries for t in e.tokens] + [0] * pad_rows, dtype=np.int64, count=n)
        row_seq = np.repeat(np.arange(s), counts)
        positions = np.arange(n) - cu[row_seq] + np.asarray(starts)[row_seq]
        first_row = {e.request: cu[i] for i, e in enumerate(entries)}
        logit_rows = np.fromiter([first_row[e.request] + w for e in given for w in e.want] + cu[real:-1].tolist(),
                                 dtype=np.int64)
        slots = [cache.slots[e.request] for e in entries] + [cache.spare_slot] * pad_rows
        single = cu[:-1][np.asarray(counts) == 1] if max(counts) > 1 else np.zeros(0, dtype=np.int64)
        pieces = StepPieces()
        for name, array in (('tokens', tokens), ('positions', positions), ('row_seq', row_seq), ('cu_seqlens', cu),
                            ('starts', starts), ('slots', slots), ('logit_rows', logit_rows), ('single_rows', single)):
            pieces.add(name, array)
        if self.previous_tokens:
            previous = np.concatenate(([-1], tokens[:-1])) if n else tokens
            last = [cache.last_tokens[e.request] for e in entries] + [None] * pad_rows
            previous[cu[:-1]] = [-1 if token is None else token for token in last]
            pieces.add('previous', previous)
        widths = []
        for index, group in enumerate(cache.kv_groups):
            tables = [cache.table(index, e.request) for e in entries] + [[cache.spare_page(index)]] * pad_rows
            width = max(len(t) for t in tables) if table_width is None else table_width
            table = np.zeros((s, width), dtype=np.int64)
            for i, t in enumerate(tables):
                table[i, :len(t)] = t
            token_slots = table[row_seq, positions // ps] * ps + positions % ps
            if (table[row_seq, positions // ps] < 0).any():
                raise RuntimeError('a new token falls into a page that was given back')
            table[table < 0] = 0          # given-back blocks lie outside every window; never read
            widths.append(width)
            pieces.add(f'tables{index}', table.reshape(-1))
            pieces.add(f'token_slots{index}', token_slots)
        facts = dict(n=n, s=s, starts=starts, counts=counts, slots=slots, cu=cu.tolist(), widths=widths,
                     max_context=int(max(st + c for st, c in zip(starts, counts))), n_logit_rows=len(logit_rows),
                     tile_seqs=sum(c > 1 for c in counts), real=real)
        return entries, pieces, facts

    def _inert(self, pieces, facts):
        """Pieces of the same layout that describe a step nobody asked for: the same numbers of tokens per sequence,
        all of them token 0 from position 0 on, every page the spare page and every state slot the spare slot.  A
        new graph warms up on these, so that the step it was made for runs once, as its first replay."""
        cache, ps = self.cache, self.cache.page_size
        spans, flat = pieces.spans(), pieces.flat().astype(np.int64)
        part = lambda name: flat[spans[name][0]:spans[name][1]]
        row_seq = part('row_seq')
        positions = part('positions') - part('starts')[row_seq]
        inert = StepPieces()
        for name in pieces.names:
            values = part(name)
            if name in ('tokens', 'starts'):
                values = np.zeros_like(values)
            elif name == 'positions':
                values = positions
            elif name == 'previous':
                values = np.full_like(values, -1)
            elif name == 'slots':
                values = np.full_like(values, cache.spare_slot)
            elif name.startswith('tables'):
                values = np.full_like(values, cache.spare_page(int(name[len('tables'):])))
            elif name.startswith('token_slots'):
                values = cache.spare_page(int(name[len('token_slots'):])) * ps + positions % ps
            inert.add(name, values)
        return inert

    def _context(self, entries, pieces, facts, device_flat, max_context=None):
        """StepContext and cache views over a device int32 array holding the pieces back to back."""
        spans = pieces.spans()
        part = lambda name: device_flat[spans[name][0]:spans[name][1]]
        s, counts = facts['s'], facts['counts']
        ctx = StepContext(
            n_tokens=facts['n'], n_seqs=s, n_logit_rows=facts['n_logit_rows'], token_ids=part('tokens'),
            positions=part('positions'), row_seq=part('row_seq'), cu_seqlens=part('cu_seqlens'), seq_starts=part('starts'),
            seq_slots=part('slots'), logit_rows=part('logit_rows'),
            single_rows=part('single_rows') if max(counts) > 1 else None, max_query=max(counts),
            max_context=max_context or facts['max_context'], host_cu_seqlens=facts['cu'], host_starts=facts['starts'],
            host_slots=facts['slots'], requests=[e.request for e in entries], tile_seqs=facts['tile_seqs'],
            previous_tokens=part('previous') if self.previous_tokens else None)
        for view in (one for view in self.views for one in (view if isinstance(view, tuple) else (view,))):
            if view is not None and hasattr(view, 'block_tables'):
                view.block_tables = part(f'tables{view.group}').view(s, facts['widths'][view.group])
                view.slots = part(f'token_slots{view.group}')
        return ctx

    def prepare(self, entries):
        """Pages, then the batch description on the device.  Does not touch the cache contents."""
        entries, pieces, facts = self._describe(entries)
        return entries, self._context(entries, pieces, facts, torch.from_numpy(pieces.flat()).to(self.model.device))

    @torch.inference_mode()
    def step(self, entries):
        """Run one batch; float32 logits [wanted, vocab] (None if nothing is wanted).

        A batch of single decoded tokens that all want their logits replays a captured HIP graph
        (``graphs.py``) when graphs are enabled; every other batch launches its kernels one by one.
        """
        replayed = self.graphs.step(entries) if self.graphs is not None and self.graphs.takes(entries) else None
        logits, entries, starts = replayed if replayed is not None else self._forward(entries)
        for entry, start in zip(entries, starts):
            self.cache.advance(entry.request, start + len(entry.tokens), entry.tokens[-1])
        self.steps += 1
        return logits

    def _forward(self, entries):
        """(logits, entries, starts) of a step that is no decode batch: from a graph of its shape if there is
        one, else launch by launch."""
        if self.graphs is not None:
            replayed = self.graphs.mixed_step(entries)
            if replayed is not None:
                return replayed
        entries, ctx = self.prepare(entries)
        return self.model.forward(ctx, self.views), entries, ctx.host_starts

    @torch.inference_mode()
    def step_and_sample(self, entries, sampler, params, counters):
        """``step``, then ``sampler``'s draw at the wanted places: the tokens as a host list (empty if nothing is
        wanted).  ``params`` and ``counters`` hold one item per wanted place, in entry order.  For a decode
        batch the draw is part of the replayed graph."""
        packed = sampler.pack(params, counters)
        replayed = self.graphs.step(entries, sampler, packed) if self.graphs is not None and self.graphs.takes(entries) else None
        if replayed is not None:
            drawn, entries, starts = replayed
        else:
            logits, entries, starts = self._forward(entries)
            drawn = None
            if logits is not None:
                if logits.shape[0] != packed.shape[1]:
                    raise ValueError('one SamplingParams and one counter per wanted place')
                out = torch.empty((2, logits.shape[0]), dtype=torch.int32, device=logits.device)
                sampler.draw(logits, torch.from_numpy(packed).to(logits.device), out)
                drawn = out.tolist()
        for entry, start in zip(entries, starts):
            self.cache.advance(entry.request, start + len(entry.tokens), entry.tokens[-1])
        self.steps += 1
        return sampler.unpack(drawn) if drawn is not None else []
