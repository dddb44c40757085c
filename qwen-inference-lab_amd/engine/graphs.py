"""HIP graphs for decode steps.

A decode step launches some ten small kernels per layer; launched one by one from Python the
host, not the GPU, sets the pace.  A batch in which every request brings exactly one token and
wants its logits has the same kernels, grids and tensor shapes whenever the number of rows and the
*bucket* of the longest context are the same, so its launches are captured once into a HIP graph
and replayed.  The number of rows is rounded up too (1, 2, 4, 8, then multiples of 4 up to 32 and of 8
beyond) and the batch filled with inert rows (token 0 at position 0 of a sequence whose only page is the
cache's spare page and whose state slot is the spare slot; their logits and draws are dropped), so that a
batch that shrinks request by request does not capture a graph for every size.  What changes from step to
step (tokens, positions, block tables, slots) lives in one static int32 device array that is overwritten
before each replay; kernels read positions from it and leave early past a row's context, so one graph
serves every context up to the bucket's end.

With a sampler the draw of the next tokens is part of the graph too (its seeds, output indices and
temperatures travel in the same array), and a step costs one upload, one replay and one download.

Steps with prompt portions have recurring shapes too (a portion of the chunk size beside so many single
tokens, step after step while a long prompt comes in), and for small models their launches cost more than
their kernels.  A shape that has been seen before (the same numbers of tokens and of wanted places per request,
largest first, and the same, wider bucket) is captured the second time and replayed from then on; the
requests are put into the graph's order and the logits back into the caller's.  The draw stays outside.

A new graph warms up (one run launch by launch, which loads the kernels and sizes the allocator) on inert
inputs of the step's shape, written to the spare page and slot, and is then captured; the step it was made for
runs once, as the graph's first replay.  A mixer therefore need not be idempotent to be captured.

Nothing in the captured region clears memory with a memset node: buffers are allocated, not
zeroed, and kernels write every element they later read.
"""
import gc
import weakref

import numpy as np
import torch

from .batch import StepEntry

BUCKET = 512          # contexts are rounded up to a multiple of this many tokens for a graph
MAX_GRAPHS = 24
DECODE_REPLACE_AT = 3   # comings of a decode batch's (rows, context bucket) before it may push a graph out of a full store
MIXED_BUCKET = 2048   # ... and of this many for a step with prompt portions (a portion moves on by its size a step)
MIXED_MOST_ROWS = 512  # steps of more rows are bound by their kernels, not by their launches
MAX_MIXED_GRAPHS = 32  # each keeps the step's activations: tens of MB at 8B sizes and 512 rows
MIXED_CAPTURE_AT = 2   # sightings of a shape before it is captured ...
MIXED_REPLACE_AT = 4   # ... and before it may push the least recently replayed graph out of a full store
MAX_SEEN = 256        # shapes remembered as seen once


def row_bucket(rows):
    """Rows of the graph that serves a decode batch of ``rows`` requests: 1, 2, 4, 8, then multiples of 4 up to 32,
    then multiples of 8."""
    for size in (1, 2, 4, 8):
        if rows <= size:
            return size
    step = 4 if rows <= 32 else 8
    return -(-rows // step) * step


class _Graph:
    def __init__(self, runner, entries, pieces, facts, bucket, sampler=None):
        self.sizes = pieces.sizes()
        self.spans = pieces.spans()
        rows = facts['s']                                   # with the inert rows that fill a decode batch
        self.rows, self.real = rows, facts['real']
        self.described = sum(self.sizes)
        total = self.described + (3 * rows if sampler is not None else 0)
        device = runner.model.device
        self.meta = torch.zeros(total, dtype=torch.int32, device=device)
        self.staging = torch.zeros(total, dtype=torch.int32).pin_memory()
        self.copied = torch.cuda.Event()
        self.widths = list(facts['widths'])
        self.written = [[(None, 0)] * rows for _ in self.widths]     # per page group and row: (table, entries uploaded)
        self.drawn = self.drawn_host = None
        if sampler is not None:
            self.drawn = torch.zeros((2, rows), dtype=torch.int32, device=device)
            self.drawn_host = torch.zeros((2, rows), dtype=torch.int32).pin_memory()
        zeros = None if sampler is None else np.zeros((3, rows), dtype=np.int32)
        self.load(runner._inert(pieces, facts), zeros)     # the warm-up's inputs: nobody's pages, nobody's state
        ctx = runner._context(entries, pieces, facts, self.meta, max_context=bucket)
        side = torch.cuda.Stream(device=device)
        side.wait_stream(torch.cuda.current_stream(device))
        with torch.cuda.stream(side):                       # launch by launch once: loads the library, sizes the allocator
            runner.model.forward(ctx, runner.views)
        torch.cuda.current_stream(device).wait_stream(side)
        self.graph = torch.cuda.CUDAGraph()
        # No garbage collection while capturing: a collected object that frees device or pinned memory
        # (an older graph, say) would issue a call the capture forbids, and the process would abort.
        collecting = gc.isenabled()
        gc.disable()
        try:
            with torch.cuda.graph(self.graph):
                self.logits = runner.model.forward(ctx, runner.views)
                if sampler is not None:
                    sampler.draw(self.logits, self.meta[self.described:].view(3, rows), self.drawn)
        finally:
            if collecting:
                gc.enable()
        self.load(pieces, zeros)                            # the step itself: it runs as the first replay

    def load(self, pieces, packed=None):
        if pieces.sizes() != self.sizes:
            raise RuntimeError('batch layout does not fit the captured graph')
        self.copied.synchronize()                           # the previous upload has left the staging buffer
        flat = self.staging.numpy()
        flat[:self.described] = pieces.flat()
        if packed is not None:
            flat[self.described:] = packed.reshape(-1)
        self.meta.copy_(self.staging, non_blocking=True)
        self.copied.record()

    def refresh(self, runner, entries, packed=None):
        """``load`` for the steps after the first, straight from the requests' state: only what changes from
        one decode step to the next is rewritten (tokens, positions, slots, and the block tables' new
        entries; a table is a list that only grows, apart from given-back entries that no kernel reads).
        Holds the pages of the new tokens.  Returns the requests' positions."""
        cache = runner.cache
        ps, spans = cache.page_size, self.spans
        starts = [cache.computed[e.request] for e in entries]
        for entry, start in zip(entries, starts):
            cache.ensure(entry.request, start + 1)
        self.copied.synchronize()
        flat = self.staging.numpy()
        count, spare_slot = len(entries), cache.spare_slot

        def put(name, values, fill):
            """The real rows' values, and ``fill`` in the rows that were real in the last step and are inert now."""
            at = spans[name][0]
            flat[at:at + count] = values
            if self.real > count:
                flat[at + count:at + self.real] = fill
        put('tokens', [e.tokens[0] for e in entries], 0)
        put('positions', starts, 0)
        put('starts', starts, 0)                            # where the requests' rows begin
        if runner.previous_tokens:
            last = [cache.last_tokens[e.request] for e in entries]
            put('previous', [-1 if token is None else token for token in last], -1)
        put('slots', [cache.slots[e.request] for e in entries], spare_slot)
        for group, width in enumerate(self.widths):
            tables_at, slots_at, written = spans[f'tables{group}'][0], spans[f'token_slots{group}'][0], self.written[group]
            for row, (entry, start) in enumerate(zip(entries, starts)):
                table = cache.table(group, entry.request)
                count_pages = len(table)
                if count_pages > width:
                    raise RuntimeError('batch layout does not fit the captured graph')
                known, done = written[row]
                if known is not table or done > count_pages:
                    done = 0
                if done < count_pages:
                    at = tables_at + row * width
                    flat[at + done:at + count_pages] = [max(page, 0) for page in table[done:]]
                    written[row] = (table, count_pages)
                page = table[start // ps]
                if page < 0:
                    raise RuntimeError('a new token falls into a page that was given back')
                flat[slots_at + row] = page * ps + start % ps
            spare = cache.spare_page(group)
            for row in range(count, self.real):             # rows that have become inert: the spare page alone
                flat[tables_at + row * width] = spare
                flat[slots_at + row] = spare * ps
                written[row] = (None, 0)
        self.real = count
        if packed is not None:
            flat[self.described:].reshape(3, self.rows)[:, :count] = packed
        self.meta.copy_(self.staging, non_blocking=True)
        self.copied.record()
        return starts

    def run(self):
        self.graph.replay()
        return self.logits

    def run_drawn(self):
        """[tokens, finite flags] of the rows, as nested host lists."""
        self.graph.replay()
        self.drawn_host.copy_(self.drawn, non_blocking=True)
        torch.cuda.current_stream(self.drawn.device).synchronize()
        return self.drawn_host.tolist()


class DecodeGraphs:
    def __init__(self, runner):
        self._runner, self.graphs, self.replays, self.captures = weakref.ref(runner), {}, 0, 0     # no cycle
        self.waiting = {}                                   # decode keys that found the store full: their comings
        self._safe = None
        self.mixed, self.seen, self.mixed_replays, self.mixed_captures = {}, {}, 0, 0

    def safe(self):
        if self._safe is None:
            blocks = self._runner().model.blocks
            self._safe = all(b.mixer is None or b.mixer.graph_safe for b in blocks)
        return self._safe

    def takes(self, entries):
        """A decode batch: every entry brings one token and wants its logits (entries may be plain tuples, whose
        third member, the wanted places, may be missing)."""
        if not entries or not self.safe():
            return False
        for entry in entries:
            if isinstance(entry, StepEntry):
                tokens, want = entry.tokens, entry.want
            else:
                tokens, want = entry[1], (entry[2] if len(entry) > 2 else ())
            if len(tokens) != 1 or tuple(want) != (0,):
                return False
        return True

    def mixed_step(self, entries):
        """(logits, entries, starts) of a step with prompt portions from a graph of its shape (a new shape is
        remembered and launched kernel by kernel, in its graph's layout), or None: the step is too large, or a mixer
        reads the host side of the step."""
        if not self.safe() or not entries:
            return None
        runner = self._runner()
        normal = [e if isinstance(e, StepEntry) else StepEntry(e[0], tuple(e[1]), tuple(e[2]) if len(e) > 2 else ())
                  for e in entries]
        if sum(len(e.tokens) for e in normal) > MIXED_MOST_ROWS or max(len(e.tokens) for e in normal) < 2:
            return None
        runner._validate(normal)
        # the graph's order: most tokens first, the caller's order among equals
        order = sorted(range(len(normal)), key=lambda i: (-len(normal[i].tokens), -len(normal[i].want), i))
        ordered = [normal[i] for i in order]
        ps = runner.cache.page_size
        longest = max(runner.cache.computed[e.request] + len(e.tokens) for e in ordered)
        bucket = -(-longest // MIXED_BUCKET) * MIXED_BUCKET
        limit = runner.max_positions
        if limit is not None:
            bucket = min(bucket, -(-limit // ps) * ps)
        width = -(-bucket // ps)
        key = (tuple(len(e.tokens) for e in ordered), tuple(len(e.want) for e in ordered), bucket)
        graph = self.mixed.get(key)
        described, pieces, facts = runner._describe(ordered, table_width=width, validate=False)
        if graph is None:
            # Capturing costs about two launched steps (the warm-up and the recording), so a shape is captured only
            # when it has come before, and it pushes another graph out only when it keeps coming: a workload that
            # cycles through more shapes than the store holds would otherwise capture at every step and never replay.
            if len(self.seen) >= MAX_SEEN and key not in self.seen:
                self.seen.clear()
            sightings = self.seen[key] = self.seen.get(key, 0) + 1
            full = len(self.mixed) >= MAX_MIXED_GRAPHS
            if sightings >= (MIXED_REPLACE_AT if full else MIXED_CAPTURE_AT):
                if full:
                    self.mixed.pop(next(iter(self.mixed)))          # the least recently replayed
                graph = self.mixed[key] = _Graph(runner, described, pieces, facts, bucket)
                self.mixed_captures += 1
                del self.seen[key]
        else:
            graph.load(pieces)
            self.mixed[key] = self.mixed.pop(key)                   # most recently replayed: last
        if graph is None:
            # Launch by launch, but described and planned exactly as the shape's graph would be (the graph's order
            # of requests, table width and context bucket), so that the kernels, their splits of the keys and the
            # order of their sums are the same whether the step is launched or replayed.
            flat = torch.from_numpy(pieces.flat()).to(runner.model.device)
            ctx = runner._context(described, pieces, facts, flat, max_context=bucket)
            logits = runner.model.forward(ctx, runner.views)
        else:
            logits = graph.run()
            self.mixed_replays += 1
        if logits is not None:
            # rows of the wanted places in the caller's order of requests
            first, at = {}, 0
            for index, entry in zip(order, ordered):
                first[index] = at
                at += len(entry.want)
            back = [first[i] + j for i in range(len(normal)) for j in range(len(normal[i].want))]
            if back != list(range(len(back))):
                logits = logits.index_select(0, torch.tensor(back, dtype=torch.int64).to(logits.device, non_blocking=True))
            else:
                logits = logits.clone()                     # the graph's own output buffer is overwritten by the next replay
        starts = {e.request: s for e, s in zip(ordered, facts['starts'])}
        return logits, normal, [starts[e.request] for e in normal]

    def step(self, entries, sampler=None, packed=None):
        """(logits, entries, starts) of a decode batch; with a sampler and its packed parameters the first
        member is the host copy of the draw ([tokens, finite flags]) instead of logits.  None: the store of graphs is
        full and this batch's shape has not come often enough to take a place (the caller launches the step)."""
        runner = self._runner()
        ps = runner.cache.page_size
        normal = [e if isinstance(e, StepEntry) else StepEntry(e[0], tuple(e[1]), tuple(e[2])) for e in entries]
        runner._validate(normal)
        longest = max(runner.cache.computed[e.request] for e in normal) + 1
        bucket = -(-longest // BUCKET) * BUCKET
        limit = runner.max_positions
        if limit is not None:
            bucket = min(bucket, -(-limit // ps) * ps)
        width = -(-bucket // ps)
        rows = row_bucket(len(normal))
        key = (rows, bucket, sampler is not None)
        graph = self.graphs.get(key)
        if graph is None:
            if len(self.graphs) >= MAX_GRAPHS:
                # a full store: the least recently replayed graph goes, but only for a batch that keeps coming
                # (capturing costs about two launched steps; the step is launched kernel by kernel meanwhile)
                if len(self.waiting) >= MAX_SEEN and key not in self.waiting:
                    self.waiting.clear()
                comings = self.waiting[key] = self.waiting.get(key, 0) + 1
                if comings < DECODE_REPLACE_AT:
                    return None
                del self.waiting[key]
                self.graphs.pop(next(iter(self.graphs)))
            described, pieces, facts = runner._describe(normal, table_width=width, validate=False,
                                                        pad_rows=rows - len(normal))
            graph = self.graphs[key] = _Graph(runner, described, pieces, facts, bucket, sampler)
            self.captures += 1
        else:
            self.graphs[key] = self.graphs.pop(key)         # most recently replayed: last
        starts = graph.refresh(runner, normal, packed)
        if sampler is not None:
            result = [values[:len(normal)] for values in graph.run_drawn()]
        else:
            result = graph.run()[:len(normal)].clone()      # the graph's own output buffer is overwritten by the next replay
        self.replays += 1
        return result, normal, starts
