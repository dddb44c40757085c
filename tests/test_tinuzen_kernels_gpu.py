"""The kernels the Tinuzen design added or changed, each alone against its plain reference (``kernel_refs``) on the same
inputs: a bias by distance and kept first keys in the attention kernels (rows alone, portions, keys in one piece and in
parts), the q/k kernels with a norm over whole rows and with values that are keys, the recurrence with a step size per
head and token and its state, the gated norm in groups, the join of gated branches with the norm behind it, the embedding
by token pairs, and one product for all that reads an input."""
import pytest
import torch

import kernel_refs as refs
from qil_amd import ops
from test_dogozen_kernels_gpu import close, ints, moved, partials
from test_kernels_gpu import build_cache

pytestmark = pytest.mark.gpu
DTYPES = [torch.float32, torch.bfloat16]


def spoil(cache, table, lengths, chunks, page_size, window, keep):
    """NaN in every key and value that no row of the step sees (a page that was given back may hold anything)."""
    k_cache, v_cache = cache
    for i, (n, c) in enumerate(zip(lengths, chunks)):
        j = torch.arange(keep, max(keep, n - c - window + 1))
        page = table[i].long().cpu()[j // page_size].cuda()
        k_cache[page, :, (j % page_size).cuda()] = float('nan')
        v_cache[page, :, :, (j % page_size).cuda()] = float('nan')


def attention_step(lengths, chunks):
    starts = [n - c for n, c in zip(lengths, chunks)]
    cu = [0]
    for c in chunks:
        cu.append(cu[-1] + c)
    single = [cu[i] for i, c in enumerate(chunks) if c == 1]
    return cu[-1], dict(row_seq=ints([i for i, c in enumerate(chunks) for _ in range(c)]),
                        positions=ints([p for s, c in zip(starts, chunks) for p in range(s, s + c)]), cu_seqlens=ints(cu),
                        seq_starts=ints(starts), single_rows=ints(single) if max(chunks) > 1 else None)


# ------------------------------------------------------------------------------------------------ bias by distance, kept keys
@pytest.mark.parametrize('dtype', DTYPES)
@pytest.mark.parametrize('lengths,chunks,page_size,d,heads,kv_heads,window,keep', [
    ([70, 33, 5, 300], [1, 1, 1, 1], 16, 56, 6, 3, 37, 20),     # rows alone: a hole of whole steps, none, no window passed yet
    ([1500, 40, 700], [1, 1, 1], 16, 64, 4, 2, 300, 70),
    ([2100, 900, 31], [1, 1, 1], 8, 128, 16, 8, 64, 1),
    ([1500, 2100], [1, 1], 16, 128, 8, 8, 1, 33),               # a window of one key
    ([3000, 2999], [1, 1], 32, 128, 16, 2, 1024, 512),          # the places in several parts
    ([300, 2], [1, 1], 4, 24, 5, 1, 7, 3),                      # sizes the matrix-core decode kernel does not take
    ([1000, 77], [1, 1], 16, 64, 4, 2, None, 0),                # no window: the slopes alone
    ([70, 70, 5, 33], [70, 2, 5, 17], 16, 56, 6, 3, 37, 10),    # portions
    ([129, 64, 1000, 16], [129, 1, 3, 16], 16, 128, 8, 2, 40, 40),
    ([257, 400], [200, 31], 3, 40, 6, 2, 64, 100),
    ([1200], [1200], 16, 128, 4, 2, 300, 65),                   # the bfloat16 kernel for heads of 128, a long prompt
    ([1500, 900], [700, 900], 16, 128, 8, 8, 64, 64),
    ([1500, 600], [2, 130], 64, 128, 4, 1, 100, 129),
    ([1500, 900], [200, 64], 16, 128, 8, 2, None, 0),
    ([1100], [1100], 16, 64, 4, 1, 512, 3),
    ([900], [900], 8, 128, 2, 2, 20, 5),                        # the kept keys and the window in one tile, then apart
])
def test_attention_with_a_bias_by_distance_and_kept_keys(dtype, lengths, chunks, page_size, d, heads, kv_heads, window, keep, monkeypatch):
    k_cache, v_cache, table, _ = build_cache(lengths, page_size, kv_heads, d, dtype)
    if window is not None:
        spoil((k_cache, v_cache), table, lengths, chunks, page_size, window, keep)
    g = torch.Generator().manual_seed(d)
    n, index = attention_step(lengths, chunks)
    index['block_tables'] = table.cpu()
    q = torch.randn(n, heads * d, generator=g).to(dtype)
    slopes = torch.tensor([2.0 ** (-8.0 * (h + 1) / heads) for h in range(heads)])
    common = dict(heads=heads, kv_heads=kv_heads, head_dim=d, page_size=page_size, n_seqs=len(lengths),
                  max_query=max(chunks), max_context=max(lengths), scale=0.3, window=window, keep_first=keep)
    caches = dict(k_cache=k_cache.cpu(), v_cache=v_cache.cpu())
    on_gpu = {k: None if v is None else v.cuda() for k, v in index.items()}
    for slope, sinks in ((slopes, None), (None, torch.linspace(-3.0, 3.0, heads)), (slopes, torch.zeros(heads))):
        want = refs.paged_attention(q, slopes=slope, sinks=sinks, accumulate=torch.float64, **caches, **index, **common)
        for forced in (None, (64, 2)):
            if forced is not None and max(chunks) == 1:
                continue
            monkeypatch.setattr(ops, 'TILE_KEY_PARTS', forced)
            got = ops.paged_attention(q.cuda(), k_cache=k_cache, v_cache=v_cache, slopes=None if slope is None else slope.cuda(),
                                      sinks=None if sinks is None else sinks.cuda(), **on_gpu, **common)
            assert torch.isfinite(got.float()).all()
            close(got, want, dtype, 0.3)
    if keep and window is not None and max(lengths) > keep + window + 64:      # the kept keys are there
        without = refs.paged_attention(q, accumulate=torch.float64, **caches, **index, **dict(common, keep_first=0))
        kept = refs.paged_attention(q, accumulate=torch.float64, **caches, **index, **common)
        assert (kept.float() - without.float()).abs().max() > 0.05


# ------------------------------------------------------------------------------------------------ the q/k kernels
def qk_inputs(n, pages, page_size, heads, kv_heads, d, extra, splits, shared, dtype, g):
    if dtype == torch.float32 and splits == 0:
        splits = 1
    positions = ints(sorted(torch.randint(0, 900, (n,), generator=g).tolist()))
    slots = torch.randperm(pages * page_size, generator=g)[:n].to(torch.int32)
    qkv = partials(torch.randn(n, (heads + (1 if shared else 2) * kv_heads) * d + extra, generator=g).to(dtype), splits, g)
    caches = [torch.zeros(pages, kv_heads, page_size, d).to(dtype), torch.zeros(pages, kv_heads, d, page_size).to(dtype)]
    return positions, slots, qkv, caches


def rotation_of(rot):
    from qil_amd.parts import RotaryFrequencies
    return (None, None) if not rot else (RotaryFrequencies(rot, 300.0).rotation(), RotaryFrequencies(rot, 300.0, device='cuda').rotation())


@pytest.mark.parametrize('dtype', DTYPES)
@pytest.mark.parametrize('heads,kv_heads,d,true_d,rot,extra,splits,shared', [
    (4, 2, 64, 64, 32, 256, 0, False), (6, 3, 56, 50, 0, 0, 3, False), (16, 4, 128, 128, 128, 64, 5, True), (5, 5, 16, 11, 6, 80, 1, True),
    (1, 1, 8, 8, 0, 0, 0, False), (32, 8, 256, 256, 0, 0, 2, False), (12, 3, 128, 128, 0, 40, 0, False), (32, 8, 128, 128, 0, 0, 0, False),
    (40, 20, 128, 128, 0, 0, 2, False), (3, 3, 56, 56, 10, 0, 2, False)])
def test_a_norm_over_whole_rows(dtype, heads, kv_heads, d, true_d, rot, extra, splits, shared):
    g = torch.Generator().manual_seed(heads * d)
    positions, slots, qkv, (kc, vc) = qk_inputs(37, 12, 8, heads, kv_heads, d, extra, splits, shared, dtype, g)
    q_weight, k_weight = torch.rand(heads * d, generator=g) + 0.5, torch.rand(kv_heads * d, generator=g) + 0.5
    rotation, on_gpu = rotation_of(rot)
    args = dict(heads=heads, kv_heads=kv_heads, head_dim=d, eps=1e-5, page_size=8, dtype=dtype, extra_columns=extra,
                q_elems=heads * true_d, k_elems=kv_heads * true_d, values_are_keys=shared)
    gk, gv = kc.cuda(), vc.cuda()
    want = refs.qk_row_norm_store(qkv, q_weight=q_weight, k_weight=k_weight, rotation=rotation, positions=positions,
                                  slots=slots, k_cache=kc, v_cache=vc, **args)
    got = ops.qk_row_norm_store(moved(qkv), q_weight=q_weight.cuda(), k_weight=k_weight.cuda(), rotation=on_gpu,
                                positions=positions.cuda(), slots=slots.cuda(), k_cache=gk, v_cache=gv, **args)
    scale = 10.0 if rot else 2.0                        # (angles of hundreds: the reference's own rounding)
    close(got, want, dtype, scale)
    close(gk, kc, dtype, scale)
    close(gv, vc, dtype)


@pytest.mark.parametrize('dtype', DTYPES)
@pytest.mark.parametrize('heads,kv_heads,d,rot,extra,splits', [(4, 2, 64, 32, 256, 0), (6, 3, 48, 20, 288, 3), (3, 1, 128, 128, 0, 2),
                                                               (2, 2, 16, 0, 32, 1)])
def test_values_that_are_keys(dtype, heads, kv_heads, d, rot, extra, splits):
    g = torch.Generator().manual_seed(heads * d)
    positions, slots, qkv, (kc, vc) = qk_inputs(37, 12, 8, heads, kv_heads, d, extra, splits, True, dtype, g)
    rotation, on_gpu = rotation_of(rot)
    args = dict(heads=heads, kv_heads=kv_heads, head_dim=d, eps=0.0, page_size=8, dtype=dtype, extra_columns=extra,
                values_are_keys=True, q_weight=None, k_weight=None)
    gk, gv = kc.cuda(), vc.cuda()
    want = refs.qk_norm_rope_store(qkv, rotation=rotation, positions=positions, slots=slots, k_cache=kc, v_cache=vc, **args)
    got = ops.qk_norm_rope_store(moved(qkv), rotation=on_gpu, positions=positions.cuda(), slots=slots.cuda(), k_cache=gk,
                                 v_cache=gv, **args)
    close(got, want, dtype, 10.0 if rot else 1.0)
    close(gk, kc, dtype, 10.0 if rot else 1.0)
    close(gv, vc, dtype)
    page, offset = slots.long() // 8, slots.long() % 8
    if rot:                                            # the values are not what the rotation made of the keys
        assert (kc[page, :, offset].float() - vc[page, :, :, offset].float()).abs().max() > 0.3


@pytest.mark.parametrize('lengths,page_size,d,heads,kv_heads,window,keep,rot,splits,extra', [
    ([2100, 1, 700, 1290, 64, 2047, 300, 33], 16, 128, 16, 4, None, 0, 64, 8, 16 * 128),
    ([1, 2, 31, 32, 33, 64, 65, 96], 8, 64, 6, 2, 20, 5, 32, 3, 0),
    ([257, 512, 513, 999], 32, 128, 8, 1, 100, 64, 128, 1, 64),
    ([400, 1000, 3000], 16, 64, 16, 4, 40, 200, 0, 2, 16 * 64),
])
def test_decoding_with_queries_made_inside_is_the_two_kernels(lengths, page_size, d, heads, kv_heads, window, keep, rot, splits, extra):
    """The decode kernel that makes its queries and new keys itself, with values that are keys, slopes, kept keys and an
    added one in the denominator: bit for bit what the q/k kernel followed by the attention kernels leave."""
    dtype, rows = torch.bfloat16, len(lengths)
    g = torch.Generator().manual_seed(d + heads)
    k_cache, v_cache, table, _ = build_cache(lengths, page_size, kv_heads, d, dtype)
    positions = ints([n - 1 for n in lengths]).cuda()
    row_seq = torch.arange(rows, dtype=torch.int32).cuda()
    slots = (table[row_seq.long(), (positions // page_size).long()] * page_size + positions % page_size).to(torch.int32)
    # as columns of a wider product
    wide = ops.Partials((torch.randn(splits, rows, 16 + (heads + kv_heads) * d + extra + 48, generator=g) * 0.7).cuda())
    qkv = ops.columns(wide, 16, (heads + kv_heads) * d + extra)
    rotation = rotation_of(rot)[1]
    sizes = dict(heads=heads, kv_heads=kv_heads, head_dim=d)
    masks = dict(scale=d ** -0.5, window=window, keep_first=keep, sinks=torch.zeros(heads).cuda(),
                 slopes=torch.tensor([2.0 ** (-8.0 * (h + 1) / heads) for h in range(heads)]).cuda())
    assert ops.decode_attention_takes(qkv, page_size=page_size, rotation=rotation, dtype=dtype, **sizes)
    common = dict(q_weight=None, k_weight=None, eps=0.0, rotation=rotation, positions=positions, page_size=page_size,
                  extra_columns=extra, values_are_keys=True, **sizes)
    k_two, v_two = k_cache.clone(), v_cache.clone()
    q = ops.qk_norm_rope_store(qkv, slots=slots, k_cache=k_two, v_cache=v_two, dtype=dtype, **common)
    want = ops.paged_attention(q, k_cache=k_two, v_cache=v_two, page_size=page_size, block_tables=table, row_seq=row_seq,
                               positions=positions, cu_seqlens=None, seq_starts=None, single_rows=None, n_seqs=rows,
                               max_query=1, max_context=max(lengths), **masks, **sizes)
    k_one, v_one = k_cache.clone(), v_cache.clone()
    got = ops.decode_attention(qkv, writes=True, k_cache=k_one, v_cache=v_one, block_tables=table, row_seq=row_seq,
                               max_context=max(lengths), **masks, **common)
    assert torch.isfinite(got.float()).all()
    torch.testing.assert_close(got, want, atol=0, rtol=0)
    same = lambda a, b: torch.equal(a.view(torch.int16), b.view(torch.int16))          # NaN-filled pages: compare the bits
    assert same(k_one, k_two) and same(v_one, v_two), 'the pages differ'
    # with an output gate, from columns of the same product: the gate multiplies before the rounding
    logits = ops.columns(wide, 8, heads * d) if extra else ops.Partials((torch.randn(2, rows, heads * d, generator=g)).cuda())
    k_gated, v_gated = k_cache.clone(), v_cache.clone()
    gated = ops.decode_attention(qkv, writes=True, k_cache=k_gated, v_cache=v_gated, block_tables=table, row_seq=row_seq,
                                 max_context=max(lengths), gate=logits, **masks, **common)
    source = logits.source.sum()[:, 8:8 + heads * d] if extra else logits.sum()
    close(gated, want.float().cpu() * torch.sigmoid(source).cpu(), dtype, 0.3)
    assert same(k_gated, k_two) and same(v_gated, v_two), 'the pages differ'


# ------------------------------------------------------------------------------------------------ the recurrence
@pytest.mark.parametrize('dtype', DTYPES)
@pytest.mark.parametrize('heads,dim,vdim,groups,splits', [(4, 128, 64, 2, 3), (6, 33, 7, 3, 0), (1, 1, 1, 1, 1), (3, 200, 70, 1, 2),
                                                          (8, 64, 128, 8, 0), (5, 16, 130, 5, 4), (16, 128, 64, 1, 0), (2, 256, 72, 2, 2),
                                                          (4, 40, 8, 2, 1)])
def test_recurrence_with_step_sizes(dtype, heads, dim, vdim, groups, splits, monkeypatch):
    """Three sequences of unequal lengths with states of their own (one begins, whatever its slot holds), in blocks side by
    side and token by token; then the second part of each from what the first left."""
    if dtype == torch.float32 and splits == 0:
        splits = 1
    g = torch.Generator().manual_seed(heads * dim + vdim)
    lengths, starts, slots = [150, 1, 70], [0, 9, 200], [2, 0, 3]
    n = sum(lengths)
    inner, shared = heads * vdim, groups * dim
    u = (torch.randn(n, inner + 2 * shared, generator=g) / dim ** 0.25).to(dtype)
    raw = partials(torch.randn(n, heads + 11, generator=g).to(dtype), splits, g)
    bias, rates = torch.randn(heads, generator=g), -torch.exp(torch.randn(heads, generator=g) * 2 - 1)
    slot = ops.state_scan_slot(heads=heads, dim=dim, vdim=vdim, mode='step')
    assert slot == heads * dim * vdim
    state = torch.randn(5, slot, generator=g)
    state[2] = float('nan')                            # the slot of the sequence that begins
    cu = ints([0, 150, 151, 221])
    columns = dict(mode='step', heads=heads, dim=dim, vdim=vdim, groups=groups, v_offset=0, k_offset=inner, q_offset=inner + shared)
    want_state = state.clone()
    want, _ = refs.state_scan(u, gates=ops.columns(raw, 5, heads), gate_bias=bias, decay=rates, state=want_state,
                              cu_seqlens=cu, seq_starts=ints(starts), seq_slots=ints(slots), n_seqs=3, **columns)
    scale = max(1.0, want.abs().max().item())
    for longest, forms in ((150, True), (150, False), (None, True)):   # the matrix cores where they take the sizes; the general kernels
        monkeypatch.setattr(ops, 'STEP_FORMS', forms)
        got_state = state.cuda()
        got, _ = ops.state_scan(u.cuda(), gates=ops.columns(moved(raw), 5, heads), gate_bias=bias.cuda(), decay=rates.cuda(),
                                state=got_state, cu_seqlens=cu.cuda(), seq_starts=ints(starts).cuda(), seq_slots=ints(slots).cuda(),
                                n_seqs=3, max_query=longest, **columns)
        torch.testing.assert_close(got.cpu(), want, atol=2e-5 * scale, rtol=2e-5)
        live = [2, 0, 3]
        torch.testing.assert_close(got_state.cpu()[live], want_state[live], atol=2e-5 * scale, rtol=2e-5)
        assert torch.equal(got_state.cpu()[[1, 4]], state[[1, 4]]), 'a slot that belongs to nobody was written'


@pytest.mark.parametrize('dtype', DTYPES)
def test_recurrence_in_long_blocks(dtype):
    """Many blocks a sequence, the second half from the state the first left; decays from a token's to thousands of tokens'."""
    g = torch.Generator().manual_seed(5)
    heads, dim, vdim, groups, n = 4, 128, 64, 2, 900
    inner, shared = heads * vdim, groups * dim
    u = (torch.randn(n, inner + 2 * shared, generator=g) / 3).to(dtype)
    raw, bias = torch.randn(n, heads, generator=g).to(dtype), torch.tensor([3.0, 0.0, -4.0, 25.0])
    rates = torch.tensor([-20.0, -1e-4, -1.0, -1e-5])
    columns = dict(mode='step', heads=heads, dim=dim, vdim=vdim, groups=groups, v_offset=0, k_offset=inner, q_offset=inner + shared)
    want_state = torch.zeros(1, heads * dim * vdim)
    want, _ = refs.state_scan(u, gates=raw, gate_bias=bias, decay=rates, state=want_state, cu_seqlens=ints([0, n]),
                              seq_starts=ints([0]), seq_slots=ints([0]), n_seqs=1, **columns)
    state, rows, at = torch.full((1, heads * dim * vdim), float('nan')).cuda(), [], 0
    for size in (513, 1, 386):
        part, _ = ops.state_scan(u[at:at + size].cuda(), gates=raw[at:at + size].cuda(), gate_bias=bias.cuda(), decay=rates.cuda(),
                                 state=state, cu_seqlens=ints([0, size]).cuda(), seq_starts=ints([at]).cuda(),
                                 seq_slots=ints([0]).cuda(), n_seqs=1, max_query=size, **columns)
        rows.append(part)
        at += size
    got = torch.cat(rows).cpu().view(n, heads, vdim)
    for h in range(heads):                             # (a head that sums everything is thousands of times larger than one that forgets)
        expected = want.view(n, heads, vdim)[:, h]
        torch.testing.assert_close(got[:, h], expected, atol=1e-5 * expected.abs().max().item(), rtol=1e-4)
    torch.testing.assert_close(state.cpu(), want_state, atol=1e-5 * want_state.abs().max().item(), rtol=1e-4)


@pytest.mark.parametrize('dtype', DTYPES)
@pytest.mark.parametrize('lengths', [1, 5])
@pytest.mark.parametrize('heads,dim,vdim,groups', [(64, 128, 64, 8), (3, 256, 256, 1), (2, 5, 4, 2), (4, 100, 32, 1)])
def test_recurrence_one_token_a_sequence(dtype, lengths, heads, dim, vdim, groups):
    g = torch.Generator().manual_seed(dim + vdim)
    n, inner, shared = lengths, heads * vdim, groups * dim
    u = torch.randn(n, inner + 2 * shared, generator=g).to(dtype)
    raw, bias, rates = torch.randn(n, heads, generator=g).to(dtype), torch.randn(heads, generator=g), -torch.rand(heads, generator=g)
    state = torch.randn(n + 2, heads * dim * vdim, generator=g)
    starts, slots = ints([0 if i == 3 else 7 + i for i in range(n)]), ints([n + 1 - i for i in range(n)])
    columns = dict(mode='step', heads=heads, dim=dim, vdim=vdim, groups=groups, v_offset=0, k_offset=inner, q_offset=inner + shared)
    want_state, got_state = state.clone(), state.cuda()
    index = dict(cu_seqlens=ints(range(n + 1)), seq_starts=starts, seq_slots=slots)
    want, _ = refs.state_scan(u, gates=raw, gate_bias=bias, decay=rates, state=want_state, n_seqs=n, **index, **columns)
    got, _ = ops.state_scan(u.cuda(), gates=raw.cuda(), gate_bias=bias.cuda(), decay=rates.cuda(), state=got_state, n_seqs=n,
                            max_query=1, **{k: v.cuda() for k, v in index.items()}, **columns)
    scale = want.abs().max().item()
    torch.testing.assert_close(got.cpu(), want, atol=1e-5 * scale, rtol=1e-4)
    torch.testing.assert_close(got_state.cpu(), want_state, atol=1e-5, rtol=1e-5)


@pytest.mark.parametrize('dtype', DTYPES)
@pytest.mark.parametrize('n,heads,vdim,groups,splits,extra', [(37, 4, 64, 2, 3, 40), (5, 6, 7, 3, 0, 3), (1, 1, 1, 1, 1, 0),
                                                              (9, 3, 16, 2, 2, 8), (3, 64, 64, 8, 0, 16), (2, 2, 5000, 1, 1, 0)])
def test_gated_norm_in_groups(dtype, n, heads, vdim, groups, splits, extra):
    if dtype == torch.float32 and splits == 0:
        splits = 1
    g = torch.Generator().manual_seed(n * vdim)
    inner = heads * vdim
    o, u = torch.randn(n, inner, generator=g), torch.randn(n, inner + extra, generator=g).to(dtype)
    z = partials((2 * torch.randn(n, inner + extra + 8, generator=g)).to(dtype), splits, g)
    skip, weight = torch.randn(heads, generator=g), torch.rand(inner, generator=g) + 0.5
    args = dict(vdim=vdim, groups=groups, eps=1e-5, out_dtype=dtype)
    want = refs.gated_group_norm(o, u, skip=skip, z=ops.columns(z, 8, inner), weight=weight, **args)
    got = ops.gated_group_norm(o.cuda(), u.cuda(), skip=skip.cuda(), z=ops.columns(moved(z), 8, inner), weight=weight.cuda(), **args)
    close(got, want, dtype, 2.0)


# ------------------------------------------------------------------------------------------------ the stream
@pytest.mark.parametrize('dtype', DTYPES)
@pytest.mark.parametrize('n,width,splits', [(7, 64, 3), (33, 2048, 0), (3, 50, 1), (1, 5120, 4), (2, 12, 2)])
@pytest.mark.parametrize('shape', ['everything', 'one mixer', 'no feed-forward', 'no gates', 'nothing'])
def test_join_of_gated_branches(dtype, n, width, splits, shape):
    if dtype == torch.float32 and splits == 0:
        splits = 1
    g = torch.Generator().manual_seed(n * width)
    value = lambda columns=width: partials(torch.randn(n, columns, generator=g).to(dtype), splits, g)
    left, right, ffn = value(), value(), value()
    both = width if shape == 'no feed-forward' else 2 * width
    gates = value(both + 24)
    bias, plus, step = torch.randn(both, generator=g), torch.randn(n, width, generator=g), torch.randn(width, generator=g)
    stream, weight = torch.randn(n, width, generator=g), torch.rand(width, generator=g) + 0.5

    def joined(move, put):
        mixed = ops.Weighted(move(left), move(right), 0.7, -1.3) if shape != 'one mixer' else move(left)
        if shape == 'nothing':
            return ops.Joined(None, None, None, None, None, put(step))
        return ops.Joined(mixed, None if shape == 'no feed-forward' else move(ffn),
                          None if shape == 'no gates' else ops.columns(move(gates), 16, both), put(bias),
                          put(plus) if shape != 'one mixer' else None, put(step) if shape != 'no gates' else None)
    on_host, on_gpu = joined(lambda t: t, lambda t: t), joined(moved, lambda t: t.cuda())
    want_stream, got_stream = stream.clone(), stream.cuda()
    rows = ints(sorted({n - 1, n // 2}))
    want_rows = refs.residual_join(want_stream, on_host, weight, 1e-5, dtype, rows=rows)
    got_rows = ops.residual_join(got_stream, on_gpu, weight.cuda(), 1e-5, dtype, rows=rows.cuda())
    assert torch.equal(got_stream.cpu(), stream)
    close(got_rows, want_rows, dtype, 2.0)
    want = refs.residual_join(want_stream, on_host, weight, 1e-5, dtype)
    got = ops.residual_join(got_stream, on_gpu, weight.cuda(), 1e-5, dtype)
    torch.testing.assert_close(got_stream.cpu(), want_stream, atol=2e-5, rtol=2e-5)        # the stream is float32 in both
    close(got, want, dtype, 2.0)


@pytest.mark.parametrize('dtype', DTYPES)
@pytest.mark.parametrize('width,buckets,mul_prev,mul_cur', [(64, 31, 7, 5), (50, 1, 0, 0), (2048, 4093, 1 << 30, 1 << 29)])
def test_embedding_by_token_pairs(dtype, width, buckets, mul_prev, mul_cur):
    """The pair's row is made in 64 bits (the products of large multipliers and tokens do not fit in 32)."""
    g = torch.Generator().manual_seed(width)
    vocab, n = 50000, 41
    table, pairs = torch.randn(vocab, width, generator=g).to(dtype), torch.randn(buckets + 1, width, generator=g).to(dtype)
    tokens, previous = torch.randint(0, vocab, (n,), generator=g).to(torch.int32), torch.randint(-1, vocab, (n,), generator=g).to(torch.int32)
    previous[0], tokens[1], previous[1] = -1, vocab - 1, vocab - 1
    args = dict(scale=3.5, buckets=buckets, mul_prev=mul_prev, mul_cur=mul_cur)
    want = refs.embed_pairs(tokens, previous, table, pairs, **args)
    got, kept = ops.embed_pairs(tokens.cuda(), previous.cuda(), table.cuda(), pairs.cuda(), keep=True, **args)
    torch.testing.assert_close(got.cpu(), want, atol=1e-6, rtol=1e-6)
    assert torch.equal(got, kept) and got.data_ptr() != kept.data_ptr()
    assert torch.equal(ops.embed_pairs(tokens.cuda(), previous.cuda(), table.cuda(), pairs.cuda(), **args), got)


# ------------------------------------------------------------------------------------------------ one product for all
@pytest.mark.parametrize('dtype', DTYPES)
@pytest.mark.parametrize('n', [1, 8, 40, 300])
def test_matrices_side_by_side_share_one_product(dtype, n):
    """Every matrix's columns of the shared product are its own product; a matrix that is not in the stack gets its own; the
    relu-gated activation and the q/k kernel read columns."""
    g = torch.Generator().manual_seed(n)
    width, sizes = 256, [96, 40, 128]
    x = torch.randn(n, width, generator=g).to(dtype)
    matrices = [(torch.randn(rows, width, generator=g) / 16).to(dtype) for rows in sizes]
    other = (torch.randn(24, width, generator=g) / 16).to(dtype).cuda()
    stack = torch.zeros(96 + 48 + 128, width, dtype=dtype).cuda()
    places, views = {}, []
    for matrix, first in zip(matrices, (0, 96, 144)):
        view = stack[first:first + matrix.shape[0]]
        view.copy_(matrix)
        places[id(view)] = first
        views.append(view)
    shared = ops.SharedInput(x.cuda(), stack, places)
    for matrix, view in zip(matrices, views):
        got = ops.linear(shared, view, None, partials=True)
        assert isinstance(got, ops.Columns) and got.shape == (n, matrix.shape[0])
        source = got.source.sum() if isinstance(got.source, ops.Partials) else got.source
        close(source[:, got.offset:got.offset + matrix.shape[0]], x.float() @ matrix.float().t(), dtype, 4.0)
    alone = ops.linear(shared, other, None)
    close(alone, x.float() @ other.cpu().float().t(), dtype, 4.0)
    gate_up = x.float() @ matrices[2].float().t()
    for interleaved in (False, True):
        got = ops.gated_linear(shared, views[2], dtype, activation='relu', interleaved=interleaved)
        close(got, refs.gated_act(gate_up, dtype, activation='relu', interleaved=interleaved), dtype, 8.0)
    odd = ops.gated_act(ops.linear(shared, views[1], None, partials=True), dtype, activation='relu')
    close(odd, refs.gated_act(x.float() @ matrices[1].float().t(), dtype, activation='relu'), dtype, 8.0)
