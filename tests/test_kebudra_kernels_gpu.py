"""The kernels the Kebudra design added or changed, each alone against its plain reference (``kernel_refs``) on the same
inputs: several residual streams with the norm behind them, paired keys and queries, the difference of two maps (whole, and
from the parts of a split context), the delta rule token by token and in chunks with its state, gated products per head, columns
passed on by the convolution, and experts without a gate branch."""
import pytest
import torch

import kernel_refs as refs
from qil_amd import ops
from test_dogozen_kernels_gpu import close, ints, moved, partials
from test_kernels_gpu import build_cache
from test_tinuzen_kernels_gpu import attention_step

pytestmark = pytest.mark.gpu
DTYPES = [torch.float32, torch.bfloat16]


def on_gpu(pending):
    if isinstance(pending, ops.StreamUpdate):
        return ops.StreamUpdate(on_gpu(pending.value), pending.mix.cuda(), pending.out.cuda())
    if isinstance(pending, ops.RoutedSum):
        return ops.RoutedSum(pending.x.cuda(), pending.pairs.cuda(), pending.chosen.cuda(), pending.weights.cuda(), pending.experts)
    return None if pending is None else moved(pending)


class Settled:
    """A routed sum for the reference."""
    def __init__(self, routed):
        n, top = routed.chosen.shape
        value = torch.where((routed.chosen >= routed.experts)[:, :, None], routed.x.float()[:, None, :], routed.pairs.view(n, top, -1))
        self.total, self.shape, self.device = (value * routed.weights[:, :, None]).sum(1), routed.shape, routed.x.device

    def materialize(self):
        return self.total


@pytest.mark.parametrize('dtype', DTYPES)
@pytest.mark.parametrize('kind', ['none', 'tensor', 'partials', 'routed'])
@pytest.mark.parametrize('streams,width,n', [(1, 44, 5), (2, 64, 3), (3, 30, 7), (4, 256, 129), (2, 2048, 70), (5, 12, 2), (16, 8, 4), (2, 7, 9)])
def test_streams_join_and_the_norm_behind_them(dtype, kind, streams, width, n):
    g = torch.Generator().manual_seed(streams * width + n)
    stream = torch.randn(n, streams * width, generator=g)
    value = None
    if kind == 'tensor':
        value = torch.randn(n, width, generator=g).to(dtype)
    elif kind == 'partials':
        value = partials(torch.randn(n, width, generator=g), 5, g)
    elif kind == 'routed':
        value = ops.RoutedSum(torch.randn(n, width, generator=g).to(dtype), torch.randn(n * 3, width, generator=g),
                              torch.randint(0, 6, (n, 3), generator=g).to(torch.int32), torch.rand(n, 3, generator=g), 5)
    mix, out = torch.randn(streams, streams, generator=g), torch.randn(streams, generator=g)
    norm = (torch.tensor(0.7), torch.randn(width, generator=g), torch.randn(width, generator=g))
    read = torch.randn(streams, generator=g)
    rows = ints([n - 1, 0, n // 2])
    updates = [value] if streams == 1 or value is None else []
    if value is not None:
        updates.append(ops.StreamUpdate(value, mix, out))
    for pending in updates:
        reference = pending
        if kind == 'routed':
            reference = Settled(value) if pending is value else ops.StreamUpdate(Settled(value), mix, out)
        for chosen_norm, chosen_read, chosen_rows in ((norm, read, None), (None, read, None), (norm, None, rows)):
            want_stream, got_stream = stream.clone(), stream.cuda()
            arguments = dict(streams=streams, out_dtype=dtype)
            want = refs.stream_join(want_stream, reference, norm=chosen_norm, read=chosen_read, rows=chosen_rows, **arguments)
            got = ops.stream_join(got_stream, on_gpu(pending), norm=None if chosen_norm is None else tuple(t.cuda() for t in chosen_norm),
                                  read=None if chosen_read is None else chosen_read.cuda(),
                                  rows=None if chosen_rows is None else chosen_rows.cuda(), **arguments)
            close(got, want, dtype, 3.0)
            close(got_stream, want_stream, torch.float32, 3.0)


@pytest.mark.parametrize('dtype', DTYPES)
@pytest.mark.parametrize('streams,width', [(2, 64), (3, 30), (4, 2048)])
def test_the_embedding_in_every_stream(dtype, streams, width):
    g = torch.Generator().manual_seed(width)
    table, tokens = torch.randn(50, width, generator=g).to(dtype), torch.randint(0, 50, (17,), generator=g).to(torch.int32)
    got = ops.embed(tokens.cuda(), table.cuda(), 2.5, streams=streams)
    torch.testing.assert_close(got.cpu(), refs.embed(tokens, table, 2.5, streams=streams), atol=0, rtol=0)


# ------------------------------------------------------------------------------------------------ two maps a head
@pytest.mark.parametrize('dtype', DTYPES)
@pytest.mark.parametrize('heads,kv_heads,dim,vdim,splits,page_size,n', [
    (4, 2, 64, 128, 0, 16, 37), (4, 2, 64, 128, 3, 16, 5), (6, 3, 9, 13, 2, 8, 20), (3, 1, 16, 64, 0, 4, 33), (8, 8, 24, 8, 4, 16, 1),
    (2, 1, 128, 256, 0, 32, 18), (5, 0, 32, 64, 2, 16, 19), (16, 4, 64, 128, 0, 16, 300)])
def test_pairs_into_the_cache(dtype, heads, kv_heads, dim, vdim, splits, page_size, n):
    if dtype == torch.float32 and splits == 0:
        splits = 1
    g = torch.Generator().manual_seed(heads * dim + n)
    padded = -(-max(2 * dim, vdim) // 8) * 8
    pages = -(-n // page_size) + 3
    columns = (heads + kv_heads) * 2 * dim + kv_heads * vdim
    x = partials(torch.randn(n, columns + 24, generator=g).to(dtype), splits, g)
    slots = torch.randperm(pages * page_size, generator=g)[:n].to(torch.int32) if kv_heads else None
    cache = [torch.full((pages, max(kv_heads, 1), page_size, padded), float('nan')).to(dtype),
             torch.full((pages, max(kv_heads, 1), padded, page_size), float('nan')).to(dtype)]
    sizes = dict(heads=heads, kv_heads=kv_heads, dim=dim, vdim=vdim, padded=padded, page_size=page_size, dtype=dtype)
    mine = [t.cuda() for t in cache]
    want = refs.pair_store(x, slots=slots, k_cache=cache[0], v_cache=cache[1], **sizes)
    got = ops.pair_store(moved(x), slots=None if slots is None else slots.cuda(), k_cache=mine[0], v_cache=mine[1], **sizes)
    close(got, want, dtype, 0.3)
    for a, b in zip(mine, cache):
        assert torch.equal(torch.isnan(a.float()).cpu(), torch.isnan(b.float())), 'a place outside the slots was written'
        close(torch.nan_to_num(a.float()), torch.nan_to_num(b.float()), dtype, 0.3)


@pytest.mark.parametrize('dtype', DTYPES)
@pytest.mark.parametrize('heads,vdim,padded,n', [(4, 128, 128, 37), (3, 13, 24, 5), (2, 256, 256, 9), (16, 64, 128, 130), (1, 1, 8, 3),
                                                 (5, 200, 256, 4), (6, 96, 96, 11)])
def test_the_difference_of_two_maps(dtype, heads, vdim, padded, n):
    g = torch.Generator().manual_seed(vdim + n)
    maps = torch.randn(n, 2 * heads * padded, generator=g).to(dtype)
    gate = partials(torch.randn(n, heads + 13, generator=g), 3, g)
    arguments = dict(heads=heads, vdim=vdim, padded=padded, factor=0.7, post=0.4, eps=1e-3, dtype=dtype)
    want = refs.difference_combine(maps, ops.columns(gate, 5, heads), **arguments)
    got = ops.difference_combine(maps.cuda(), ops.columns(moved(gate), 5, heads), **arguments)
    close(got, want, dtype, 1.0)


@pytest.mark.parametrize('dtype', DTYPES)
@pytest.mark.parametrize('lengths,chunks,page_size,dim,vdim,heads,kv_heads', [
    ([2100, 1, 700, 1290], [1, 1, 1, 1], 16, 64, 128, 8, 4), ([900, 31], [1, 1], 16, 9, 13, 6, 3), ([3000], [1], 16, 32, 64, 4, 1),
    ([300, 2, 50], [1, 1, 1], 4, 128, 200, 4, 2), ([70, 70, 5, 33], [70, 2, 5, 1], 16, 64, 128, 4, 2), ([1200, 40], [1200, 1], 16, 64, 128, 4, 2),
    ([500, 300], [17, 300], 8, 24, 56, 6, 2)])
def test_two_maps_over_the_paged_cache(dtype, lengths, chunks, page_size, dim, vdim, heads, kv_heads):
    """Paired queries through the attention kernels (rows alone with their contexts in parts, portions) and their difference,
    against two attentions of their own per head."""
    padded = -(-max(2 * dim, vdim) // 8) * 8
    k_cache, v_cache, table, histories = build_cache(lengths, page_size, kv_heads, padded, dtype)
    k_cache[..., 2 * dim:] = 0.0
    v_cache[:, :, vdim:] = 0.0
    g = torch.Generator().manual_seed(dim)
    n, index = attention_step(lengths, chunks)
    x = torch.randn(n, heads * 2 * dim, generator=g).to(dtype)
    gate = torch.randn(n, heads, generator=g)
    q = ops.pair_store(x.cuda(), heads=heads, kv_heads=0, dim=dim, vdim=vdim, padded=padded, slots=None, k_cache=None, v_cache=None,
                       page_size=page_size, dtype=dtype)
    step = {k: None if v is None else v.cuda() for k, v in index.items()}
    maps = ops.paged_attention(q, heads=2 * heads, kv_heads=kv_heads, head_dim=padded, k_cache=k_cache, v_cache=v_cache, page_size=page_size,
                               block_tables=table, n_seqs=len(lengths), max_query=max(chunks), max_context=max(lengths), scale=0.2,
                               window=None, unmerged=True, **step)
    if max(chunks) == 1 and max(lengths) >= 2000:
        assert isinstance(maps, ops.Unmerged)
    got = ops.difference_combine(maps, gate.cuda(), heads=heads, vdim=vdim, padded=padded, factor=0.6, post=0.5, eps=1e-2, dtype=dtype)
    want = torch.zeros(n, heads, vdim, dtype=torch.float64)
    for row in range(n):
        k, v = (t[:int(index['positions'][row]) + 1].double() for t in histories[int(index['row_seq'][row])])
        for h in range(heads):
            a = [torch.softmax(k[:, h // (heads // kv_heads), m * dim:(m + 1) * dim] @
                               x[row].double().reshape(heads, 2, dim)[h, m] * 0.2, dim=0) @ v[:, h // (heads // kv_heads), :vdim] for m in (0, 1)]
            o = a[0] - 0.6 * a[1]
            want[row, h] = o / torch.sqrt(o.square().mean() + 1e-2) * 0.5 * torch.sigmoid(gate[row, h].double())
    close(got, want.reshape(n, -1), dtype, 0.5)


# ------------------------------------------------------------------------------------------------ the delta rule
def delta_inputs(n, heads, kv_heads, dim, vdim, splits, dtype, g):
    if dtype == torch.float32 and splits == 0:
        splits = 1
    channels = 2 * kv_heads * dim + heads * vdim
    u = torch.randn(n, channels + 8, generator=g).to(dtype)
    raised = partials(torch.randn(n, heads * (dim + vdim) + 8, generator=g).to(dtype), splits, g)
    steps = partials(torch.randn(n, heads + 11, generator=g).to(dtype), splits, g)
    fixed = dict(decay_bias=torch.randn(heads * dim, generator=g) * 2 - 1, rates=-torch.exp(torch.randn(heads, generator=g) * 2 - 2),
                 weight=torch.rand(vdim, generator=g) + 0.5)
    sizes = dict(heads=heads, kv_heads=kv_heads, dim=dim, vdim=vdim, k_offset=0, q_offset=kv_heads * dim, v_offset=2 * kv_heads * dim, eps=1e-4)
    return u, raised, steps, fixed, sizes


def delta_columns(raised, steps, sizes):
    heads, dim, vdim = sizes['heads'], sizes['dim'], sizes['vdim']
    return dict(decays=ops.columns(raised, 8, heads * dim), steps=ops.columns(steps, 5, heads),
                gate=ops.columns(raised, 8 + heads * dim, heads * vdim))


@pytest.mark.parametrize('dtype', DTYPES)
@pytest.mark.parametrize('heads,kv_heads,dim,vdim,splits', [(4, 2, 128, 128, 0), (6, 3, 33, 7, 3), (1, 1, 1, 1, 1), (3, 1, 200, 72, 2), (2, 2, 64, 64, 0),
                                                            (4, 1, 16, 300, 0), (2, 2, 256, 256, 0), (5, 5, 40, 130, 2), (2, 1, 96, 48, 0)])
def test_the_delta_rule(dtype, heads, kv_heads, dim, vdim, splits):
    """Three sequences of unequal lengths with states of their own (one begins, whatever its slot holds), in chunks beside a row
    that is alone, all in chunks, and token by token."""
    g = torch.Generator().manual_seed(heads * dim + vdim)
    lengths, starts, slots = [150, 70, 1], [0, 200, 9], [2, 3, 0]
    n = sum(lengths)
    u, raised, steps, fixed, sizes = delta_inputs(n, heads, kv_heads, dim, vdim, splits, dtype, g)
    state = torch.randn(5, heads * dim * vdim, generator=g)
    state[2] = float('nan')
    sequences = dict(cu_seqlens=ints([0, 150, 220, 221]), seq_starts=ints(starts), seq_slots=ints(slots))
    want_state = state.clone()
    want = refs.delta_rule(u.float(), state=want_state, n_seqs=3, accumulate=torch.float64, **delta_columns(raised, steps, sizes),
                           **fixed, **sequences, **sizes)
    u_gpu, columns = u.cuda(), delta_columns(moved(raised), moved(steps), sizes)
    there = {k: v.cuda() for k, v in {**fixed, **sequences}.items()}
    for longest, tiles in ((150, 2), (150, None), (31, None)):
        got_state = state.cuda()
        got = ops.delta_rule(u_gpu, state=got_state, n_seqs=3, max_query=longest, tile_seqs=tiles, **columns, **there, **sizes)
        close(got, want, dtype, 5.0 if dtype == torch.float32 else 1.0)
        live = [2, 3, 0]
        scale = want_state[live].abs().max().item()
        torch.testing.assert_close(got_state.cpu()[live], want_state[live], atol=2e-5 * scale, rtol=1e-4)
        assert torch.equal(got_state.cpu()[[1, 4]], state[[1, 4]]), 'a slot that belongs to nobody was written'


@pytest.mark.parametrize('dtype', DTYPES)
@pytest.mark.parametrize('dim,vdim', [(128, 128), (64, 96), (20, 12)])
def test_the_delta_rule_over_many_chunks(dtype, dim, vdim):
    """Many chunks a sequence, the rest from the state the first portion left; heads that forget within a token, within a chunk
    and hardly at all."""
    g = torch.Generator().manual_seed(5)
    heads, kv_heads, n = 4, 2, 900
    u, raised, steps, fixed, sizes = delta_inputs(n, heads, kv_heads, dim, vdim, 0, dtype, g)
    fixed['rates'] = torch.tensor([-20.0, -1e-4, -1.0, -0.02])
    fixed['decay_bias'] = torch.linspace(-8.0, 25.0, heads * dim)[torch.randperm(heads * dim, generator=g)]
    want_state = torch.zeros(1, heads * dim * vdim)
    want = refs.delta_rule(u.float(), state=want_state, n_seqs=1, cu_seqlens=ints([0, n]), seq_starts=ints([0]), seq_slots=ints([0]),
                           accumulate=torch.float64, **delta_columns(raised, steps, sizes), **fixed, **sizes)
    state, rows, at = torch.full((1, heads * dim * vdim), float('nan')).cuda(), [], 0
    there = {k: v.cuda() for k, v in fixed.items()}
    value = lambda x: x.sum() if isinstance(x, ops.Partials) else x
    for size in (513, 1, 7, 379):
        cut = lambda x: value(x)[at:at + size].contiguous().cuda()
        rows.append(ops.delta_rule(cut(u), state=state, n_seqs=1, max_query=size, cu_seqlens=ints([0, size]).cuda(), seq_starts=ints([at]).cuda(),
                                   seq_slots=ints([0]).cuda(), **delta_columns(cut(raised), cut(steps), sizes), **there, **sizes))
        at += size
    close(torch.cat(rows), want, dtype, 5.0 if dtype == torch.float32 else 1.0)
    torch.testing.assert_close(state.cpu(), want_state, atol=2e-5 * want_state.abs().max().item(), rtol=1e-4)


# ------------------------------------------------------------------------------------------------ changed kernels
@pytest.mark.parametrize('dtype', DTYPES)
@pytest.mark.parametrize('n,heads,k,o', [(5, 4, 64, 32), (70, 3, 40, 13), (300, 4, 128, 64), (300, 2, 24, 5), (1, 16, 512, 128)])
def test_a_gated_product_per_head(dtype, n, heads, k, o):
    g = torch.Generator().manual_seed(n)
    x, w = torch.randn(n, heads * k, generator=g), (torch.randn(heads, k, o, generator=g) / k ** 0.5).to(dtype)
    gate = partials(torch.randn(n, heads * o + 16, generator=g), 2 if n < 100 or dtype == torch.float32 else 0, g)
    want = refs.head_product(x, w, heads=heads, out_dtype=dtype, gate=ops.columns(gate, 8, heads * o))
    got = ops.head_product(x.cuda(), w.cuda(), heads=heads, out_dtype=dtype, gate=ops.columns(moved(gate), 8, heads * o))
    close(got, want, dtype, 1.0)


@pytest.mark.parametrize('dtype', DTYPES)
def test_latents_from_a_wider_product(dtype):
    """The latents' kernel on the leading columns of a stacked product whose other columns belong to someone else."""
    g = torch.Generator().manual_seed(3)
    n, q_rank, rank, rot = 19, 24, 40, 8
    from qil_amd.parts import RotaryFrequencies
    down = partials(torch.randn(n, q_rank + rank + rot + 56, generator=g), 3, g)
    weights = dict(q_weight=torch.rand(q_rank, generator=g) + 0.5, c_weight=torch.rand(rank, generator=g) + 0.5)
    places = dict(positions=ints(range(5, 5 + n)), slots=torch.randperm(32, generator=g)[:n].to(torch.int32))
    caches = dict(latent=torch.zeros(4, 8, rank).to(dtype), rope=torch.zeros(4, 8, rot).to(dtype))
    mine = {k: v.cuda() for k, v in caches.items()}
    sizes = dict(q_rank=q_rank, rank=rank, rot=rot, eps=1e-5, dtype=dtype)
    f = RotaryFrequencies(rot, 100.0).frequencies()
    want = refs.latent_prepare(ops.columns(down, 0, q_rank + rank + rot), frequencies=f, **weights, **places, **caches, **sizes)
    got = ops.latent_prepare(ops.columns(moved(down), 0, q_rank + rank + rot), frequencies=f.cuda(), **{k: v.cuda() for k, v in {**weights, **places}.items()},
                             **mine, **sizes)
    close(got, want, dtype, 1.0)
    for name in caches:
        close(mine[name], caches[name], dtype, 1.0)


@pytest.mark.parametrize('dtype', DTYPES)
@pytest.mark.parametrize('columns,pass_from,passed,splits', [(64, 64, 64, 3), (61, 64, 5, 2), (48, 56, 8, 0), (13, 14, 70, 1)])
def test_columns_passed_on_by_the_convolution(dtype, columns, pass_from, passed, splits):
    if dtype == torch.float32 and splits == 0:
        splits = 1
    g = torch.Generator().manual_seed(columns)
    lengths, starts, taps = [9, 1, 3], [0, 5, 1], 4
    n = sum(lengths)
    width = -(-(pass_from + passed) // 8) * 8
    x = partials(torch.randn(n, width, generator=g).to(dtype), splits, g)
    w, state = torch.randn(taps, columns, generator=g), torch.randn(4, taps - 1, columns, generator=g)
    step = dict(cu_seqlens=ints([0, 9, 10, 13]), seq_starts=ints(starts), seq_slots=ints([2, 0, 3]), row_seq=ints([0] * 9 + [1] + [2] * 3))
    sizes = dict(columns=columns, n_seqs=3, activation='silu', out_dtype=dtype, pass_from=pass_from, passed=passed)
    mine = state.cuda()
    want, through = refs.channel_conv(x, w, None, state=state, **step, **sizes)
    got, mine_through = ops.channel_conv(moved(x), w.cuda(), None, state=mine, **{k: v.cuda() for k, v in step.items()}, **sizes)
    close(got, want, dtype, 1.0)
    close(mine_through, through, dtype, 0.3)
    close(mine[[0, 2, 3]], state[[0, 2, 3]], torch.float32, 1.0)


@pytest.mark.parametrize('dtype', DTYPES)
@pytest.mark.parametrize('n,width,ff,experts,top', [(5, 64, 32, 8, 2), (9, 44, 20, 5, 3), (200, 128, 48, 4, 2), (300, 256, 160, 3, 2), (1, 512, 96, 16, 4),
                                                    (130, 40, 24, 2, 1), (260, 96, 272, 2, 2)])
def test_experts_without_a_gate_branch(dtype, n, width, ff, experts, top):
    g = torch.Generator().manual_seed(n + width)
    x = torch.randn(n, width, generator=g).to(dtype)
    up = (torch.randn(experts, 1, ff, width, generator=g) / width ** 0.5).to(dtype)
    down = (torch.randn(experts, width, ff, generator=g) / ff ** 0.5).to(dtype)
    chosen = torch.stack([torch.randperm(experts, generator=g)[:top] for _ in range(n)]).to(torch.int32)
    weights = torch.rand(n, top, generator=g)
    want = refs.moe_experts(x, chosen, weights, up, down, activation='relu_squared')
    arguments = (x.cuda(), chosen.cuda(), weights.cuda(), up.cuda(), down.cuda())
    close(ops.moe_experts(*arguments, activation='relu_squared'), want, dtype, 2.0)
    close(ops.moe_experts(*arguments, activation='relu_squared', lazy=True).materialize(), want, dtype, 2.0)


@pytest.mark.parametrize('dtype', DTYPES)
@pytest.mark.parametrize('n,outputs,identity,groups,keep,top', [(1, 32, 0, 1, 1, 4), (8, 16, 0, 1, 1, 2), (17, 40, 8, 4, 2, 6), (64, 7, 0, 1, 1, 7),
                                                                (64, 300, 0, 1, 1, 16), (65, 16, 0, 1, 1, 2)])
def test_choice_and_grouping_in_one_kernel(dtype, n, outputs, identity, groups, keep, top):
    """Steps of few rows are chosen and grouped by one kernel: the same choices and weights as by the two, bit for bit, and the
    experts' results from its grouping are those of the grouping made from the choices."""
    g = torch.Generator().manual_seed(n + outputs)
    width, ff, experts = 96, 32, outputs - identity
    x, router = torch.randn(n, width, generator=g).to(dtype).cuda(), torch.randn(outputs, width, generator=g).cuda()
    up = (torch.randn(experts, 1, ff, width, generator=g) / 10).to(dtype).cuda()
    down = (torch.randn(experts, width, ff, generator=g) / 6).to(dtype).cuda()
    rules = dict(groups=groups, keep=keep, top=top, renormalize=True)
    chosen, weights = ops.moe_route(x, router, None, **rules)
    same, share, grouping = ops.moe_route(x, router, None, align_for=experts, **rules)
    assert (grouping is not None) == (n <= 64 and outputs <= 300)
    assert torch.equal(chosen, same) and torch.equal(weights, share)
    want = ops.moe_experts(x, chosen, weights, up, down, activation='relu_squared')
    got = ops.moe_experts(x, same, share, up, down, activation='relu_squared', grouping=grouping)
    assert torch.equal(want, got)
