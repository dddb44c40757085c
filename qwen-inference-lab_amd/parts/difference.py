"""Attention with two softmax maps a head over the same values, the second taken off the first."""
import torch

from .base import Mixer, ParamSpec, KVNeed
from .. import ops


class DifferenceAttention(Mixer):
    """Per head two queries, per key/value head two keys (each of ``head_dim``, laid out head by head as [first, second]) and
    one value (``value_dim``); each pair is a causal attention of its own over the same values:

        a_m(h, i) = softmax_j(scale q_m,h,i . k_m,g,j) v_g,j,   m = 1, 2,   g = h // (heads / kv_heads)
        o = a_1 - factor a_2,   o <- o / sqrt(mean(o^2) + eps) (1 - diff),   times sigmoid(W_g x)_h
        factor = exp(sum(lq1 lk1)) - exp(sum(lq2 lk2)) + diff      (stored vectors; one number for the layer)

    No rotation and no biases; positions enter through the mask only.

    The paged attention kernels run on it as they are.  A key head's two keys are one cached key [k1 | k2] of padded_dim
    elements, and a head's queries become two query heads [q1 | 0] and [0 | q2] of that size (``ops.pair_store``): a product
    with the cached key is exactly that of one map, both maps share a group's keys and values, and nothing is cached twice.
    ``padded_dim``: the larger of 2 head_dim and value_dim, padded with zeros to a multiple of 8.  The difference, its norm and the
    gate are one kernel (``ops.difference_combine``), which also merges the parts of a split context.
    ``own_kv=False``: no key and value projections; the schedule entry reads another entry's cache."""
    graph_safe = True

    def __init__(self, *, width, heads, kv_heads, head_dim, value_dim, scale, diff, eps, own_kv=True, dtype=torch.bfloat16):
        super().__init__()
        for name, value in (('heads', heads), ('kv_heads', kv_heads), ('head_dim', head_dim), ('value_dim', value_dim)):
            if type(value) is not int or value < 1:
                raise ops.UnsupportedShape(f'{name} must be a positive integer, not {value!r}')
        if heads % kv_heads:
            raise ValueError('heads must be a multiple of kv_heads')
        self.width, self.heads, self.kv_heads, self.head_dim, self.value_dim = int(width), heads, kv_heads, head_dim, value_dim
        self.scale, self.diff, self.eps, self.own_kv, self.dtype = float(scale), float(diff), float(eps), bool(own_kv), dtype
        self.padded_dim = -(-max(2 * head_dim, value_dim) // 8) * 8
        ops.check_attention_geometry(heads=2 * heads, kv_heads=kv_heads, head_dim=self.padded_dim, dtype=dtype)

    def param_specs(self):
        pair, d = 2 * self.head_dim, self.head_dim
        specs = {'q_proj.weight': ParamSpec((self.heads * pair, self.width)),
                 'o_proj.weight': ParamSpec((self.width, self.heads * self.value_dim)),
                 'g_proj.weight': ParamSpec((self.heads, self.width))}
        if self.own_kv:
            specs['k_proj.weight'] = ParamSpec((self.kv_heads * pair, self.width))
            specs['v_proj.weight'] = ParamSpec((self.kv_heads * self.value_dim, self.width))
        specs.update({name: ParamSpec((d,), 'vector') for name in ('lq1', 'lk1', 'lq2', 'lk2')})
        return specs

    def cache_need(self):
        return KVNeed(self.kv_heads, self.padded_dim)

    def finalize(self):
        p = self.p
        stacked = [p.pop(f'{name}_proj.weight') for name in (('q', 'k', 'v') if self.own_kv else ('q',))]
        self.gate_offset = 0
        for piece in (None, p.pop('g_proj.weight')):     # the gate's rows at a multiple of 8, the stack too
            if piece is not None:
                self.gate_offset = sum(matrix.shape[0] for matrix in stacked)
                stacked.append(piece)
            pad = -sum(matrix.shape[0] for matrix in stacked) % 8
            if pad:
                stacked.append(stacked[0].new_zeros((pad, self.width)))
        p['in_proj.weight'] = torch.cat(stacked).contiguous()
        lq1, lk1, lq2, lk2 = (p[name].double().cpu() for name in ('lq1', 'lk1', 'lq2', 'lk2'))
        self.factor = float(torch.exp((lq1 * lk1).sum()) - torch.exp((lq2 * lk2).sum())) + self.diff

    def forward(self, h, ctx, cache):
        if cache.writes and not self.own_kv:
            raise ValueError("an attention part without keys and values of its own reads another entry's cache")
        proj = ops.linear(h, self.p['in_proj.weight'], None, partials=True)
        q = ops.pair_store(proj, heads=self.heads, kv_heads=self.kv_heads if self.own_kv else 0, dim=self.head_dim,
                           vdim=self.value_dim, padded=self.padded_dim, slots=cache.slots if cache.writes else None,
                           k_cache=cache.k, v_cache=cache.v, page_size=cache.page_size, dtype=self.dtype)
        maps = ops.paged_attention(
            q, heads=2 * self.heads, kv_heads=self.kv_heads, head_dim=self.padded_dim, k_cache=cache.k, v_cache=cache.v,
            page_size=cache.page_size, block_tables=cache.block_tables, row_seq=ctx.row_seq, positions=ctx.positions,
            cu_seqlens=ctx.cu_seqlens, seq_starts=ctx.seq_starts, single_rows=ctx.single_rows, n_seqs=ctx.n_seqs,
            max_query=ctx.max_query, max_context=ctx.max_context, tile_seqs=ctx.tile_seqs, scale=self.scale, window=None,
            unmerged=True)
        out = ops.difference_combine(maps, ops.columns(proj, self.gate_offset, self.heads), heads=self.heads, vdim=self.value_dim,
                                     padded=self.padded_dim, factor=self.factor, post=1.0 - self.diff, eps=self.eps, dtype=self.dtype)
        return ops.linear(out, self.p['o_proj.weight'], None, partials=True)
