"""A matrix memory per head that is corrected towards each new value (the delta rule), with a decay per key channel."""
import torch

from .base import Mixer, ParamSpec, StateNeed, CompoundNeed
from .. import ops


class DeltaRule(Mixer):
    """With h the mixer's input, ``kv_heads`` heads of queries and keys [dim] and ``heads`` heads of values [vdim] (head h reads
    queries and keys of head h // (heads / kv_heads)):

        [q | k | v] = silu(conv(W h))    (W_q, W_k, W_v; causal, per channel, ``taps`` taps, no bias, zeros before the start)
        q, k <- unit vectors per head, x / sqrt(sum(x^2) + 1e-6);   q also times dim^(-1/2)
        beta = sigmoid(W_b h) per head,   g = exp(-exp(A_log) softplus(W_up W_down h + dt_bias)) per head and key channel
        S <- diag(g) S;   w = beta (v - S^T k);   S <- S + k w^T;   o = S^T q
        result = W_o (o / sqrt(mean(o^2) + eps) * norm * sigmoid(V_up V_down h))      (the mean over a head's vdim)

    The projections and the convolution with its activation run in the model's type; the unit norms, beta, the decays with
    their logarithms, the state and everything that touches it, the head norm and its gate are float32.  A request keeps the
    convolution's last ``taps - 1`` inputs and the state [heads, dim, vdim], each in a slot of its own kind (``cache_need``: a
    ``CompoundNeed``, or the state alone for a single tap).  The inner sizes of the two low-rank products are the
    checkpoint's (``decay_rank``, ``gate_rank`` are what random weights get).

    ``finalize`` stacks [W_q W_k W_v | W_down V_down | W_b] into one matrix (parts at multiples of 8 rows), lays W_up and V_up on
    the diagonal of one matrix, so that a second product makes the decays' and the gate's numbers at once, turns the
    convolutions' weights to [taps, channels] and makes -exp(A_log) once, in float32."""
    graph_safe = True

    def __init__(self, *, width, heads, kv_heads, dim, vdim, taps, eps, decay_rank=16, gate_rank=16, dtype=torch.bfloat16):
        super().__init__()
        for name, value in (('heads', heads), ('kv_heads', kv_heads), ('dim', dim), ('vdim', vdim), ('taps', taps)):
            if type(value) is not int or value < 1:
                raise ops.UnsupportedShape(f'{name} must be a positive integer, not {value!r}')
        ops.check_delta_geometry(heads=heads, kv_heads=kv_heads, dim=dim, vdim=vdim)
        self.width, self.heads, self.kv_heads, self.dim, self.vdim = int(width), heads, kv_heads, dim, vdim
        self.taps, self.eps, self.dtype = taps, float(eps), dtype
        self.decay_rank, self.gate_rank = int(decay_rank), int(gate_rank)
        self.channels = 2 * kv_heads * dim + heads * vdim

    def param_specs(self):
        qk, v, d, w = self.kv_heads * self.dim, self.heads * self.vdim, self.heads * self.dim, self.width
        specs = {}
        for name, rows in (('q', qk), ('k', qk), ('v', v)):
            specs[f'{name}_proj.weight'] = ParamSpec((rows, w))
            specs[f'{name}_conv.weight'] = ParamSpec((rows, self.taps), 'vector')
        specs.update({'b_proj.weight': ParamSpec((self.heads, w)), 'A_log': ParamSpec((self.heads,), 'vector'),
                      'dt_bias': ParamSpec((d,), 'vector'), 'out_norm.weight': ParamSpec((self.vdim,), 'vector', 'one_plus_normal'),
                      'decay_down.weight': ParamSpec((self.decay_rank, w), free=(0,)),
                      'decay_up.weight': ParamSpec((d, self.decay_rank), free=(1,)),
                      'gate_down.weight': ParamSpec((self.gate_rank, w), free=(0,)),
                      'gate_up.weight': ParamSpec((v, self.gate_rank), free=(1,)),
                      'o_proj.weight': ParamSpec((w, v))})
        return specs

    def cache_need(self):
        memory = StateNeed((self.heads * self.dim * self.vdim,), 'float32')
        if self.taps == 1:
            return memory
        return CompoundNeed((StateNeed((self.taps - 1, self.channels), 'float32'), memory))

    def finalize(self):
        p = self.p
        down, up = [], []
        for name in ('decay', 'gate'):
            down.append(p.pop(f'{name}_down.weight'))
            up.append(p.pop(f'{name}_up.weight'))
            if down[-1].shape[0] != up[-1].shape[1]:
                raise ValueError(f"the {name}'s two matrices do not fit: {tuple(down[-1].shape)} and {tuple(up[-1].shape)}")
        even = lambda rows: -(-rows // 8) * 8
        self.low = -(-sum(matrix.shape[0] for matrix in down) // 64) * 64       # whole stages of the product kernels
        self.low_offset = even(self.channels)
        self.beta_offset = self.low_offset + self.low
        w_in = down[0].new_zeros((self.beta_offset + even(self.heads), self.width))
        at = 0
        for name in ('q', 'k', 'v'):
            matrix = p.pop(f'{name}_proj.weight')
            w_in[at:at + matrix.shape[0]].copy_(matrix)
            at += matrix.shape[0]
        self.gate_offset = even(self.heads * self.dim)
        w_up = up[0].new_zeros((self.gate_offset + even(self.heads * self.vdim), self.low))
        row, column = 0, 0
        for matrix_down, matrix_up in zip(down, up):
            rank = matrix_down.shape[0]
            w_in[self.low_offset + column:self.low_offset + column + rank].copy_(matrix_down)
            w_up[row:row + matrix_up.shape[0], column:column + rank].copy_(matrix_up)
            row, column = self.gate_offset, column + rank
        w_in[self.beta_offset:self.beta_offset + self.heads].copy_(p.pop('b_proj.weight'))
        p['in_proj.weight'], p['up_proj.weight'] = w_in, w_up
        p['conv.weight'] = torch.cat([p.pop(f'{name}_conv.weight') for name in ('q', 'k', 'v')]).t().contiguous()
        p['rates'] = (-torch.exp(p.pop('A_log').to(torch.float32))).contiguous()

    def forward(self, h, ctx, cache):
        p = self.p
        conv_cache, memory = (None, cache) if self.taps == 1 else cache
        sequences = dict(cu_seqlens=ctx.cu_seqlens, seq_starts=ctx.seq_starts, seq_slots=ctx.seq_slots, n_seqs=ctx.n_seqs)
        proj = ops.linear(h, p['in_proj.weight'], None, partials=True)
        u, low = ops.channel_conv(proj, p['conv.weight'], None, columns=self.channels,
                                  state=conv_cache.state if conv_cache is not None else None, activation='silu', out_dtype=self.dtype,
                                  row_seq=ctx.row_seq, pass_from=self.low_offset, passed=self.low, **sequences)
        raised = ops.linear(low, p['up_proj.weight'], None, partials=True)
        qk = self.kv_heads * self.dim
        y = ops.delta_rule(u, ops.columns(raised, 0, self.heads * self.dim), ops.columns(proj, self.beta_offset, self.heads),
                           heads=self.heads, kv_heads=self.kv_heads, dim=self.dim, vdim=self.vdim, q_offset=0, k_offset=qk,
                           v_offset=2 * qk, decay_bias=p['dt_bias'], rates=p['rates'], state=memory.state, max_query=ctx.max_query,
                           gate=ops.columns(raised, self.gate_offset, self.heads * self.vdim), weight=p['out_norm.weight'],
                           eps=self.eps, tile_seqs=ctx.tile_seqs, **sequences)
        return ops.linear(y, p['o_proj.weight'], None, partials=True)
