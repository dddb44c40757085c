"""Decode and prefill throughput of the engine at Qwen3-8B sizes on one MI355X.

    python bench.py [--gpus 1] [--steps K] [--warmup W] [--layers L] [--batch B] [--dtype bfloat16] [--sizes 8b]

Random weights, seeded uniform-random token ids.  A step is one decode step of the
serving loop (scheduler plan, one batched model step, greedy sampling, events) with
every request decoding at a 2,048-token history.  Prints ONE JSON line.

The protocol follows the reference's (benchmarks/compare_independent.py:148-159: a warm-up, the median of five
runs, the outputs of the runs compared): every decode point is measured --repeats times, each time from fresh
requests with the same prompts (W untimed steps, then exactly K timed steps between two synchronisations); the
line carries the median with the fastest and the slowest repeat, and says whether all repeats drew the same tokens.
"""
import argparse
import json
import random
import statistics
import sys
import time

HBM_GBPS = 8000.0                                   # MI355X published peaks
PEAK_TFLOPS = {'bfloat16': 2500.0, 'float32': 157.3}

SIZES = dict(vocab_size=151936, hidden_size=4096, intermediate_size=12288, num_hidden_layers=36,
             num_attention_heads=32, num_key_value_heads=8, head_dim=128, max_position_embeddings=4096,
             rms_norm_eps=1e-6, rope_theta=1000000.0, attention_bias=False, tie_word_embeddings=False,
             model_type='qwen3', architectures=['Qwen3ForCausalLM'], hidden_act='silu', eos_token_id=None)


# Other layer sizes to measure with --sizes (the default line is always the 8B set above).
OTHER_SIZES = {
    '8b': {},
    '32b': dict(hidden_size=5120, intermediate_size=25600, num_hidden_layers=64, num_attention_heads=64),
    '0.6b': dict(hidden_size=1024, intermediate_size=3072, num_hidden_layers=28, num_attention_heads=16,
                 tie_word_embeddings=True),
}
NAMES = {'8b': 'Qwen3-8B', '32b': 'Qwen3-32B', '0.6b': 'Qwen3-0.6B'}


def matrix_params_per_layer(c):
    qkv = (c['num_attention_heads'] + 2 * c['num_key_value_heads']) * c['head_dim'] * c['hidden_size']
    out = c['num_attention_heads'] * c['head_dim'] * c['hidden_size']
    return qkv + out + 3 * c['hidden_size'] * c['intermediate_size']


def decode_bytes(c, element, contexts):
    """Every weight the step uses once, and the cache of the live requests."""
    layers = c['num_hidden_layers']
    weights = layers * (matrix_params_per_layer(c) * element + (2 * c['hidden_size'] + 2 * c['head_dim']) * 4)
    weights += c['vocab_size'] * c['hidden_size'] * element + c['hidden_size'] * 4
    kv = sum(contexts) * layers * 2 * c['num_key_value_heads'] * c['head_dim'] * element
    return weights + kv + len(contexts) * c['hidden_size'] * element          # + the embedding rows


def prefill_flops(c, tokens):
    layers = c['num_hidden_layers']
    linear = 2 * tokens * layers * matrix_params_per_layer(c) + 2 * c['vocab_size'] * c['hidden_size']
    attention = layers * 4 * c['num_attention_heads'] * c['head_dim'] * tokens * (tokens + 1) // 2
    return linear + attention


def products_phase(args, torch, config):
    """The four matrix products of a layer at --prefill-tokens rows, each alone on data that the caches hold: the GPU
    BLAS (``torch.mm``) against this library's kernel for products of many rows, microseconds (the median of 3 replays of
    a graph of --steps calls) and PFLOP/s, with random operands and with zeros (the clock under load depends on the operands)."""
    import statistics as st
    from qil_amd import ops
    device = 'cuda:0'
    generator = torch.Generator(device=device).manual_seed(53)
    rows, hidden, inner = args.prefill_tokens, config['hidden_size'], config['intermediate_size']
    qkv = (config['num_attention_heads'] + 2 * config['num_key_value_heads']) * config['head_dim']
    shapes = {'qkv': (qkv, hidden), 'attention_output': (hidden, config['num_attention_heads'] * config['head_dim']),
              'gate_up': (2 * inner, hidden), 'down': (hidden, inner)}

    def timed(call):
        """Microseconds a call on the GPU: --steps calls recorded into a HIP graph and replayed, so that the host's
        time to launch (three times longer for the BLAS than for a kernel of this library) is not in it."""
        side = torch.cuda.Stream()
        side.wait_stream(torch.cuda.current_stream())
        with torch.cuda.stream(side):
            for _ in range(3):
                call()
        torch.cuda.current_stream().wait_stream(side)
        graph = torch.cuda.CUDAGraph()
        with torch.cuda.graph(graph):
            for _ in range(args.steps):
                call()
        graph.replay()
        out = []
        for _ in range(3):
            start, end = torch.cuda.Event(enable_timing=True), torch.cuda.Event(enable_timing=True)
            start.record()
            graph.replay()
            end.record()
            end.synchronize()
            out.append(start.elapsed_time(end) * 1000 / args.steps)
        return st.median(out)

    report = {'phase': 'products', 'rows': rows, 'sizes': NAMES[args.sizes]}
    for operands in ('random', 'zeros'):
        for name, (n, k) in shapes.items():
            if operands == 'random':
                x = torch.randn((rows, k), generator=generator, device=device).bfloat16()
                w = (torch.randn((n, k), generator=generator, device=device) * 0.02).bfloat16()
            else:
                x = torch.zeros((rows, k), dtype=torch.bfloat16, device=device)
                w = torch.zeros((n, k), dtype=torch.bfloat16, device=device)
            ops.OWN_LARGE_PRODUCTS = False
            blas = timed(lambda: ops.linear(x, w))
            ops.OWN_LARGE_PRODUCTS = True
            own = timed(lambda: ops.linear(x, w))
            ops.OWN_LARGE_PRODUCTS = False
            flops = 2.0 * rows * n * k
            report[f'{name}_{operands}'] = {'blas_us': round(blas, 1), 'own_us': round(own, 1),
                                            'blas_pflops': round(flops / blas / 1e9, 2), 'own_pflops': round(flops / own / 1e9, 2)}
    print(json.dumps(report))
    return 0


def attention_phase(args, torch, config, dtype):
    """The attention kernels alone.  (1) Decode attention at the shapes of the reference's own micro-benchmark
    (benchmarks/profile_paged.py:21-38: four requests, 16 query heads over 8 kv heads of 128, 16-token pages, 256
    pages, contexts of 128 x 4, 512 x 4, 17/63/255/511 and 32/128/512/2048; the median of 7 samples of 30 calls).
    (2) Prompt attention of one --prefill-tokens sequence at the benchmark configuration's heads, and decode attention
    of --batch rows at --history tokens, each called --steps times (a profiler's counters then see these kernels)."""
    import statistics as st
    from qil_amd import ops
    device = 'cuda:0'
    generator = torch.Generator(device=device).manual_seed(51)
    page_size = 16

    def timed(call, calls, samples=7):
        for _ in range(5):
            call()
        out = []
        for _ in range(samples):
            start, end = torch.cuda.Event(enable_timing=True), torch.cuda.Event(enable_timing=True)
            start.record()
            for _ in range(calls):
                call()
            end.record()
            end.synchronize()
            out.append(start.elapsed_time(end) * 1000 / calls)
        return round(st.median(out), 2)

    def caches(pages, kv_heads, d):
        k = torch.randn((pages, kv_heads, page_size, d), generator=generator, device=device, dtype=torch.float32).to(dtype)
        v = torch.randn((pages, kv_heads, d, page_size), generator=generator, device=device, dtype=torch.float32).to(dtype)
        return k, v

    def decode_call(lengths, heads, kv_heads, d):
        rows = len(lengths)
        per_row = [-(-n // page_size) for n in lengths]
        k, v = caches(max(256, sum(per_row)), kv_heads, d)
        width = max(per_row)
        table = torch.zeros((rows, width), dtype=torch.int32)
        at = 0
        for r, count in enumerate(per_row):
            table[r, :count] = torch.arange(at, at + count, dtype=torch.int32)
            at += count
        table = table.to(device)
        q = torch.randn((rows, heads * d), generator=generator, device=device, dtype=torch.float32).to(dtype)
        int32 = lambda values: torch.tensor(values, dtype=torch.int32, device=device)
        positions, row_seq = int32([n - 1 for n in lengths]), int32(list(range(rows)))
        return lambda: ops.paged_attention(
            q, heads=heads, kv_heads=kv_heads, head_dim=d, k_cache=k, v_cache=v, page_size=page_size, block_tables=table,
            row_seq=row_seq, positions=positions, cu_seqlens=None, seq_starts=None, single_rows=None, n_seqs=rows,
            max_query=1, max_context=max(lengths), scale=d ** -0.5, window=None)

    report = {'phase': 'attention', 'dtype': args.dtype, 'reference_shapes_us': {}}
    for lengths in ([128] * 4, [512] * 4, [17, 63, 255, 511], [32, 128, 512, 2048]):
        report['reference_shapes_us']['/'.join(map(str, lengths))] = timed(decode_call(lengths, 16, 8, 128), 30)
    heads, kv_heads, d = config['num_attention_heads'], config['num_key_value_heads'], config['head_dim']
    report[f'decode_{args.batch}x{args.history}_us'] = timed(decode_call([args.history] * args.batch, heads, kv_heads, d),
                                                             args.steps, samples=3)
    tokens = args.prefill_tokens
    pages = -(-tokens // page_size)
    k, v = caches(pages, kv_heads, d)
    q = torch.randn((tokens, heads * d), generator=generator, device=device, dtype=torch.float32).to(dtype)
    int32 = lambda values: torch.tensor(values, dtype=torch.int32, device=device)
    table = torch.arange(pages, dtype=torch.int32, device=device).view(1, pages)
    described = dict(row_seq=torch.zeros(tokens, dtype=torch.int32, device=device),
                     positions=torch.arange(tokens, dtype=torch.int32, device=device), cu_seqlens=int32([0, tokens]),
                     seq_starts=int32([0]), single_rows=int32([]))
    prompt_call = lambda: ops.paged_attention(
        q, heads=heads, kv_heads=kv_heads, head_dim=d, k_cache=k, v_cache=v, page_size=page_size, block_tables=table,
        n_seqs=1, max_query=tokens, max_context=tokens, scale=d ** -0.5, window=None, tile_seqs=1, **described)
    microseconds = timed(prompt_call, args.steps, samples=3)
    flops = 4 * heads * d * tokens * (tokens + 1) // 2
    report[f'prompt_{tokens}_us'] = microseconds
    report[f'prompt_{tokens}_tflops_causal'] = round(flops / microseconds / 1e6, 1)
    print(json.dumps(report))
    return 0



# ---------------------------------------------------------------------------------------------------------------
# --phase designs: the Fubapel design beside dense Qwen3 at equal sizes (width, feed-forward, layers, heads x head size)
DESIGN_SIZES = {
    # width, feed-forward, heads, head size of the attention; the latent's ranks; the memories' heads and head sizes
    '1b': dict(width=2048, ff=6144, heads=16, dim=128, rot_dim=64, kv_rank=512, q_rank=1536, memory_heads=8, memory_dim=128,
               memory_vdim=256),
    '8b': dict(width=4096, ff=12288, heads=32, dim=128, rot_dim=64, kv_rank=512, q_rank=1536, memory_heads=16, memory_dim=128,
               memory_vdim=256),
}


def fubapel_config(z, layers, vocab):
    """`layers` layers in turns of latent attention, gated memory, decaying memory; a feed-forward behind each."""
    ffn = dict(kind='dense', ff=z['ff'], limit=7.0)
    kinds = [
        dict(type='latent_attention', mlp=ffn,
             mixer=dict(heads=z['heads'], dim=z['dim'], rot_dim=z['rot_dim'], vdim=z['dim'], kv_rank=z['kv_rank'],
                        q_rank=z['q_rank'], rot=dict(base=10000.0, dims=z['rot_dim']), scale=(z['dim'] + z['rot_dim']) ** -0.5)),
        dict(type='mlstm', mlp=ffn, mixer=dict(heads=z['memory_heads'], dim=z['memory_dim'], vdim=z['memory_vdim'], gate_cap=15.0)),
        dict(type='retention', mlp=ffn,
             mixer=dict(heads=z['memory_heads'], dim=z['memory_dim'], vdim=z['memory_vdim'],
                        decay=[1 - 2.0 ** (-5 - i % 8) for i in range(z['memory_heads'])],
                        rot=dict(base=10000.0, dims=z['memory_dim']))),
    ]
    return dict(architecture='Fubapel', vocab=vocab, width=z['width'], layers=[kinds[i % 3] for i in range(layers)],
                loop=dict(start=0, stop=0, times=1), norm=dict(eps=1e-5), residual_mult=1.0)


def gerivik_config(z, layers, vocab):
    """`layers` layers in turns of gated linear attention and capped attention, a routed feed-forward behind each: 30
    experts and 2 identity experts in 4 groups of which 2 are kept, 4 chosen, every expert a quarter of the dense
    feed-forward (a token's experts together are as large as the dense one)."""
    ffn = dict(kind='moe', expert=dict(ff=z['ff'] // 4, limit=7.0),
               router=dict(experts=30, identity=2, top=4, groups=dict(count=4, keep=2)))
    kinds = [
        dict(type='gla', mlp=ffn, mixer=dict(heads=z['memory_heads'], dim=z['memory_dim'], vdim=z['memory_vdim'], tau=8.0)),
        dict(type='attention', mlp=ffn,
             mixer=dict(heads=z['heads'], kv_heads=max(1, z['heads'] // 4), dim=z['dim'], vdim=z['dim'],
                        rot=dict(base=10000.0, dims=z['rot_dim']), scale=z['dim'] ** -0.5, softcap=30.0)),
    ]
    return dict(architecture='Gerivik', vocab=vocab, width=z['width'], embedding=dict(scale=1.0),
                layers=[kinds[i % 2] for i in range(layers)], norm=dict(eps=1e-6))


def zinesun_config(z, layers, vocab, window, kind='turns'):
    """`layers` layers of windowed latent attention at the sizes of Fubapel's, a four-tap convolution in front of each;
    behind them a dense xielu feed-forward one and a half times as wide as the gated ones beside it (two matrices
    instead of three: equal weights and arithmetic), or a routed one (32 experts of a quarter of the gated
    feed-forward's inner size, 4 chosen: a token's experts are as large as the gated one), or both in turns."""
    mixer = dict(heads=z['heads'], dim=z['dim'], rot_dim=z['rot_dim'], vdim=z['dim'], kv_rank=z['kv_rank'], q_rank=z['q_rank'],
                 rot=dict(base=10000.0, dims=z['rot_dim']), scale=(z['dim'] + z['rot_dim']) ** -0.5, mask=dict(size=window))
    dense = dict(kind='dense', ff=z['ff'] * 3 // 2)
    routed = dict(kind='moe', expert=dict(ff=z['ff'] // 4), router=dict(experts=32, top=4))
    feeds = dict(turns=[dense, routed], dense=[dense], routed=[routed])[kind]
    return dict(architecture='Zinesun', vocab=vocab, width=z['width'], embedding=dict(scale=z['width'] ** 0.5), canon=dict(taps=4),
                layers=[dict(type='latent_attention', mixer=mixer, mlp=feeds[i % len(feeds)]) for i in range(layers)],
                norm=dict(eps=1e-5))


def dogozen_config(z, layers, vocab, window, kind='turns'):
    """`layers` layers of the Dogozen design: gated attention without a rotation (queries with a temperature) behind a
    routed feed-forward (32 experts in 4 groups of which 2 are kept, 4 chosen, each a quarter of the dense one, and a
    shared expert of that size), or windowed attention with sinks beside a selective scan (inner size twice the
    width, 16 states, four taps) behind a dense gated feed-forward, or both in turns; every fourth attention layer of
    the turns reads the keys and values of the one before it."""
    attention = dict(heads=z['heads'], kv_heads=max(1, z['heads'] // 4), dim=z['dim'], vdim=z['dim'], scale=z['dim'] ** -0.5,
                     q_temp=dict(coef=0.1, every=256))
    left = dict(heads=z['heads'], kv_heads=max(1, z['heads'] // 4), dim=z['dim'], vdim=z['dim'], scale=z['dim'] ** -0.5,
                rot=dict(base=10000.0, dims=z['rot_dim'], scaling=dict(factor=8.0, low=1.0, high=4.0, original=8192)),
                mask=dict(size=window))
    right = dict(inner=2 * z['width'], state=16, conv=4, dt_rank=z['width'] // 16)
    dense = dict(kind='dense', ff=z['ff'])
    routed = dict(kind='moe', expert=dict(ff=z['ff'] // 4), shared=dict(ff=z['ff'] // 4),
                  router=dict(experts=32, top=4, scale=2.5, groups=dict(count=4, keep=2)))
    gated = dict(type='attention', mixer=attention, mlp=routed)
    both = dict(type='parallel', mixer=dict(left=left, right=right, left_scale=0.5, right_scale=0.5), mlp=dense)
    if kind == 'turns':
        made = [both if i % 2 == 0 else gated for i in range(layers)]
        if layers >= 4:
            made[3] = dict(gated, mixer=dict(attention, kv_from=1))
    elif kind == 'attention':
        made = [dict(gated, mlp=dense)] * layers
    elif kind == 'attention-routed':
        made = [gated] * layers
    elif kind == 'window':
        made = [dict(both, mixer=dict(both['mixer'], right_scale=0.5, right=dict(inner=16, state=1, conv=1, dt_rank=1)))] * layers
    else:
        made = [both] * layers
    return dict(architecture='Dogozen', vocab=vocab, width=z['width'], layers=made, norm=dict(eps=1e-6), logit_softcap=30.0)


def tinuzen_config(z, layers, vocab, window, kind='turns'):
    """`layers` layers of the Tinuzen design, a relu-gated feed-forward beside the mixer of each: attention whose values
    are its keys beside a state-space recurrence (twice the width in heads of 64 channels, 128 states, 8 groups, four
    taps), or attention with a bias by distance and a window behind 64 kept first keys, or both in turns ('loop': the turns,
    half as many layers run twice); every bigram has a row of its own table of 8,191."""
    kv = max(1, z['heads'] // 4)
    left = dict(heads=z['heads'], kv_heads=kv, dim=z['dim'], vdim=z['dim'], scale=z['dim'] ** -0.5, rot=dict(base=10000.0, dims=z['rot_dim']))
    right = dict(heads=2 * z['width'] // 64, vdim=64, state=128, groups=8, conv=4, norm_groups=8)
    dense = dict(kind='dense', ff=z['ff'])
    both = dict(type='parallel', mlp=dense, mixer=dict(left=left, right=right, left_scale=0.5, right_scale=0.5))
    attention = dict(type='attention', mlp=dense,
                     mixer=dict(heads=z['heads'], kv_heads=kv, dim=z['dim'], vdim=z['dim'], scale=z['dim'] ** -0.5,
                                mask=dict(size=window, keep_first=64)))
    small = dict(both, mixer=dict(both['mixer'], right=dict(heads=1, vdim=64, state=16, groups=1, conv=4, norm_groups=1)))
    kinds = dict(turns=[both, attention], loop=[both, attention], parallel=[both], attention=[attention], left=[small])[kind]
    out = dict(architecture='Tinuzen', vocab=vocab, width=z['width'], norm=dict(eps=1e-6),
               embedding=dict(scale=z['width'] ** 0.5, bigram=dict(buckets=8191, mul_prev=31, mul_cur=17)),
               layers=[kinds[i % len(kinds)] for i in range(layers)])
    if kind == 'loop':
        out['layers'] = out['layers'][:max(1, layers // 2)]
        out['loop'] = dict(start=0, stop=max(1, layers // 2), times=2)
    return out


def kebudra_config(z, layers, vocab, kind='turns'):
    """`layers` layers of the Kebudra design with four residual streams, a routed feed-forward behind each (32 experts
    without a gate branch of which 4 are chosen, three eighths of the gated feed-forward's inner size each: a token's
    experts have its weights): the delta rule with a decay per key channel (heads of 128 x 128, a state as large as that of the
    other designs' memories), attention as the difference of two maps (two queries and two keys of half a head's size a
    head), latent attention at the sizes of Fubapel's, or the three in turns (the second difference layer of six reads the
    first one's cache)."""
    moe = dict(kind='moe', expert=dict(ff=z['ff'] * 3 // 8), router=dict(experts=32, top=4))
    heads = max(1, z['memory_heads'] * z['memory_vdim'] // 128)
    delta = dict(type='channel_delta', mlp=moe, mixer=dict(heads=heads, kv_heads=heads, dim=128, vdim=128, conv=4))
    difference = dict(type='attention', mlp=moe,
                      mixer=dict(heads=z['heads'], kv_heads=max(1, z['heads'] // 4), dim=z['dim'] // 2, vdim=z['dim'],
                                 scale=(z['dim'] // 2) ** -0.5, diff=0.5))
    latent = dict(type='latent_attention', mlp=moe,
                  mixer=dict(heads=z['heads'], dim=z['dim'], rot_dim=z['rot_dim'], vdim=z['dim'], kv_rank=z['kv_rank'], q_rank=z['q_rank'],
                             rot=dict(base=10000.0, dims=z['rot_dim']), scale=(z['dim'] + z['rot_dim']) ** -0.5))
    kinds = dict(turns=[delta, difference, latent], delta=[delta], difference=[difference], latent=[latent])[kind]
    made = [kinds[i % len(kinds)] for i in range(layers)]
    if kind == 'turns' and layers >= 5:
        made[4] = dict(difference, mixer=dict(difference['mixer'], kv_from=1))
    return dict(architecture='Kebudra', vocab=vocab, width=z['width'], streams=4, embedding=dict(scale=z['width'] ** 0.5),
                layers=made, norm=dict(eps=1e-6))


def designs_phase(args, torch, dtype):
    """Prefill tokens a second and decode milliseconds a step of a design's models whose layers are all of one kind
    (and of its kinds in turns), beside dense Qwen3 of the same width, feed-forward, depth and attention heads."""
    from qil_amd import Engine, Qwen3
    from qil_amd.engine import ModelRunner, StepEntry
    z, layers, vocab, page_size = DESIGN_SIZES[args.design_sizes], args.layers or 6, 32768, 16
    generator = torch.Generator().manual_seed(99)
    if args.design == 'zinesun':
        # beside it the closest models of the engine: Fubapel's latent attention (no window, no gate, no convolution, a
        # gated feed-forward, pre-norm) and Gerivik's capped attention with the routed feed-forward
        models = {f'zinesun ({name}, window {args.design_window})': zinesun_config(z, layers, vocab, args.design_window, kind)
                  for kind, name in (('turns', 'feed-forwards in turns'), ('dense', 'dense feed-forwards'), ('routed', 'routed feed-forwards'))}
        models[f'zinesun (dense feed-forwards, window {8 * args.design_window})'] = zinesun_config(z, layers, vocab, 8 * args.design_window, 'dense')
        models['fubapel (latent attention only)'] = dict(fubapel_config(z, layers, vocab), layers=[fubapel_config(z, 1, vocab)['layers'][0]] * layers)
        models['gerivik (capped attention only)'] = dict(gerivik_config(z, layers, vocab), layers=[gerivik_config(z, 2, vocab)['layers'][1]] * layers)
    elif args.design == 'dogozen':
        # beside it the closest model of the engine: Gerivik's capped attention with the routed feed-forward (the same
        # arrangement of norms, grouped-query attention of the same sizes, a routed feed-forward of the same sizes)
        names = (('turns', 'kinds in turns'), ('attention', 'gated attention, dense feed-forwards'),
                 ('attention-routed', 'gated attention, routed feed-forwards'),
                 ('parallel', f'window {args.design_window} beside a scan, dense feed-forwards'),
                 ('window', f'window {args.design_window} beside a scan of one channel group, dense feed-forwards'))
        models = {f'dogozen ({name})': dogozen_config(z, layers, vocab, args.design_window, kind) for kind, name in names}
        models['gerivik (capped attention only)'] = dict(gerivik_config(z, layers, vocab), layers=[gerivik_config(z, 2, vocab)['layers'][1]] * layers)
    elif args.design == 'tinuzen':
        # beside it the closest models of the engine: Dogozen's two kinds of layer with dense feed-forwards (two mixers side
        # by side, one of them a state-space scan; gated attention) and Fubapel's memory with fixed decays (a matrix
        # state per head)
        names = (('turns', f'kinds in turns, window {args.design_window}'), ('loop', 'kinds in turns, half the layers twice'),
                 ('parallel', 'attention beside a recurrence'), ('attention', f'window {args.design_window} with a bias by distance'),
                 ('left', 'attention beside a recurrence of one head'))
        models = {f'tinuzen ({name})': tinuzen_config(z, layers, vocab, args.design_window, kind) for kind, name in names}
        models['dogozen (window beside a scan)'] = dogozen_config(z, layers, vocab, args.design_window, 'parallel')
        models['dogozen (gated attention)'] = dogozen_config(z, layers, vocab, args.design_window, 'attention')
        models['fubapel (decaying memory only)'] = dict(fubapel_config(z, layers, vocab), layers=[fubapel_config(z, 3, vocab)['layers'][2]] * layers)
    elif args.design == 'kebudra':
        # beside it the closest models of the engine: Gerivik's memory with a decay per row (a matrix state of the same size
        # per layer, a routed feed-forward), its attention, and Fubapel's latent attention
        names = (('turns', 'kinds in turns'), ('delta', 'delta rule'), ('difference', 'difference of two maps'), ('latent', 'latent attention'))
        models = {f'kebudra ({name})': kebudra_config(z, layers, vocab, kind) for kind, name in names}
        gerivik = gerivik_config(z, layers, vocab)
        for index, name in enumerate(('gated linear attention', 'capped attention')):
            models[f'gerivik ({name} only)'] = dict(gerivik, layers=[gerivik['layers'][index]] * layers)
        models['fubapel (latent attention only)'] = dict(fubapel_config(z, layers, vocab), layers=[fubapel_config(z, 1, vocab)['layers'][0]] * layers)
    elif args.design == 'gerivik':
        mixed = gerivik_config(z, layers, vocab)
        models = {'gerivik (kinds in turns)': mixed}
        for index, name in enumerate(('gated linear attention', 'capped attention')):
            models[f'gerivik ({name} only)'] = dict(mixed, layers=[mixed['layers'][index]] * layers)
    else:
        mixed = fubapel_config(z, layers, vocab)
        models = {'fubapel (kinds in turns)': mixed}
        for index, name in enumerate(('latent attention', 'gated memory', 'decaying memory')):
            models[f'fubapel ({name} only)'] = dict(mixed, layers=[mixed['layers'][index]] * layers)
    models['qwen3 (equal sizes)'] = dict(SIZES, vocab_size=vocab, hidden_size=z['width'], intermediate_size=z['ff'],
                                         num_hidden_layers=layers, num_attention_heads=z['heads'],
                                         num_key_value_heads=max(1, z['heads'] // 4), head_dim=z['dim'],
                                         max_position_embeddings=max(args.history + args.steps + args.warmup + 64, args.prefill_tokens))
    if args.design_only:
        models = {name: config for name, config in models.items() if args.design_only in name}
    report = {'phase': 'designs', 'design': args.design, 'sizes': args.design_sizes, 'layers': layers, 'dtype': args.dtype,
              'prefill_tokens': args.prefill_tokens, 'batch': args.batch, 'history': args.history, 'models': {}}
    for name, config in models.items():
        model = Qwen3.from_config(config, seed=0, dtype=dtype, device='cuda:0', on_device=True)
        tokens = lambda n: torch.randint(0, vocab, (n,), generator=generator).tolist()
        runner = ModelRunner(model, num_pages=-(-args.prefill_tokens // page_size) + 1, page_size=page_size, max_requests=1)
        times = []
        for attempt in range(4):
            runner.admit(attempt)
            ids = tuple(tokens(args.prefill_tokens))
            torch.cuda.synchronize()
            started = time.perf_counter()
            logits = runner.step([StepEntry(attempt, ids, (args.prefill_tokens - 1,))])
            torch.cuda.synchronize()
            times.append(time.perf_counter() - started)
            assert torch.isfinite(logits).all()
            runner.release(attempt)
        prefill_s = statistics.median(times[1:])
        del runner
        new_tokens = args.warmup + args.steps + 8
        pages = args.batch * (-(-(args.history + new_tokens) // page_size) + 1)
        engine = Engine(model, num_pages=pages, page_size=page_size, token_budget=args.history + args.batch,
                        prefill_chunk=args.history, max_active=args.batch)
        ids = [engine.submit(tokens(args.history), max_new_tokens=new_tokens, ignore_eos=True) for _ in range(args.batch)]
        while any(engine.result(i)['state'] == 'waiting' or engine.scheduler.computed(i) < args.history for i in ids):
            engine.step()
        for _ in range(args.warmup):
            engine.step()
        torch.cuda.synchronize()
        started = time.perf_counter()
        for _ in range(args.steps):
            assert len(engine.step()) == args.batch
        torch.cuda.synchronize()
        step_s = (time.perf_counter() - started) / args.steps
        engine.close()
        report['models'][name] = {'prefill_ms': round(prefill_s * 1e3, 3), 'prefill_tokens_per_s': round(args.prefill_tokens / prefill_s, 1),
                                  'decode_ms_per_step': round(step_s * 1e3, 4), 'decode_tokens_per_s': round(args.batch / step_s, 1),
                                  'parameter_mb': round(model.parameter_bytes() / 1e6, 1)}
        print(f'[bench] {name}: prefill {prefill_s * 1e3:.2f} ms, decode {step_s * 1e3:.3f} ms/step', file=sys.stderr, flush=True)
        del engine, model
        torch.cuda.empty_cache()
    print(json.dumps(report))
    return 0


def main():
    parser = argparse.ArgumentParser()
    parser.add_argument('--gpus', type=int, default=1)
    parser.add_argument('--steps', type=int, default=128)
    parser.add_argument('--warmup', type=int, default=8)
    parser.add_argument('--sizes', default='8b', choices=sorted(OTHER_SIZES), help='layer sizes (default: the benchmark\'s)')
    parser.add_argument('--layers', type=int, default=None, help='fewer layers than the size set has (both numbers are reported)')
    parser.add_argument('--batch', type=int, default=8)
    parser.add_argument('--repeats', type=int, default=5, help='timed regions per decode point (the median is reported)')
    parser.add_argument('--history', type=int, default=2048)
    parser.add_argument('--dtype', default='bfloat16', choices=['bfloat16', 'float32'])
    parser.add_argument('--points', default='1,64', help='other decode batch sizes to report, comma separated')
    parser.add_argument('--prefill-tokens', type=int, default=2048)
    parser.add_argument('--phase', default='all', choices=['all', 'decode', 'prefill', 'e2e', 'mixed', 'attention', 'products', 'designs'],
                        help='measure only one phase (for profiling); the JSON line then lacks the other.  e2e: the '
                             'reference\'s own workloads (output tokens over the wall time of whole requests).  '
                             'mixed: steps of one prompt portion (--portion tokens) beside --batch decoded rows.  attention: the '
                             'attention kernels alone, at the reference\'s own shapes and at the benchmark\'s.  products: a layer\'s '
                             'matrix products at --prefill-tokens rows alone, GPU BLAS against own kernel.  designs: prefill and decode of the '
                             'design named by --design at --design-sizes beside dense Qwen3 of equal sizes (--layers, default 6)')
    parser.add_argument('--design', default='fubapel', choices=['fubapel', 'gerivik', 'zinesun', 'dogozen', 'tinuzen', 'kebudra'], help='the design of --phase designs')
    parser.add_argument('--design-window', type=int, default=512, help='the attention window of --design zinesun, dogozen and tinuzen')
    parser.add_argument('--design-only', default=None, help='of the models of --phase designs, only those whose name holds this (for profiling)')
    parser.add_argument('--design-sizes', default='1b', choices=sorted(DESIGN_SIZES), help='layer sizes of --phase designs')
    parser.add_argument('--portion', type=int, default=128, help='tokens of the prompt portion of a mixed step')
    parser.add_argument('--own-products', action='store_true',
                        help='bfloat16 matrix products of many rows on this library\'s kernels instead of the GPU BLAS '
                             '(qil_amd.ops.OWN_LARGE_PRODUCTS)')
    args = parser.parse_args()
    if args.gpus != 1:
        print(f'bench.py measures one GPU: this engine runs on a single MI355X (asked for {args.gpus})')
        return 2

    import torch
    from qil_amd import Engine, Qwen3
    from qil_amd import ops
    from qil_amd.engine import ModelRunner, StepEntry
    ops.OWN_LARGE_PRODUCTS = args.own_products
    if args.phase == 'designs':
        return designs_phase(args, torch, getattr(torch, args.dtype))

    sizes = dict(SIZES, **OTHER_SIZES[args.sizes])
    if args.layers is None:
        args.layers = sizes['num_hidden_layers']
    config = dict(sizes, num_hidden_layers=args.layers)
    longest = args.history + args.warmup + args.steps + 2 * max([args.batch] + [int(b) for b in args.points.split(',') if b]) + 8
    longest = max(longest, args.prefill_tokens)
    if longest > config['max_position_embeddings']:             # --history or --prefill-tokens beyond the size set's context
        config['max_position_embeddings'] = longest
    dtype = getattr(torch, args.dtype)
    element = 2 if args.dtype == 'bfloat16' else 4
    if args.phase == 'attention':
        return attention_phase(args, torch, config, dtype)
    if args.phase == 'products':
        return products_phase(args, torch, config)
    model = Qwen3.from_config(config, seed=0, dtype=dtype, device='cuda:0', on_device=True)
    generator = torch.Generator().manual_seed(1234)
    page_size = 16

    def prompt(length, seed=None):
        """Uniform-random token ids: from the run's generator, or (seed given) the same ids whenever asked."""
        source = generator if seed is None else torch.Generator().manual_seed(seed)
        return torch.randint(0, config['vocab_size'], (length,), generator=source).tolist()

    def decode_once(batch):
        """(seconds per step, contexts at the middle of the timed steps, drawn tokens) of `batch` requests decoding
        together: fresh requests, the same prompts every time."""
        # requests that finish their prompt early decode while the others still prefill (about one
        # prompt a step): leave room for that many extra tokens
        new_tokens = args.warmup + args.steps + 2 * batch + 8
        pages = batch * (-(-(args.history + new_tokens) // page_size) + 1)
        engine = Engine(model, num_pages=pages, page_size=page_size, token_budget=args.history + batch,
                        prefill_chunk=args.history, max_active=batch)
        ids = [engine.submit(prompt(args.history, seed=5000 + index), max_new_tokens=new_tokens, ignore_eos=True)
               for index in range(batch)]
        computed = engine.scheduler.computed
        drawn = []
        while any(engine.result(i)['state'] == 'waiting' or computed(i) < args.history for i in ids):      # untimed: histories into the cache
            drawn += [(e['request_id'], e['token_id']) for e in engine.step()]
        for _ in range(args.warmup):
            drawn += [(e['request_id'], e['token_id']) for e in engine.step()]
        torch.cuda.synchronize()
        started = time.perf_counter()
        events = []
        for _ in range(args.steps):
            events.append(engine.step())
        torch.cuda.synchronize()
        elapsed = time.perf_counter() - started
        assert sum(len(e) for e in events) == batch * args.steps, 'a decode step must produce one token per request'
        drawn += [(e['request_id'], e['token_id']) for step in events for e in step]
        contexts = [computed(i) - args.steps // 2 for i in ids]
        engine.close()
        engine.cache.check()
        assert engine.cache.free_pages == [pages], 'pages leaked'
        del engine
        torch.cuda.empty_cache()
        return elapsed / args.steps, contexts, drawn

    def decode_run(batch):
        """The median of --repeats such runs: (seconds per step, contexts, [fastest, slowest], whether every repeat
        drew the same tokens)."""
        runs = [decode_once(batch) for _ in range(max(1, args.repeats))]
        times = sorted(run[0] for run in runs)
        agree = all(run[2] == runs[0][2] for run in runs)
        if not agree:
            note(f'decode batch {batch}: the repeats did not draw the same tokens')
        return statistics.median(times), runs[0][1], [times[0], times[-1]], agree

    def prefill_run(tokens):
        runner = ModelRunner(model, num_pages=-(-tokens // page_size) + 1, page_size=page_size, max_requests=1)
        times = []
        for attempt in range(4):
            ids = tuple(prompt(tokens))
            runner.admit(attempt)
            torch.cuda.synchronize()
            started = time.perf_counter()
            logits = runner.step([StepEntry(attempt, ids, (tokens - 1,))])
            torch.cuda.synchronize()
            times.append(time.perf_counter() - started)
            assert torch.isfinite(logits).all()
            runner.release(attempt)
        return statistics.median(times[1:])

    def note(text):
        print(f'[bench] {text}', file=sys.stderr, flush=True)

    if args.phase == 'e2e':
        # The reference's published workloads (docs/prefill-gpu-validation-2026-09-20.md:26-31, README.md:38-41):
        # 1 or 4 requests with prompts of 128 / 512 / 2048 tokens, 32 output tokens each, greedy, 16-token pages,
        # token budget 512, portions of 128, 4 active; one warm-up, the median of five runs; output tokens over
        # the wall time of the whole batch (prefill and decode).
        table = {}
        for length in (128, 512, 2048):
            for count in (1, 4):
                engine = Engine(model, num_pages=640 if length == 2048 else 256, page_size=16, token_budget=512,
                                prefill_chunk=128, max_active=4)
                times = []
                for attempt in range(6):
                    prompts = [prompt(length) for _ in range(count)]
                    torch.cuda.synchronize()
                    started = time.perf_counter()
                    results = engine.generate(prompts, max_new_tokens=32, ignore_eos=True)
                    times.append(time.perf_counter() - started)
                    assert all(len(r['token_ids']) == 32 for r in results)
                engine.close()
                table[f'{length}x{count}'] = round(32 * count / statistics.median(times[1:]), 1)
        # A mixed batch: 8 requests with prompts of 16 to 2,048 tokens (seeded), portions of 128 under a budget of 512
        # tokens, 8 active, 32 output tokens each.
        lengths = [random.Random(7 + i).randrange(16, 2049) for i in range(8)]
        engine = Engine(model, num_pages=sum(-(-(n + 32) // 16) for n in lengths) + 8, page_size=16, token_budget=512,
                        prefill_chunk=128, max_active=8)
        times = []
        for attempt in range(4):
            prompts = [prompt(n) for n in lengths]
            torch.cuda.synchronize()
            started = time.perf_counter()
            results = engine.generate(prompts, max_new_tokens=32, ignore_eos=True)
            times.append(time.perf_counter() - started)
            assert all(len(r['token_ids']) == 32 for r in results)
        # once more, step by step with a synchronisation after every step: where the time of this workload goes
        ids = [engine.submit(prompt(n), max_new_tokens=32, ignore_eos=True) for n in lengths]
        kinds = {'portions': [], 'portions beside decoded rows': [], 'decoded rows only': []}
        while not engine.idle:
            torch.cuda.synchronize()
            started = time.perf_counter()
            events = engine.step()
            torch.cuda.synchronize()
            elapsed = time.perf_counter() - started
            stats = engine.stats()
            tokens, requests = stats['last_step_tokens'], stats['last_step_requests']
            kind = 'decoded rows only' if tokens == requests else \
                'portions beside decoded rows' if len(events) > 1 or requests > -(-tokens // 128) else 'portions'
            kinds[kind].append((elapsed, tokens))
        breakdown = {kind: {'steps': len(rows), 'ms_per_step': round(1e3 * sum(t for t, _ in rows) / len(rows), 3),
                            'tokens_per_step': round(sum(n for _, n in rows) / len(rows), 1),
                            'ms': round(1e3 * sum(t for t, _ in rows), 2)} for kind, rows in kinds.items() if rows}
        engine.close()
        table['16-2048x8'] = round(32 * 8 / statistics.median(times[1:]), 1)
        print(json.dumps({'e2e_output_tokens_per_s': table, 'mixed_batch_steps': breakdown, 'sizes': NAMES[args.sizes],
                          'layers': args.layers, 'dtype': args.dtype}))
        return 0
    if args.phase == 'mixed':
        # One request's prompt arrives in portions while `batch` others decode: every step is one batch of
        # portion + batch rows, the decoding requests at --history tokens, the prompt growing from --history on.
        steps = min(args.steps, 12)
        room = args.history + (steps + 1) * args.portion + 16
        config_room = config['max_position_embeddings']
        if room > config_room:
            raise SystemExit(f'--history {args.history} and {steps} portions of {args.portion} need {room} positions, the model has {config_room}')
        runner = ModelRunner(model, num_pages=(args.batch + 1) * (-(-room // page_size) + 1), page_size=page_size,
                             max_requests=args.batch + 1)
        for request in range(args.batch + 1):
            runner.admit(request)
            runner.step([StepEntry(request, tuple(prompt(args.history)), ())])
        feed, times = prompt(room), []
        for index in range(steps + 1):
            entries = [StepEntry(args.batch, tuple(feed[index * args.portion:(index + 1) * args.portion]), (args.portion - 1,))]
            entries += [StepEntry(request, (feed[request + index],), (0,)) for request in range(args.batch)]
            torch.cuda.synchronize()
            started = time.perf_counter()
            logits = runner.step(entries)
            torch.cuda.synchronize()
            times.append(time.perf_counter() - started)
            assert logits.shape[0] == args.batch + 1 and torch.isfinite(logits).all()
        print(json.dumps({'mixed_ms_per_step': round(statistics.median(times[1:]) * 1e3, 3), 'portion': args.portion,
                          'decoded_rows': args.batch, 'history': args.history, 'layers': args.layers,
                          'sizes': NAMES[args.sizes], 'dtype': args.dtype}))
        return 0
    if args.phase == 'prefill':
        prefill_s = prefill_run(args.prefill_tokens)
        print(json.dumps({'prefill_ms': round(prefill_s * 1e3, 3), 'tokens': args.prefill_tokens, 'layers': args.layers}))
        return 0
    step_s, contexts, spread, agree = decode_run(args.batch)
    note(f'decode batch {args.batch}: {step_s * 1e3:.3f} ms/step ({spread[0] * 1e3:.3f} to {spread[1] * 1e3:.3f} over {args.repeats} repeats)')
    if args.phase == 'decode':
        achieved = decode_bytes(config, element, contexts) / step_s / 1e9
        print(json.dumps({'decode_ms_per_step': round(step_s * 1e3, 4), 'batch': args.batch, 'layers': args.layers,
                          'ms_per_step_min': round(spread[0] * 1e3, 4), 'ms_per_step_max': round(spread[1] * 1e3, 4),
                          'repeats': args.repeats, 'repeats_agree': agree,
                          'tokens_per_s': round(args.batch / step_s, 1), 'hbm_gb_per_s': round(achieved, 1),
                          'hbm_frac': round(achieved / HBM_GBPS, 4)}))
        return 0
    points, point_times = {}, {f'decode_b{args.batch}': [round(step_s * 1e3, 4)] + [round(t * 1e3, 4) for t in spread]}
    agreed = {f'decode_b{args.batch}': agree}
    for batch in [int(b) for b in args.points.split(',') if b]:
        seconds, _, point_spread, point_agree = decode_run(batch)
        points[f'decode_b{batch}'] = round(batch / seconds, 1)
        point_times[f'decode_b{batch}'] = [round(seconds * 1e3, 4)] + [round(t * 1e3, 4) for t in point_spread]
        agree = agree and point_agree
        agreed[f'decode_b{batch}'] = point_agree
        note(f'decode batch {batch}: {seconds * 1e3:.3f} ms/step ({point_spread[0] * 1e3:.3f} to {point_spread[1] * 1e3:.3f})')
    prefill_s = prefill_run(args.prefill_tokens)
    note(f'prefill {args.prefill_tokens}: {prefill_s * 1e3:.2f} ms')

    value = args.batch / step_s
    bytes_read = decode_bytes(config, element, contexts)
    achieved = bytes_read / step_s / 1e9
    flops = prefill_flops(config, args.prefill_tokens)
    line = {
        'metric': f'decode tok/s at batch {args.batch} ({NAMES[args.sizes]} sizes, {args.history}-token histories)',
        'value': round(value, 1),
        'unit': 'tokens/s', 'n_gpus': 1, 'steps': args.steps, 'warmup': args.warmup,
        'ms_per_step': round(step_s * 1e3, 4), 'ms_per_step_min': round(spread[0] * 1e3, 4),
        'ms_per_step_max': round(spread[1] * 1e3, 4), 'repeats': args.repeats, 'repeats_agree': agree,
        'higher_is_better': True, 'scaling': 'weak', 'vs_baseline': None,
        'dtype': 'bf16' if args.dtype == 'bfloat16' else 'fp32', 'data': 'synthetic',
        'config': {'model': f'{NAMES[args.sizes]} sizes, random weights', 'layers': args.layers,
                   'layers_of_model': sizes['num_hidden_layers'], 'hidden': config['hidden_size'],
                   'heads': config['num_attention_heads'], 'kv_heads': config['num_key_value_heads'],
                   'head_dim': config['head_dim'], 'intermediate': config['intermediate_size'],
                   'vocab': config['vocab_size'], 'global_batch': args.batch, 'seq_len': args.history,
                   'context': config['max_position_embeddings'], 'page_size': page_size,
                   'prefill_tokens': args.prefill_tokens, 'parallelism': 'single GPU',
                   'large_products': 'own kernels' if args.own_products else 'GPU BLAS'},
        'prefill': {'value': round(args.prefill_tokens / prefill_s, 1), 'tokens': args.prefill_tokens,
                    'ms': round(prefill_s * 1e3, 3), 'frac': round(flops / prefill_s / (PEAK_TFLOPS[args.dtype] * 1e12), 4)},
        'roofline': {'bound': 'hbm', 'achieved': round(achieved, 1), 'peak': HBM_GBPS, 'unit': 'GB/s',
                     'frac': round(achieved / HBM_GBPS, 4)},
        'points': points,
        'points_ms_per_step': point_times,           # per point: median, fastest, slowest repeat
        'points_repeats_agree': agreed,
    }
    print(json.dumps(line))
    return 0


if __name__ == '__main__':
    sys.exit(main())
