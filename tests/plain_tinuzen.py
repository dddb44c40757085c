"""A plain, slow Tinuzen in float64: one function per mechanism, whole sequences at once or token by token.

Nothing here is shared with the engine.  ``weights`` maps checkpoint names to float64 tensors; ``config`` is the
dict of config.json.  A sequence is run alone; ``states`` (a dict per layer run, and one for the embedding) carries what
decoding needs, so that the same functions serve whole prompts and single tokens.
"""
import math

import torch

F = torch.float64


def rms(x, eps):
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def silu(z):
    return z * torch.sigmoid(z)


def softplus(z):
    return torch.where(z > 30, z, torch.log1p(torch.exp(torch.clamp(z, max=30.0))))


def bigram_rows(tokens, previous, b):
    """The bigram table's row of every token; ``previous``: the token before the first one (None at a sequence's start,
    whose row is the table's last)."""
    out = []
    for token in tokens:
        out.append(b['buckets'] if previous is None else (previous * b['mul_prev'] + token * b['mul_cur']) % b['buckets'])
        previous = token
    return out


def embed(tokens, w, e, state):
    x = w['embed'][torch.as_tensor(tokens)] * e['scale']
    if e.get('bigram') is not None:
        x = x + w['bigram'][torch.as_tensor(bigram_rows(tokens, state.get('previous'), e['bigram']))]
    state['previous'] = tokens[-1]
    return x


def rotate_neighbours(x, positions, dims, base):
    """x [T, heads, d]: elements 2 i and 2 i + 1 of the first ``dims`` are a pair, turned by position * base^(-2 i / dims)."""
    freqs = torch.tensor([base ** (-2.0 * i / dims) for i in range(dims // 2)], dtype=F)
    a = positions.to(F)[:, None] * freqs[None, :]
    c, s = torch.cos(a)[:, None, :], torch.sin(a)[:, None, :]
    u, v = x[..., 0:dims:2], x[..., 1:dims:2]
    out = x.clone()
    out[..., 0:dims:2] = u * c - v * s
    out[..., 1:dims:2] = v * c + u * s
    return out


def attend(q, k, v, q_pos, k_pos, scale, window=None, keep_first=0, slopes=None, one=False):
    """q [T, H, d], k [S, G, d], v [S, G, dv] -> [T, H * dv]; key j is visible to query i iff j <= i and, with a window,
    i - j < window or j < keep_first.  ``slopes`` [H]: slopes[h] * (i - j) is taken off the scaled score.  ``one``: the
    softmax's denominator is one larger."""
    T, H, _ = q.shape
    rep = H // k.shape[1]
    out = torch.zeros(T, H, v.shape[-1], dtype=F)
    diff = q_pos[:, None] - k_pos[None, :]
    visible = diff >= 0
    if window is not None:
        visible = visible & ((diff < window) | (k_pos[None, :] < keep_first))
    for h in range(H):
        s = (q[:, h] @ k[:, h // rep].T) * scale
        if slopes is not None:
            s = s - slopes[h] * diff
        s = s.masked_fill(~visible, -math.inf)
        m = s.max(-1, keepdim=True).values
        if one:
            m = torch.clamp(m, min=0.0)
        e = torch.exp(s - m)
        below = e.sum(-1, keepdim=True)
        if one:
            below = below + torch.exp(-m)
        out[:, h] = (e / below) @ v[:, h // rep]
    return out.reshape(T, -1)


def head_slopes(heads):
    return [2.0 ** (-8.0 * (h + 1) / heads) for h in range(heads)]


def remember(state, name, new):
    state[name] = new if name not in state else torch.cat([state[name], new])
    return state[name]


def key_value_attention(h, positions, w, p, m, state):
    """The left half of the 'parallel' mixer: the values are the keys as they were before the rotation, one more term 1
    in the denominator, an output gate."""
    H, G, d = m['heads'], m['kv_heads'], m['dim']
    T = h.shape[0]
    q = (h @ w[p + 'q'].T).reshape(T, H, d)
    k = (h @ w[p + 'k'].T).reshape(T, G, d)
    v = k
    if m.get('rot') is not None:
        q = rotate_neighbours(q, positions, m['rot']['dims'], m['rot']['base'])
        k = rotate_neighbours(k, positions, m['rot']['dims'], m['rot']['base'])
    keys, values = remember(state, 'k', k), remember(state, 'v', v)
    out = attend(q, keys, values, positions, torch.arange(keys.shape[0]), m['scale'], one=True)
    return (out * torch.sigmoid(h @ w[p + 'g'].T)) @ w[p + 'o'].T


def dual_scan(h, w, p, m, eps, state):
    """The right half: a state-space recurrence with one decay a head and token, token by token.  ``state``: {'conv':
    the convolution's last taps - 1 inputs, 'S': [heads, n, vdim]}."""
    H, dv, n, G, taps = m['heads'], m['vdim'], m['state'], m['groups'], m['conv']
    inner, T = H * dv, h.shape[0]
    proj = h @ w[p + 'in'].T
    z, xbc, dt = proj[:, :inner], proj[:, inner:2 * inner + 2 * G * n], proj[:, 2 * inner + 2 * G * n:]
    past = state.get('conv', torch.zeros(taps - 1, xbc.shape[1], dtype=F))
    padded = torch.cat([past, xbc])
    conv = torch.zeros_like(xbc)
    for j in range(taps):
        conv += padded[j:j + T] * w[p + 'conv'][:, j]
    if taps > 1:
        state['conv'] = padded[-(taps - 1):]
    u = silu(conv + w[p + 'conv.b'])
    x = u[:, :inner].reshape(T, H, dv)
    B = u[:, inner:inner + G * n].reshape(T, G, n)
    C = u[:, inner + G * n:].reshape(T, G, n)
    dt = softplus(dt + w[p + 'dt_bias'])                            # [T, H]
    keep = torch.exp(-torch.exp(w[p + 'A_log']) * dt)
    S = state.get('S', torch.zeros(H, n, dv, dtype=F))
    group = torch.arange(H) // (H // G)
    y = torch.zeros(T, H, dv, dtype=F)
    for t in range(T):
        S = keep[t][:, None, None] * S + dt[t][:, None, None] * B[t][group][:, :, None] * x[t][:, None, :]
        y[t] = (S * C[t][group][:, :, None]).sum(1) + w[p + 'D'][:, None] * x[t]
    state['S'] = S
    gated = y.reshape(T, inner) * silu(z)
    parts = rms(gated.reshape(T, m['norm_groups'], -1), eps).reshape(T, inner)
    return (parts * w[p + 'norm']) @ w[p + 'o'].T


def parallel_mixer(h, positions, w, p, m, eps, state):
    left = key_value_attention(h, positions, w, p + 'left.', m['left'], state.setdefault('left', {}))
    right = dual_scan(h, w, p + 'right.', m['right'], eps, state.setdefault('right', {}))
    return m['left_scale'] * left + m['right_scale'] * right


def attention_mixer(h, positions, w, p, m, eps, state):
    """The 'attention' mixer: norms over the whole projections, no rotation, a bias by distance, a window with kept
    first tokens."""
    H, G, d, dv = m['heads'], m['kv_heads'], m['dim'], m['vdim']
    T = h.shape[0]
    q = (rms(h @ w[p + 'q'].T, eps) * w[p + 'q.norm']).reshape(T, H, d)
    k = (rms(h @ w[p + 'k'].T, eps) * w[p + 'k.norm']).reshape(T, G, d)
    v = (h @ w[p + 'v'].T).reshape(T, G, dv)
    keys, values = remember(state, 'k', k), remember(state, 'v', v)
    mask = m.get('mask') or {'size': None, 'keep_first': 0}
    out = attend(q, keys, values, positions, torch.arange(keys.shape[0]), m['scale'], window=mask['size'],
                 keep_first=mask['keep_first'], slopes=head_slopes(H))
    return out @ w[p + 'o'].T


MIXERS = {'parallel': parallel_mixer, 'attention': attention_mixer}


def feed_forward(h, w, p):
    return (torch.relu(h @ w[p + 'gate'].T) * (h @ w[p + 'up'].T)) @ w[p + 'down'].T


def layer_runs(config):
    """(layer, pass of the loop if this run begins one, else None) in the order of running."""
    loop, count = config.get('loop'), len(config['layers'])
    if loop is None:
        return [(i, None) for i in range(count)]
    runs = [(i, None) for i in range(loop['start'])]
    for t in range(loop['times']):
        runs += [(i, t if i == loop['start'] else None) for i in range(loop['start'], loop['stop'])]
    return runs + [(i, None) for i in range(loop['stop'], count)]


def forward(config, w, tokens, start=0, states=None, collect=None):
    """(logits [T, vocab], states) of ``tokens`` at positions start ..; ``states``: what earlier calls for the same
    sequence left, or None.  ``collect``: a list that receives the residual stream after every layer run."""
    eps = config['norm']['eps']
    runs = layer_runs(config)
    states = states if states is not None else [dict() for _ in range(len(runs) + 1)]
    embedded = embed(list(tokens), w, config['embedding'], states[-1])
    x = embedded
    positions = torch.arange(start, start + len(tokens))
    for run, (i, begins) in enumerate(runs):
        layer, p = config['layers'][i], f'l{i}.'
        if begins is not None:
            if begins > 0:
                x = x + embedded
            x = x + w['loop.step'][begins]
        h = rms(x, eps) * w[p + 'norm1']
        added = torch.sigmoid(h @ w[p + 'rg1'].T + w[p + 'rg1.b']) * \
            MIXERS[layer['type']](h, positions, w, p + 'mix.', layer['mixer'], eps, states[run])
        if layer['mlp'] is not None:
            added = added + torch.sigmoid(h @ w[p + 'rg2'].T + w[p + 'rg2.b']) * feed_forward(h, w, p + 'mlp.')
        x = x + added
        if collect is not None:
            collect.append(x.clone())
    return (rms(x, eps) * w['final.norm']) @ w['head'].T, states


# ------------------------------------------------------------------------------------------------ making models
def parallel_layer(*, heads, kv_heads, dim, scale, rot_dims=None, base=10000.0, scan_heads, vdim, state, groups=1, conv=4,
                   norm_groups=1, left_scale=1.0, right_scale=1.0, ff=None):
    left = dict(heads=heads, kv_heads=kv_heads, dim=dim, vdim=dim, scale=scale)
    if rot_dims is not None:
        left['rot'] = dict(base=base, dims=rot_dims)
    right = dict(heads=scan_heads, vdim=vdim, state=state, groups=groups, conv=conv, norm_groups=norm_groups)
    return dict(type='parallel', mixer=dict(left=left, right=right, left_scale=left_scale, right_scale=right_scale),
                mlp=dict(kind='dense', ff=ff) if ff is not None else None)


def attention_layer(*, heads, kv_heads, dim, vdim, scale, window=None, keep_first=0, ff=None):
    mixer = dict(heads=heads, kv_heads=kv_heads, dim=dim, vdim=vdim, scale=scale)
    if window is not None:
        mixer['mask'] = dict(size=window, keep_first=keep_first)
    return dict(type='attention', mixer=mixer, mlp=dict(kind='dense', ff=ff) if ff is not None else None)


def make_config(layers, *, vocab, width, eps=1e-5, embedding_scale=1.0, bigram=None, loop=None):
    embedding = dict(scale=embedding_scale)
    if bigram is not None:
        embedding['bigram'] = dict(zip(('buckets', 'mul_prev', 'mul_cur'), bigram))
    out = dict(architecture='Tinuzen', vocab=vocab, width=width, embedding=embedding, layers=layers, norm=dict(eps=eps))
    if loop is not None:
        out['loop'] = dict(zip(('start', 'stop', 'times'), loop))
    return out


def random_weights(config, seed, spread=1.0):
    """float64 tensors whose values bfloat16 holds exactly, by checkpoint name."""
    g = torch.Generator().manual_seed(seed)
    width = config['width']
    w = {}

    def held(t):
        return t.to(torch.bfloat16).to(F)

    def matrix(name, rows, columns, gain=1.0):
        w[name] = held(torch.randn(rows, columns, generator=g, dtype=F) * (gain * spread / math.sqrt(columns)))

    def vector(name, size, std=0.1, mean=0.0):
        w[name] = held(mean + std * torch.randn(size, generator=g, dtype=F))

    e = config['embedding']
    w['embed'] = held(torch.randn(config['vocab'], width, generator=g, dtype=F) / e['scale'])
    if e.get('bigram') is not None:
        w['bigram'] = held(torch.randn(e['bigram']['buckets'] + 1, width, generator=g, dtype=F))
    if config.get('loop') is not None:
        w['loop.step'] = held(torch.randn(config['loop']['times'], width, generator=g, dtype=F) * 0.5)
    matrix('head', config['vocab'], width)
    vector('final.norm', width, 0.2, 1.0)
    for i, layer in enumerate(config['layers']):
        p, m = f'l{i}.', layer['mixer']
        vector(p + 'norm1', width, 0.2, 1.0)
        for name in ('rg1',) + (('rg2',) if layer['mlp'] is not None else ()):
            matrix(p + name, width, width)
            vector(p + name + '.b', width, 0.5)
        if layer['type'] == 'attention':
            H, G, d, dv = m['heads'], m['kv_heads'], m['dim'], m['vdim']
            matrix(p + 'mix.q', H * d, width)
            matrix(p + 'mix.k', G * d, width)
            matrix(p + 'mix.v', G * dv, width)
            vector(p + 'mix.q.norm', H * d, 0.3, 1.0)
            vector(p + 'mix.k.norm', G * d, 0.3, 1.0)
            matrix(p + 'mix.o', width, H * dv)
        else:
            a, r = m['left'], m['right']
            H, G, d = a['heads'], a['kv_heads'], a['dim']
            matrix(p + 'mix.left.q', H * d, width)
            matrix(p + 'mix.left.k', G * d, width)
            matrix(p + 'mix.left.g', H * d, width, 2.0)
            matrix(p + 'mix.left.o', width, H * d)
            H, dv, n, G, taps = r['heads'], r['vdim'], r['state'], r['groups'], r['conv']
            inner, channels = H * dv, H * dv + 2 * G * n
            matrix(p + 'mix.right.in', inner + channels + H, width)
            w[p + 'mix.right.conv'] = held(torch.randn(channels, taps, generator=g, dtype=F) * 0.6)
            vector(p + 'mix.right.conv.b', channels, 0.2)
            vector(p + 'mix.right.dt_bias', H, 1.0, -1.0)
            w[p + 'mix.right.A_log'] = held(torch.log(torch.rand(H, generator=g, dtype=F) * 2.0 + 0.02))
            vector(p + 'mix.right.D', H, 0.5, 1.0)
            vector(p + 'mix.right.norm', inner, 0.2, 1.0)
            matrix(p + 'mix.right.o', width, inner)
        if layer['mlp'] is not None:
            matrix(p + 'mlp.gate', layer['mlp']['ff'], width)
            matrix(p + 'mlp.up', layer['mlp']['ff'], width)
            matrix(p + 'mlp.down', width, layer['mlp']['ff'], 1.5)
    return w


def logits(tokens, weights, config):
    """Logits [T, vocab] of a whole sequence."""
    return forward(config, weights, tokens)[0]


def greedy(prompt, count, weights, config):
    tokens = list(prompt)
    for _ in range(count):
        tokens.append(int(logits(tokens, weights, config)[-1].argmax()))
    return tokens[len(prompt):]
