"""A plain, slow Kebudra in float64: one function per mechanism, whole sequences at once or token by token.

Nothing here is shared with the engine.  ``weights`` maps checkpoint names to float64 tensors; ``config`` is the
dict of config.json.  A sequence is run alone; ``states`` (a dict per layer) carries what decoding needs, so that the
same functions serve whole prompts and single tokens.
"""
import math

import torch

F = torch.float64
UNIT_EPS = 1e-6


def rms(x, eps):
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def silu(z):
    return z * torch.sigmoid(z)


def softplus(z):
    return torch.where(z > 30, z, torch.log1p(torch.exp(torch.clamp(z, max=30.0))))


def tanh_norm(x, w, name):
    return torch.tanh(w[name + '.alpha'] * x) * w[name] + w[name + '.b']


def streams_in(streams, w, p):
    """u = sum_s in[s] x_s of streams [S, T, width]."""
    return (w[p + 'in'][:, None, None] * streams).sum(0)


def streams_out(streams, y, w, p):
    """x_t <- sum_s mix[s, t] x_s + out[t] y."""
    mix, out = w[p + 'mix'], w[p + 'out']
    new = []
    for t in range(streams.shape[0]):
        x = out[t] * y
        for s in range(streams.shape[0]):
            x = x + mix[s, t] * streams[s]
        new.append(x)
    return torch.stack(new)


def remember(state, name, new):
    state[name] = new if name not in state else torch.cat([state[name], new])
    return state[name]


def softmax_over(scores, q_pos, count):
    """scores [T, count] with the keys 0 .. count - 1 behind a query's position hidden -> the weights."""
    hidden = torch.arange(count)[None, :] > q_pos[:, None]
    return torch.softmax(scores.masked_fill(hidden, -math.inf), dim=-1)


def difference_factor(w, p, m):
    return torch.exp((w[p + 'lq1'] * w[p + 'lk1']).sum()) - torch.exp((w[p + 'lq2'] * w[p + 'lk2']).sum()) + m['diff']


def attention_mixer(h, positions, w, p, m, eps, state, owner):
    """Two softmax maps a head over the same values, the second one taken off with a factor.  ``owner``: the state of the
    layer whose keys and values are read (this layer's own unless 'kv_from' names another)."""
    H, G, d, dv = m['heads'], m['kv_heads'], m['dim'], m['vdim']
    T = h.shape[0]
    q = (h @ w[p + 'q'].T).reshape(T, H, 2, d)
    if m.get('kv_from') is None:
        remember(state, 'k', (h @ w[p + 'k'].T).reshape(T, G, 2, d))
        remember(state, 'v', (h @ w[p + 'v'].T).reshape(T, G, dv))
        owner = state
    k, v = owner['k'], owner['v']
    factor = difference_factor(w, p, m)
    gate = torch.sigmoid(h @ w[p + 'g'].T)
    out = torch.zeros(T, H, dv, dtype=F)
    for head in range(H):
        g = head // (H // G)
        maps = [softmax_over((q[:, head, i] @ k[:, g, i].T) * m['scale'], positions, k.shape[0]) @ v[:, g] for i in (0, 1)]
        out[:, head] = rms(maps[0] - factor * maps[1], eps) * (1.0 - m['diff']) * gate[:, head:head + 1]
    return out.reshape(T, H * dv) @ w[p + 'o'].T


def rotate_neighbours(x, positions, dims, base):
    """x [T, .., d]: elements 2 i and 2 i + 1 of the first ``dims`` are a pair, turned by position * base^(-2 i / dims)."""
    freqs = torch.tensor([base ** (-2.0 * i / dims) for i in range(dims // 2)], dtype=F)
    a = positions.to(F)[:, None] * freqs[None, :]
    a = a.reshape(a.shape[0], *([1] * (x.ndim - 2)), a.shape[1])
    c, s = torch.cos(a), torch.sin(a)
    u, v = x[..., 0:dims:2], x[..., 1:dims:2]
    out = x.clone()
    out[..., 0:dims:2] = u * c - v * s
    out[..., 1:dims:2] = v * c + u * s
    return out


def latent_mixer(h, positions, w, p, m, eps, state, owner=None):
    H, d, r, dv, rank = m['heads'], m['dim'], m['rot_dim'], m['vdim'], m['kv_rank']
    T = h.shape[0]
    cq = rms(h @ w[p + 'dq'].T, eps) * w[p + 'dq.norm']
    q = (cq @ w[p + 'uq'].T).reshape(T, H, d + r)
    q_rot = rotate_neighbours(q[..., d:], positions, m['rot']['dims'], m['rot']['base'])
    down = h @ w[p + 'dkv'].T
    c = remember(state, 'c', rms(down[:, :rank], eps) * w[p + 'dkv.norm'])
    k_rot = remember(state, 'kr', rotate_neighbours(down[:, rank:], positions, m['rot']['dims'], m['rot']['base']))
    k = (c @ w[p + 'uk'].T).reshape(-1, H, d)
    v = (c @ w[p + 'uv'].T).reshape(-1, H, dv)
    out = torch.zeros(T, H, dv, dtype=F)
    for head in range(H):
        scores = (q[:, head, :d] @ k[:, head].T + q_rot[:, head] @ k_rot.T) * m['scale']
        out[:, head] = softmax_over(scores, positions, c.shape[0]) @ v[:, head]
    return (out.reshape(T, H * dv) * torch.sigmoid(h @ w[p + 'g'].T)) @ w[p + 'o'].T


def short_conv(x, weight, state, name):
    """A causal convolution over time per channel, zeros before the start; weight [channels, taps]."""
    T, taps = x.shape[0], weight.shape[1]
    padded = torch.cat([state.get(name, torch.zeros(taps - 1, x.shape[1], dtype=F)), x])
    out = torch.zeros_like(x)
    for j in range(taps):
        out += padded[j:j + T] * weight[:, j]
    if taps > 1:
        state[name] = padded[-(taps - 1):]
    return out


def unit(x):
    return x / torch.sqrt((x * x).sum(-1, keepdim=True) + UNIT_EPS)


def delta_scan(q, k, v, g, beta, S):
    """q, k, g [T, H, d] (g the decays), v [T, H, dv], beta [T, H], S [H, d, dv] -> (o [T, H, dv], S), token by token."""
    out = torch.zeros_like(v)
    for t in range(q.shape[0]):
        S = g[t][:, :, None] * S
        u = beta[t][:, None] * (v[t] - (S * k[t][:, :, None]).sum(1))
        S = S + k[t][:, :, None] * u[:, None, :]
        out[t] = (S * q[t][:, :, None]).sum(1)
    return out, S


def delta_mixer(h, positions, w, p, m, eps, state, owner=None):
    H, G, d, dv = m['heads'], m['kv_heads'], m['dim'], m['vdim']
    T = h.shape[0]
    q, k, v = (silu(short_conv(h @ w[p + name].T, w[p + name + '.conv'], state, name)) for name in ('q', 'k', 'v'))
    share = torch.arange(H) // (H // G)
    q = (unit(q.reshape(T, G, d)) * d ** -0.5)[:, share]
    k = unit(k.reshape(T, G, d))[:, share]
    beta = torch.sigmoid(h @ w[p + 'b'].T)
    raw = softplus(h @ w[p + 'a1'].T @ w[p + 'a2'].T + w[p + 'dt_bias']).reshape(T, H, d)
    decay = torch.exp(-torch.exp(w[p + 'A_log'])[:, None] * raw)
    S = state.get('S', torch.zeros(H, d, dv, dtype=F))
    o, state['S'] = delta_scan(q, k, v.reshape(T, H, dv), decay, beta, S)
    o = rms(o, eps) * w[p + 'norm'] * torch.sigmoid(h @ w[p + 'g1'].T @ w[p + 'g2'].T).reshape(T, H, dv)
    return o.reshape(T, H * dv) @ w[p + 'o'].T


MIXERS = {'attention': attention_mixer, 'latent_attention': latent_mixer, 'channel_delta': delta_mixer}


def feed_forward(h, w, p, f):
    z = h @ w[p + 'router'].T
    out = torch.zeros_like(h)
    best, chosen = torch.topk(z, f['router']['top'], dim=-1)
    weights = torch.softmax(best, dim=-1)
    for t in range(h.shape[0]):
        for e, weight in zip(chosen[t].tolist(), weights[t]):
            hidden = torch.relu(h[t] @ w[p + f'e{e}.up'].T) ** 2
            out[t] += weight * (hidden @ w[p + f'e{e}.down'].T)
    return out


def forward(config, w, tokens, start=0, states=None, collect=None):
    """(logits [T, vocab], states) of ``tokens`` at positions start ..; ``states``: what earlier calls for the same
    sequence left, or None.  ``collect``: a list that receives the sum of the streams after every layer."""
    eps = config['norm']['eps']
    states = states if states is not None else [dict() for _ in config['layers']]
    x = w['embed'][torch.as_tensor(list(tokens))] * config['embedding']['scale']
    streams = torch.stack([x] * config['streams'])
    positions = torch.arange(start, start + len(tokens))
    for i, layer in enumerate(config['layers']):
        p, m = f'l{i}.', layer['mixer']
        owner = states[m['kv_from']] if m.get('kv_from') is not None else None
        h = tanh_norm(streams_in(streams, w, p + 'hc1.'), w, p + 'norm1')
        y = MIXERS[layer['type']](h, positions, w, p + 'mix.', m, eps, states[i], owner)
        streams = streams_out(streams, y, w, p + 'hc1.')
        if layer['mlp'] is not None:
            h = tanh_norm(streams_in(streams, w, p + 'hc2.'), w, p + 'norm2')
            streams = streams_out(streams, feed_forward(h, w, p + 'mlp.', layer['mlp']), w, p + 'hc2.')
        if collect is not None:
            collect.append(streams.sum(0))
    return tanh_norm(streams.sum(0), w, 'final.norm') @ w['head'].T, states


# ------------------------------------------------------------------------------------------------ making models
def moe(experts, top, ff):
    return dict(kind='moe', expert=dict(ff=ff), router=dict(experts=experts, top=top))


def attention_layer(*, heads, kv_heads, dim, vdim, scale, diff, kv_from=None, mlp=None):
    mixer = dict(heads=heads, kv_heads=kv_heads, dim=dim, vdim=vdim, scale=scale, diff=diff)
    if kv_from is not None:
        mixer['kv_from'] = kv_from
    return dict(type='attention', mixer=mixer, mlp=mlp)


def latent_layer(*, heads, dim, rot_dim, vdim, kv_rank, q_rank, scale, base=10000.0, mlp=None):
    return dict(type='latent_attention', mlp=mlp,
                mixer=dict(heads=heads, dim=dim, rot_dim=rot_dim, vdim=vdim, kv_rank=kv_rank, q_rank=q_rank, scale=scale,
                           rot=dict(base=base, dims=rot_dim)))


def delta_layer(*, heads, kv_heads, dim, vdim, conv, mlp=None):
    return dict(type='channel_delta', mixer=dict(heads=heads, kv_heads=kv_heads, dim=dim, vdim=vdim, conv=conv), mlp=mlp)


def make_config(layers, *, vocab, width, streams, eps=1e-5, embedding_scale=1.0):
    return dict(architecture='Kebudra', vocab=vocab, width=width, streams=streams, embedding=dict(scale=embedding_scale),
                layers=layers, norm=dict(eps=eps))


def random_weights(config, seed, spread=1.0, ranks=(5, 11), clear_routers=False):
    """float64 tensors whose values bfloat16 holds exactly, by checkpoint name.  ``ranks``: inner sizes of the low-rank
    products of the decays and of the gate.  ``clear_routers``: no router is ever close to choosing otherwise (for engines that
    round: an expert more or less is no rounding error).  Every token then has one of 16 sign patterns in the last four
    channels, which no sub-layer writes to and which the routers read alone, and the routers are drawn until every pattern's
    choice is clear."""
    g = torch.Generator().manual_seed(seed)
    width, streams = config['width'], config['streams']
    w = {}

    def held(t):
        return t.to(torch.bfloat16).to(F)

    def normal(*shape):
        return torch.randn(*shape, generator=g, dtype=F)

    def matrix(name, rows, columns, gain=1.0):
        w[name] = held(normal(rows, columns) * (gain * spread / math.sqrt(columns)))

    def vector(name, size, std=0.1, mean=0.0):
        w[name] = held(mean + std * normal(size))

    def norm(name):
        vector(name, width, 0.2, 1.0)
        vector(name + '.b', width, 0.1)
        w[name + '.alpha'] = held(0.5 + 0.2 * torch.rand((), generator=g, dtype=F))

    w['embed'] = held(normal(config['vocab'], width) / config['embedding']['scale'])
    matrix('head', config['vocab'], width)
    norm('final.norm')
    for i, layer in enumerate(config['layers']):
        p, m = f'l{i}.', layer['mixer']
        for q in (1, 2) if layer['mlp'] is not None else (1,):
            norm(p + f'norm{q}')
            vector(p + f'hc{q}.in', streams, 0.3, 1.0 / streams)
            vector(p + f'hc{q}.out', streams, 0.3, 1.0)
            w[p + f'hc{q}.mix'] = held(0.8 * torch.eye(streams, dtype=F) + 0.15 * normal(streams, streams))
        p += 'mix.'
        if layer['type'] == 'attention':
            H, G, d, dv = m['heads'], m['kv_heads'], m['dim'], m['vdim']
            matrix(p + 'q', H * 2 * d, width, 1.5)
            if m.get('kv_from') is None:
                matrix(p + 'k', G * 2 * d, width, 1.5)
                matrix(p + 'v', G * dv, width)
            for name in ('lq1', 'lk1', 'lq2', 'lk2'):
                vector(p + name, d, 0.25)
            matrix(p + 'g', H, width, 2.0)
            matrix(p + 'o', width, H * dv)
        elif layer['type'] == 'latent_attention':
            H, d, r, dv = m['heads'], m['dim'], m['rot_dim'], m['vdim']
            matrix(p + 'dq', m['q_rank'], width)
            vector(p + 'dq.norm', m['q_rank'], 0.2, 1.0)
            matrix(p + 'uq', H * (d + r), m['q_rank'], 1.5)
            matrix(p + 'dkv', m['kv_rank'] + r, width)
            vector(p + 'dkv.norm', m['kv_rank'], 0.2, 1.0)
            matrix(p + 'uk', H * d, m['kv_rank'], 1.5)
            matrix(p + 'uv', H * dv, m['kv_rank'])
            matrix(p + 'g', H * dv, width, 2.0)
            matrix(p + 'o', width, H * dv)
        else:
            H, G, d, dv = m['heads'], m['kv_heads'], m['dim'], m['vdim']
            for name, rows in (('q', G * d), ('k', G * d), ('v', H * dv)):
                matrix(p + name, rows, width)
                w[p + name + '.conv'] = held(normal(rows, m['conv']) * 0.6)
            matrix(p + 'b', H, width, 2.0)
            w[p + 'A_log'] = held(torch.log(torch.rand(H, generator=g, dtype=F) * 1.5 + 0.01))
            vector(p + 'dt_bias', H * d, 1.0, -2.0)
            vector(p + 'norm', dv, 0.2, 1.0)
            matrix(p + 'a1', ranks[0], width)
            matrix(p + 'a2', H * d, ranks[0])
            matrix(p + 'g1', ranks[1], width)
            matrix(p + 'g2', H * dv, ranks[1], 2.0)
            matrix(p + 'o', width, H * dv)
        if layer['mlp'] is not None:
            p, f = f'l{i}.mlp.', layer['mlp']
            matrix(p + 'router', f['router']['experts'], width, 2.0)
            for e in range(f['router']['experts']):
                matrix(p + f'e{e}.up', f['expert']['ff'], width)
                matrix(p + f'e{e}.down', width, f['expert']['ff'], 1.5)
    if clear_routers:
        signs = torch.tensor([[1.0 if token >> bit & 1 else -1.0 for bit in range(4)] for token in range(config['vocab'])], dtype=F)
        w['embed'][:, -4:] = held(3.0 / config['embedding']['scale'] * signs)
        for name in w:
            if name.endswith('.mix.o') or name.endswith('.down'):
                w[name][-4:] = 0.0
            elif name.endswith('.norm2'):
                w[name][-4:], w[name + '.b'][-4:] = 1.0, 0.0
        for i, layer in enumerate(config['layers']):
            if layer['mlp'] is None:
                continue
            r = layer['mlp']['router']
            while True:
                router = held(normal(r['experts'], 4))
                z = (signs[:16] @ router.T).sort(dim=-1, descending=True).values
                if r['top'] == r['experts'] or (z[:, r['top'] - 1] - z[:, r['top']]).min() > 0.12:
                    break
            w[f'l{i}.mlp.router'] = torch.zeros(r['experts'], width, dtype=F)
            w[f'l{i}.mlp.router'][:, -4:] = router
    return w


def logits(tokens, weights, config):
    """Logits [T, vocab] of a whole sequence."""
    return forward(config, weights, tokens)[0]


def greedy(prompt, count, weights, config):
    tokens = list(prompt)
    for _ in range(count):
        tokens.append(int(logits(tokens, weights, config)[-1].argmax()))
    return tokens[len(prompt):]
