"""The Kebudra design in the engine against its plain restatement (``plain_kebudra``), under every way of cutting the work:
whole prompts, token-by-token decoding, portions down to two tokens, unequal batches, pages and state slots that are freed
and used again, and generation through the serving loop; then each mechanism alone, with weights or inputs made so that a fault
shows (a far key that only one of two maps looks for, a factor that takes the second map off, a memory that must survive
hundreds of tokens or forget within one, a key written twice, streams that must not be mixed up).

Each model test runs three ways, as the step function's own tests do: on the CPU with the kernels' plain references
substituted, and on the GPU with the HIP kernels in float32 and in bfloat16 (marked ``gpu``).  Page and state storage
is filled with NaN first.  Configurations are small and their sizes differ from one another in every field.
"""
import json
import random

import pytest
import torch

import plain_kebudra as plain
from conftest import write_model_folder
from qil_amd.engine import ModelRunner, StepEntry
from qil_amd.weights import load_model

GPU = [pytest.param(('cuda', torch.float32), id='gpu-f32', marks=pytest.mark.gpu),
       pytest.param(('cuda', torch.bfloat16), id='gpu-bf16', marks=pytest.mark.gpu)]
BACKENDS = [pytest.param(('cpu', torch.float32), id='cpu-refs')] + GPU


def _mixed():
    # three streams; every kind of layer with and without a feed-forward; sizes that are multiples of nothing much
    layers = [
        plain.latent_layer(heads=3, dim=10, rot_dim=6, vdim=14, kv_rank=21, q_rank=18, scale=0.3, base=300.0, mlp=plain.moe(6, 3, 20)),
        plain.attention_layer(heads=6, kv_heads=3, dim=9, vdim=13, scale=0.5, diff=0.3, mlp=plain.moe(9, 1, 12)),
        plain.delta_layer(heads=6, kv_heads=2, dim=11, vdim=7, conv=4, mlp=plain.moe(5, 5, 18)),
        plain.attention_layer(heads=4, kv_heads=4, dim=6, vdim=20, scale=0.4, diff=0.7),
        plain.attention_layer(heads=6, kv_heads=3, dim=9, vdim=13, scale=0.7, diff=0.45, kv_from=1, mlp=plain.moe(4, 2, 33)),
        plain.delta_layer(heads=3, kv_heads=3, dim=16, vdim=24, conv=2),
    ]
    return plain.make_config(layers, vocab=97, width=44, streams=3, embedding_scale=6.6)


def _wide():
    # heads of 64 and 128 once paired, memories of a real model's head sizes, a latent of the matrix-core kernel's sizes; four
    # streams; the first layer's keys are read by the last
    layers = [
        plain.attention_layer(heads=4, kv_heads=1, dim=64, vdim=128, scale=0.125, diff=0.2, mlp=plain.moe(8, 2, 32)),
        plain.delta_layer(heads=4, kv_heads=2, dim=128, vdim=128, conv=4, mlp=plain.moe(3, 3, 64)),
        plain.latent_layer(heads=4, dim=32, rot_dim=32, vdim=40, kv_rank=128, q_rank=64, scale=0.12, mlp=plain.moe(16, 4, 16)),
        plain.attention_layer(heads=4, kv_heads=2, dim=32, vdim=64, scale=0.2, diff=0.9, mlp=plain.moe(2, 1, 48)),
        plain.delta_layer(heads=2, kv_heads=2, dim=64, vdim=96, conv=3, mlp=plain.moe(8, 2, 32)),
        plain.attention_layer(heads=4, kv_heads=1, dim=64, vdim=128, scale=0.1, diff=0.6, kv_from=0),
    ]
    return plain.make_config(layers, vocab=61, width=64, streams=4, eps=1e-6, embedding_scale=8.0)


def _plainest():
    # one stream, no feed-forwards, every count one
    layers = [plain.delta_layer(heads=1, kv_heads=1, dim=10, vdim=14, conv=1),
              plain.attention_layer(heads=1, kv_heads=1, dim=12, vdim=5, scale=12 ** -0.5, diff=0.5),
              plain.latent_layer(heads=1, dim=7, rot_dim=2, vdim=9, kv_rank=13, q_rank=11, scale=0.4)]
    return plain.make_config(layers, vocab=50, width=24, streams=1)


# (configuration, seed, page size, spread of the matrices)
CONFIGS = {'mixed': (_mixed(), 21, 8, 1.0), 'wide': (_wide(), 22, 16, 0.9), 'plainest': (_plainest(), 23, 4, 1.2)}


def tokens_for(config, length, seed):
    r = random.Random(seed)
    return [r.randrange(config['vocab']) for _ in range(length)]


def row_errors(actual, expected):
    """Every row's error: root mean square over the vocabulary of the difference (its mean taken off), over the root
    mean square of the expected logits."""
    difference = actual.double().cpu() - expected.double()
    difference = difference - difference.mean(dim=-1, keepdim=True)
    return difference.square().mean(dim=-1).sqrt() / expected.double().square().mean().sqrt()


def error(actual, expected):
    return row_errors(actual, expected).max().item()


# The engine in float32 is 1e-6 to 1e-5 from the float64 plain model on these configurations; in bfloat16 (activations
# between kernels rounded; memories, decays, scores, norms, streams and their sums float32) about 0.01 to 0.04.
LIMIT = {torch.float32: 1e-4, torch.bfloat16: 0.07}


class Case:
    def __init__(self, name, config, weights, model, page_size, dtype):
        self.name, self.config, self.weights, self.model, self.page_size, self.dtype = name, config, weights, model, page_size, dtype
        self._expected = {}

    def expected(self, tokens):
        key = tuple(tokens)
        if key not in self._expected:
            self._expected[key] = plain.logits(tokens, self.weights, self.config)
        return self._expected[key]

    def runner(self, pages, requests=4, graphs=False):
        runner = ModelRunner(self.model, num_pages=pages, page_size=self.page_size, max_requests=requests, graphs=graphs)
        for group in runner.cache.kv_groups:
            for tensor in group['tensors'].values() if 'tensors' in group else (group['k'], group['v']):
                tensor.fill_(float('nan'))
        for group in runner.cache.state_groups:
            group['state'].fill_(float('nan'))
        return runner

    def close(self, actual, expected, what='', slack=1.0):
        """Every row within the limit; in bfloat16 one row in ten may lie beyond it while the median stays within half."""
        assert torch.isfinite(actual).all(), what
        errors = row_errors(actual, expected)
        limit = LIMIT[self.dtype] * slack
        if self.dtype == torch.bfloat16 and len(errors) >= 10:
            over = int((errors > limit).sum())
            assert over * 10 <= len(errors) and errors.median().item() <= limit / 2, \
                f'{what}: {over} of {len(errors)} rows over {limit}, median {errors.median().item():.3e} ({self.dtype})'
            return
        e = errors.max().item()
        assert e <= limit, f'{what}: error {e:.3e} ({self.dtype})'


@pytest.fixture(params=BACKENDS)
def backend(request):
    device, dtype = request.param
    if device == 'cpu':
        request.getfixturevalue('cpu_kernels')
    return device, dtype


def weights_of(name, dtype):
    """Random weights of a configuration; in bfloat16 none whose routers hesitate."""
    config, seed, _, spread = CONFIGS[name]
    return plain.random_weights(config, seed, spread, clear_routers=dtype == torch.bfloat16)


def make_case(name, config, weights, backend, folder, page_size):
    device, dtype = backend
    write_model_folder(folder, config, weights, torch.bfloat16)
    return Case(name, config, weights, load_model(folder, dtype=dtype, device=device), page_size, dtype)


@pytest.fixture(params=sorted(CONFIGS))
def case(request, backend, tmp_path):
    config, seed, page_size, spread = CONFIGS[request.param]
    return make_case(request.param, config, weights_of(request.param, backend[1]), backend, tmp_path / request.param, page_size)


def feed(runner, name, tokens, cuts, want=None):
    """One request alone, its tokens in steps of the given sizes (the rest one by one); the logits of every place (or
    of the places in ``want``)."""
    runner.admit(name)
    rows, at, sizes = [], 0, list(cuts)
    while at < len(tokens):
        size = min(sizes.pop(0) if sizes else 1, len(tokens) - at)
        places = tuple(range(size)) if want is None else tuple(p - at for p in want if at <= p < at + size)
        out = runner.step([StepEntry(name, tuple(tokens[at:at + size]), places)])
        if out is not None:
            rows.append(out)
        at += size
    runner.release(name)
    return torch.cat(rows)


# ------------------------------------------------------------------------------------------------ whole models
def test_whole_prompts(case):
    runner = case.runner(pages=64)
    for length, seed in ((1, 1), (2, 2), (37, 3), (110, 4)):
        tokens = tokens_for(case.config, length, seed)
        case.close(feed(runner, 'r', tokens, [length]), case.expected(tokens), f'{length} tokens')
    runner.cache.check()


def test_decoding_token_by_token_equals_the_prompt(case):
    """The first tokens of a sequence one by one, then a long run of single tokens behind a prompt."""
    runner = case.runner(pages=64)
    tokens = tokens_for(case.config, 45, 5)
    case.close(feed(runner, 'r', tokens, []), case.expected(tokens), 'one by one from the first token')
    tokens = tokens_for(case.config, 130, 6)
    case.close(feed(runner, 'r', tokens, [60]), case.expected(tokens), '60, then 70 single tokens')


@pytest.mark.parametrize('where', GPU)
@pytest.mark.parametrize('name', sorted(CONFIGS))
def test_a_long_prompt(name, where, tmp_path):
    """Several hundred tokens at once (the memory's chunks side by side, the attention's keys in many tiles), then two
    long portions and single tokens; the late places are compared."""
    config, seed, page_size, spread = CONFIGS[name]
    case = make_case(name, config, weights_of(name, where[1]), where, tmp_path / name, page_size)
    runner = case.runner(pages=-(-700 // case.page_size) + 2)
    tokens = tokens_for(case.config, 650, 10)
    late = list(range(560, 650))
    expected = case.expected(tokens)[late]
    case.close(feed(runner, 'r', tokens, [650], late), expected, 'whole')
    case.close(feed(runner, 'r', tokens, [130, 470, 3], late), expected, 'two long portions, then single tokens')


@pytest.mark.parametrize('where', GPU)
@pytest.mark.parametrize('name', sorted(CONFIGS))
def test_graphs_replay_the_same_logits(name, where, tmp_path):
    """Decode steps from captured graphs, between them a
    second request's portion, and a batch that shrinks."""
    config, seed, page_size, spread = CONFIGS[name]
    case = make_case(name, config, weights_of(name, where[1]), where, tmp_path / name, page_size)
    runner = case.runner(pages=64, graphs=True)
    tokens = tokens_for(case.config, 70, 7)
    case.close(feed(runner, 'r', tokens, [20]), case.expected(tokens), 'decode steps from graphs')
    assert runner.graphs.safe() and runner.graphs.replays >= 20
    a, b = tokens_for(case.config, 50, 8), tokens_for(case.config, 41, 9)
    runner.admit('a')
    runner.admit('b')
    runner.step([StepEntry('a', tuple(a[:11]))])
    runner.step([StepEntry('b', tuple(b[:3]))])
    rows = {'a': [], 'b': []}
    for i in range(38):
        both = runner.step([StepEntry('b', (b[3 + i],), (0,)), StepEntry('a', (a[11 + i],), (0,))])
        rows['b'].append(both[0])
        rows['a'].append(both[1])
    rows['a'].append(runner.step([StepEntry('a', (a[49],), (0,))])[0])
    case.close(torch.stack(rows['a']), case.expected(a)[11:], 'two rows, then one')
    case.close(torch.stack(rows['b']), case.expected(b)[3:], 'two rows')


@pytest.mark.parametrize('cuts', [[2] * 40, [3, 2, 17, 2, 5, 31, 2, 2, 9], [16, 16, 1, 15, 33, 7], [63, 2, 1, 1, 2],
                                  [64, 64, 65, 2]])
def test_portions_of_changing_size(case, cuts):
    """Portions down to two tokens, cut inside pages and the memory's chunks and at their borders, shorter than the convolution's
    state and longer; the rest one by one."""
    if case.model.device.type == 'cpu' and cuts[0] in (16, 64):
        pytest.skip('the GPU runs these')
    runner = case.runner(pages=64)
    tokens = tokens_for(case.config, max(90, sum(cuts) + 3), 8)
    case.close(feed(runner, 'r', tokens, cuts), case.expected(tokens), f'cuts {cuts[:6]}')


def test_unequal_requests_together_and_slots_used_again(case):
    """Up to three live requests of unequal lengths, portions beside single tokens; requests end and others take their
    pages and state slots (three slots, six requests); some steps leave a live request out."""
    lengths = dict(a=71, b=9, c=38, d=1, e=55, f=20)
    sequences = {name: tokens_for(case.config, n, 20 + i) for i, (name, n) in enumerate(lengths.items())}
    pages = -(-(71 + 55 + 38) // case.page_size) + 3
    runner = case.runner(pages=pages, requests=3)
    waiting, live = list(sequences), []
    fed = {name: 0 for name in sequences}
    got = {name: [] for name in sequences}
    r = random.Random(3)
    used_slots = []
    while waiting or live:
        while waiting and len(live) < 3:
            name = waiting.pop(0)
            assert runner.admit(name)
            used_slots.append(runner.cache.slots[name])
            live.append(name)
        entries = []
        for name in live:
            if len(live) > 1 and r.random() < 0.2:
                continue                                      # left out of this step
            left = len(sequences[name]) - fed[name]
            size = min(left, r.choice([1, 1, 2, 3, 7, 16, 29, 40]))
            entries.append(StepEntry(name, tuple(sequences[name][fed[name]:fed[name] + size]), tuple(range(size))))
        if not entries:
            continue
        logits = runner.step(entries)
        at = 0
        for entry in entries:
            size = len(entry.tokens)
            got[entry.request].append(logits[at:at + size])
            at += size
            fed[entry.request] += size
            if fed[entry.request] == len(sequences[entry.request]):
                runner.release(entry.request)
                live.remove(entry.request)
        runner.cache.check()
    assert sorted(set(used_slots)) == [0, 1, 2] and len(used_slots) == 6
    assert runner.cache.free_pages == [pages] * len(runner.cache.kv_groups)
    for name, tokens in sequences.items():
        case.close(torch.cat(got[name]), case.expected(tokens), f'request {name}')


def test_a_batch_changes_nothing(case):
    """The same request alone and beside others gives the same logits (beyond rounding: the same kernels may split
    their sums differently)."""
    a, b, c = (tokens_for(case.config, n, 40 + n) for n in (33, 12, 50))
    alone = feed(case.runner(pages=32), 'a', a, [20, 2])
    runner = case.runner(pages=32)
    for name in 'abc':
        runner.admit(name)
    rows = [runner.step([StepEntry('b', tuple(b[:5])), StepEntry('a', tuple(a[:20]), tuple(range(20))), StepEntry('c', tuple(c[:31]))])]
    rows.append(runner.step([StepEntry('a', tuple(a[20:22]), (0, 1)), StepEntry('c', tuple(c[31:32])), StepEntry('b', tuple(b[5:]))])[:2])
    for i in range(22, 33):
        rows.append(runner.step([StepEntry('c', (c[i + 10],)), StepEntry('a', (a[i],), (0,))]))
    together = torch.cat(rows)
    between = row_errors(together, alone.cpu())
    assert (between.max() if case.dtype == torch.float32 else between.median()) <= LIMIT[case.dtype] / 2
    case.close(together, case.expected(a), 'beside others')


def test_generation_through_the_serving_loop(case):
    """Greedy generation by the engine's own entry point and scheduler: every drawn token is (within the dtype's
    rounding) the best one of the plain logits of the engine's own sequence so far."""
    from qil_amd.engine import Engine
    prompts = [tokens_for(case.config, n, 60 + n) for n in (5, 1, 23, 12, 9)]
    engine = Engine(case.model, num_pages=24, page_size=case.page_size, token_budget=20, prefill_chunk=7, max_active=3)
    reports = engine.generate(prompts, max_new_tokens=12, ignore_eos=True)
    engine.cache.check()
    assert engine.cache.free_pages == [24] * len(engine.cache.kv_groups)
    slack = 1e-4 if case.dtype == torch.float32 else 0.06
    good = total = 0
    for prompt, report in zip(prompts, reports):
        output = report['token_ids']
        assert len(output) == 12 and report['finish_reason'] == 'length'
        rows = plain.logits(prompt + output, case.weights, case.config)
        spread = rows.std().item()
        for index, token in enumerate(output):
            row = rows[len(prompt) + index - 1]
            best = bool(row[token] >= row.max() - slack * spread)
            assert best or case.dtype == torch.bfloat16, f'token {index} of {prompt}'
            good, total = good + best, total + 1
    assert good * 10 >= total * 9


# ------------------------------------------------------------------------------------------------ each mechanism alone
def _difference(**changes):
    base = dict(heads=2, kv_heads=1, dim=8, vdim=12, scale=0.5, diff=0.4)
    base.update(changes)
    return plain.attention_layer(**base)


def _latent(**changes):
    base = dict(heads=2, dim=8, rot_dim=4, vdim=6, kv_rank=16, q_rank=12, scale=0.4)
    base.update(changes)
    return plain.latent_layer(**base)


def _delta(**changes):
    base = dict(heads=2, kv_heads=1, dim=8, vdim=12, conv=3)
    base.update(changes)
    return plain.delta_layer(**base)


def _one(layer, width=24, streams=2, **changes):
    return plain.make_config([layer], vocab=40, width=width, streams=streams, **changes)


ALONE = {
    'difference-one-head': _one(_difference(heads=1, kv_heads=1, dim=5, vdim=7)),
    'difference-values-narrower-than-keys': _one(_difference(heads=6, kv_heads=2, dim=20, vdim=3, scale=0.3)),
    'difference-values-wider-than-pairs': _one(_difference(heads=4, kv_heads=4, dim=8, vdim=52, diff=0.0)),
    'difference-large-eps': _one(_difference(heads=3, kv_heads=1, dim=16, vdim=16), eps=0.3),
    'difference-pairs-of-64': _one(_difference(heads=4, kv_heads=2, dim=32, vdim=64, scale=0.2), width=32),
    'difference-pairs-of-128': _one(_difference(heads=8, kv_heads=2, dim=64, vdim=128, scale=0.125, diff=0.8), width=48),
    'difference-pairs-of-256': _one(_difference(heads=2, kv_heads=1, dim=128, vdim=200, scale=0.09), width=40),
    'difference-diff-beyond-one': _one(_difference(diff=1.5)),
    'latent-one-head': _one(_latent(heads=1, dim=3, rot_dim=2, vdim=5, kv_rank=9, q_rank=7)),
    'latent-matrix-core-sizes': _one(_latent(heads=4, dim=64, rot_dim=32, vdim=24, kv_rank=128, q_rank=40, scale=0.1), width=32),
    'latent-many-heads': _one(_latent(heads=16, dim=16, rot_dim=8, vdim=16, kv_rank=64, q_rank=48, scale=0.2), width=40),
    'memory-one-of-each': _one(_delta(heads=1, kv_heads=1, dim=1, vdim=1, conv=1)),
    'memory-odd-sizes': _one(_delta(heads=6, kv_heads=3, dim=17, vdim=35, conv=7)),
    'memory-shared-keys': _one(_delta(heads=8, kv_heads=2, dim=32, vdim=16, conv=2), width=32),
    'memory-heads-of-64': _one(_delta(heads=2, kv_heads=2, dim=64, vdim=64, conv=4), width=32),
    'memory-heads-of-128': _one(_delta(heads=3, kv_heads=1, dim=128, vdim=128, conv=4), width=32),
    'memory-wide-keys': _one(_delta(heads=2, kv_heads=1, dim=200, vdim=40, conv=3), width=32),
    'memory-wide-values': _one(_delta(heads=2, kv_heads=1, dim=24, vdim=300, conv=3), width=32),
    'one-stream': _one(_difference(mlp=plain.moe(4, 2, 20)), streams=1),
    'five-streams': _one(_delta(mlp=plain.moe(4, 2, 20)), streams=5),
    'every-expert': _one(_latent(mlp=plain.moe(7, 7, 20)), width=36),
    'one-expert': _one(_difference(mlp=plain.moe(1, 1, 9)), width=20),
    'many-experts': _one(_delta(mlp=plain.moe(70, 3, 16)), width=32),
    'experts-of-eight-elements': _one(_delta(mlp=plain.moe(2, 1, 8)), width=16),
}


@pytest.mark.parametrize('name', sorted(ALONE))
def test_each_mechanism_alone(name, backend, tmp_path):
    """Models of one layer: one mechanism each, at sizes where fields that often coincide differ (key size and value size,
    heads and key/value heads, ranks, experts and chosen ones) and where counts are 1."""
    config = ALONE[name]
    case = make_case(name, config, plain.random_weights(config, 5, 1.3), backend, tmp_path / name, 8)
    tokens = tokens_for(config, 100, 9)
    runner = case.runner(pages=16)
    case.close(feed(runner, 'r', tokens, [100]), case.expected(tokens), 'whole')
    case.close(feed(runner, 'r', tokens, [13, 2, 9, 8, 40]), case.expected(tokens), 'portions, then single tokens')


def _marked(config, w, key_channel=5, query_channel=7):
    """Token 10's input excites one channel that no other token's does, token 11's another."""
    embed = w['embed'].clone()
    embed[:, key_channel] = embed[:, query_channel] = 0.0
    embed[10], embed[11] = 0.0, 0.0
    embed[10, key_channel], embed[11, query_channel] = 8.0, 8.0
    w['embed'] = embed
    width, streams = config['width'], config['streams']
    w['l0.norm1'], w['l0.norm1.b'] = torch.ones(width, dtype=torch.float64), torch.zeros(width, dtype=torch.float64)
    w['l0.norm1.alpha'] = torch.tensor(1.0, dtype=torch.float64)
    w['l0.hc1.in'] = torch.full((streams,), 1.0 / streams, dtype=torch.float64)
    return w


def _held(t):
    return t.to(torch.bfloat16).double()


def _far_key(config, w, backend, folder):
    """A key at the last place of the first page decides what late rows get: in a prompt, in portions, and decoded."""
    case = make_case('far', config, w, backend, folder, 16)
    tokens = [t % 10 for t in tokens_for(config, 420, 2)]
    tokens[15] = 10
    asking = [300, 401, 419]
    for place in asking:
        tokens[place] = 11
    expected = case.expected(tokens)
    other = list(tokens)
    other[15] = 3
    moved = error(plain.logits(other, w, config)[asking], expected[asking])
    assert moved > 0.05, f'the test lost its point: the far key does not matter ({moved})'
    runner = case.runner(pages=40)
    case.close(feed(runner, 'r', tokens, [420], asking), expected[asking], 'in a prompt')
    if case.model.device.type == 'cuda':
        case.close(feed(runner, 'r', tokens, [128, 130, 100, 42], asking), expected[asking], 'in portions')
    case.close(feed(runner, 'r', tokens, [400], asking[1:]), expected[asking[1:]], 'decoded')


@pytest.mark.parametrize('dim', [12, 32, 64])
@pytest.mark.parametrize('which', [0, 1])
def test_a_far_key_of_one_map_decides(which, dim, backend, tmp_path):
    """Only one of the two maps looks for the far key (the other's query of the asking token is zero): maps that were
    exchanged, or keys of one map read by the other, show."""
    if backend[0] == 'cpu' and dim != 12:
        pytest.skip('the GPU kernels differ by head size')
    config = plain.make_config([_difference(heads=2, kv_heads=1, dim=dim, vdim=2 * dim, scale=20.0 / dim, diff=0.5)], vocab=12, width=48,
                               streams=2)
    w = _marked(config, plain.random_weights(config, 3, 1.0))
    key, query = w['l0.mix.k'].clone(), w['l0.mix.q'].clone()
    key[:, 5] *= 16.0
    query[:, 7] = 0.0
    for h in range(2):
        rows = slice((h * 2 + which) * dim, (h * 2 + which + 1) * dim)
        query[rows, 7] = key[which * dim:(which + 1) * dim, 5] / 16.0
    w['l0.mix.k'], w['l0.mix.q'] = key, query
    _far_key(config, w, backend, tmp_path / 'far')


@pytest.mark.parametrize('sizes', [dict(dim=20, rot_dim=6, kv_rank=24, q_rank=18), dict(dim=32, rot_dim=32, kv_rank=128, q_rank=64)])
def test_a_far_latent_decides(sizes, backend, tmp_path):
    """The same for keys made from a cached latent: the query is made for the unrotated key of the marked token's latent."""
    config = plain.make_config([_latent(heads=3, vdim=16, scale=1.0, **sizes)], vocab=12, width=48, streams=2)
    w = _marked(config, plain.random_weights(config, 3, 1.0))
    rank, dim, rot = sizes['kv_rank'], sizes['dim'], sizes['rot_dim']
    p = 'l0.mix.'
    latent = plain.rms(w[p + 'dkv'][:rank, 5], 1e-5) * w[p + 'dkv.norm']
    asked = plain.rms(w[p + 'dq'][:, 7], 1e-5) * w[p + 'dq.norm']
    query = w[p + 'uq'].clone().reshape(3, dim + rot, -1)
    for h in range(3):
        key = w[p + 'uk'][h * dim:(h + 1) * dim] @ latent
        query[h] = 0.0
        query[h, :dim] = _held(14.0 / (key @ key) * torch.outer(key, asked) / (asked @ asked))
    w[p + 'uq'] = query.reshape(3 * (dim + rot), -1)
    _far_key(config, w, backend, tmp_path / 'far')


def test_the_factor_of_the_second_map(backend, tmp_path):
    """Stored vectors whose products are large: the factor is far from the configuration's constant, and the first two and the
    last two are not exchangeable."""
    config = _one(_difference(heads=4, kv_heads=2, dim=10, vdim=16, diff=0.25))
    w = plain.random_weights(config, 6, 1.0)
    m = config['layers'][0]['mixer']
    w['l0.mix.lq1'], w['l0.mix.lk1'] = torch.full((10,), 0.5, dtype=torch.float64), torch.full((10,), 0.25, dtype=torch.float64)
    w['l0.mix.lq2'], w['l0.mix.lk2'] = torch.full((10,), -0.5, dtype=torch.float64), torch.full((10,), 0.25, dtype=torch.float64)
    factor = plain.difference_factor(w, 'l0.mix.', m)
    assert abs(float(factor) - (3.4903 - 0.2865 + 0.25)) < 1e-3
    tokens = tokens_for(config, 60, 3)
    turned = dict(w, **{'l0.mix.lq1': w['l0.mix.lq2'], 'l0.mix.lq2': w['l0.mix.lq1']})
    assert error(plain.logits(tokens, turned, config), plain.logits(tokens, w, config)) > 0.1
    case = make_case('factor', config, w, backend, tmp_path / 'factor', 8)
    runner = case.runner(pages=16)
    case.close(feed(runner, 'r', tokens, [60]), case.expected(tokens), 'whole')
    case.close(feed(runner, 'r', tokens, [20, 2, 7]), case.expected(tokens), 'portions and single tokens')


def _steady(config, w, beta_logit, h_channel=0):
    """A norm whose output has a constant 1 in one channel, which the step sizes read alone."""
    w['l0.norm1'][h_channel] = 0.0
    w['l0.norm1.b'][h_channel] = 1.0
    w['l0.mix.b'] = torch.zeros_like(w['l0.mix.b'])
    w['l0.mix.b'][:, h_channel] = beta_logit
    return w


@pytest.mark.parametrize('sizes', [dict(dim=8, vdim=12), dict(dim=64, vdim=48)])
def test_a_memory_lasts(sizes, backend, tmp_path):
    """Decays almost 1 and small step sizes: what the first tokens wrote still decides the output three hundred tokens later, in
    a prompt, across portions and through decoding (a memory that is lost, or zeroed at a portion's start, shows)."""
    config = _one(_delta(heads=2, kv_heads=1, conv=3, **sizes), width=16)
    w = _steady(config, plain.random_weights(config, 7, 1.0), -3.0)
    w['l0.mix.A_log'] = torch.full_like(w['l0.mix.A_log'], -9.0)
    tokens = tokens_for(config, 330, 5)
    other = [(t + 1) % 30 for t in tokens[:20]] + tokens[20:]
    late = list(range(300, 330))
    assert error(plain.logits(other, w, config)[late], plain.logits(tokens, w, config)[late]) > 0.01
    case = make_case('memory', config, w, backend, tmp_path / 'memory', 16)
    runner = case.runner(pages=32)
    expected = case.expected(tokens)
    case.close(feed(runner, 'r', tokens, [330], late), expected[late], 'whole')
    case.close(feed(runner, 'r', tokens, [2, 70, 2, 130, 100, 3], late), expected[late], 'portions and single tokens')


def test_a_key_written_again_replaces_its_value(backend, tmp_path):
    """Step sizes near 1, no forgetting, two tokens only and no convolution: a key's value is replaced, not added to, so a late
    output equals an early one; sums would grow with the length."""
    config = _one(_delta(heads=2, kv_heads=2, dim=8, vdim=12, conv=1), width=16)
    w = _steady(config, plain.random_weights(config, 11, 1.0), 6.0)
    w['l0.mix.A_log'] = torch.full_like(w['l0.mix.A_log'], -12.0)
    tokens = [3, 9] * 80
    expected = plain.logits(tokens, w, config)
    assert error(expected[[158, 159]], expected[[20, 21]]) < 0.02
    case = make_case('again', config, w, backend, tmp_path / 'again', 16)
    runner = case.runner(pages=16)
    case.close(feed(runner, 'r', tokens, [160]), expected, 'whole')
    case.close(feed(runner, 'r', tokens, [33, 2, 64]), expected, 'portions and single tokens')


def test_fast_and_slow_decays_together(backend, tmp_path):
    """Channels that forget within a token beside channels that hardly forget, in one head: a chunk's sums of log decays reach
    thousands, and what is left of the slow ones must be exact."""
    config = _one(_delta(heads=4, kv_heads=2, dim=8, vdim=12, conv=2), width=16)
    w = plain.random_weights(config, 9, 1.0)
    w['l0.mix.A_log'] = torch.tensor([1.5, -6.0, 3.0, -1.0], dtype=torch.float64)
    w['l0.mix.dt_bias'] = torch.tensor([6.0, 0.0, -3.0, 30.0, -9.0, 2.0, 1.0, -6.0] * 4, dtype=torch.float64)
    case = make_case('decays', config, w, backend, tmp_path / 'decays', 16)
    tokens = tokens_for(config, 150, 5)
    runner = case.runner(pages=16)
    case.close(feed(runner, 'r', tokens, [150]), case.expected(tokens), 'whole')
    case.close(feed(runner, 'r', tokens, [65, 2, 63]), case.expected(tokens), 'portions and single tokens')


def test_the_convolution_sees_the_step_before(backend, tmp_path):
    """Another token two places back changes a token's logits through the convolution; portions that begin anywhere, also
    shorter than the taps, read the inputs that earlier steps left, and a request that takes over a slot starts from zeros."""
    config = _one(_delta(heads=2, kv_heads=1, dim=8, vdim=12, conv=5), width=16)
    w = plain.random_weights(config, 10, 1.0)
    tokens = tokens_for(config, 24, 4)
    case = make_case('conv', config, w, backend, tmp_path / 'conv', 4)
    runner = case.runner(pages=12, requests=1)
    for cuts in ([24], [10, 14], [2] * 12, [], [1, 9, 1, 2, 11]):
        case.close(feed(runner, 'r', tokens, cuts), case.expected(tokens), f'cuts {cuts}')
    case.close(feed(runner, 'r', tokens[5:], []), case.expected(tokens[5:]), 'another sequence in the same slot')


def test_streams_are_mixed_from_and_to(backend, tmp_path):
    """Mixing matrices far from symmetric, one stream read by nobody but through the mix: a transposed matrix, streams updated one
    after another, or an update from the new values would show."""
    config = plain.make_config([_difference(mlp=plain.moe(3, 2, 12)), _delta()], vocab=30, width=16, streams=3)
    w = plain.random_weights(config, 12, 1.0)
    for i, q in ((0, 1), (0, 2), (1, 1)):
        w[f'l{i}.hc{q}.mix'] = torch.tensor([[0.5, 1.0, -0.75], [0.0, 0.25, 1.5], [1.0, 0.0, 0.5]], dtype=torch.float64)
        w[f'l{i}.hc{q}.in'] = torch.tensor([1.0, 0.0, 0.5], dtype=torch.float64)
        w[f'l{i}.hc{q}.out'] = torch.tensor([0.0, 2.0, -0.5], dtype=torch.float64)
    tokens = tokens_for(config, 40, 3)
    base = plain.logits(tokens, w, config)
    turned = {name: t.T.contiguous() if name.endswith('.mix') else t for name, t in w.items()}
    assert error(plain.logits(tokens, turned, config), base) > 0.3
    case = make_case('streams', config, w, backend, tmp_path / 'streams', 8)
    runner = case.runner(pages=12)
    case.close(feed(runner, 'r', tokens, [40]), base, 'whole')
    case.close(feed(runner, 'r', tokens, [17, 2]), base, 'portions and single tokens')


def test_a_layer_reads_another_layers_cache(backend, tmp_path):
    """Two layers read the keys and values of the first, with queries, factors and gates of their own; the readers hold nothing."""
    layers = [_difference(heads=4, kv_heads=2, dim=8, vdim=16), _delta(), _difference(heads=4, kv_heads=2, dim=8, vdim=16, scale=1.0, diff=0.1, kv_from=0),
              _difference(heads=4, kv_heads=2, dim=8, vdim=16, scale=0.2, diff=0.8, kv_from=0)]
    config = plain.make_config(layers, vocab=30, width=24, streams=2)
    w = plain.random_weights(config, 13, 1.0)
    case = make_case('reader', config, w, backend, tmp_path / 'reader', 8)
    runner = case.runner(pages=12)
    assert [len(g['entries']) for g in runner.cache.kv_groups] == [1]
    tokens = tokens_for(config, 70, 3)
    case.close(feed(runner, 'r', tokens, [70]), case.expected(tokens), 'whole')
    case.close(feed(runner, 'r', tokens, [31, 2, 16]), case.expected(tokens), 'portions and single tokens')


def test_the_streams_sum_layer_by_layer(backend, tmp_path):
    """The sum of the streams after every layer against the plain model's."""
    import kernel_refs
    config, seed, page_size, spread = CONFIGS['mixed']
    case = make_case('layers', config, weights_of('mixed', backend[1]), backend, tmp_path / 'layers', page_size)
    tokens = tokens_for(config, 30, 2)
    collected = []
    plain.forward(config, case.weights, tokens, collect=collected)

    def settled(stream, pending):
        return kernel_refs.stream_join(stream.clone(), pending, streams=config['streams'], out_dtype=torch.float32).cpu()
    seen = []
    case.model.observer = lambda position, stream, pending, scale: seen.append(settled(stream, pending))
    try:
        feed(case.runner(pages=16), 'r', tokens, [30])
    finally:
        case.model.observer = None
    assert len(seen) == len(collected)
    for run, (actual, expected) in enumerate(zip(seen, collected)):
        case.close(actual, expected, f'layer {run}')


# ------------------------------------------------------------------------------------------------ the oracle, the configuration
def test_the_plain_model_cuts_like_its_parts():
    """The oracle itself: a prefix's logits do not depend on what follows, and tokens fed one by one through the
    states give what the whole sequence gives."""
    config, seed, _, spread = CONFIGS['mixed']
    weights = plain.random_weights(config, seed, spread)
    tokens = tokens_for(config, 30, 1)
    whole = plain.logits(tokens, weights, config)
    assert torch.allclose(whole[:17], plain.logits(tokens[:17], weights, config), atol=1e-9)
    states, rows = None, []
    for start, size in ((0, 1), (1, 2), (3, 9), (12, 1), (13, 17)):
        out, states = plain.forward(config, weights, tokens[start:start + size], start=start, states=states)
        rows.append(out)
    assert torch.allclose(torch.cat(rows), whole, atol=1e-9)


def test_the_plain_mechanisms_on_numbers_made_by_hand():
    F = torch.float64
    num = lambda *values: torch.tensor(values, dtype=F)
    # tanh(alpha x) w + b
    w = {'n': num(2.0, 3.0), 'n.b': num(0.5, -1.0), 'n.alpha': torch.tensor(0.5, dtype=F)}
    assert torch.allclose(plain.tanh_norm(num(2.0, 0.0), w, 'n'), num(2.0 * torch.tanh(num(1.0)).item() + 0.5, -1.0))
    # two streams of one token and one channel: u = 3 x_1 + 5 x_2; x_1 <- m11 x_1 + m21 x_2 + o1 y
    hc = {'in': num(3.0, 5.0), 'mix': torch.tensor([[1.0, 2.0], [4.0, 8.0]], dtype=F), 'out': num(0.5, 0.25)}
    x = num(1.0, 10.0).reshape(2, 1, 1)
    assert plain.streams_in(x, hc, '').item() == 53.0
    assert plain.streams_out(x, num(100.0).reshape(1, 1), hc, '').flatten().tolist() == [91.0, 107.0]
    # a memory of one number: forget, correct, read
    one = torch.ones(2, 1, 1, dtype=F)
    o, S = plain.delta_scan(2.0 * one, one, torch.stack([3.0 * one[0], 7.0 * one[0]]), 0.5 * one, num(0.5, 1.0).reshape(2, 1),
                            torch.zeros(1, 1, 1, dtype=F))
    # S: 0 -> 1.5; 0.75 -> 0.75 + (7 - 0.75) = 7
    assert o.flatten().tolist() == [3.0, 14.0] and S.item() == 7.0
    assert torch.allclose(plain.unit(num(3.0, 4.0)), num(0.6, 0.8), atol=1e-7)
    # a convolution of two taps, the last column the current token's
    state = {}
    first = plain.short_conv(num(1.0, 2.0).reshape(2, 1), num(10.0, 1.0).reshape(1, 2), state, 'x')
    assert first.flatten().tolist() == [1.0, 12.0]
    assert plain.short_conv(num(3.0).reshape(1, 1), num(10.0, 1.0).reshape(1, 2), state, 'x').item() == 23.0
    # neighbours turn together: a quarter turn takes (u, v) to (-v, u)
    turned = plain.rotate_neighbours(num(1.0, 2.0, 3.0, 4.0).reshape(1, 4), torch.tensor([1]), 4, (2 / torch.pi) ** 2)
    c, s = torch.cos(num(1.0)).item(), torch.sin(num(1.0)).item()
    assert torch.allclose(turned[0], num(c - 2 * s, 2 * c + s, -4.0, 3.0))
    # the router: softmax over the chosen logits, squared relu inside
    moe = {'router': torch.tensor([[1.0], [0.0], [-9.0]], dtype=F)}
    for e, up in enumerate((2.0, -3.0, 5.0)):
        moe[f'e{e}.up'], moe[f'e{e}.down'] = num(up).reshape(1, 1), num(1.0).reshape(1, 1)
    share = torch.sigmoid(num(1.0)).item()
    out = plain.feed_forward(num(1.0).reshape(1, 1), moe, '', plain.moe(3, 2, 1))
    assert torch.isclose(out, num(share * 4.0)).all()


def test_config_round_trip_and_refusals():
    from qil_amd.config import ConfigError, KebudraConfig
    from qil_amd.registry import architecture_for
    config = CONFIGS['mixed'][0]
    typed = KebudraConfig.from_dict(config)
    assert architecture_for(config).name == 'Kebudra'
    assert KebudraConfig.from_dict(json.loads(json.dumps(typed.to_dict()))) == typed
    layers = config['layers']

    def with_mixer(index, **changes):
        return dict(config, layers=layers[:index] + [dict(layers[index], mixer=dict(layers[index]['mixer'], **changes))] + layers[index + 1:])

    for broken in (dict(config, window=4), dict(config, norm=dict(eps=1e-6, kind='rms')), dict(config, norm=dict(eps=0)),
                   dict(config, streams=0), dict(config, streams=1.5), dict(config, embedding=dict(scale=0.0)), dict(config, embedding={}),
                   dict(config, layers=[]), dict(config, layers=[dict(layers[0], type='conv')]),
                   with_mixer(0, rot=dict(base=10.0, dims=4)), with_mixer(0, rot_dim=5), with_mixer(0, sink=True), with_mixer(0, q_rank=0),
                   with_mixer(1, heads=4), with_mixer(1, diff='x'), with_mixer(1, kv_from=1), with_mixer(4, kv_from=2), with_mixer(4, kv_from=3),
                   with_mixer(4, dim=8), with_mixer(2, conv=0), with_mixer(2, kv_heads=4), with_mixer(2, scale=1.0),
                   dict(config, layers=[dict(layers[0], mlp=dict(kind='dense', ff=8))]),
                   dict(config, layers=[dict(layers[0], mlp=plain.moe(2, 3, 8))]), dict(config, layers=[dict(layers[0], mlp=plain.moe(2, 1, 0))])):
        with pytest.raises(ConfigError):
            KebudraConfig.from_dict(broken)


def test_sizes_beyond_the_kernels_are_refused_when_the_model_is_built():
    from qil_amd import ops
    from qil_amd.config import KebudraConfig
    from qil_amd.models.kebudra import build_kebudra
    for config in (_one(_difference(dim=130)), _one(_difference(vdim=300)), _one(_delta(dim=257)), _one(_delta(), streams=17)):
        with pytest.raises(ops.UnsupportedShape):
            build_kebudra(KebudraConfig.from_dict(config), device='cpu')


def test_the_bench_makes_valid_configurations():
    """The configurations that ``bench.py --phase designs --design kebudra`` measures are ones the design accepts."""
    import bench
    from qil_amd.config import KebudraConfig
    for sizes in bench.DESIGN_SIZES.values():
        for kind in ('turns', 'delta', 'difference', 'latent'):
            assert len(KebudraConfig.from_dict(bench.kebudra_config(sizes, 6, 100, kind)).layers) == 6


def test_random_weights_load(tmp_path, cpu_kernels):
    """A folder written from a configuration and a seed holds every tensor of the design, and loads and runs; the inner sizes of
    the low-rank products are the folder's."""
    from qil_amd.weights import write_random_model
    config = CONFIGS['mixed'][0]
    folder = write_random_model(tmp_path / 'random', config, 4)
    from safetensors import safe_open
    with safe_open(str(folder / 'model.safetensors'), framework='pt') as f:
        stored = {name: tuple(f.get_slice(name).get_shape()) for name in f.keys()}
    mine = {name: tuple(t.shape) for name, t in plain.random_weights(config, 1).items()}
    assert set(stored) == set(mine)
    low = ('.a1', '.a2', '.g1', '.g2')
    assert all(stored[name] == mine[name] for name in mine if not name.endswith(low))
    model = load_model(folder, dtype=torch.float32, device='cpu')
    runner = ModelRunner(model, num_pages=8, page_size=8, max_requests=1)
    runner.admit('r')
    assert torch.isfinite(runner.step([StepEntry('r', (1, 2, 3), (2,))])).all()


def test_low_rank_matrices_that_do_not_fit_are_refused(tmp_path, cpu_kernels):
    config = CONFIGS['mixed'][0]
    w = plain.random_weights(config, 1)
    w['l2.mix.a2'] = w['l2.mix.a2'][:, :-1]
    folder = write_model_folder(tmp_path / 'model', config, w, torch.bfloat16)
    with pytest.raises(ValueError, match='do not fit'):
        load_model(folder, dtype=torch.float32, device='cpu')


@pytest.mark.gpu
def test_command_line(tmp_path):
    """``python -m qil_amd`` on a Kebudra folder: greedy generation through the scheduler in portions of two tokens
    equals the plain model's, and a folder written from a configuration with a seed generates with a temperature."""
    import subprocess
    import sys
    from pathlib import Path
    root = Path(__file__).resolve().parent.parent
    config, seed, _, spread = CONFIGS['mixed']
    weights = plain.random_weights(config, seed, spread)
    folder = write_model_folder(tmp_path / 'model', config, weights, torch.bfloat16)
    prompt, out = [5, 17, 3, 41, 8, 8, 30], tmp_path / 'result.json'
    run = subprocess.run([sys.executable, '-m', 'qil_amd', '--model', str(folder), '--token-ids', json.dumps(prompt),
                          '--dtype', 'float32', '--max-new-tokens', '6', '--pages', '8', '--page-size', '4',
                          '--chunk-size', '2', '--ignore-eos', '--output', str(out)],
                         cwd=root, capture_output=True, text=True, timeout=300)
    assert run.returncode == 0, run.stderr[-2000:]
    result = json.loads(out.read_text())
    assert result['token_ids'] == plain.greedy(prompt, 6, weights, config) and result['state'] == 'completed'
    run = subprocess.run([sys.executable, '-m', 'qil_amd', '--model', str(tmp_path / 'random'), '--random-config',
                          json.dumps(CONFIGS['wide'][0]), '--random-seed', '3', '--token-ids', '[1, 2, 3]', '--dtype',
                          'bfloat16', '--max-new-tokens', '5', '--temperature', '0.8', '--ignore-eos', '--output', str(out)],
                         cwd=root, capture_output=True, text=True, timeout=300)
    assert run.returncode == 0, run.stderr[-2000:]
    assert len(json.loads(out.read_text())['token_ids']) == 5


@pytest.mark.gpu
@pytest.mark.parametrize('dtype', ['float32', 'bfloat16'])
def test_trace_replay_program(tmp_path, dtype):
    """``bin/trace_run`` on a Kebudra folder: requests alone and whole, their last tokens one by one, portions down to
    two tokens, and up to four live requests in a pool of pages and state slots that is used again."""
    from test_engine_gpu import collect, replay, traces
    config, seed, _, _ = CONFIGS['mixed']
    weights = weights_of('mixed', getattr(torch, dtype))
    folder = write_model_folder(tmp_path / 'model', config, weights, torch.bfloat16)
    prompts, shapes = traces(dict(vocab_size=config['vocab']), seed)
    judge = Case('replay', config, weights, None, 16, getattr(torch, dtype))
    for shape, (steps, max_tokens) in shapes.items():
        out = tmp_path / shape
        replay(folder, dtype, steps, out, max_tokens)
        rows = collect(out, steps, config['vocab'])
        assert rows, shape
        for request, items in rows.items():
            got = torch.stack([row for _, row in items])
            judge.close(got, judge.expected(prompts[request])[[position for position, _ in items]], f'{shape} {request}')
