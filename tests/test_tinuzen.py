"""The Tinuzen design in the engine against its plain restatement (``plain_tinuzen``), under every way of cutting the
work: whole prompts, token-by-token decoding, portions down to two tokens, unequal batches, pages and state slots that
are freed and used again, and generation through the serving loop; then each mechanism alone, with weights or inputs
made so that a fault shows (a far key that decides the answer, the keys just inside and just outside a window and the kept
first ones, a denominator whose added one takes most of the weight, a state that must survive hundreds of tokens, a pair
of tokens that is cut by a step).

Each model test runs three ways, as the step function's own tests do: on the CPU with the kernels' plain references
substituted, and on the GPU with the HIP kernels in float32 and in bfloat16 (marked ``gpu``).  Page and state storage
is filled with NaN first.  Configurations are small and their sizes differ from one another in every field.
"""
import json
import random

import pytest
import torch

import plain_tinuzen as plain
from conftest import write_model_folder
from qil_amd.engine import ModelRunner, StepEntry
from qil_amd.weights import load_model

GPU = [pytest.param(('cuda', torch.float32), id='gpu-f32', marks=pytest.mark.gpu),
       pytest.param(('cuda', torch.bfloat16), id='gpu-bf16', marks=pytest.mark.gpu)]
BACKENDS = [pytest.param(('cpu', torch.float32), id='cpu-refs')] + GPU


def _mixed():
    # a loop in the middle, run three times; sizes that are multiples of nothing much
    layers = [
        plain.attention_layer(heads=6, kv_heads=3, dim=20, vdim=12, scale=0.3, window=11, keep_first=5, ff=44),
        plain.parallel_layer(heads=4, kv_heads=2, dim=24, scale=0.25, rot_dims=10, base=300.0, scan_heads=6, vdim=10, state=7,
                             groups=3, conv=4, norm_groups=4, left_scale=0.7, right_scale=1.3, ff=56),
        plain.attention_layer(heads=5, kv_heads=1, dim=8, vdim=16, scale=0.4, window=30, keep_first=17),
        plain.parallel_layer(heads=3, kv_heads=3, dim=12, scale=0.4, rot_dims=12, scan_heads=2, vdim=18, state=20, groups=1,
                             conv=2, norm_groups=1, ff=24),
    ]
    return plain.make_config(layers, vocab=97, width=44, embedding_scale=6.6, bigram=(53, 31, 5), loop=(1, 3, 3))


def _wide():
    # heads of 64 and 128 (sizes with kernels of their own), states and values of a real model's sizes, five taps, windows of
    # a page and more with kept keys below, at and above a page's size; the loop begins at the first layer
    layers = [
        plain.parallel_layer(heads=4, kv_heads=1, dim=64, scale=0.125, rot_dims=32, base=1e4, scan_heads=4, vdim=64, state=128,
                             groups=2, conv=4, norm_groups=2, left_scale=0.9, right_scale=0.5, ff=72),
        plain.attention_layer(heads=4, kv_heads=2, dim=128, vdim=128, scale=0.09, window=70, keep_first=33, ff=32),
        plain.parallel_layer(heads=2, kv_heads=2, dim=128, scale=0.08, rot_dims=64, base=500.0, scan_heads=8, vdim=32, state=40,
                             groups=8, conv=5, norm_groups=8, left_scale=0.4, right_scale=0.6, ff=40),
        plain.attention_layer(heads=8, kv_heads=2, dim=64, vdim=64, scale=0.125, window=16, keep_first=1, ff=80),
    ]
    return plain.make_config(layers, vocab=61, width=64, eps=1e-6, embedding_scale=8.0, bigram=(11, 3, 2), loop=(0, 2, 2))


def _plainest():
    # no token pairs, no loop, no window, no rotation, nothing beside the first mixer, every count one
    layers = [plain.attention_layer(heads=3, kv_heads=1, dim=12, vdim=12, scale=12 ** -0.5),
              plain.parallel_layer(heads=1, kv_heads=1, dim=10, scale=0.6, scan_heads=1, vdim=14, state=5, conv=1, ff=16)]
    return plain.make_config(layers, vocab=50, width=24)


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
# between kernels rounded; state, step sizes, decays, scores, norms and residual sums float32) about 0.01 to 0.04.
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
            group['k'].fill_(float('nan'))
            group['v'].fill_(float('nan'))
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


def make_case(name, config, weights, backend, folder, page_size):
    device, dtype = backend
    write_model_folder(folder, config, weights, torch.bfloat16)
    return Case(name, config, weights, load_model(folder, dtype=dtype, device=device), page_size, dtype)


@pytest.fixture(params=sorted(CONFIGS))
def case(request, backend, tmp_path):
    config, seed, page_size, spread = CONFIGS[request.param]
    return make_case(request.param, config, plain.random_weights(config, seed, spread), backend, tmp_path / request.param, page_size)


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
    """Several hundred tokens at once (the recurrence in blocks side by side, the attention's keys in many tiles), then two
    long portions and single tokens; the late places are compared."""
    config, seed, page_size, spread = CONFIGS[name]
    case = make_case(name, config, plain.random_weights(config, seed, spread), where, tmp_path / name, page_size)
    runner = case.runner(pages=-(-700 // case.page_size) + 2)
    tokens = tokens_for(case.config, 650, 10)
    late = list(range(560, 650))
    expected = case.expected(tokens)[late]
    case.close(feed(runner, 'r', tokens, [650], late), expected, 'whole')
    case.close(feed(runner, 'r', tokens, [130, 470, 3], late), expected, 'two long portions, then single tokens')


@pytest.mark.parametrize('where', GPU)
@pytest.mark.parametrize('name', sorted(CONFIGS))
def test_graphs_replay_the_same_logits(name, where, tmp_path):
    """Decode steps from captured graphs (the previous token travels with the other pieces of a step), between them a
    second request's portion, and a batch that shrinks."""
    config, seed, page_size, spread = CONFIGS[name]
    case = make_case(name, config, plain.random_weights(config, seed, spread), where, tmp_path / name, page_size)
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
    """Portions down to two tokens, cut inside pages and windows and at their borders, shorter than the convolution's
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
def _beside(**changes):
    base = dict(heads=2, kv_heads=1, dim=8, scale=0.5, rot_dims=8, scan_heads=2, vdim=4, state=4, conv=2)
    base.update(changes)
    return plain.parallel_layer(**base)


ALONE = {
    'keys-as-values-one-head': plain.make_config(
        [_beside(heads=1, kv_heads=1, dim=14, rot_dims=6, scale=0.9, right_scale=0.0)], vocab=40, width=24),
    'keys-as-values-unrotated': plain.make_config(
        [_beside(heads=9, kv_heads=3, dim=11, rot_dims=None, scale=0.4, right_scale=0.0)], vocab=40, width=36),
    'keys-as-values-heads-of-64': plain.make_config(
        [_beside(heads=4, kv_heads=2, dim=64, rot_dims=64, scale=0.125, right_scale=0.01)], vocab=40, width=32),
    'keys-as-values-heads-of-128': plain.make_config(
        [_beside(heads=4, kv_heads=4, dim=128, rot_dims=32, scale=0.09, base=50.0, right_scale=0.01)], vocab=40, width=32),
    'recurrence-one-of-each': plain.make_config(
        [_beside(scan_heads=1, vdim=1, state=1, conv=1, left_scale=0.0)], vocab=40, width=16),
    'recurrence-odd-sizes': plain.make_config(
        [_beside(scan_heads=6, vdim=7, state=33, groups=2, conv=7, norm_groups=3, left_scale=0.0)], vocab=40, width=24),
    'recurrence-many-states': plain.make_config(
        [_beside(scan_heads=2, vdim=70, state=200, groups=2, conv=3, norm_groups=1, left_scale=0.01)], vocab=40, width=40),
    'recurrence-norm-groups-across-heads': plain.make_config(
        [_beside(scan_heads=3, vdim=16, state=16, groups=1, conv=4, norm_groups=2, left_scale=0.0)], vocab=40, width=24),
    'distance-one-head': plain.make_config(
        [plain.attention_layer(heads=1, kv_heads=1, dim=10, vdim=14, scale=0.9)], vocab=40, width=24),
    'distance-odd-heads': plain.make_config(
        [plain.attention_layer(heads=7, kv_heads=7, dim=36, vdim=4, scale=0.2, window=19, keep_first=2, ff=20)], vocab=40, width=36),
    'distance-heads-of-128': plain.make_config(
        [plain.attention_layer(heads=8, kv_heads=2, dim=128, vdim=128, scale=0.09, window=40, keep_first=40)], vocab=40, width=48),
    'distance-heads-of-128-unwindowed': plain.make_config(
        [plain.attention_layer(heads=4, kv_heads=4, dim=128, vdim=128, scale=0.09)], vocab=40, width=48),
    'window-of-one-and-a-kept-key': plain.make_config(
        [plain.attention_layer(heads=4, kv_heads=2, dim=16, vdim=8, scale=0.8, window=1, keep_first=1)], vocab=40, width=16),
    'window-without-kept-keys': plain.make_config(
        [plain.attention_layer(heads=4, kv_heads=2, dim=64, vdim=32, scale=0.2, window=9)], vocab=40, width=32),
    'window-wider-than-the-sequence': plain.make_config(
        [plain.attention_layer(heads=2, kv_heads=1, dim=16, vdim=16, scale=0.5, window=500, keep_first=300)], vocab=40, width=16),
    'loop-of-one-layer': plain.make_config(
        [plain.attention_layer(heads=2, kv_heads=1, dim=8, vdim=8, scale=0.5, ff=12), _beside(ff=8)], vocab=40, width=16,
        bigram=(7, 9, 4), loop=(1, 2, 4)),
    'loop-once': plain.make_config([_beside()], vocab=40, width=16, embedding_scale=3.0, loop=(0, 1, 1)),
    'pairs-in-one-bucket': plain.make_config([_beside(ff=70)], vocab=40, width=20, embedding_scale=0.5, bigram=(1, 0, 1)),
}


@pytest.mark.parametrize('name', sorted(ALONE))
def test_each_mechanism_alone(name, backend, tmp_path):
    """Models of one or two layers: one mechanism each, at sizes where fields that often coincide differ (key size and
    value size, heads and key/value heads, rotated part and head, states and a wave's lanes) and where counts are 1."""
    config = ALONE[name]
    case = make_case(name, config, plain.random_weights(config, 5, 1.3), backend, tmp_path / name, 8)
    tokens = tokens_for(config, 100, 9)
    runner = case.runner(pages=16)
    case.close(feed(runner, 'r', tokens, [100]), case.expected(tokens), 'whole')
    case.close(feed(runner, 'r', tokens, [13, 2, 9, 8, 40]), case.expected(tokens), 'portions, then single tokens')


def _marked(config, w, layer, q_name, k_name, heads, dim, key_channel=5, query_channel=7):
    """Weights in which token 10's key is what token 11's query looks for: the marked token's input excites one channel
    and the asking token's another, and the query matrix's column for the second is the key matrix's column for the
    first (for every query head)."""
    width = config['width']
    embed = w['embed'].clone()
    embed[10], embed[11] = 0.0, 0.0
    embed[10, key_channel], embed[11, query_channel] = 8.0, 8.0
    w['embed'] = embed
    w[f'l{layer}.norm1'] = torch.ones(width, dtype=torch.float64)
    query = w[q_name].clone()
    for h in range(heads):
        query[h * dim:(h + 1) * dim, query_channel] = w[k_name][:dim, key_channel]
    w[q_name] = query
    return w


def test_a_far_key_decides(backend, tmp_path):
    """One key hundreds of tokens back, at a page's last place, is the only one a late query likes: its value, which is the
    key before its rotation, must come through, in a prompt, in portions and in decoding.  (Two rotated elements of 32 stay
    out of the marked score.)"""
    config = plain.make_config([plain.parallel_layer(heads=2, kv_heads=1, dim=32, scale=1.5, rot_dims=2, scan_heads=1, vdim=4,
                                                     state=2, conv=2, right_scale=0.02)], vocab=12, width=48)
    w = plain.random_weights(config, 3, 1.0)
    w['l0.mix.left.k'][:2] = 0.0
    w = _marked(config, w, 0, 'l0.mix.left.q', 'l0.mix.left.k', 2, 32)
    case = make_case('far', config, w, backend, tmp_path / 'far', 16)
    tokens = [t % 10 for t in tokens_for(config, 420, 2)]
    tokens[15] = 10                                   # the last place of the first page
    asking = [300, 401, 419]
    for place in asking:
        tokens[place] = 11
    expected = case.expected(tokens)
    other = list(tokens)
    other[15] = 3
    moved = error(plain.logits(other, w, config)[asking], expected[asking])
    assert moved > 0.05, 'the test lost its point: the far key does not matter'
    runner = case.runner(pages=40)
    case.close(feed(runner, 'r', tokens, [420], asking), expected[asking], 'in a prompt')
    if case.model.device.type == 'cuda':
        case.close(feed(runner, 'r', tokens, [128, 130, 100, 42], asking), expected[asking], 'in portions')
    case.close(feed(runner, 'r', tokens, [400], asking[1:]), expected[asking[1:]], 'decoded')


@pytest.mark.parametrize('dim', [16, 64, 128])
@pytest.mark.parametrize('window,keep', [(5, 3), (16, 16), (23, 40), (70, 1)])
def test_the_edges_of_a_window_and_of_the_kept_keys(window, keep, dim, backend, tmp_path):
    """The marked key lies exactly window - 1 places back (the last one seen) or window places back (the first one
    not seen), or is the last of the kept keys (seen from any distance) or the first behind them (not seen); the asking
    rows are in a prompt, in the first rows of a portion, and decoded; the window is shorter than a page, a page, and
    longer, and so are the kept keys.  One query head: its slope 2^-8 leaves far scores standing."""
    if backend[0] == 'cpu' and dim != 16:
        pytest.skip('the GPU kernels differ by head size')
    config = plain.make_config([plain.attention_layer(heads=1, kv_heads=1, dim=dim, vdim=8, scale=10.0 / dim, window=window,
                                                      keep_first=keep)], vocab=12, width=32)
    w = plain.random_weights(config, 4, 1.0)
    for name in ('q', 'k'):
        w[f'l0.mix.{name}.norm'] = torch.ones_like(w[f'l0.mix.{name}.norm'])
    w = _marked(config, w, 0, 'l0.mix.q', 'l0.mix.k', 1, dim)
    case = make_case('edge', config, w, backend, tmp_path / 'edge', 16)
    r = random.Random(window)
    at_window = {}                                    # asking place -> marked place
    for marked, inside in ((140, True), (150 + window, False), (180 + 2 * window, True)):
        at_window[marked + (window - 1 if inside else window)] = marked
    # the last kept key, the one behind it, the window's edges: a sequence each (marked keys are alike, and one that is
    # seen would hide another)
    for asking in ({120: keep - 1, 399: keep - 1}, {120: keep, 399: keep}, at_window):
        tokens = [r.randrange(10) for _ in range(400)]
        for marked in asking.values():
            tokens[marked] = 10
        for at in asking:
            tokens[at] = 11
        places = sorted(asking)
        expected = case.expected(tokens)
        for at, marked in asking.items():             # the point: seen, the marked key matters; unseen, it does not
            other = list(tokens)
            other[marked] = 3
            moved = error(plain.logits(other, w, config)[[at]], expected[[at]])
            seen = at - marked < window or marked < keep
            assert (moved > 0.05) == seen, (at, marked, moved)
        runner = case.runner(pages=32)
        case.close(feed(runner, 'r', tokens, [400], places), expected[places], 'in a prompt')
        cuts = [places[0] - 1, 2, places[1] - places[0] - 1, 40]         # portions that begin at and before asking rows
        case.close(feed(runner, 'r', tokens, cuts, places), expected[places], 'in portions')
        if case.model.device.type == 'cuda':
            case.close(feed(runner, 'r', tokens, [20], places), expected[places], 'decoded')


def test_kept_pages_stay_and_others_go_back(backend, tmp_path):
    """A windowed layer with kept keys gives the pages between back while the request lives, keeps the first ones, and the
    pages that came back serve another request."""
    config = plain.make_config([plain.attention_layer(heads=2, kv_heads=1, dim=16, vdim=16, scale=0.6, window=9, keep_first=13)],
                               vocab=40, width=16)
    case = make_case('pages', config, plain.random_weights(config, 8, 1.3), backend, tmp_path / 'pages', 4)
    runner = case.runner(pages=14)
    a, b = tokens_for(config, 90, 1), tokens_for(config, 20, 2)
    runner.admit('a')
    rows = []
    for at in range(0, 90, 10):                        # 23 blocks of keys pass through 14 pages
        rows.append(runner.step([StepEntry('a', tuple(a[at:at + 10]), tuple(range(10)))]))
    assert len(runner.cache.kv_groups[0]['pool'].held('a')) <= 4 + 3 + 1
    assert runner.cache.table(0, 'a')[:4] == [page for page in runner.cache.table(0, 'a')[:4] if page >= 0]
    case.close(torch.cat(rows), case.expected(a), 'through few pages')
    case.close(feed(runner, 'b', b, [7, 2]), case.expected(b), 'in pages that came back')
    runner.release('a')
    runner.cache.check()


def test_one_in_the_denominator(backend, tmp_path):
    """Scores far below zero: the added one takes nearly all of the weight, which an engine that left it out (or shifted it
    with the scores) would not give."""
    config = plain.make_config([_beside(heads=4, kv_heads=2, dim=8, scale=0.6, rot_dims=2, base=1e9, right_scale=0.0)], vocab=30, width=16)
    w = plain.random_weights(config, 6, 1.0)
    w['l0.norm1'] = w['l0.norm1'].abs()
    w['embed'] = (w['embed'].abs() + 0.5).to(torch.bfloat16).double()      # every channel positive: a negative query matrix lowers every score
    w['l0.mix.left.k'] = w['l0.mix.left.k'].abs()
    w['l0.mix.left.q'] = -w['l0.mix.left.q'].abs()
    tokens = tokens_for(config, 80, 3)
    m = config['layers'][0]['mixer']['left']
    h = plain.rms(w['embed'][tokens], 1e-5) * w['l0.norm1']
    with_one = plain.key_value_attention(h, torch.arange(80), w, 'l0.mix.left.', m, {})
    shifted = dict(w)
    shifted['l0.mix.left.q'] = -w['l0.mix.left.q']     # positive scores: the one hardly counts
    assert with_one.abs().mean() < 0.5 * plain.key_value_attention(h, torch.arange(80), shifted, 'l0.mix.left.', m, {}).abs().mean()
    for name, weights in (('low', w), ('high', shifted)):
        case = make_case(name, config, weights, backend, tmp_path / name, 8)
        runner = case.runner(pages=16)
        case.close(feed(runner, 'r', tokens, [80]), case.expected(tokens), f'{name}, whole')
        case.close(feed(runner, 'r', tokens, [30, 2, 7]), case.expected(tokens), f'{name}, portions and single tokens')


def test_a_state_lasts(backend, tmp_path):
    """A recurrence whose decays are almost 1: what the first tokens wrote still decides the output three hundred tokens
    later, in a prompt, across portions and through decoding (a state that is lost, or zeroed at a portion's start,
    shows)."""
    config = plain.make_config([_beside(scan_heads=2, vdim=8, state=8, conv=3, left_scale=0.0)], vocab=30, width=16)
    w = plain.random_weights(config, 7, 1.0)
    w['l0.mix.right.A_log'] = torch.full_like(w['l0.mix.right.A_log'], -7.0)       # decay exp(-d * 0.0009)
    tokens = tokens_for(config, 330, 5)
    other = [(t + 1) % 30 for t in tokens[:20]] + tokens[20:]
    late = list(range(300, 330))
    assert error(plain.logits(other, w, config)[late], plain.logits(tokens, w, config)[late]) > 0.01
    case = make_case('state', config, w, backend, tmp_path / 'state', 16)
    runner = case.runner(pages=32)
    expected = case.expected(tokens)
    case.close(feed(runner, 'r', tokens, [330], late), expected[late], 'whole')
    case.close(feed(runner, 'r', tokens, [2, 70, 2, 130, 100, 3], late), expected[late], 'portions and single tokens')


def test_fast_and_slow_decays_together(backend, tmp_path):
    """Steps so large that a head forgets within a token beside heads that hardly forget: the sums of a block's decays
    reach hundreds, and their differences must not lose the small ones."""
    config = plain.make_config([_beside(scan_heads=4, vdim=8, state=8, groups=2, conv=2, left_scale=0.0)], vocab=30, width=16)
    w = plain.random_weights(config, 9, 1.0)
    w['l0.mix.right.dt_bias'] = torch.tensor([6.0, 0.0, -3.0, 30.0], dtype=torch.float64)
    w['l0.mix.right.A_log'] = torch.tensor([1.5, -6.0, 2.0, -9.0], dtype=torch.float64)
    case = make_case('decays', config, w, backend, tmp_path / 'decays', 16)
    tokens = tokens_for(config, 150, 5)
    runner = case.runner(pages=16)
    case.close(feed(runner, 'r', tokens, [150]), case.expected(tokens), 'whole')
    case.close(feed(runner, 'r', tokens, [65, 2, 63]), case.expected(tokens), 'portions and single tokens')


def test_a_pair_is_not_cut_by_a_step(backend, tmp_path):
    """The row of the pair table depends on the token of the step before: another token there changes the logits, and
    steps that begin anywhere read the right row; a request that takes over a slot starts with the last row."""
    config = plain.make_config([_beside(left_scale=0.1, right_scale=0.1)], vocab=30, width=16, embedding_scale=0.3, bigram=(101, 37, 3))
    w = plain.random_weights(config, 10, 1.0)
    tokens = tokens_for(config, 24, 4)
    rows = plain.bigram_rows(tokens, None, config['embedding']['bigram'])
    assert rows[0] == 101 and max(rows[1:]) < 101 and rows[1] == (tokens[0] * 37 + tokens[1] * 3) % 101
    other = list(tokens)
    other[9] = (other[9] + 1) % 30
    assert error(plain.logits(other, w, config)[[10]], plain.logits(tokens, w, config)[[10]]) > 0.3
    case = make_case('pair', config, w, backend, tmp_path / 'pair', 4)
    runner = case.runner(pages=12, requests=1)
    for cuts in ([24], [10, 14], [2] * 12, [], [1, 9, 1, 2, 11]):
        case.close(feed(runner, 'r', tokens, cuts), case.expected(tokens), f'cuts {cuts}')
    expected = case.expected(tokens[5:])
    case.close(feed(runner, 'r', tokens[5:], []), expected, 'another sequence in the same slot')


def test_pass_vectors_and_the_embedding_join_once(backend, tmp_path):
    """A loop whose stored vectors and embedding are large against what the layers add: one added twice, in the wrong
    pass, or on the stream of the pass before shows at once."""
    config = plain.make_config([plain.attention_layer(heads=2, kv_heads=1, dim=8, vdim=8, scale=0.5),
                                _beside(), plain.attention_layer(heads=1, kv_heads=1, dim=8, vdim=8, scale=0.5)],
                               vocab=30, width=16, embedding_scale=2.0, bigram=(19, 2, 3), loop=(1, 2, 3))
    w = plain.random_weights(config, 12, 1.0)
    w['loop.step'] = w['loop.step'] * 8.0
    tokens = tokens_for(config, 40, 3)
    base = plain.logits(tokens, w, config)
    moved = dict(w)
    moved['loop.step'] = w['loop.step'].flip(0)
    assert error(plain.logits(tokens, dict(w, **{'loop.step': w['loop.step'] * 0}), config), base) > 0.3
    # (the order of the vectors matters too: the passes between see other streams)
    assert error(plain.logits(tokens, moved, config), base) > 0.01
    case = make_case('passes', config, w, backend, tmp_path / 'passes', 8)
    runner = case.runner(pages=12)
    case.close(feed(runner, 'r', tokens, [40]), base, 'whole')
    case.close(feed(runner, 'r', tokens, [17, 2]), base, 'portions and single tokens')


def test_the_residual_stream_layer_by_layer(backend, tmp_path):
    """The stream after every layer run against the plain model's."""
    config, seed, page_size, spread = CONFIGS['mixed']
    case = make_case('layers', config, plain.random_weights(config, seed, spread), backend, tmp_path / 'layers', page_size)
    tokens = tokens_for(config, 30, 2)
    collected = []
    plain.forward(config, case.weights, tokens, collect=collected)
    import kernel_refs

    def settled(stream, joined):
        host = {}
        for name in ('mixed', 'ffn', 'gates', 'bias'):
            value = getattr(joined, name)
            host[name] = value
        copy = stream.clone()
        kernel_refs.residual_join(copy, joined, torch.ones(stream.shape[1], device=stream.device), 1e-6, torch.float32)
        return copy.cpu()
    seen = []
    case.model.observer = lambda position, stream, pending, scale: seen.append(settled(stream, pending))
    try:
        feed(case.runner(pages=16), 'r', tokens, [30])
    finally:
        case.model.observer = None
    assert len(seen) == len(collected)
    for run, (actual, expected) in enumerate(zip(seen, collected)):
        case.close(actual, expected, f'run {run}')


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
    # neighbours turn together: a quarter turn takes (u, v) to (-v, u), and the rest passes
    x = torch.tensor([[[1.0, 2.0, 3.0, 4.0, 5.0]]], dtype=F)
    turned = plain.rotate_neighbours(x, torch.tensor([1]), 4, (2 / torch.pi) ** 2)      # angles 1 and pi / 2
    c, s = torch.cos(torch.tensor(1.0, dtype=F)), torch.sin(torch.tensor(1.0, dtype=F))
    assert torch.allclose(turned[0, 0], torch.stack([c - 2 * s, 2 * c + s, torch.tensor(-4.0, dtype=F), torch.tensor(3.0, dtype=F),
                                                     torch.tensor(5.0, dtype=F)]))
    # one key of score s: e^s / (1 + e^s); two heads' slopes at distance 3; a hidden and a kept key
    q, k, v = torch.full((1, 1, 1), 2.0, dtype=F), torch.full((1, 1, 1), -1.0, dtype=F), torch.ones(1, 1, 1, dtype=F)
    one = plain.attend(q, k, v, torch.tensor([0]), torch.tensor([0]), 0.5, one=True)
    assert torch.isclose(one[0, 0], torch.sigmoid(torch.tensor(-1.0, dtype=F)))
    keys, values = torch.zeros(4, 1, 1, dtype=F), torch.tensor([1.0, 10.0, 100.0, 1000.0], dtype=F)[:, None, None]
    far = plain.attend(torch.zeros(1, 1, 1, dtype=F), keys, values, torch.tensor([3]), torch.arange(4), 1.0, window=1, keep_first=1,
                       slopes=[0.5])
    e = torch.exp(torch.tensor(-1.5, dtype=F))
    assert torch.isclose(far[0, 0], (1000.0 + e) / (1.0 + e))
    assert plain.head_slopes(2) == [2.0 ** -4, 2.0 ** -8]
    assert plain.layer_runs(dict(layers=[0] * 4, loop=dict(start=1, stop=3, times=2))) == \
        [(0, None), (1, 0), (2, None), (1, 1), (2, None), (3, None)]


def test_config_round_trip_and_refusals():
    from qil_amd.config import ConfigError, TinuzenConfig
    from qil_amd.registry import architecture_for
    config = CONFIGS['mixed'][0]
    typed = TinuzenConfig.from_dict(config)
    assert architecture_for(config).name == 'Tinuzen'
    assert TinuzenConfig.from_dict(json.loads(json.dumps(typed.to_dict()))) == typed
    assert typed.layer_runs() == plain.layer_runs(config)
    layers = config['layers']

    def with_mixer(index, **changes):
        return dict(layers[index], mixer=dict(layers[index]['mixer'], **changes))

    def with_half(index, half, **changes):
        return with_mixer(index, **{half: dict(layers[index]['mixer'][half], **changes)})

    for broken in (dict(config, window=4), dict(config, norm=dict(eps=1e-6, kind='layer')), dict(config, norm=dict(eps=0)),
                   dict(config, loop=dict(start=1, stop=5, times=2)), dict(config, loop=dict(start=2, stop=2, times=2)),
                   dict(config, loop=dict(start=0, stop=1, times=0)), dict(config, loop=dict(start=0, stop=1)),
                   dict(config, embedding=dict(scale=0.0)), dict(config, embedding=dict(scale=1.0, bigram=dict(buckets=0, mul_prev=1, mul_cur=1))),
                   dict(config, embedding=dict(scale=1.0, bigram=dict(buckets=5, mul_prev=1))),
                   dict(config, layers=[dict(layers[0], type='conv')]), dict(config, layers=[with_mixer(0, rot=None)]),
                   dict(config, layers=[with_mixer(0, heads=4)]), dict(config, layers=[with_mixer(0, mask=dict(size=0, keep_first=1))]),
                   dict(config, layers=[with_mixer(0, mask=dict(size=4, keep_first=-1))]),
                   dict(config, layers=[with_half(1, 'left', vdim=12)]),
                   dict(config, layers=[with_half(1, 'left', rot=dict(base=10.0, dims=26))]),
                   dict(config, layers=[with_half(1, 'right', groups=4)]), dict(config, layers=[with_half(1, 'right', norm_groups=7)]),
                   dict(config, layers=[with_half(1, 'right', inner=60)]),
                   dict(config, layers=[dict(layers[0], mlp=dict(kind='moe', ff=8))])):
        with pytest.raises(ConfigError):
            TinuzenConfig.from_dict(broken)


def test_the_bench_makes_valid_configurations():
    """The configurations that ``bench.py --phase designs --design tinuzen`` measures are ones the design accepts."""
    import bench
    from qil_amd.config import TinuzenConfig
    sizes = dict(width=512, ff=96, heads=4, dim=16, rot_dim=8)
    for kind in ('turns', 'loop', 'parallel', 'attention', 'left'):
        typed = TinuzenConfig.from_dict(bench.tinuzen_config(sizes, 6, 100, 32, kind))
        assert len(typed.layer_runs()) == 6


def test_random_weights_load(tmp_path, cpu_kernels):
    """A folder written from a configuration and a seed holds every tensor of the design, and loads and runs."""
    from qil_amd.weights import write_random_model
    config = CONFIGS['mixed'][0]
    folder = write_random_model(tmp_path / 'random', config, 4)
    from safetensors import safe_open
    with safe_open(str(folder / 'model.safetensors'), framework='pt') as f:
        stored = {name: tuple(f.get_slice(name).get_shape()) for name in f.keys()}
    assert stored == {name: tuple(t.shape) for name, t in plain.random_weights(config, 1).items()}
    model = load_model(folder, dtype=torch.float32, device='cpu')
    runner = ModelRunner(model, num_pages=8, page_size=8, max_requests=1)
    runner.admit('r')
    assert torch.isfinite(runner.step([StepEntry('r', (1, 2, 3), (2,))])).all()


@pytest.mark.gpu
def test_command_line(tmp_path):
    """``python -m qil_amd`` on a Tinuzen folder: greedy generation through the scheduler in portions of two tokens
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
    """``bin/trace_run`` on a Tinuzen folder: requests alone and whole, their last tokens one by one, portions down to
    two tokens, and up to four live requests in a pool of pages and state slots that is used again."""
    from test_engine_gpu import collect, replay, traces
    config, seed, _, spread = CONFIGS['mixed']
    weights = plain.random_weights(config, seed, spread)
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
