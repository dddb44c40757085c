"""Typed configuration of the Tinuzen design, read from its own config.json keys.

    architecture   'Tinuzen'
    vocab, width   sizes of the embedding and of the head
    embedding      {'scale'}, optionally 'bigram': {'buckets', 'mul_prev', 'mul_cur'} (a second table by token pairs)
    layers         list; each entry: 'type' ('parallel' | 'attention'), 'mixer' (its sizes and constants) and 'mlp' (null, or
                   {'kind': 'dense', 'ff'})
      parallel     {'left': {'heads', 'kv_heads', 'dim', 'vdim', 'scale'} and optionally 'rot': {'base', 'dims'} (the
                   values are the keys: vdim == dim), 'right': {'heads', 'vdim', 'state', 'groups', 'conv',
                   'norm_groups'}, 'left_scale', 'right_scale'}
      attention    {'heads', 'kv_heads', 'dim', 'vdim', 'scale'}, optionally 'mask': {'size', 'keep_first'}
    loop           {'start', 'stop', 'times'}: layers start .. stop - 1 run 'times' times in a row with the same weights
                   (every pass with caches and states of its own), then the rest follow; absent: every layer once
    norm           {'eps'}

Every size and constant comes from here; a key the design does not know is refused, so that a model this engine would
run differently does not load silently.
"""
import copy
import math
from dataclasses import dataclass

from .base import ConfigError, check_positive_int, check_positive_finite, read_config_json

_TOP_KEYS = {'architecture', 'architectures', 'model_type', 'vocab', 'width', 'embedding', 'layers', 'loop', 'norm'}


def _keys(where, value, required, optional=()):
    if not isinstance(value, dict) or not set(required) <= set(value) <= set(required) | set(optional):
        raise ConfigError(f'{where} must have the keys {sorted(required)}' +
                          (f' and at most {sorted(optional)} besides' if optional else ''))


def _finite(name, value):
    if isinstance(value, bool) or not isinstance(value, (int, float)) or not math.isfinite(value):
        raise ConfigError(f'{name} must be a finite number, got {value!r}')


def _not_negative(name, value):
    if type(value) is not int or value < 0:
        raise ConfigError(f'{name} must be a non-negative integer, got {value!r}')


def _check_heads(where, m):
    for name in ('heads', 'kv_heads', 'dim', 'vdim'):
        check_positive_int(f'{where}.{name}', m[name])
    if m['heads'] % m['kv_heads']:
        raise ConfigError(f'{where}: heads must be a multiple of kv_heads')
    check_positive_finite(f'{where}.scale', m['scale'])


def _check_parallel(where, m):
    _keys(where, m, {'left', 'right', 'left_scale', 'right_scale'})
    _finite(f'{where}.left_scale', m['left_scale'])
    _finite(f'{where}.right_scale', m['right_scale'])
    left, right = m['left'], m['right']
    _keys(f'{where}.left', left, {'heads', 'kv_heads', 'dim', 'vdim', 'scale'}, {'rot'})
    _check_heads(f'{where}.left', left)
    if left['vdim'] != left['dim']:
        raise ConfigError(f'{where}.left: the values are the keys, vdim must be dim')
    if left.get('rot') is not None:
        _keys(f'{where}.left.rot', left['rot'], {'base', 'dims'})
        check_positive_finite(f'{where}.left.rot.base', left['rot']['base'])
        check_positive_int(f'{where}.left.rot.dims', left['rot']['dims'])
        if left['rot']['dims'] % 2 or left['rot']['dims'] > left['dim']:
            raise ConfigError(f'{where}.left.rot.dims must be even and at most dim')
    names = ('heads', 'vdim', 'state', 'groups', 'conv', 'norm_groups')
    _keys(f'{where}.right', right, set(names))
    for name in names:
        check_positive_int(f'{where}.right.{name}', right[name])
    if right['heads'] % right['groups']:
        raise ConfigError(f'{where}.right: heads must be a multiple of groups')
    if right['heads'] * right['vdim'] % right['norm_groups']:
        raise ConfigError(f'{where}.right: heads * vdim must be a multiple of norm_groups')


def _check_attention(where, m):
    _keys(where, m, {'heads', 'kv_heads', 'dim', 'vdim', 'scale'}, {'mask'})
    _check_heads(where, m)
    if m.get('mask') is not None:
        _keys(f'{where}.mask', m['mask'], {'size'}, {'keep_first'})
        check_positive_int(f'{where}.mask.size', m['mask']['size'])
        _not_negative(f'{where}.mask.keep_first', m['mask'].get('keep_first', 0))


_MIXERS = {'parallel': _check_parallel, 'attention': _check_attention}


def _check_layer(index, layer):
    where = f'layers[{index}]'
    _keys(where, layer, {'type', 'mixer', 'mlp'})
    if layer['type'] not in _MIXERS:
        raise ConfigError(f"{where}.type {layer['type']!r} is not one of {sorted(_MIXERS)}")
    _MIXERS[layer['type']](f'{where}.mixer', layer['mixer'])
    mlp = layer['mlp']
    if mlp is not None:
        _keys(f'{where}.mlp', mlp, {'kind', 'ff'})
        if mlp['kind'] != 'dense':
            raise ConfigError(f"{where}.mlp.kind must be 'dense'")
        check_positive_int(f'{where}.mlp.ff', mlp['ff'])


@dataclass(frozen=True)
class TinuzenConfig:
    vocab: int
    width: int
    embedding: dict               # {'scale', 'bigram'}, checked
    layers: tuple                 # of dicts as in config.json, checked
    norm_eps: float
    loop: dict | None = None      # {'start', 'stop', 'times'}

    architecture = 'Tinuzen'
    model_type = 'tinuzen'

    def __post_init__(self):
        check_positive_int('vocab', self.vocab)
        check_positive_int('width', self.width)
        _keys('embedding', self.embedding, {'scale'}, {'bigram'})
        check_positive_finite('embedding.scale', self.embedding['scale'])
        if self.embedding.get('bigram') is not None:
            _keys('embedding.bigram', self.embedding['bigram'], {'buckets', 'mul_prev', 'mul_cur'})
            check_positive_int('embedding.bigram.buckets', self.embedding['bigram']['buckets'])
            for name in ('mul_prev', 'mul_cur'):
                _not_negative(f'embedding.bigram.{name}', self.embedding['bigram'][name])
        if not self.layers:
            raise ConfigError('layers must not be empty')
        for index, layer in enumerate(self.layers):
            _check_layer(index, layer)
        check_positive_finite('norm.eps', self.norm_eps)
        if self.loop is not None:
            _keys('loop', self.loop, {'start', 'stop', 'times'})
            _not_negative('loop.start', self.loop['start'])
            _not_negative('loop.stop', self.loop['stop'])
            check_positive_int('loop.times', self.loop['times'])
            if not self.loop['start'] < self.loop['stop'] <= len(self.layers):
                raise ConfigError('loop: 0 <= start < stop <= number of layers')

    @property
    def vocab_size(self):
        return self.vocab

    @property
    def eos_ids(self):
        return frozenset()

    def layer_runs(self):
        """(layer index, number of the pass that begins before this run, or None) in the order the layers run."""
        if self.loop is None:
            return [(index, None) for index in range(len(self.layers))]
        start, stop = self.loop['start'], self.loop['stop']
        runs = [(index, None) for index in range(start)]
        for number in range(self.loop['times']):
            runs += [(index, number if index == start else None) for index in range(start, stop)]
        return runs + [(index, None) for index in range(stop, len(self.layers))]

    @classmethod
    def from_dict(cls, data):
        if data.get('architecture', (data.get('architectures') or [None])[0]) != cls.architecture:
            raise ConfigError(f"architecture must be {cls.architecture!r}")
        unknown = sorted(set(data) - _TOP_KEYS)
        if unknown:
            raise ConfigError(f'config.json has keys this design does not know: {unknown}')
        missing = [name for name in ('vocab', 'width', 'embedding', 'layers', 'norm') if name not in data]
        if missing:
            raise ConfigError(f'config.json lacks required keys: {missing}')
        if not isinstance(data['layers'], list):
            raise ConfigError('layers must be a list')
        _keys('norm', data['norm'], {'eps'})
        return cls(vocab=data['vocab'], width=data['width'], embedding=copy.deepcopy(data['embedding']),
                   layers=tuple(copy.deepcopy(data['layers'])), norm_eps=data['norm']['eps'],
                   loop=copy.deepcopy(data.get('loop')))

    @classmethod
    def read(cls, directory):
        return cls.from_dict(read_config_json(directory))

    def to_dict(self):
        out = dict(architecture=self.architecture, vocab=self.vocab, width=self.width, embedding=copy.deepcopy(self.embedding),
                   layers=copy.deepcopy(list(self.layers)), norm=dict(eps=self.norm_eps))
        if self.loop is not None:
            out['loop'] = dict(self.loop)
        return out
