"""Typed configuration of the Kebudra design, read from its own config.json keys.

    architecture   'Kebudra'
    vocab, width   sizes of the embedding and of the head
    streams        residual streams side by side
    embedding      {'scale'}
    layers         list; each entry: 'type' ('attention' | 'latent_attention' | 'channel_delta'), 'mixer' (its sizes and
                   constants) and 'mlp' (null, or {'kind': 'moe', 'expert': {'ff'}, 'router': {'experts', 'top'}})
      attention         {'heads', 'kv_heads', 'dim', 'vdim', 'scale', 'diff'}, optionally 'kv_from' (an earlier attention layer,
                        with keys and values of its own, whose cache this one reads)
      latent_attention  {'heads', 'dim', 'rot_dim', 'vdim', 'kv_rank', 'q_rank', 'scale', 'rot': {'base', 'dims'}}
      channel_delta     {'heads', 'kv_heads', 'dim', 'vdim', 'conv'}
    norm           {'eps'}

Every size and constant comes from here or from a tensor's shape; a key the design does not know is refused, so that a
model this engine would run differently does not load silently.
"""
import copy
import math
from dataclasses import dataclass

from .base import ConfigError, check_positive_int, check_positive_finite, read_config_json

_TOP_KEYS = {'architecture', 'architectures', 'model_type', 'vocab', 'width', 'streams', 'embedding', 'layers', 'norm'}


def _keys(where, value, required, optional=()):
    if not isinstance(value, dict) or not set(required) <= set(value) <= set(required) | set(optional):
        raise ConfigError(f'{where} must have the keys {sorted(required)}' +
                          (f' and at most {sorted(optional)} besides' if optional else ''))


def _finite(name, value):
    if isinstance(value, bool) or not isinstance(value, (int, float)) or not math.isfinite(value):
        raise ConfigError(f'{name} must be a finite number, got {value!r}')


def _check_groups(where, m):
    if m['heads'] % m['kv_heads']:
        raise ConfigError(f'{where}: heads must be a multiple of kv_heads')


def _check_attention(where, m):
    sizes = ('heads', 'kv_heads', 'dim', 'vdim')
    _keys(where, m, {*sizes, 'scale', 'diff'}, {'kv_from'})
    for name in sizes:
        check_positive_int(f'{where}.{name}', m[name])
    _check_groups(where, m)
    check_positive_finite(f'{where}.scale', m['scale'])
    _finite(f'{where}.diff', m['diff'])


def _check_latent_attention(where, m):
    sizes = ('heads', 'dim', 'rot_dim', 'vdim', 'kv_rank', 'q_rank')
    _keys(where, m, {*sizes, 'scale', 'rot'})
    for name in sizes:
        check_positive_int(f'{where}.{name}', m[name])
    check_positive_finite(f'{where}.scale', m['scale'])
    _keys(f'{where}.rot', m['rot'], {'base', 'dims'})
    check_positive_finite(f'{where}.rot.base', m['rot']['base'])
    if m['rot_dim'] % 2 or m['rot']['dims'] != m['rot_dim']:
        raise ConfigError(f'{where}: rot_dim must be even, and rot.dims must be rot_dim')


def _check_channel_delta(where, m):
    sizes = ('heads', 'kv_heads', 'dim', 'vdim', 'conv')
    _keys(where, m, set(sizes))
    for name in sizes:
        check_positive_int(f'{where}.{name}', m[name])
    _check_groups(where, m)


_MIXERS = {'attention': _check_attention, 'latent_attention': _check_latent_attention, 'channel_delta': _check_channel_delta}


def _check_layer(index, layers):
    where, layer = f'layers[{index}]', layers[index]
    _keys(where, layer, {'type', 'mixer', 'mlp'})
    if layer['type'] not in _MIXERS:
        raise ConfigError(f"{where}.type {layer['type']!r} is not one of {sorted(_MIXERS)}")
    m = layer['mixer']
    _MIXERS[layer['type']](f'{where}.mixer', m)
    source = m.get('kv_from')
    if source is not None:
        if type(source) is not int or not 0 <= source < index or layers[source]['type'] != 'attention' or \
                layers[source]['mixer'].get('kv_from') is not None:
            raise ConfigError(f'{where}.mixer.kv_from must name an earlier attention layer that has keys and values of its own')
        if any(layers[source]['mixer'][name] != m[name] for name in ('heads', 'kv_heads', 'dim', 'vdim')):
            raise ConfigError(f'{where}.mixer: the layer named by kv_from has other heads')
    mlp = layer['mlp']
    if mlp is not None:
        _keys(f'{where}.mlp', mlp, {'kind', 'expert', 'router'})
        if mlp['kind'] != 'moe':
            raise ConfigError(f"{where}.mlp.kind must be 'moe'")
        _keys(f'{where}.mlp.expert', mlp['expert'], {'ff'})
        check_positive_int(f'{where}.mlp.expert.ff', mlp['expert']['ff'])
        _keys(f'{where}.mlp.router', mlp['router'], {'experts', 'top'})
        for name in ('experts', 'top'):
            check_positive_int(f'{where}.mlp.router.{name}', mlp['router'][name])
        if mlp['router']['top'] > mlp['router']['experts']:
            raise ConfigError(f'{where}.mlp.router: top must be at most experts')


@dataclass(frozen=True)
class KebudraConfig:
    vocab: int
    width: int
    streams: int
    embedding_scale: float
    layers: tuple                 # of dicts as in config.json, checked
    norm_eps: float

    architecture = 'Kebudra'
    model_type = 'kebudra'

    def __post_init__(self):
        for name in ('vocab', 'width', 'streams'):
            check_positive_int(name, getattr(self, name))
        check_positive_finite('embedding.scale', self.embedding_scale)
        if not self.layers:
            raise ConfigError('layers must not be empty')
        for index in range(len(self.layers)):
            _check_layer(index, self.layers)
        check_positive_finite('norm.eps', self.norm_eps)

    @property
    def vocab_size(self):
        return self.vocab

    @property
    def eos_ids(self):
        return frozenset()

    @classmethod
    def from_dict(cls, data):
        if data.get('architecture', (data.get('architectures') or [None])[0]) != cls.architecture:
            raise ConfigError(f"architecture must be {cls.architecture!r}")
        unknown = sorted(set(data) - _TOP_KEYS)
        if unknown:
            raise ConfigError(f'config.json has keys this design does not know: {unknown}')
        missing = [name for name in ('vocab', 'width', 'streams', 'embedding', 'layers', 'norm') if name not in data]
        if missing:
            raise ConfigError(f'config.json lacks required keys: {missing}')
        if not isinstance(data['layers'], list):
            raise ConfigError('layers must be a list')
        _keys('embedding', data['embedding'], {'scale'})
        _keys('norm', data['norm'], {'eps'})
        return cls(vocab=data['vocab'], width=data['width'], streams=data['streams'], embedding_scale=data['embedding']['scale'],
                   layers=tuple(copy.deepcopy(data['layers'])), norm_eps=data['norm']['eps'])

    @classmethod
    def read(cls, directory):
        return cls.from_dict(read_config_json(directory))

    def to_dict(self):
        return dict(architecture=self.architecture, vocab=self.vocab, width=self.width, streams=self.streams,
                    embedding=dict(scale=self.embedding_scale), layers=copy.deepcopy(list(self.layers)),
                    norm=dict(eps=self.norm_eps))
