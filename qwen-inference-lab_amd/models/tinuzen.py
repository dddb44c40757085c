"""Tinuzen assembled from parts.

Token embedding times a constant plus a second table read by the pair (previous token, token); layers of two kinds,
chosen layer by layer by the configuration: 'parallel' (two mixers on the same input whose results are added with a
factor each: attention whose values are its keys before the rotation of neighbouring elements, with one added to the
softmax's denominator and an output gate; and a state-space recurrence with a matrix state and one decay a head and
token behind a short convolution) and 'attention' (grouped-query attention without a rotation, queries and keys normed over
the whole projection, a bias by distance with a slope per head, a sliding window behind first keys that stay visible).
Mixer and feed-forward (gated, relu) stand side by side on one RMS norm, each multiplied per channel by a sigmoid gate
made from the same input.  A span of layers may run several times with the same weights, every pass with caches and
states of its own; before a pass a stored vector is added to the stream, and before each pass but the first the
embedding's output too.  Final RMS norm and an untied head.
"""
import torch

from ..config.tinuzen import TinuzenConfig
from ..parts import (RMSNorm, RotaryFrequencies, Attention, DualStateSpace, ParallelMixers, GatedMLP, ParallelBlock, Embedding,
                     PairEmbedding, PassVectors, LMHead, CausalLM, ScheduleEntry)
from ..registry import register_architecture


def head_slopes(heads):
    """The bias by distance: 2^(-8 (h + 1) / heads) for head h."""
    return [2.0 ** (-8.0 * (h + 1) / heads) for h in range(heads)]


def _parallel(width, m, eps, dtype, device):
    a, r = m['left'], m['right']
    rot = a.get('rot')
    position = RotaryFrequencies(rot['dims'], rot['base'], device=device) if rot is not None else None
    left = Attention(width=width, heads=a['heads'], kv_heads=a['kv_heads'], head_dim=a['dim'], value_dim=a['vdim'], bias=False,
                     qk_norm_eps=None, scale=a['scale'], position=position, pairing='neighbours', values_are_keys=True,
                     sink_value=0.0, gate=True, dtype=dtype)
    right = DualStateSpace(width=width, heads=r['heads'], vdim=r['vdim'], state=r['state'], groups=r['groups'], taps=r['conv'],
                           norm_groups=r['norm_groups'], eps=eps, dtype=dtype)
    return ParallelMixers(left=left, right=right, left_scale=m['left_scale'], right_scale=m['right_scale'], summed=False)


def _attention(width, m, eps, dtype, device):
    mask = m.get('mask') or {'size': None}
    return Attention(width=width, heads=m['heads'], kv_heads=m['kv_heads'], head_dim=m['dim'], value_dim=m['vdim'], bias=False,
                     qk_norm_eps=eps, qk_norm='row', scale=m['scale'], position=None, window=mask['size'],
                     keep_first=mask.get('keep_first', 0), distance_slopes=head_slopes(m['heads']), dtype=dtype)


def _dense(width, f, dtype):
    return GatedMLP(width=width, intermediate=f['ff'], activation='relu', dtype=dtype)


MIXERS = {'parallel': _parallel, 'attention': _attention}
FEED_FORWARDS = {'dense': _dense}

# checkpoint suffix -> the part's own tensor name
_MIXER_TENSORS = {
    'parallel': {'left.q': 'left.q_proj.weight', 'left.k': 'left.k_proj.weight', 'left.g': 'left.g_proj.weight',
                 'left.o': 'left.o_proj.weight', 'right.in': 'right.in_proj.weight', 'right.conv': 'right.conv.weight',
                 'right.conv.b': 'right.conv.bias', 'right.dt_bias': 'right.dt_bias', 'right.A_log': 'right.A_log',
                 'right.D': 'right.D', 'right.norm': 'right.norm.weight', 'right.o': 'right.o_proj.weight'},
    'attention': {'q': 'q_proj.weight', 'k': 'k_proj.weight', 'v': 'v_proj.weight', 'q.norm': 'q_norm.weight',
                  'k.norm': 'k_norm.weight', 'o': 'o_proj.weight'},
}
_MLP_TENSORS = {'gate': 'gate_proj.weight', 'up': 'up_proj.weight', 'down': 'down_proj.weight'}


def build_tinuzen(config, *, dtype=torch.bfloat16, device='cuda'):
    width, eps, bigram = config.width, config.norm_eps, config.embedding.get('bigram')
    if bigram is not None:
        embedding = PairEmbedding(config.vocab, width, scale=config.embedding['scale'], buckets=bigram['buckets'],
                                  mul_prev=bigram['mul_prev'], mul_cur=bigram['mul_cur'])
    else:
        embedding = Embedding(config.vocab, width, scale=config.embedding['scale'])
    names = {'embed': (embedding, 'weight')}
    if bigram is not None:
        names['bigram'] = (embedding, 'pairs.weight')
    blocks = []
    for index, layer in enumerate(config.layers):
        mixer = MIXERS[layer['type']](width, layer['mixer'], eps, dtype, device)
        ffn = FEED_FORWARDS[layer['mlp']['kind']](width, layer['mlp'], dtype) if layer['mlp'] is not None else None
        block = ParallelBlock(norm=RMSNorm(width, eps), mixer=mixer, ffn=ffn, gated=True, width=width, dtype=dtype)
        blocks.append(block)
        names[f'l{index}.norm1'] = (block.norm, 'weight')
        names[f'l{index}.rg1'] = (block, 'mixer_gate.weight')
        names[f'l{index}.rg1.b'] = (block, 'mixer_gate.bias')
        for suffix, local in _MIXER_TENSORS[layer['type']].items():
            names[f'l{index}.mix.{suffix}'] = (mixer, local)
        if ffn is not None:
            names[f'l{index}.rg2'] = (block, 'ffn_gate.weight')
            names[f'l{index}.rg2.b'] = (block, 'ffn_gate.bias')
            for suffix, local in _MLP_TENSORS.items():
                names[f'l{index}.mlp.{suffix}'] = (ffn, local)
    vectors = None
    if config.loop is not None:
        vectors = PassVectors(config.loop['times'], width)
        names['loop.step'] = (vectors, 'weight')
    final_norm, head = RMSNorm(width, eps), LMHead(config.vocab, width)
    names['final.norm'] = (final_norm, 'weight')
    names['head'] = (head, 'weight')
    # a looped layer appears once per pass; every run owns a cache (or state) of its mixer's need
    schedule = [ScheduleEntry(index, add_embedding=begins is not None and begins > 0, add_vector=begins)
                for index, begins in config.layer_runs()]
    return CausalLM(config=config, embedding=embedding, blocks=blocks, schedule=schedule, final_norm=final_norm, head=head,
                    names=names, dtype=dtype, device=device, pass_vectors=vectors)


register_architecture('Tinuzen', model_type='tinuzen', config_class=TinuzenConfig, build=build_tinuzen, replace=True)
