"""Kebudra assembled from parts.

Token embedding times a constant, copied into several residual streams; layers of three kinds of mixer, chosen layer by layer
by the configuration: 'attention' (two softmax maps a head over the same values, the second taken off the first, a head
norm and a gate per head, no rotation; a layer may read an earlier layer's cached keys and values), 'latent_attention' (keys
and values expanded from a cached latent, queries through a latent of their own, neighbouring elements rotated, an output
gate element by element) and 'channel_delta' (a matrix memory corrected by the delta rule with a decay per key channel,
behind short convolutions); each followed by a routed feed-forward (experts without a gate branch, squared relu, weights by
the softmax over the chosen logits) or by nothing.  Every sub-layer reads a weighted sum of the streams through tanh(alpha x)
weight + bias and joins all streams, which are mixed at the same time; a last norm of that kind over the streams' sum and an
untied head.
"""
import torch

from ..config.kebudra import KebudraConfig
from ..parts import (TanhNorm, RotaryFrequencies, DifferenceAttention, LatentAttention, DeltaRule, RoutedExperts, StreamsBlock,
                     Embedding, LMHead, CausalLM, ScheduleEntry)
from ..registry import register_architecture


def _attention(width, m, eps, dtype, device):
    return DifferenceAttention(width=width, heads=m['heads'], kv_heads=m['kv_heads'], head_dim=m['dim'], value_dim=m['vdim'],
                               scale=m['scale'], diff=m['diff'], eps=eps, own_kv=m.get('kv_from') is None, dtype=dtype)


def _latent_attention(width, m, eps, dtype, device):
    return LatentAttention(width=width, heads=m['heads'], dim=m['dim'], rot_dim=m['rot_dim'], vdim=m['vdim'],
                           kv_rank=m['kv_rank'], q_rank=m['q_rank'], scale=m['scale'], eps=eps, sink=False, gate='element',
                           pairing='neighbours', position=RotaryFrequencies(m['rot']['dims'], m['rot']['base'], device=device),
                           dtype=dtype)


def _channel_delta(width, m, eps, dtype, device):
    # (the inner sizes of the low-rank products are the checkpoint's; random weights get a head's sizes)
    return DeltaRule(width=width, heads=m['heads'], kv_heads=m['kv_heads'], dim=m['dim'], vdim=m['vdim'], taps=m['conv'], eps=eps,
                     decay_rank=m['dim'], gate_rank=m['vdim'], dtype=dtype)


def _moe(width, f, dtype):
    return RoutedExperts(width=width, experts=f['router']['experts'], top=f['router']['top'], intermediate=f['expert']['ff'],
                         activation='relu_squared', renormalize=True, dtype=dtype)


MIXERS = {'attention': _attention, 'latent_attention': _latent_attention, 'channel_delta': _channel_delta}
FEED_FORWARDS = {'moe': _moe}

# checkpoint suffix -> the part's own tensor name
_MIXER_TENSORS = {
    'attention': {'q': 'q_proj.weight', 'k': 'k_proj.weight', 'v': 'v_proj.weight', 'lq1': 'lq1', 'lk1': 'lk1', 'lq2': 'lq2',
                  'lk2': 'lk2', 'g': 'g_proj.weight', 'o': 'o_proj.weight'},
    'latent_attention': {'dq': 'q_down.weight', 'dq.norm': 'q_norm.weight', 'uq': 'q_up.weight', 'dkv': 'kv_down.weight',
                         'dkv.norm': 'kv_norm.weight', 'uk': 'k_up.weight', 'uv': 'v_up.weight', 'g': 'g_proj.weight',
                         'o': 'o_proj.weight'},
    'channel_delta': {'q': 'q_proj.weight', 'q.conv': 'q_conv.weight', 'k': 'k_proj.weight', 'k.conv': 'k_conv.weight',
                      'v': 'v_proj.weight', 'v.conv': 'v_conv.weight', 'b': 'b_proj.weight', 'A_log': 'A_log',
                      'norm': 'out_norm.weight', 'a1': 'decay_down.weight', 'a2': 'decay_up.weight', 'dt_bias': 'dt_bias',
                      'g1': 'gate_down.weight', 'g2': 'gate_up.weight', 'o': 'o_proj.weight'},
}
_EXPERT_TENSORS = {'up': 'up_proj.weight', 'down': 'down_proj.weight'}
_STREAM_TENSORS = ('in', 'mix', 'out')


def build_kebudra(config, *, dtype=torch.bfloat16, device='cuda'):
    width, eps, streams = config.width, config.norm_eps, config.streams
    embedding = Embedding(config.vocab, width, scale=config.embedding_scale, streams=streams)
    blocks, names = [], {'embed': (embedding, 'weight')}

    def name_norm(name, norm):
        names.update({name: (norm, 'weight'), f'{name}.b': (norm, 'bias'), f'{name}.alpha': (norm, 'alpha')})

    for index, layer in enumerate(config.layers):
        mixer = MIXERS[layer['type']](width, layer['mixer'], eps, dtype, device)
        ffn = FEED_FORWARDS[layer['mlp']['kind']](width, layer['mlp'], dtype) if layer['mlp'] is not None else None
        block = StreamsBlock(mixer_norm=TanhNorm(width), mixer=mixer, ffn_norm=TanhNorm(width) if ffn is not None else None, ffn=ffn,
                             streams=streams, dtype=dtype)
        blocks.append(block)
        name_norm(f'l{index}.norm1', block.mixer_norm)
        names.update({f'l{index}.hc1.{name}': (block, f'mixer_{name}') for name in _STREAM_TENSORS})
        declared = mixer.param_specs()
        for suffix, local in _MIXER_TENSORS[layer['type']].items():
            if local in declared:                       # (a layer that reads another's keys and values has none)
                names[f'l{index}.mix.{suffix}'] = (mixer, local)
        if ffn is None:
            continue
        name_norm(f'l{index}.norm2', block.ffn_norm)
        names.update({f'l{index}.hc2.{name}': (block, f'ffn_{name}') for name in _STREAM_TENSORS})
        names[f'l{index}.mlp.router'] = (ffn, 'router.weight')
        for e in range(ffn.experts):
            for suffix, local in _EXPERT_TENSORS.items():
                names[f'l{index}.mlp.e{e}.{suffix}'] = (ffn, f'experts.{e}.{local}')
    final_norm, head = TanhNorm(width, streams=streams), LMHead(config.vocab, width)
    name_norm('final.norm', final_norm)
    names['head'] = (head, 'weight')
    # a layer with kv_from reads the cache that the named layer's run owns (schedule positions are layer indices)
    schedule = [ScheduleEntry(index, cache_of=layer['mixer'].get('kv_from')) for index, layer in enumerate(config.layers)]
    return CausalLM(config=config, embedding=embedding, blocks=blocks, schedule=schedule, final_norm=final_norm, head=head,
                    names=names, dtype=dtype, device=device)


register_architecture('Kebudra', model_type='kebudra', config_class=KebudraConfig, build=build_kebudra, replace=True)
