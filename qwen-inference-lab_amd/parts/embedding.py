"""Token embedding into the float32 stream, and the output head."""
from .base import Part, ParamSpec
from .. import ops


class Embedding(Part):
    """stream[n] = float32(table[token[n]]) * scale; no scaling (scale 1) in qil/model.py:126.  ``streams``: so many
    copies of it, for a model with several residual streams."""

    def __init__(self, vocab, width, scale=1.0, streams=1):
        super().__init__()
        ops.check_streams(streams)
        self.vocab, self.width, self.scale, self.streams = vocab, width, float(scale), streams

    def param_specs(self):
        return {'weight': ParamSpec((self.vocab, self.width))}

    def forward(self, token_ids):
        if self.streams > 1:
            return ops.embed(token_ids, self.p['weight'], self.scale, streams=self.streams)
        return ops.embed(token_ids, self.p['weight'], self.scale)

    def forward_step(self, ctx):
        """The float32 stream [N, width] of a step's rows.  What the model calls; an embedding that also needs
        the rows' positions (learned absolute positions, say) finds them in ``ctx`` (engine/batch.py)."""
        return self.forward(ctx.token_ids)


    def forward_step_kept(self, ctx):
        """``forward_step``'s stream and a copy of it that nobody changes (for models that add it again later)."""
        stream = self.forward_step(ctx)
        return stream, stream.clone()


class PairEmbedding(Embedding):
    """stream[n] = table[token] * scale + pairs[row]: a second table (``pairs.weight`` [buckets + 1, width]) is read by the
    token and the one before it in the sequence, row = (previous * mul_prev + token * mul_cur) mod buckets; a
    sequence's first token reads the last row.  The step function brings every row's previous token
    (``StepContext.previous_tokens``; across steps the cache manager keeps it per request)."""
    needs_previous_tokens = True

    def __init__(self, vocab, width, *, buckets, mul_prev, mul_cur, scale=1.0):
        super().__init__(vocab, width, scale)
        self.buckets, self.mul_prev, self.mul_cur = int(buckets), int(mul_prev), int(mul_cur)
        if self.buckets < 1 or self.mul_prev < 0 or self.mul_cur < 0:
            raise ValueError('buckets must be positive and the multipliers not negative')

    def param_specs(self):
        return {**super().param_specs(), 'pairs.weight': ParamSpec((self.buckets + 1, self.width))}

    def _embed(self, ctx, keep):
        return ops.embed_pairs(ctx.token_ids, ctx.previous_tokens, self.p['weight'], self.p['pairs.weight'], scale=self.scale,
                               buckets=self.buckets, mul_prev=self.mul_prev, mul_cur=self.mul_cur, keep=keep)

    def forward_step(self, ctx):
        return self._embed(ctx, False)

    def forward_step_kept(self, ctx):
        return self._embed(ctx, True)


class PassVectors(Part):
    """One stored vector per pass of a loop over layers (``weight`` [passes, width], float32 on the device): what is added
    to the stream before a pass's first layer."""

    def __init__(self, passes, width):
        super().__init__()
        self.passes, self.width = int(passes), int(width)

    def param_specs(self):
        return {'weight': ParamSpec((self.passes, self.width), 'vector')}

    def finalize(self):
        self.vectors = [self.p['weight'][t].contiguous() for t in range(self.passes)]


class LMHead(Part):
    """float32 logits = rows @ weight^T, no bias (qil/model.py:134).

    ``tied_to`` names an Embedding whose table is the head's matrix too
    (qil/model.py:96-98); the head then declares no tensor of its own.
    ``softcap`` c: the logits become c * tanh(logits / c), in float32.
    """

    def __init__(self, vocab, width, tied_to=None, softcap=None):
        super().__init__()
        self.vocab, self.width, self.tied_to = vocab, width, tied_to
        self.softcap = None if softcap is None else float(softcap)
        if self.softcap is not None and not self.softcap > 0:
            raise ValueError('softcap must be positive')

    def param_specs(self):
        return {} if self.tied_to is not None else {'weight': ParamSpec((self.vocab, self.width))}

    @property
    def weight(self):
        return self.tied_to.p['weight'] if self.tied_to is not None else self.p['weight']

    def forward(self, rows):
        import torch
        logits = ops.linear(rows, self.weight, None, out_dtype=torch.float32)
        return logits if self.softcap is None else ops.soft_cap(logits, self.softcap)
