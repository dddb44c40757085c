"""What every part is: a holder of declared tensors with a forward of its kind.

A part never learns which model it sits in.  It receives its sizes and constants
as constructor arguments, declares its tensors in ``param_specs()``, gets them
through ``set_param`` (from a checkpoint or a random generator), may re-lay them
out once in ``finalize()``, and computes with the kernels of ``qil_amd.ops``.

Tensor kinds (``ParamSpec.kind``):
  matrix  -> stored in the model's dtype (bfloat16 or float32)
  vector  -> norm scales and biases, and small matrices whose products are float32 in every model (a router);
             always float32 on the device, which holds a bfloat16 or a float32 checkpoint value exactly
  table   -> integer tables; int32
"""
from dataclasses import dataclass


@dataclass(frozen=True)
class ParamSpec:
    shape: tuple
    kind: str = 'matrix'          # matrix | vector | table
    init: str = 'normal'          # normal | one_plus_normal | zeros
    free: tuple = ()              # axes whose size the checkpoint decides (no configuration key gives it); the size
                                  # in ``shape`` is what random weights get, and the part checks in ``finalize`` that
                                  # the sizes it was given fit each other

    def fits(self, shape):
        shape = tuple(shape)
        return len(shape) == len(self.shape) and all(a == b or axis in self.free
                                                     for axis, (a, b) in enumerate(zip(shape, self.shape)))


@dataclass(frozen=True)
class KVNeed:
    """Per-token keys and values in pages.  ``window`` None keeps every key; ``keep_first``: behind a window, the first
    so many tokens are kept for good."""
    kv_heads: int
    head_dim: int
    window: int | None = None
    keep_first: int = 0


@dataclass(frozen=True)
class PagedNeed:
    """Per-token data in pages, in tensors of the mixer's own: ``tensors`` is a tuple of (name, shape of one
    token's entry, 'model' or 'float32').  The cache manager keeps ``[pages, page_size, *shape]`` per name and entry
    and gives the mixer a ``PagedView`` with the step's block tables and the new tokens' slots (slot = page *
    page_size + position % page_size, an index into the first two axes taken together).  ``window`` None keeps every
    token; needs that are equal share a page pool and block tables."""
    tensors: tuple
    window: int | None = None


@dataclass(frozen=True)
class StateNeed:
    """Fixed-size per-request state, one slot per live request.

    dtype: 'float32' or 'model'.  The slot of a request that starts (start == 0)
    must be treated as empty by the mixer; the cache manager does not clear it.
    """
    shape: tuple
    dtype: str = 'float32'


@dataclass(frozen=True)
class CompoundNeed:
    """Several needs of one schedule entry: ``needs`` is a tuple of KVNeed | PagedNeed | StateNeed (a block whose
    mixer keeps pages while another of its parts keeps a fixed-size state).  Each need joins the group of its kind as
    if it stood alone; the entry's view is the tuple of their views, in the same order."""
    needs: tuple


class Part:
    def __init__(self):
        self.p = {}

    def param_specs(self):
        """dict local name -> ParamSpec."""
        return {}

    def set_param(self, name, tensor):
        spec = self.param_specs()[name]
        if not spec.fits(tensor.shape):
            raise ValueError(f'{type(self).__name__}.{name}: shape {tuple(tensor.shape)} != {tuple(spec.shape)}')
        self.p[name] = tensor

    def finalize(self):
        """Called once after every declared tensor is set."""

    def after_finalize(self):
        """Called once after ``finalize`` of every part of the model (a block may lay its parts' tensors together)."""

    def input_matrices(self):
        """Names in ``p`` of the matrices whose products with the part's input the part asks ``ops.linear`` (or
        ``ops.gated_linear``) for, without a bias: a block whose parts read the same input may lay them one behind
        another (``ops.SharedInput``).  Empty: the part's input must be a tensor."""
        return ()

    def matrix(self, name):
        return self.p[name]

    def place_matrix(self, name, tensor):
        """``tensor`` holds what ``p[name]`` holds, in memory that other parts' matrices share; use it from now on."""
        self.p[name] = tensor

    def parameter_bytes(self):
        return sum(t.numel() * t.element_size() for t in self.p.values())


class Norm(Part):
    """[N, width] float32 stream -> normalised [N, width] in ``out_dtype``.

    ``forward(stream, delta, out_dtype)``: if ``delta`` is given it is first added
    into ``stream`` in place (float32 sum), then the sum is normalised.
    ``forward_rows(stream, delta, rows, out_dtype)``: the same for the selected
    rows only, leaving ``stream`` untouched.
    A block whose residual sums are scaled (x + m * sublayer(x)) passes ``delta_scale=m`` to both; blocks that do not
    scale never pass it.
    """
    def forward(self, stream, delta, out_dtype):
        raise NotImplementedError

    def forward_lazy(self, stream, out_dtype, added):
        """The norm of a stream that ``added`` (an ``ops.Added``) has just completed, as an object that a consumer's
        kernel computes while it stages its operand (``ops.Normed``), or None where that does not apply.  Asked for
        only by blocks whose consumer says it takes such an object (``takes_lazy_norm``)."""
        return None

    def forward_rows(self, stream, delta, rows, out_dtype):
        raise NotImplementedError


    def forward_streams(self, stream, pending, out_dtype, *, streams, read):
        """Several residual streams [N, streams * width]: what is pending (``ops.StreamUpdate`` or None) joins them in place,
        and the norm of u = sum_s read[s] x_s comes back.  This form makes u first; a norm with a kernel for it overrides it."""
        from .. import ops
        import torch
        joined = ops.stream_join(stream, pending, streams=streams, read=read, out_dtype=torch.float32)
        return self.forward(joined, None, out_dtype)


class PositionEncoding(Part):
    """Something the mixer applies to queries and keys by absolute position.

    ``rotation()`` returns None (nothing to apply) or a ``Rotation`` record that
    the fused query/key kernel understands.
    """
    def rotation(self):
        return None


@dataclass(frozen=True)
class Rotation:
    cos: object            # float32 [positions, rot_dim/2]; None with ``frequencies``
    sin: object
    rot_dim: int           # leading rot_dim elements of each head are rotated, pairs (i, i + rot_dim/2)
    frequencies: object = None   # float32 [rot_dim/2]: the kernels make the angle position * frequency themselves


class Mixer(Part):
    """Token mixer: [N, width] -> [N, width] over the step's batch and the cache.

    The result is a tensor of the model's type or ``ops.Partials`` (float32 partial sums that the
    next norm adds).
    ``cache_need()`` says what it keeps between steps (KVNeed, StateNeed or None);
    ``forward(h, ctx, cache)`` gets the step context (engine/batch.py) and the
    cache view of its schedule entry (cache/manager.py: KVView or StateView).
    Its result must not depend on how a request's tokens were cut into steps.
    """
    # True if forward reads only device tensors of the step context (and shapes), never its host lists: then a step
    # may be captured into a HIP graph and replayed with other contents.  A step's forward runs once per step (a new
    # graph warms up on inert rows that write to the cache's spare page and spare state slot), so a mixer that adds
    # into its state may be captured as well.  Captured decode batches are filled up with such inert rows (one
    # token at position 0, ``seq_starts`` 0): a mixer must cope with them as with any request that begins.
    graph_safe = False
    # True if forward takes ``h`` as an ``ops.Normed`` (a norm not computed yet) as well as a tensor.
    takes_lazy_norm = False

    def cache_need(self):
        return None

    def forward(self, h, ctx, cache):
        raise NotImplementedError


class FeedForward(Part):
    """Per-token map [N, width] -> [N, width] (tensor of the model's type or ``ops.Partials``).

    A part that sets ``adds_to_stream`` is called as ``forward(h, add_to=stream)`` and may add its result into
    the float32 residual stream itself; it then returns the ``ops.Added`` that its last product gave."""
    adds_to_stream = False

    def forward(self, h):
        raise NotImplementedError


class Block(Part):
    """Arrangement of parts around the residual stream.

    ``forward(stream, pending, ctx, cache)`` -> pending: ``stream`` is the float32
    residual stream [N, width], changed in place; ``pending`` is a sub-layer
    output not yet added to it (or None), which lets the add fuse into the next
    norm.  The block returns its own last sub-layer output as the new pending; an
    ``ops.Added`` says that the output is in the stream already.
    """
    mixer = None
    # True if forward takes an ``ops.Joined`` as pending: then a schedule entry of the block may add the embedding's
    # output or a pass's vector to the stream before the run.
    takes_pass_start = False

    def parts(self):
        """dict local prefix -> Part (for naming tensors)."""
        return {}

    def cache_need(self):
        """What a run of the block keeps between steps: its mixer's need, unless the block has parts of its own
        that keep something too (then a ``CompoundNeed``, and ``forward`` gets the tuple of views)."""
        return self.mixer.cache_need() if self.mixer is not None else None

    def forward(self, stream, pending, ctx, cache):
        raise NotImplementedError
