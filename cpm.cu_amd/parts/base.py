"""Interfaces of the parts a layer is put together from, and their registries.

A part owns its sizes and constants (given to its constructor), says which
checkpoint tensors it needs (``weight_specs``), takes them (``bind``) and runs
(``forward``).  No part knows which model it is in: a model file only chooses
parts by name and hands them numbers from its configuration.

Kinds of parts and what each must provide:

* ``Norm``:      forward(x, branch, branch_scale, ctx, rows=None) -> normed [n or R, H]
                 (adds ``branch_scale * branch`` into the float residual ``x`` first)
* ``PositionEncoding``: rotary_params() -> (inv_freq, magnitude) or None, and
                 apply(q, k, ctx) for encodings that are not a plain rotation, and/or
                 score_bias() -> per-head slopes for encodings that bias the scores by distance
* ``Mixer``:     cache_needs() and forward(h, ctx, cache, writes_cache) -> branch [n, H] or [P, n, H]
* ``FeedForward``: forward(h, ctx) -> branch [n, H] or [P, n, H]
* ``Block``:     forward(stream, ctx, cache, writes_cache): the arrangement of the above
                 around the residual stream

A branch may have a norm of its own before it joins the residual (``NormedBranch``; ``Norm.normalize``), or a
bias that its consumer adds (``BiasedBranch``).

Two optional protocols let neighbouring parts share a kernel without knowing each other: a norm may leave
its row factor to the product that follows (``forward_unscaled`` / ``takes_row_scale``), and a part may leave
its last product to the norm that follows (``DeferredBranch``: ``can_defer_last`` /
``takes_deferred_branch``).  A part that implements neither is handed plain tensors.

Branches may come back as float partial sums ``[P, n, H]`` of a split matrix
product; whoever adds them to the residual sums them.
"""
from __future__ import annotations

from dataclasses import dataclass, field
from typing import Callable, Dict, List, Mapping, Optional, Sequence, Tuple

import torch

from ..cache.paged import CacheNeeds, CacheView, SequenceCache


# ---------------------------------------------------------------------------
# weights
# ---------------------------------------------------------------------------
@dataclass(frozen=True)
class WeightSpec:
    """A checkpoint tensor a part needs.  ``init`` names the rule by which the random-weights writer draws it
    (weights.register_init_rule; built in: 'matrix' and 'table' N(0, std), 'norm' 1 + N(0, norm_std)).
    ``storage`` is the dtype it is written in and kept in by the loader ('bfloat16', 'float32' or 'int32')."""
    name: str
    shape: Tuple[int, ...]
    init: str = "matrix"
    storage: str = "bfloat16"


# ---------------------------------------------------------------------------
# run-time objects handed to parts
# ---------------------------------------------------------------------------
class Workspace:
    """Named scratch buffers that live as long as the engine: a part asks for
    ``get(name, shape, dtype)`` and receives the same memory at every step (it
    grows when a larger shape is asked for), so steps allocate nothing and a
    captured step replays on fixed addresses."""

    def __init__(self, device):
        self.device = torch.device(device)
        self._buf: Dict[str, torch.Tensor] = {}
        self.generation = 0           # counts the times a buffer moved (captured graphs hold the old address)
        self.sealed = False           # set by the engine once it is built: what is asked for later is noted
        self.grown: List[str] = []    # names of buffers made or enlarged after that

    def get(self, name: str, shape: Sequence[int], dtype: torch.dtype) -> torch.Tensor:
        n = 1
        for s in shape:
            n *= int(s)
        nbytes = n * torch.empty((), dtype=dtype).element_size()
        buf = self._buf.get(name)
        if buf is None or buf.numel() < nbytes:
            if buf is not None:
                self.generation += 1
            buf = torch.empty(max(nbytes, 256), dtype=torch.uint8, device=self.device)
            self._buf[name] = buf
            if self.sealed and name not in self.grown:
                self.grown.append(name)
        return buf[:nbytes].view(dtype).view(*shape)

    def bytes(self) -> int:
        return sum(b.numel() for b in self._buf.values())


@dataclass
class Runtime:
    """What an engine gives every part at bind time."""
    device: torch.device
    dtype: torch.dtype            # element type of activations, weights and cache: float32 or bfloat16
    workspace: Workspace
    max_seq_len: int              # longest sequence the engine holds
    tiled_weights: bool = True    # keep a second copy of linear weights in the decode product's layout
    page_size: int = 64           # tokens a cache page


class _NoTimer:
    def __enter__(self):
        return self

    def __exit__(self, *exc):
        return False


_NO_TIMER = _NoTimer()


@dataclass
class StepContext:
    """One step's batch as every part sees it: packed tokens of several sequences."""
    n_tokens: int
    n_seqs: int
    token_ids: torch.Tensor       # int32 [n]
    positions: torch.Tensor       # int32 [n] absolute position of each token in its sequence
    tok_slot: torch.Tensor        # int32 [n] cache slot of each token
    cu_q: torch.Tensor            # int32 [B+1] start of each sequence's tokens in the packed batch
    seq_slot: torch.Tensor        # int32 [B]
    seq_len: torch.Tensor         # int32 [B] tokens each sequence holds after this step
    q_lens: List[int]             # host copies
    kv_lens: List[int]
    max_pos: int                  # largest position in the step
    single_token: bool            # every sequence brings exactly one token
    ws: Workspace
    cache: Optional[SequenceCache]
    logit_rows: Optional[torch.Tensor] = None     # int32 [R]: packed token rows whose logits are wanted
    extras: Dict[str, object] = field(default_factory=dict)   # what kernels derive from the batch once a step
    perf: Optional[object] = None                 # label-keyed timers (utils.perf.PerfTimers) when switched on

    def timed(self, label: str):
        """A context manager that times the GPU work inside it under ``prefill_<label>`` or ``decode_<label>``
        while the timers are switched on, and does nothing otherwise.  The reference's labels make the same
        distinction (src/model/minicpm4/minicpm4_layer.cuh:46-83, minicpm4_attn.cuh:107-202)."""
        if self.perf is None or not self.perf.enabled:
            return _NO_TIMER
        return self.perf.gpu(("decode_" if self.single_token else "prefill_") + label)


class DeferredBranch:
    """A branch whose last linear layer has not run yet: branch = ``linear``(``a``).  A part that is asked to
    (``forward(..., defer_last=True)``) may hand this back instead of a tensor; a norm that knows a kernel which
    runs that product together with the residual add takes it as it is (``Norm.takes_deferred_branch``), for
    everybody else ``evaluate()`` runs the product as the part would have and gives the tensor."""

    def __init__(self, linear, a: torch.Tensor, ctx: "StepContext", tag: str):
        self.linear, self.a, self.ctx, self.tag = linear, a, ctx, tag
        self._value: Optional[torch.Tensor] = None

    def evaluate(self) -> torch.Tensor:
        if self._value is None:
            self._value = self.linear.forward(self.a, self.ctx, self.tag, out_dtype=torch.float32, partials=True)
        return self._value


class NormedBranch:
    """A branch that passes a norm of its own before it joins the residual: x += ``norm``(``branch``) (the
    arrangement with a norm before and after every sub-layer).  A norm that knows a kernel which does this
    together with its own work takes it as it is (``Norm.takes_normed_branch``); for everybody else
    ``evaluate()`` runs ``norm.normalize`` and gives the tensor to add."""

    def __init__(self, branch, norm: "Norm", ctx: "StepContext", tag: str):
        self.branch, self.norm, self.ctx, self.tag = branch, norm, ctx, tag
        self._value: Optional[torch.Tensor] = None

    def evaluate(self) -> torch.Tensor:
        if self._value is None:
            self._value = self.norm.normalize(branch_tensor(self.branch), self.ctx, self.tag)
        return self._value


class BiasedBranch:
    """A branch whose last product has a bias that is not added yet: branch = ``branch`` + ``bias`` (float32 [H]),
    ``branch`` a tensor [n, H] or float partial sums [P, n, H].  A consumer that adds the bias in a kernel of its
    own takes the two as they are (a parallel layer's gate kernel does; ``Norm.takes_biased_branch``); for
    everybody else ``evaluate()`` gives the float sum."""

    def __init__(self, branch: torch.Tensor, bias: torch.Tensor, ctx: "StepContext", tag: str):
        self.branch, self.bias, self.ctx, self.tag = branch, bias, ctx, tag
        self._value: Optional[torch.Tensor] = None

    def evaluate(self) -> torch.Tensor:
        if self._value is None:
            from .. import ops
            n, H = self.branch.shape[-2], self.branch.shape[-1]
            self._value = self.ctx.ws.get(self.tag + ".biased", (n, H), torch.float32)
            ops.bias_sum(self.branch, self.bias, self._value)
        return self._value


class ReplacingBranch:
    """What takes the residual's place: x <- ``branch`` + ``bias`` (tensor [n, H] or float partial sums [P, n, H];
    bias float32 [H] or None), left pending like every branch for the norm that follows (Norm.takes_replacing_branch);
    for everybody else ``evaluate()`` does it and leaves nothing to add (None)."""

    def __init__(self, x: torch.Tensor, branch: torch.Tensor, bias: Optional[torch.Tensor] = None):
        self.x, self.branch, self.bias = x, branch, bias

    def evaluate(self) -> None:
        from .. import ops
        if self.branch is not None:
            ops.norm_rows(self.x, None, None, branch=self.branch, branch_bias=self.bias, replace=True)
            self.branch = None


class StreamsBranch:
    """A sub-layer's result that joins a residual of several streams (hyper-connections): all streams at once,
    x_t <- sum_s ``mix``[s, t] x_s + ``out``[t] * ``scale`` * ``branch`` (mix float32 [S, S] indexed [from, to], out
    float32 [S]).  ``branch`` is a tensor [n, H], float partial sums [P, n, H] or a BiasedBranch.  It is left pending like
    every branch and added by the norm that follows (``Norm.forward_streams``)."""

    def __init__(self, branch, mix: torch.Tensor, out: torch.Tensor, scale: float = 1.0):
        self.branch, self.mix, self.out, self.scale = branch, mix, out, float(scale)
        if isinstance(branch, BiasedBranch) and self.scale != 1.0:
            self.branch = branch.evaluate()             # the kernel scales the branch before its bias joins

    def pieces(self):
        """(tensor, bias or None) of the branch."""
        if isinstance(self.branch, BiasedBranch):
            return self.branch.branch, self.branch.bias
        return branch_tensor(self.branch), None


def branch_tensor(branch):
    """The branch as a tensor (or None), whatever form it was handed over in."""
    if isinstance(branch, (DeferredBranch, NormedBranch, BiasedBranch, ReplacingBranch)):
        return branch.evaluate()
    return branch


def branch_for(norm: "Norm", branch):
    """The branch in a form that ``norm.forward`` accepts: as it is if the norm declares that it takes that
    form, else as a tensor."""
    if isinstance(branch, DeferredBranch) and not norm.takes_deferred_branch:
        return branch.evaluate()
    if isinstance(branch, NormedBranch) and not norm.takes_normed_branch:
        return branch.evaluate()
    if isinstance(branch, BiasedBranch) and not norm.takes_biased_branch:
        return branch.evaluate()
    if isinstance(branch, ReplacingBranch) and not norm.takes_replacing_branch:
        return branch.evaluate()
    return branch


class ResidualStream:
    """The float residual ``x`` [n, H] and a branch not yet added to it.  ``pending`` reads as a tensor;
    ``take_pending()`` gives it in the form it was left in, which may be a DeferredBranch."""

    def __init__(self, x: torch.Tensor, pending=None, pending_scale: float = 1.0):
        self.x = x
        self._pending = pending
        self.pending_scale = pending_scale

    @property
    def pending(self) -> Optional[torch.Tensor]:
        self._pending = branch_tensor(self._pending)
        return self._pending

    @pending.setter
    def pending(self, value):
        self._pending = value

    def take_pending(self):
        return self._pending


# ---------------------------------------------------------------------------
# the part interfaces
# ---------------------------------------------------------------------------
class Part:
    def parts(self) -> List["Part"]:
        return []

    def weight_specs(self) -> List[WeightSpec]:
        return []

    def bind(self, tensors: Mapping[str, torch.Tensor], rt: Runtime):
        """Take the tensors named by weight_specs (already on the device) and prepare for forward."""

    # False for a part whose forward reads device data on the host, allocates, or launches different work from
    # step to step (a router that counts tokens per expert, a recurrence that loops in Python over lengths):
    # such a forward cannot be recorded once and replayed.  An engine whose model holds one runs every step
    # eagerly, whatever its hip_graph option says.
    graph_capturable = True

    def reserve_workspace(self, ws: "Workspace", rt: Runtime, max_step_tokens: int, max_slots: int):
        """Called once when the engine is built, after bind: ask ``ws`` for the scratch whose size grows with the
        context (``rt.max_seq_len``) rather than with the step, so that it is part of the engine's memory figure
        and no later step has to grow it.  Scratch that depends on the step's tokens only is sized by the
        engine's rehearsal passes and needs nothing here."""

    # helpers over the tree
    def all_parts(self) -> List["Part"]:
        out: List["Part"] = [self]
        for p in self.parts():
            out.extend(p.all_parts())
        return out

    def all_weight_specs(self) -> List[WeightSpec]:
        out = list(self.weight_specs())
        for p in self.parts():
            out.extend(p.all_weight_specs())
        return out

    def bind_all(self, tensors: Mapping[str, torch.Tensor], rt: Runtime):
        self.bind(tensors, rt)
        for p in self.parts():
            p.bind_all(tensors, rt)


class Norm(Part):
    def forward(self, x: torch.Tensor, branch: Optional[torch.Tensor], branch_scale: float, ctx: StepContext,
                rows: Optional[torch.Tensor] = None, tag: str = "norm") -> torch.Tensor:
        raise NotImplementedError

    def forward_unscaled(self, x: torch.Tensor, branch: Optional[torch.Tensor], branch_scale: float,
                         ctx: StepContext, tag: str = "norm"):
        """For a norm whose result is (one number a row) * (something computed column by column), and a consumer
        that begins with a linear layer: add the branch as forward does and return (rows without the row
        factor, ops.RowScale that yields it), for the consumer's product to multiply its result by.  None if
        this norm, or this step, has no such form; the caller then uses forward.  Only called when the
        consumer's takes_row_scale() said yes."""
        return None

    # True if forward and forward_unscaled accept a DeferredBranch as ``branch``
    takes_deferred_branch = False
    # True if forward and forward_unscaled accept a NormedBranch as ``branch``
    takes_normed_branch = False
    # True if forward and forward_unscaled accept a BiasedBranch as ``branch``
    takes_biased_branch = False
    # True if forward and forward_unscaled accept a ReplacingBranch as ``branch``
    takes_replacing_branch = False

    # True if forward accepts ``out_dtype=`` (the element type of the normed rows; None: the engine's)
    takes_out_dtype = False

    def forward_convolved(self, x: torch.Tensor, branch, branch_scale: float, ctx: StepContext, convs, conv_state,
                          tags: Sequence[str]) -> Optional[List[torch.Tensor]]:
        """For a step in which every row is a sequence's only token, and a norm that knows a kernel for it: add the
        branch as forward does, norm, and run the short convolutions ``convs`` over the normed rows, h + conv(h) each,
        with the sequences' earlier rows from ``conv_state`` (ops.norm_rows).  None: the caller does it in steps."""
        return None

    def forward_streams(self, x: torch.Tensor, pending: Optional["StreamsBranch"], read: Optional[torch.Tensor],
                        ctx: StepContext, rows: Optional[torch.Tensor] = None, tag: str = "norm") -> torch.Tensor:
        """For a residual of several streams x float32 [S, n, H]: add the pending StreamsBranch into the streams
        (in place, unless ``rows`` selects rows), read u = sum_s read[s] x_s (read float32 [S]; None: the plain
        sum) and return this norm of u.  A norm that a model with such a residual uses defines it."""
        raise NotImplementedError(f"{type(self).__name__} does not read a residual of several streams")

    def normalize(self, t: torch.Tensor, ctx: StepContext, tag: str = "norm.plain") -> torch.Tensor:
        """The norm of the rows of ``t`` alone, float32 [n, H]: no residual, nothing added (what a branch that
        has a norm of its own passes through, NormedBranch)."""
        raise NotImplementedError


class PositionEncoding(Part):
    # which features a rotation pairs: 'halves' pairs feature i with i + r/2 of the r rotated features (rotate-half),
    # 'interleaved' pairs neighbours 2i and 2i + 1.  A mixer whose kernels know only one of them refuses the other.
    pairs = "halves"

    def rotary_params(self) -> Optional[Tuple[torch.Tensor, float]]:
        """(inv_freq float32 [head_dim/2], magnitude) if this encoding is a rotation of feature pairs (``pairs``) by
        position * inv_freq, which the fused kernel applies while it writes the cache; else None."""
        return None

    def apply(self, q: torch.Tensor, k: Optional[torch.Tensor], ctx: StepContext):
        """Encode positions into q [n, heads, hd] and k [n, kv_heads, hd] in place (used when
        rotary_params() is None and a subclass defines it)."""
        raise NotImplementedError

    def score_bias(self) -> Optional[torch.Tensor]:
        """float32 [heads] on the device, or None: an encoding that lowers the score of key j for the query at
        position p by slope[head] * (p - j) instead of (or beside) changing q and k.  The attention kernels
        take it as it is; nothing about positions is then stored in the cache."""
        return None

    def rewrites_vectors(self) -> bool:
        """Whether ``apply`` is this encoding's own (an encoding that only biases scores leaves it out)."""
        return type(self).apply is not PositionEncoding.apply


class Mixer(Part):
    def cache_needs(self) -> CacheNeeds:
        return CacheNeeds()

    def forward(self, h: torch.Tensor, ctx: StepContext, cache: Optional[CacheView], writes_cache: bool = True
                ) -> torch.Tensor:
        raise NotImplementedError

    def takes_row_scale(self, n: int, ctx: StepContext, cache: Optional[CacheView], writes_cache: bool) -> bool:
        """True if forward, for this step of n tokens, accepts ``row_scale=`` (Norm.forward_unscaled) beside h.
        A subclass that overrides forward of a mixer that says yes takes the argument too, or says no here."""
        return False

    # True (set in the class that defines ``forward``) if that forward accepts ``defer_last=True`` and may then
    # return a DeferredBranch
    can_defer_last = False


class FeedForward(Part):
    def forward(self, h: torch.Tensor, ctx: StepContext) -> torch.Tensor:
        raise NotImplementedError

    def takes_row_scale(self, n: int, ctx: StepContext) -> bool:
        """True if forward, for this step of n tokens, accepts ``row_scale=`` (Norm.forward_unscaled) beside h."""
        return False

    # True if forward accepts ``defer_last=True`` and may then return a DeferredBranch
    can_defer_last = False
    # True (set in the class that defines ``forward``) if forward accepts ``join=`` (ops.Join): its result, the other
    # result of a parallel layer and the residual are then summed in its last kernel, and it returns None.  ``joins``
    # says whether it would for a given other result
    can_join = False

    def joins(self, other: Optional[torch.Tensor]) -> bool:
        return self.can_join


def forward_declares(part: Part, flag: str) -> bool:
    """Whether the class that defines ``part.forward`` sets the class attribute ``flag`` itself.  Optional
    protocols that add a keyword to ``forward`` (``can_defer_last``) are declared beside the ``forward`` that
    implements them: a subclass that overrides ``forward`` and says nothing is not handed the keyword."""
    for cls in type(part).__mro__:
        if "forward" in cls.__dict__:
            return bool(cls.__dict__.get(flag, False))
    return False


class Block(Part):
    mixer: Mixer

    def cache_needs(self) -> CacheNeeds:
        """What a run of this block keeps per sequence: its mixer's needs, and the block's own."""
        return self.mixer.cache_needs()

    def forward(self, stream: ResidualStream, ctx: StepContext, cache: Optional[CacheView], writes_cache: bool = True):
        raise NotImplementedError


# ---------------------------------------------------------------------------
# registries: kind name -> constructor
# ---------------------------------------------------------------------------
class Registry:
    def __init__(self, what: str):
        self.what = what
        self._items: Dict[str, Callable] = {}

    def register(self, name: str, ctor: Optional[Callable] = None):
        def deco(c):
            if name in self._items and self._items[name] is not c:
                raise ValueError(f"{self.what} '{name}' is already registered")
            self._items[name] = c
            return c
        return deco if ctor is None else deco(ctor)

    def unregister(self, name: str):
        self._items.pop(name, None)

    def get(self, name: str) -> Callable:
        try:
            return self._items[name]
        except KeyError:
            raise KeyError(f"unknown {self.what} '{name}' (registered: {sorted(self._items)})") from None

    def build(self, kind: str, /, **params):
        return self.get(kind)(**params)

    def names(self):
        return sorted(self._items)


NORMS = Registry("norm")
POSITION_ENCODINGS = Registry("position encoding")
MIXERS = Registry("mixer")
FEED_FORWARDS = Registry("feed-forward")
BLOCKS = Registry("block")


@dataclass(frozen=True)
class PartSpec:
    """A part chosen by name with its parameters: what a model file writes per layer."""
    kind: str
    params: Tuple[Tuple[str, object], ...] = ()

    @staticmethod
    def of(kind: str, **params) -> "PartSpec":
        return PartSpec(kind, tuple(sorted(params.items())))

    def build(self, registry: Registry, **extra):
        return registry.build(self.kind, **dict(self.params), **extra)
