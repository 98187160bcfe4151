"""What a mixer asks of the cache, and what a layer is handed at run time."""
from __future__ import annotations

from dataclasses import dataclass, replace
from typing import Optional, Tuple

import torch


@dataclass(frozen=True)
class PagedNeed:
    """Memory per token, in pages: the mixer names the tensors it keeps and the shape of one block of
    each. ``tensors`` is a tuple of (name, shape of one block, dtype or None for the model's dtype), a -1
    in a shape standing for the engine's block size; the
    engine allocates ``[blocks, *shape]`` for each and hands them over in ``LayerCache.tensors`` by name;
    token slot s of the step (``batch.slots[group]``) is slot ``s % block_size`` of block ``s // block_size``,
    wherever in its block's shape the mixer puts it. ``window`` W > 0: only the last W tokens are read, the
    blocks behind them go back to the pool, but for those that hold the request's first ``keep`` tokens.
    ``chunked``: read are the tokens of the same chunk of W, counted from position 0; the chunks behind go back."""
    tensors: Tuple[Tuple[str, Tuple[int, ...], Optional[torch.dtype]], ...]
    window: int = 0
    keep: int = 0
    chunked: bool = False

    def block_tensors(self, block_size: int):
        return tuple((name, tuple(block_size if n == -1 else n for n in shape), dtype)
                     for name, shape, dtype in self.tensors)


@dataclass(frozen=True)
class KVNeed:
    """Keys and values of every token (``window`` 0) or of the last ``window`` tokens (and of a request's first
    ``keep`` tokens), as the attention kernels read them: tensors "k" and "v", a block of each ``[kv_heads, block_size // 16, 16 * head_dim]``,
    tiles of 16 slots in matrix-core operand order (:mod:`reinfer_amd.cache.layout`)."""
    num_kv_heads: int
    head_dim: int
    window: int = 0
    keep: int = 0           # first tokens that a window keeps in sight
    chunked: bool = False   # the window is the query's own chunk of that many tokens, counted from position 0

    def block_tensors(self, block_size: int):
        from ..cache.layout import cache_shape
        shape = cache_shape(1, self.num_kv_heads, block_size, self.head_dim)[1:]
        return (("k", shape, None), ("v", shape, None))


@dataclass(frozen=True)
class StateNeed:
    """Per-request state of fixed size: one ``shape`` tensor per live request."""
    shape: Tuple[int, ...]
    dtype: torch.dtype = torch.float32


@dataclass(frozen=True)
class JointNeed:
    """What a layer keeps when it holds several mixers: each member's own need (None for a member that keeps
    nothing), in the members' order. At most one member may keep pages (keys and values or other paged
    tensors): the layer's block tables and window are that member's. The layer's :class:`LayerCache` then
    has one cache per member in ``members``."""
    members: Tuple[Optional[object], ...]

    def paged(self):
        found = [m for m in self.members if isinstance(m, (KVNeed, PagedNeed))]
        if len(found) > 1:
            raise ValueError("a layer's mixers may keep pages in one of them only")
        return found[0] if found else None


def covering(need, other):
    """``need`` with a window that also covers what a layer of need ``other`` reads of the same pages: the wider of
    two windows; of two chunk sizes the larger if it is a multiple of the smaller, else (and for a chunk beside a window: no
    chunk reaches further back than its size) a sliding window of the larger; everything where either reads everything."""
    a, b = (need.window, need.chunked), (other.window, other.chunked)
    keep = max(need.keep, other.keep)
    if not a[0] or not b[0]:
        return replace(need, window=0, keep=0, chunked=False)
    wide, narrow = max(a[0], b[0]), min(a[0], b[0])
    chunked = a[1] and b[1] and wide % narrow == 0 and not keep
    return replace(need, window=wide, keep=keep, chunked=chunked)


def paged_need(need):
    """The part of ``need`` that lives in pages (KVNeed or PagedNeed), or None."""
    if isinstance(need, (KVNeed, PagedNeed)):
        return need
    if isinstance(need, JointNeed):
        return need.paged()
    return None


@dataclass
class LayerCache:
    """The cache of one run-order entry, as its mixer sees it.

    Paged memory: ``tensors[name]`` is ``[blocks, *shape of one block]`` as the mixer's need named it;
    for keys and values (:class:`KVNeed`) ``k``/``v`` are the same tensors,
    ``[blocks, kv_heads, block_size // 16, 16 * head_dim]``, tiles of 16 slots in the order of
    :mod:`reinfer_amd.cache.layout`; ``group`` picks the step's block tables and slots, ``writes`` is
    False for an entry that reads another entry's cache. For state: ``state`` is
    ``[max_seqs, *shape]``, indexed by the step's ``state_slots``.
    """
    k: Optional[torch.Tensor] = None
    v: Optional[torch.Tensor] = None
    group: int = 0
    writes: bool = True
    state: Optional[torch.Tensor] = None
    tensors: Optional[dict] = None      # every paged tensor by the name its mixer gave it ("k" and "v" among them)
    members: Optional[list] = None      # for a :class:`JointNeed`: one LayerCache (or None) per member mixer

    def flat(self):
        """This cache and, for a joint one, its members' caches."""
        out = [self]
        for m in self.members or ():
            if m is not None:
                out += m.flat()
        return out


@dataclass
class RowScaled:
    """Rows whose RMSNorm is half done: ``x`` = bfloat16(stream * norm weight) [T, width]; the
    row factor rsqrt(sum_p ss[p, t] / width + eps) is applied by the product that takes them
    (y = rstd * ((x .* w) . W^T): the norm costs no kernel of its own). A part that declares
    ``takes_row_scaled = True`` may be handed this instead of a tensor."""
    x: torch.Tensor
    ss: torch.Tensor            # float32 [parts, T]
    eps: float
    width: int

    @property
    def row_sums(self):
        return self.ss, self.eps, self.width


@dataclass
class NormTarget:
    """Buffers that a part's last product fills for the norm that follows it, when it adds its
    result into the stream itself: ``x`` = bfloat16(new stream * norm.weight), ``ss`` = partial
    sums of squares of the new stream's rows. A part that declares ``emits_for_norm = True``
    may be given one (``emit=``); it returns it if it filled it.

    ``finished``: with more rows than a product behind the norm could scale (they are the library's), the
    part is asked for the whole norm instead, ``x`` = bfloat16(norm(new stream) * norm.weight), and there are
    no sums; it returns the target only if its product could do that."""
    norm: object
    x: torch.Tensor
    ss: Optional[torch.Tensor]
    finished: bool = False

    @property
    def emit(self):
        return self.norm.weight, self.x, self.ss

    @property
    def finish(self):
        return self.norm.weight, self.x, self.norm.eps


@dataclass
class StreamCopy:
    """What a block hands on in place of a pending addend when everything is in the stream already and it also
    holds the stream in the activations' type (``x`` [T, width]): a block whose parts read the stream itself takes
    it as their operand; any other block treats it as "nothing pending"."""
    x: torch.Tensor


@dataclass
class StreamMix:
    """What a block of several residual streams hands on: a sublayer's result ``y`` that is not in the streams yet, with
    the sublayer's ``mix`` [from, to] and ``w_out``, X_t <- sum_s mix[s, t] X_s + w_out[t] y; ``base`` [T, width]: every
    stream is still this row (the model's start), the streams' own buffer holds nothing yet."""
    base: Optional[torch.Tensor] = None
    y: Optional[torch.Tensor] = None
    mix: Optional[torch.Tensor] = None
    w_out: Optional[torch.Tensor] = None

    def norm_of(self, ops, streams: torch.Tensor, w_in: Optional[torch.Tensor], weight: Optional[torch.Tensor], eps: float,
                dtype: torch.dtype, rows: Optional[torch.Tensor] = None, store: bool = True) -> torch.Tensor:
        """The norm of the weighted sum of the streams (``w_in`` None: their sum; ``weight`` None: no norm) after what is
        pending; the new streams are kept where there was something pending, unless ``rows`` asks for some rows alone."""
        T, _, width = streams.shape
        out = torch.empty((T if rows is None else rows.numel(), width), dtype=dtype, device=streams.device)
        ops.hyper_step(streams, self.base, self.y, self.mix, self.w_out, w_in, weight, eps, out, rows=rows,
                       store=store and rows is None and self.y is not None)
        return out

    def stored(self) -> "StreamMix":
        """What is left pending once :meth:`norm_of` has kept the new streams."""
        return self if self.y is None else StreamMix()


@dataclass
class ScaledTerms:
    """A part's result left as a sum to be formed, sum_i scales[i] * terms[i] ([T, width] tensors of one dtype):
    handed back by a part that declares ``returns_terms`` to a caller that asked with ``terms_ok=True`` and adds
    the terms up itself, in float, in the kernel that consumes the sum."""
    terms: list
    scales: list


def project_out(ops, x: torch.Tensor, weight: torch.Tensor, resid: Optional[torch.Tensor], emit: Optional[NormTarget]):
    """A part's last product x . W^T. Where it can add into the stream ``resid`` it does and None comes back, or ``emit`` if it
    also prepared the norm that follows; otherwise the product, in the type of ``x``."""
    can_add = getattr(ops, "can_accumulate", None)
    if resid is not None and can_add and can_add(x, weight):
        # resid += x . W^T in the epilogue, which can also prepare the norm that follows
        if emit is not None and emit.finished:
            done = ops.linear_skinny(x, weight, resid, accumulate=True, finish=emit.finish)
            return emit if done else None
        if emit is not None:
            written = ops.linear_skinny(x, weight, resid, accumulate=True, emit=emit.emit)
            emit.ss = emit.ss[:written]          # as many partial sums a row as the kernel that ran has workgroups
            return emit
        ops.linear_skinny(x, weight, resid, accumulate=True)
        return None
    out = torch.empty((x.shape[0], weight.shape[0]), dtype=x.dtype, device=x.device)
    ops.linear(x, weight, out)
    return out


def split_input(x):
    """(tensor, row sums or None) of a part's input, plain or :class:`RowScaled`."""
    if isinstance(x, RowScaled):
        return x.x, x.row_sums
    return x, None
