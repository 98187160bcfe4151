"""Tensor-level entry points of the kernel library.

Each function checks on the host that shapes, dtypes, devices and strides are
what the kernel assumes, and only then launches on torch's current stream. The
parts call these through :func:`reinfer_amd.kernels.current`.
"""
from __future__ import annotations

import heapq
from typing import Optional

import torch

from . import library

_TAG = {torch.float32: 0, torch.bfloat16: 1}


def _tag(t: torch.Tensor, what: str) -> int:
    try:
        return _TAG[t.dtype]
    except KeyError:
        raise TypeError(f"{what}: dtype {t.dtype} is not float32 or bfloat16") from None


def _dev(*tensors) -> None:
    for t in tensors:
        if t is None:
            continue
        if not t.is_cuda:
            raise library.KernelLibraryError(
                "the kernels run on the GPU only: got a tensor on " + str(t.device))


def _ptr(t: Optional[torch.Tensor]) -> Optional[int]:
    return None if t is None else t.data_ptr()


def _stream() -> int:
    return torch.cuda.current_stream().cuda_stream


def _int32(t: torch.Tensor, what: str, n: Optional[int] = None) -> None:
    if t.dtype != torch.int32 or not t.is_contiguous():
        raise TypeError(f"{what}: expected a contiguous int32 tensor, got {t.dtype}")
    if n is not None and t.numel() < n:
        raise ValueError(f"{what}: {t.numel()} entries, need {n}")


class HipKernels:
    """The product's kernels. Stateless apart from the loaded library."""

    name = "hip-gfx950"

    def __init__(self):
        library.load()
        self._decode_slots = {}     # (heads, KV heads, head size) -> workgroups of the decode kernel's grid
        self._cu_count = {}
        self._side_streams = {}     # device -> the stream for the second kernel of a mixed step

    # ------------------------------------------------------------------ rows
    def embed(self, table: torch.Tensor, ids: torch.Tensor, out: torch.Tensor, scale: float = 1.0) -> None:
        _dev(table, ids, out)
        T, h = out.shape
        if table.dim() != 2 or table.shape[1] != h or not table.is_contiguous():
            raise ValueError(f"embed: table {tuple(table.shape)} does not have rows of width {h}")
        if out.dtype != torch.float32 or not out.is_contiguous():
            raise TypeError("embed: the residual stream is contiguous float32")
        _int32(ids, "embed ids", T)
        library.call("ra_embed", table.data_ptr(), _tag(table, "embed table"), ids.data_ptr(),
                     out.data_ptr(), T, h, float(scale), _stream())

    def add_rmsnorm(self, resid: torch.Tensor, delta: Optional[torch.Tensor], weight: torch.Tensor,
                    eps: float, out: torch.Tensor, rows: Optional[torch.Tensor] = None,
                    delta_scale: float = 1.0, groups: int = 1) -> None:
        """``groups`` > 1: the row is normed in that many equal consecutive parts, each over its own root mean
        square."""
        _dev(resid, delta, weight, out, rows)
        h = resid.shape[-1]
        n = out.shape[0]
        if resid.dtype != torch.float32 or not resid.is_contiguous():
            raise TypeError("add_rmsnorm: the residual stream is contiguous float32")
        if weight.shape != (h,) or out.shape[-1] != h or not out.is_contiguous():
            raise ValueError(f"add_rmsnorm: width {h}, weight {tuple(weight.shape)}, out {tuple(out.shape)}")
        if delta is not None:
            if delta.shape != resid.shape or delta.dtype != out.dtype or not delta.is_contiguous():
                raise ValueError("add_rmsnorm: delta must match the residual's shape and the output's dtype")
        if rows is None:
            if n != resid.shape[0]:
                raise ValueError("add_rmsnorm: in-place form needs one output row per residual row")
        else:
            _int32(rows, "add_rmsnorm rows", n)
        if groups != 1:
            if groups < 1 or h % groups:
                raise ValueError(f"add_rmsnorm: width {h} does not split into {groups} equal groups")
            library.call("ra_add_group_rmsnorm", resid.data_ptr(), _ptr(delta), weight.data_ptr(),
                         _tag(weight, "norm weight"), out.data_ptr(), _tag(out, "add_rmsnorm out"),
                         _ptr(rows), n, h, int(groups), float(eps), float(delta_scale), _stream())
            return
        library.call("ra_add_rmsnorm", resid.data_ptr(), _ptr(delta), weight.data_ptr(),
                     _tag(weight, "norm weight"), out.data_ptr(), _tag(out, "add_rmsnorm out"),
                     _ptr(rows), n, h, float(eps), float(delta_scale), _stream())

    def qk_norm_rope_cache(self, qkv: torch.Tensor, q_weight: Optional[torch.Tensor],
                           k_weight: Optional[torch.Tensor], eps: float, positions: torch.Tensor,
                           inv_freq: torch.Tensor, rotary_dim: int, rope_style: int,
                           slots: torch.Tensor, kcache: torch.Tensor, vcache: torch.Tensor,
                           num_heads: int, num_kv_heads: int, head_dim: int, values_are_keys: bool = False) -> None:
        """Head norm and rotation of q (in place) and k, k and v into the cache. ``values_are_keys``: the rows hold
        q and k alone, and the value that is cached is the key as it stands there, before norm and rotation.
        ``qkv`` may be wider than its heads (they stand at the start of a row). ``num_kv_heads`` 0: queries alone,
        nothing is cached (``kcache`` and ``vcache`` None, ``k_weight`` as ``q_weight``)."""
        _dev(qkv, q_weight, k_weight, positions, inv_freq, slots, kcache, vcache)
        T = qkv.shape[0]
        width = (num_heads + (1 if values_are_keys else 2) * num_kv_heads) * head_dim
        if qkv.dim() != 2 or qkv.shape[1] < width or qkv.stride(1) != 1 or qkv.stride(0) < width:
            raise ValueError(f"qk_norm_rope_cache: qkv {tuple(qkv.shape)}, expected rows of at least {width}")
        if num_kv_heads:
            self._check_cache("qk_norm_rope_cache", kcache, vcache, num_kv_heads, head_dim)
            if kcache.dtype != qkv.dtype or vcache.dtype != qkv.dtype:
                raise TypeError("qk_norm_rope_cache: the cache has the activations' dtype")
        _int32(positions, "positions", T)
        _int32(slots, "cache slots", T)
        if inv_freq.dtype != torch.float32 or inv_freq.numel() < rotary_dim // 2:
            raise ValueError("qk_norm_rope_cache: inv_freq is float32 with rotary_dim/2 entries")
        wtag = 0
        for w in (q_weight, k_weight):
            if w is not None:
                if w.shape != (head_dim,):
                    raise ValueError(f"qk_norm_rope_cache: head-norm weight {tuple(w.shape)}, expected [{head_dim}]")
                wtag = _tag(w, "head-norm weight")
        if q_weight is not None and k_weight is not None and q_weight.dtype != k_weight.dtype:
            raise TypeError("qk_norm_rope_cache: q and k norm weights differ in dtype")
        library.call("ra_qk_norm_rope_cache", qkv.data_ptr(), _tag(qkv, "qkv"), _ptr(q_weight),
                     _ptr(k_weight), wtag, float(eps), positions.data_ptr(), inv_freq.data_ptr(),
                     int(rotary_dim), int(rope_style), slots.data_ptr(), _ptr(kcache) if num_kv_heads else None,
                     _ptr(vcache) if num_kv_heads else None, kcache.shape[2] * 16 if num_kv_heads else 16, T, num_heads,
                     num_kv_heads, head_dim, 1 if values_are_keys else 0, qkv.stride(0), _stream())

    # ---- the q/k/v product left in K ranges for the kernel that consumes it
    def linear_ranges(self, x: torch.Tensor, weight: torch.Tensor):
        """x . weight^T as the float results of the K ranges it was cut into, [ranges, M, N], not yet
        added, or None where that does not pay: only the products the split kernel takes (bfloat16,
        17 to 64 rows) and cuts (few output features), whose adding kernel a consumer can save by
        adding the ranges itself (``qk_norm_rope_cache(..., ranges=)``)."""
        if not (x.is_cuda and x.dtype == torch.bfloat16 and weight.dtype == torch.bfloat16 and x.dim() == 2):
            return None
        M, K = x.shape
        N = weight.shape[0]
        if not (self.NORM_SKINNY_ROWS < M <= 64) or K % 8 or x.stride(1) != 1 or x.stride(0) % 8 \
                or weight.shape != (N, K) or not weight.is_contiguous():
            return None
        lib = library.load()
        S = int(lib.ra_gemm_wide_ranges(M, N, K))
        if S < 2 or not lib.ra_gemm_wide_preferred(0, M, N, K):
            return None
        parts = torch.empty((S, M, N), dtype=torch.float32, device=x.device)
        library.call("ra_gemm_wide_partial", x.data_ptr(), weight.data_ptr(), parts.data_ptr(), parts.numel(),
                     M, N, K, x.stride(0), _stream())
        return parts

    def qk_norm_rope_cache_ranges(self, ranges: torch.Tensor, row_sums, q_out: torch.Tensor,
                                  q_weight: Optional[torch.Tensor], k_weight: Optional[torch.Tensor], eps: float,
                                  positions: torch.Tensor, inv_freq: torch.Tensor, rotary_dim: int,
                                  rope_style: int, slots: torch.Tensor, kcache: torch.Tensor,
                                  vcache: torch.Tensor, num_heads: int, num_kv_heads: int, head_dim: int) -> None:
        """``qk_norm_rope_cache`` on the result of ``linear_ranges``: the ranges are added here (in
        range order), the rows scaled by the RMSNorm that the product carried (``row_sums`` = (ss
        [parts, T], eps, width) or None), q normalised and rotated into ``q_out`` [T, heads * head_dim]."""
        _dev(ranges, q_weight, k_weight, positions, inv_freq, slots, kcache, vcache, q_out)
        S, T, width = ranges.shape
        if width != (num_heads + 2 * num_kv_heads) * head_dim or ranges.dtype != torch.float32 \
                or not ranges.is_contiguous():
            raise ValueError(f"qk_norm_rope_cache: ranges {tuple(ranges.shape)} {ranges.dtype}, expected float32 "
                             f"[ranges, T, {(num_heads + 2 * num_kv_heads) * head_dim}]")
        self._check_cache("qk_norm_rope_cache", kcache, vcache, num_kv_heads, head_dim)
        if q_out.dtype != kcache.dtype or q_out.shape != (T, num_heads * head_dim) or q_out.stride(1) != 1:
            raise ValueError("qk_norm_rope_cache: q_out is [T, heads * head_dim] in the cache's dtype")
        _int32(positions, "positions", T)
        _int32(slots, "cache slots", T)
        if inv_freq.dtype != torch.float32 or inv_freq.numel() < rotary_dim // 2:
            raise ValueError("qk_norm_rope_cache: inv_freq is float32 with rotary_dim/2 entries")
        wtag = 0
        for w in (q_weight, k_weight):
            if w is not None:
                if w.shape != (head_dim,):
                    raise ValueError(f"qk_norm_rope_cache: head-norm weight {tuple(w.shape)}, expected [{head_dim}]")
                wtag = _tag(w, "head-norm weight")
        ss = None
        parts, in_eps, in_width = 0, 0.0, 0
        if row_sums is not None:
            ss, in_eps, in_width = row_sums
            _dev(ss)
            if ss.dtype != torch.float32 or ss.dim() != 2 or ss.shape[1] != T or not ss.is_contiguous():
                raise ValueError(f"qk_norm_rope_cache: row sums {tuple(ss.shape)} {ss.dtype}, expected float32 [parts, {T}]")
            parts = ss.shape[0]
        library.call("ra_qk_norm_rope_cache_sums", ranges.data_ptr(), S, _ptr(ss), parts, float(in_eps),
                     int(in_width), q_out.data_ptr(), q_out.stride(0), _tag(q_out, "q"), _ptr(q_weight),
                     _ptr(k_weight), wtag, float(eps), positions.data_ptr(), inv_freq.data_ptr(),
                     int(rotary_dim), int(rope_style), slots.data_ptr(), kcache.data_ptr(), vcache.data_ptr(),
                     kcache.shape[2] * 16, T, num_heads, num_kv_heads, head_dim, 0, _stream())

    GATE_ACTS = {"silu": 0, "gelu_tanh": 1, "swish_bounded": 2}

    def silu_mul(self, gate_up: torch.Tensor, out: torch.Tensor, group: int = 0, act: str = "silu",
                 limit: float = 0.0) -> None:
        """out = act(gate) * up, act "silu" or "gelu_tanh" (0.5 z (1 + tanh(sqrt(2/pi) (z + 0.044715 z^3)))), or
        "swish_bounded": g <- min(gate, limit), u <- clamp(up, -limit, limit), out = g sigmoid(1.702 g) (u + 1).
        ``group`` 0: gate_up is [gate | up]; ``group`` g > 0: runs of g gate columns and g up columns alternate."""
        _dev(gate_up, out)
        T, I = out.shape
        if gate_up.shape != (T, 2 * I) or gate_up.dtype != out.dtype \
                or not gate_up.is_contiguous() or not out.is_contiguous():
            raise ValueError(f"silu_mul: gate_up {tuple(gate_up.shape)} against out {tuple(out.shape)}")
        if group < 0 or (group > 0 and I % group != 0):
            raise ValueError(f"silu_mul: width {I} is not a whole number of runs of {group}")
        if act not in self.GATE_ACTS:
            raise ValueError(f"silu_mul: activation {act!r}; built: {sorted(self.GATE_ACTS)}")
        if act == "swish_bounded" and not limit > 0.0:
            raise ValueError("silu_mul: the bounded activation needs a positive limit")
        library.call("ra_act_mul_bounded", gate_up.data_ptr(), out.data_ptr(), _tag(out, "silu_mul"), T, I,
                     int(group), self.GATE_ACTS[act], float(limit), _stream())

    # ------------------------------------------------------------- attention
    SHORT_PORTION = 4     # portions up to this many tokens go token by token through the decode kernel
    TWO_STREAMS_FROM = 8  # decode tokens of a mixed step from which their attention runs beside the prompt portions'

    def attention(self, q: torch.Tensor, q_stride: int, out: torch.Tensor, kcache: torch.Tensor,
                  vcache: torch.Tensor, batch, num_heads: int, num_kv_heads: int, head_dim: int,
                  scale: float, window: int, group: int, softcap: float = 0.0, distance=None,
                  keep: int = 0, aligned: bool = False, sink=None, gate=None) -> None:
        """Attention of every token of the step over its request's cache.

        ``softcap`` > 0: score <- softcap * tanh(score / softcap); ``distance`` = (r1, r2), two float32 vectors
        with one entry a query head: score <- score - r1[h] * ln(1 + r2[h] * (query position - key position)),
        behind the cap. ``keep`` > 0 with a window: a request's first ``keep`` keys are seen as well, however far
        the window has moved on. ``aligned``: the keys are cut into chunks of ``window`` from position 0 and a query
        sees those of its own chunk alone. ``sink`` (float32, one entry a query head): the softmax's denominator holds
        one more term exp(sink[h]). ``gate`` ([T, at least the query heads] rows of the activations' dtype, unit column
        stride): a head's result is multiplied by the sigmoid of its number. Every kernel below applies them alike.

        ``q`` is the buffer whose row ``t`` holds the query heads of token t at
        its start (row stride ``q_stride`` elements); ``batch`` is the step's
        :class:`reinfer_amd.engine.batch.StepBatch`; ``group`` picks the block
        tables of the cache group this layer belongs to. bfloat16: single tokens
        and short portions take the split-KV decode kernel, longer portions the
        MFMA prefill kernel in tiles of queries; sizes neither takes, and
        float32, go to the plain kernel.
        """
        lib = library.load()
        mod = self._score_mod(softcap, distance, num_heads, q.device)
        # handed on only where there is a change, so that the kernels' callers of old need not know of it
        changed = {"mod": mod} if (mod[0] > 0.0 or mod[1] is not None) else {}
        if keep < 0:
            raise ValueError("attention: a negative number of kept keys")
        if keep and window:
            changed["keep"] = int(keep)
        if aligned and window:
            if keep:
                raise ValueError("attention: chunks keep no first keys")
            changed["aligned"] = True
        if sink is not None or gate is not None:
            changed["head_out"] = self._head_out(sink, gate, q, num_heads)
        if q.dtype != torch.bfloat16:
            return self.attention_plain(q, q_stride, out, kcache, vcache, batch, num_heads, num_kv_heads,
                                        head_dim, scale, window, group, **changed)
        bs = kcache.shape[2] * 16
        tile = lib.ra_attention_prefill_tile(num_heads, num_kv_heads, head_dim)
        # query tiles that give every CU one workgroup
        room = self._cus(q.device) // max(1, lib.ra_attention_prefill_groups(num_heads, num_kv_heads, head_dim))
        halves = lib.ra_attention_prefill_columns(num_heads, num_kv_heads, head_dim) == 2
        # the plan's fixed costs are priced in rounds of this shape: a round's time goes with the columns of a
        # query tile times the head size the kernel is built for
        cols = 128 * max(1, lib.ra_attention_prefill_columns(num_heads, num_kv_heads, head_dim))
        built_for = 64 if head_dim <= 64 else 128 if head_dim <= 128 else 256
        plan = self._attention_plan(batch, q.device, tile, room, halves, (256 * 128) / (cols * built_for),
                                    int(window) if aligned else 0)
        dec_ok = bool(lib.ra_attention_decode_supports(num_heads, num_kv_heads, head_dim, bs))
        pre_ok = bool(lib.ra_attention_prefill_supports(num_heads, num_kv_heads, head_dim, bs))
        side = None
        if plan["n_decode"] >= self.TWO_STREAMS_FROM and plan["n_tiles"] and dec_ok and pre_ok \
                and not torch.cuda.is_current_stream_capturing():
            # a mixed step: the decoding requests' attention streams keys and values, the prompt
            # portions' attention computes; on two streams (both of default priority) the two kernels
            # share the chip (128 requests at the Qwen3-4B shape, 2048-token steps: 0.7 ms a mixed step)
            side = self._side_stream(q.device)
            cur = torch.cuda.current_stream()
            side.wait_stream(cur)
            with torch.cuda.stream(side):           # its scratch comes from, and goes back to, the side stream's pool
                self.attention_decode(q, q_stride, out, kcache, vcache, batch, num_heads, num_kv_heads,
                                      head_dim, scale, window, group, plan["decode_list"], plan["n_decode"],
                                      plan["decode_max_ctx"], **changed)
        elif plan["n_decode"]:
            if dec_ok:
                self.attention_decode(q, q_stride, out, kcache, vcache, batch, num_heads, num_kv_heads,
                                      head_dim, scale, window, group, plan["decode_list"], plan["n_decode"],
                                      plan["decode_max_ctx"], **changed)
            else:
                self.attention_plain(q, q_stride, out, kcache, vcache, batch, num_heads, num_kv_heads,
                                     head_dim, scale, window, group, plan["decode_list"], plan["n_decode"], **changed)
        if plan["n_tiles"]:
            if pre_ok:
                self.attention_prefill(q, q_stride, out, kcache, vcache, batch, num_heads, num_kv_heads,
                                       head_dim, scale, window, group, plan["tiles"], plan["n_tiles"],
                                       plan.get("ranges"), plan.get("merge"), plan.get("n_merge", 0),
                                       plan.get("n_slots", 0), **changed)
            else:
                self.attention_plain(q, q_stride, out, kcache, vcache, batch, num_heads, num_kv_heads,
                                     head_dim, scale, window, group, plan["prefill_list"], plan["n_prefill"], **changed)
        if side is not None:
            torch.cuda.current_stream().wait_stream(side)

    @staticmethod
    def _score_mod(softcap: float, distance, num_heads: int, device):
        """(softcap, r1 pointer or None, r2 pointer or None) for the kernels' ``_mod`` entry points, checked."""
        if softcap < 0.0:
            raise ValueError("attention: a negative score cap")
        if distance is None:
            return (float(softcap), None, None)
        r1, r2 = distance
        for r in (r1, r2):
            if r.dtype != torch.float32 or r.shape != (num_heads,) or not r.is_contiguous() or r.device != device:
                raise ValueError(f"attention: the distance term takes two float32 vectors of {num_heads} entries")
        return (float(softcap), r1.data_ptr(), r2.data_ptr())

    @staticmethod
    def _head_out(sink, gate, q, num_heads: int):
        """(sink pointer or None, gate pointer or None, gate row stride) for the kernels' ``_mod`` entry points, checked."""
        if sink is not None and (sink.dtype != torch.float32 or sink.shape != (num_heads,) or not sink.is_contiguous()
                                 or sink.device != q.device):
            raise ValueError(f"attention: the sink is a float32 vector of {num_heads} entries")
        if gate is not None and (gate.dtype != q.dtype or gate.dim() != 2 or gate.shape[0] != q.shape[0]
                                 or gate.shape[1] < num_heads or gate.stride(1) != 1 or gate.device != q.device):
            raise ValueError(f"attention: the gate is [T, at least {num_heads}] in the queries' dtype, unit column stride")
        return (_ptr(sink), _ptr(gate), gate.stride(0) if gate is not None else 0)

    def shared_head_limit(self, head_dim: int, block_size: int = 16) -> int:
        """Query heads that may share one KV head in a call of :meth:`attention` and still take the
        matrix-core kernels (the decode kernel's waves add their results through LDS, which bounds heads times
        head size); 0: no number of heads does at this head size. A mixer all of whose heads read one cached
        row (a shared latent) splits its heads into groups of at most this many."""
        lib = library.load()
        for g in range(16, 0, -1):
            if lib.ra_attention_decode_supports(g, 1, int(head_dim), int(block_size)) \
                    and lib.ra_attention_prefill_supports(g, 1, int(head_dim), int(block_size)):
                return g
        return 0

    def _side_stream(self, device):
        s = self._side_streams.get(device)
        if s is None:
            s = self._side_streams[device] = torch.cuda.Stream(device=device)      # default priority
        return s

    def _cus(self, device) -> int:
        n = self._cu_count.get(device)
        if n is None:
            n = self._cu_count[device] = int(torch.cuda.get_device_properties(device).multi_processor_count)
        return n

    # What the prompt kernel's plan is chosen by, in rounds of 64 keys of a whole query tile of 256 columns
    # and head size 128 (2.1 us: 64 queries of 4 heads): a tile listed with half of its heads costs 0.76 of the
    # whole one, every listed item one such round to start and end, and the kernel that adds the parts of cut
    # tiles 3 rounds and 0.15 for each part; for another shape the three fixed costs are scaled by how much
    # shorter or longer its rounds are (``fixed``: the reference round's work over this shape's) (measured: a portion of 512 tokens behind 3584: 142 us as it is, 115 with the tiles
    # listed twice, 57 cut by keys; 256 behind 7936: 277 / 223 / 58; a whole prompt of 2048: 83 / 69 / 83,
    # of 1024: 43 / 35 / 40; 2048 behind 2048: 152 / 195 / 146)
    PREFILL_ROUND = 64
    PREFILL_HALF_HEADS = 0.76
    PREFILL_ITEM = 1.0
    PREFILL_MERGE = (3.0, 0.15)
    PREFILL_PART_ROUNDS = 4     # a part of a cut tile has at least this many rounds
    PREFILL_MAX_PARTS = 8

    @staticmethod
    def _span(costs, room: int) -> float:
        """When the last of ``costs`` ends if ``room`` run at a time, the heaviest started first and each
        further one where room is first free."""
        if len(costs) <= room:
            return max(costs)
        costs = sorted(costs, reverse=True)
        ends = costs[:room]
        heapq.heapify(ends)
        for c in costs[room:]:
            heapq.heappush(ends, heapq.heappop(ends) + c)
        return max(ends)

    def _prefill_items(self, tiles, room: int, halves: bool, fixed: float = 1.0, chunk: int = 0):
        """The prompt kernel's work items for ``tiles`` of (request, row, queries, position), and the list
        for the kernel that adds the parts of tiles cut by keys: ``(items, merge, n_slots)``, an item being
        (cost, tile, first key, one past the last key, slot or -1).

        A launch lasts as long as its heaviest item while the CUs of the light ones idle: a whole prompt of
        2048 tokens is one tile a CU, the last with 32 times the keys of the first; a portion of 512 tokens
        deep in a long prompt is eight tiles of thousands of keys each on a chip with room for 32. Three
        ways to list the tiles are priced by ``_span`` and the cheapest is taken. As they are. Where the
        kernel can give a workgroup half of a tile's heads (``halves``), the tiles with the most keys
        twice, each time with half of the heads (as many as there is room for and at
        least a quarter of ``room``; from ``room`` to 5/4 of it 3/16 of ``room``): a half that queues behind
        a light tile still ends before a whole heavy one would, which pays for a prompt from its start. Or,
        while there are fewer tiles than ``room``, the heaviest cut by keys into parts, each an item whose
        float sums a second kernel adds up; the spare room goes, one part at a time, to the tile whose
        parts are longest. (Windows are not known here, one plan serving all layers: a part below a
        layer's window finds nothing to do. ``chunk`` > 0: the plan of layers whose queries see the keys of their own chunk
        of that many alone; a tile's rounds then begin at the chunk of its first query.)"""
        R = self.PREFILL_ROUND
        n = len(tiles)
        item_cost = self.PREFILL_ITEM * fixed
        begin = [pos // chunk * chunk // R if chunk else 0 for (_, _, _, pos) in tiles]      # a tile's first round
        rounds = [-(-(pos + q) // R) - b for (_, _, q, pos), b in zip(tiles, begin)]
        whole = [(r + item_cost, tl, 0, 0, -1) for tl, r in zip(tiles, rounds)]
        if room <= 0 or n == 0:
            return whole, [], 0
        best, best_span = (whole, [], 0), self._span([it[0] for it in whole], room)
        # the heaviest twice, by heads
        n_twice = 0
        if not halves:
            pass
        elif n <= room:
            n_twice = min(n, max(room - n, room // 4))
        elif n <= room + room // 4:
            n_twice = (3 * room) // 16
        if n_twice:
            twice = set(sorted(range(n), key=lambda k: -rounds[k])[:n_twice])
            items = []
            for k, (tl, r) in enumerate(zip(tiles, rounds)):
                if k in twice:
                    i, row, q, pos = tl
                    c = r * self.PREFILL_HALF_HEADS + item_cost
                    items.append((c, (i, row, q | (1 << 16), pos), 0, 0, -1))
                    items.append((c, (i, row, q | (2 << 16), pos), 0, 0, -1))
                else:
                    items.append(whole[k])
            span = self._span([it[0] for it in items], room)
            if span < best_span:
                best, best_span = (items, [], 0), span
        # the heaviest cut by keys
        if n < room:
            parts = [1] * n
            heap = [(-r, k) for k, r in enumerate(rounds)]
            heapq.heapify(heap)
            used = n
            while used < room and heap:
                _, k = heapq.heappop(heap)
                if parts[k] >= self.PREFILL_MAX_PARTS or rounds[k] < self.PREFILL_PART_ROUNDS * (parts[k] + 1):
                    continue
                parts[k] += 1
                used += 1
                heapq.heappush(heap, (-rounds[k] / parts[k], k))
            items, merge, n_slots = [], [], 0
            for k, (tl, r) in enumerate(zip(tiles, rounds)):
                per = -(-r // parts[k])
                p = -(-r // per)
                if p <= 1:
                    items.append(whole[k])
                    continue
                merge.extend((tl[1], tl[2], n_slots, p))
                for j in range(p):
                    lo = (begin[k] + j * per) * R if j else 0
                    hi = (begin[k] + (j + 1) * per) * R if j + 1 < p else 1 << 30
                    items.append((min(per, r - j * per) + item_cost, tl, lo, hi, n_slots + j))
                n_slots += p
            if n_slots:
                span = self._span([it[0] for it in items], room) + (self.PREFILL_MERGE[0]
                                                                      + self.PREFILL_MERGE[1] * n_slots) * fixed
                if span < best_span:
                    best, best_span = (items, merge, n_slots), span
        return best

    def plan_captured_step(self, batch, num_rows: int, ctx_cap: int) -> None:
        """The attention plan of a captured decode step: ``num_rows`` single tokens over contexts of at most
        ``ctx_cap``, whatever the step that is replayed holds (the grids are chosen from these)."""
        batch.extra["attention_plan"] = {
            "n_decode": num_rows, "decode_max_ctx": ctx_cap, "decode_list": None, "n_prefill": 0,
            "prefill_list": None, "n_tiles": 0, "tiles": None}

    def _attention_plan(self, batch, device, tile: int, room: int = 0, halves: bool = False, fixed: float = 1.0,
                        chunk: int = 0):
        """Which tokens go to which kernel; made once per step and query-tile size, shared by the
        layers. ``room`` is the number of query tiles whose workgroups fill the chip once (0: the tiles
        are listed as they are)."""
        plan = batch.extra.get("attention_plan")
        if plan is not None and plan.get("tile", tile) == tile:
            return plan
        plan = batch.extra.get(("attention_plan", tile, room, halves, fixed, chunk))
        if plan is not None:
            return plan
        dec, pre, tiles = [], [], []
        dec_max_ctx = 0
        t = 0
        for i, (ql, st) in enumerate(zip(batch.q_lens, batch.starts)):
            if ql <= self.SHORT_PORTION:
                dec.extend(range(t, t + ql))
                dec_max_ctx = max(dec_max_ctx, st + ql)
            else:
                pre.extend(range(t, t + ql))
                for q0 in range(0, ql, tile):
                    tiles.append((i, t + q0, min(tile, ql - q0), st + q0))
            t += ql
        items, merge, n_slots = self._prefill_items(tiles, room, halves, fixed, chunk)
        items.sort(key=lambda it: it[0])                     # the heaviest last: the kernel starts the last listed first
        listed = [v for it in items for v in it[1]]
        ranges = [v for it in items for v in ((it[2], it[3], it[4]) if it[4] >= 0 else (0, 1 << 30, -1))] if merge else []
        all_decode = len(dec) == batch.num_tokens
        flat = ([] if all_decode else dec) + pre + listed + ranges + merge
        dev = torch.tensor(flat, dtype=torch.int32).to(device, non_blocking=True) if flat else None
        n_dec_listed = 0 if all_decode else len(dec)
        o_tiles = n_dec_listed + len(pre)
        o_ranges = o_tiles + len(listed)
        o_merge = o_ranges + len(ranges)
        plan = {
            "n_decode": len(dec), "decode_max_ctx": dec_max_ctx,
            "decode_list": None if all_decode or not dec else dev[:n_dec_listed],
            "n_prefill": len(pre),
            "prefill_list": dev[n_dec_listed:o_tiles] if pre else None,
            "n_tiles": len(items),
            "tiles": dev[o_tiles:o_ranges] if items else None,
            "ranges": dev[o_ranges:o_merge] if merge else None,
            "merge": dev[o_merge:] if merge else None,
            "n_merge": len(merge) // 4, "n_slots": n_slots,
            "tile": tile,
        }
        batch.extra[("attention_plan", tile, room, halves, fixed, chunk)] = plan
        return plan

    @staticmethod
    def _check_cache(what: str, kcache, vcache, num_kv_heads: int, head_dim: int) -> None:
        """K and V of a layer: [blocks, kv heads, block_size // 16, 16 * head_dim], tiled."""
        if kcache.dim() != 4 or kcache.shape != vcache.shape or kcache.shape[1] != num_kv_heads \
                or head_dim % 16 != 0 or kcache.shape[3] != 16 * head_dim \
                or not kcache.is_contiguous() or not vcache.is_contiguous():
            raise ValueError(f"{what}: cache K {tuple(kcache.shape)}, V {tuple(vcache.shape)}: expected "
                             f"[blocks, {num_kv_heads}, block_size // 16, 16 * {head_dim}] "
                             "(head sizes in steps of 16)")

    def _check_attention(self, q, q_stride, out, kcache, vcache, batch, num_heads, num_kv_heads, head_dim, group):
        _dev(q, out, kcache, vcache)
        T = batch.num_tokens
        tables = batch.block_tables[group]
        if out.shape != (T, num_heads * head_dim) or out.stride(1) != 1 or out.dtype != q.dtype:
            raise ValueError(f"attention: out {tuple(out.shape)}, expected [{T}, {num_heads * head_dim}] with "
                             "contiguous rows (it may be a column range of a wider buffer)")
        if q.shape[0] != T or q_stride < num_heads * head_dim or q.stride(0) != q_stride:
            raise ValueError("attention: query rows do not match the step's tokens")
        if kcache.dtype != q.dtype or vcache.dtype != q.dtype:
            raise TypeError("attention: the cache has the activations' dtype")
        self._check_cache("attention", kcache, vcache, num_kv_heads, head_dim)
        _int32(tables, "block tables")
        if tables.dim() != 2 or tables.shape[0] < batch.num_seqs:
            raise ValueError("attention: one block-table row per request of the step")
        # every key a query may read must have a table entry
        if tables.shape[1] * kcache.shape[2] * 16 < batch.max_ctx_len:
            raise ValueError("attention: block tables shorter than the longest context")
        return tables

    def attention_plain(self, q, q_stride, out, kcache, vcache, batch, num_heads, num_kv_heads, head_dim,
                        scale, window, group, token_list=None, n_listed=None, mod=(0.0, None, None), keep: int = 0,
                        aligned: bool = False, head_out=(None, None, 0)) -> None:
        tables = self._check_attention(q, q_stride, out, kcache, vcache, batch, num_heads, num_kv_heads,
                                       head_dim, group)
        n = batch.num_tokens if token_list is None else int(n_listed)
        library.call("ra_attention_plain_mod", q.data_ptr(), q_stride, out.data_ptr(), out.stride(0),
                     kcache.data_ptr(), vcache.data_ptr(), _tag(q, "attention"), tables.data_ptr(),
                     tables.shape[1], _ptr(token_list), batch.seq_of_token.data_ptr(),
                     batch.positions.data_ptr(), n, kcache.shape[2] * 16, num_heads, num_kv_heads, head_dim,
                     float(scale), int(window), int(aligned), int(keep), mod[0], mod[1], mod[2], *head_out, _stream())

    # The decode kernel runs in workgroups of 12 waves from this many (token, KV head) pairs on, or over
    # contexts longer than this; below both, in workgroups of 4 (measured with 32 query heads over 8 KV
    # heads of 128, flash decode and merge together: 2200 keys a token, 1 / 4 / 8 / 16 / 32 / 64 tokens: 4 waves
    # 10.6 / 13.1 / 23.3 / 40.4 / 61.3 / 107 us, 12 waves 13.6 / 14.5 / 21.5 / 33.8 / 56.2 / 107; 8000 keys,
    # 1 / 4 / 16 / 64 tokens: 17.9 / 35.9 / 113 / 370 against 14.7 / 31.2 / 101 / 364)
    DECODE_WIDE_PAIRS = 64
    DECODE_WIDE_CTX = 4096      # keys of head size 128: what counts is the bytes of a (token, KV head) pair
    DECODE_WIDE_FILL = 0.9      # of the last round of large workgroups that the pairs must fill
    # Fewer pairs than the chip holds large workgroups: one large workgroup a pair, nothing to merge, from this
    # share of them on (20 to 28 requests over 8 KV heads, 1000 to 7000 keys: 8 to 14 % faster than the small
    # workgroups with their chunks and merge, 16 requests: equal), and at any number over contexts up to
    # DECODE_SHORT_CTX keys of head size 128 (600 keys, 1 to 24 requests: 7.8 to 15.2 us against 9.3 to 20.6)
    DECODE_WIDE_FILL_ONE = 0.6
    DECODE_SHORT_CTX = 768

    def _slots_of_decode(self, num_heads: int, num_kv_heads: int, head_dim: int, waves: int) -> int:
        """Workgroups of the decode kernel's form with ``waves`` waves that the chip holds at once (0: that
        form does not take these sizes)."""
        key = (num_heads, num_kv_heads, head_dim, waves)
        slots = self._decode_slots.get(key)
        if slots is None:
            slots = int(library.load().ra_attention_decode_slots(num_heads, num_kv_heads, head_dim, waves))
            self._decode_slots[key] = slots
        return slots

    def decode_chunk(self, n_tokens: int, num_heads: int, num_kv_heads: int, head_dim: int, max_ctx: int):
        """How the decode kernel cuts a token's keys: (least chunk length, most chunks a token, waves a
        workgroup). The kernel cuts every token into equal chunks of its own length, so only their
        number is chosen here: as many as fill the kernel's grid once (the workgroups the chip holds at
        once, whatever the batch). Then all work items run side by side and the launch lasts as long as
        one of them; more items than that cost a start and a partial result each (measured at 2200
        and 8000 keys a token, 1 to 128 tokens). Workgroups of 12 waves, one a CU, each with three times
        the keys in flight, need a third of the chunks to keep the memory as busy, which leaves fewer
        partial results to merge (none at 32 tokens and more); a small step over short contexts has too
        little work for them, and a step with more (token, KV head) pairs than the chip holds such
        workgroups would give some of them two pairs one after the other while the rest idle (33
        requests over 8 KV heads: 68 us a layer against 47 with the small workgroups, of which three fit
        a CU)."""
        pairs = max(1, n_tokens * num_kv_heads)
        waves = 4
        wide = self._slots_of_decode(num_heads, num_kv_heads, head_dim, 12)
        if 0 < pairs <= wide and (pairs >= self.DECODE_WIDE_FILL_ONE * wide
                                  or max_ctx * head_dim <= self.DECODE_SHORT_CTX * 128):
            return 512, 1, 12
        if pairs >= self.DECODE_WIDE_PAIRS or max_ctx * head_dim > self.DECODE_WIDE_CTX * 128:
            # whole rounds of the large workgroups, or nearly (64 requests over 8 KV heads are two rounds
            # of 256: 8.45 ms a step against 8.65 with the small workgroups)
            if wide > 0 and pairs >= self.DECODE_WIDE_FILL * (-(-pairs // wide) * wide):
                waves = 12
        slots = self._slots_of_decode(num_heads, num_kv_heads, head_dim, waves) or 768
        least = 256 if waves == 4 else 512
        return least, max(1, min(slots // pairs, -(-max_ctx // least))), waves

    def attention_decode(self, q, q_stride, out, kcache, vcache, batch, num_heads, num_kv_heads, head_dim,
                         scale, window, group, token_list=None, n_listed=None, max_ctx=None,
                         chunk=None, waves=None, mod=(0.0, None, None), keep: int = 0, aligned: bool = False,
                         head_out=(None, None, 0)) -> None:
        tables = self._check_attention(q, q_stride, out, kcache, vcache, batch, num_heads, num_kv_heads,
                                       head_dim, group)
        if q.dtype != torch.bfloat16:
            raise TypeError("attention_decode: bfloat16 only")
        n = batch.num_tokens if token_list is None else int(n_listed)
        max_ctx = int(max_ctx or batch.max_ctx_len)
        if window > 0:
            # no token reads more than its window (from the tile that holds its first key) and the kept keys' tiles
            max_ctx = min(max_ctx, int(window) + 15 + -(-int(keep) // 16) * 16)
            if aligned:
                # nor more than its chunk, of which it sees half on average: the cut is chosen for three quarters of one (any
                # cut is right for any number of keys). 1 to 32 requests over chunks of 1024: one part of keys a token, and
                # nothing to merge, takes 8 to 15 us from the chunk's start to its end, several parts 11 to 18
                max_ctx = min(max_ctx, max(16, 3 * int(window) // 4))
        if chunk is None:
            chunk, max_chunks, waves = self.decode_chunk(n, num_heads, num_kv_heads, head_dim, max_ctx)
        else:
            waves = int(waves or 4)
            max_chunks = max(1, -(-max_ctx // int(chunk)))
        part_o = part_ml = None
        if max_chunks > 1:
            pairs = n * num_kv_heads
            G = num_heads // num_kv_heads
            part_o = torch.empty((pairs, max_chunks, G, head_dim), dtype=torch.float32, device=q.device)
            part_ml = torch.empty((pairs, max_chunks, G, 2), dtype=torch.float32, device=q.device)
        # every request of the step brings one token: token t is request t, and the kernel need not look it up
        one_each = token_list is None and batch.num_tokens == batch.num_seqs
        library.call("ra_attention_decode_mod", q.data_ptr(), q_stride, out.data_ptr(), out.stride(0),
                     kcache.data_ptr(), vcache.data_ptr(), tables.data_ptr(), tables.shape[1],
                     _ptr(token_list), None if one_each else batch.seq_of_token.data_ptr(), batch.positions.data_ptr(), n,
                     kcache.shape[2] * 16, num_heads, num_kv_heads, head_dim, float(scale), int(window), int(aligned),
                     int(keep), int(chunk), int(max_chunks), int(waves), _ptr(part_o), _ptr(part_ml), mod[0], mod[1], mod[2],
                     *head_out, _stream())

    def attention_prefill(self, q, q_stride, out, kcache, vcache, batch, num_heads, num_kv_heads, head_dim,
                          scale, window, group, tiles, n_tiles, ranges=None, merge=None, n_merge: int = 0,
                          n_slots: int = 0, mod=(0.0, None, None), keep: int = 0, aligned: bool = False,
                          head_out=(None, None, 0)) -> None:
        """``tiles``: four ints a listed query tile (request row, first token row, queries, first
        position). With ``ranges`` (three ints a listed tile: first key, one past the last, the part's
        slot or -1) some tiles are listed in several parts by keys, and ``merge`` (four ints a cut tile:
        first token row, queries, first slot, parts) says which to add up."""
        tables = self._check_attention(q, q_stride, out, kcache, vcache, batch, num_heads, num_kv_heads,
                                       head_dim, group)
        if q.dtype != torch.bfloat16:
            raise TypeError("attention_prefill: bfloat16 only")
        _int32(tiles, "query tiles", 4 * n_tiles)
        if ranges is not None:
            _int32(ranges, "key ranges", 3 * n_tiles)
            _int32(merge, "cut tiles", 4 * n_merge)
            if n_merge <= 0 or n_slots <= 0:
                raise ValueError("attention_prefill: key ranges without cut tiles")
            lib = library.load()
            part_o = torch.empty(int(lib.ra_attention_prefill_part_floats(num_heads, num_kv_heads, head_dim, n_slots, 0)),
                                 dtype=torch.float32, device=q.device)
            part_ml = torch.empty(int(lib.ra_attention_prefill_part_floats(num_heads, num_kv_heads, head_dim, n_slots, 1)),
                                  dtype=torch.float32, device=q.device)
            library.call("ra_attention_prefill_split_mod", q.data_ptr(), q_stride, out.data_ptr(), out.stride(0),
                         kcache.data_ptr(), vcache.data_ptr(), tables.data_ptr(), tables.shape[1],
                         tiles.data_ptr(), int(n_tiles), ranges.data_ptr(), merge.data_ptr(), int(n_merge),
                         part_o.data_ptr(), part_ml.data_ptr(), kcache.shape[2] * 16, num_heads, num_kv_heads,
                         head_dim, float(scale), int(window), int(aligned), int(keep), mod[0], mod[1], mod[2], *head_out,
                         _stream())
            return
        library.call("ra_attention_prefill_mod", q.data_ptr(), q_stride, out.data_ptr(), out.stride(0),
                     kcache.data_ptr(), vcache.data_ptr(), tables.data_ptr(), tables.shape[1],
                     tiles.data_ptr(), int(n_tiles), kcache.shape[2] * 16, num_heads, num_kv_heads, head_dim,
                     float(scale), int(window), int(aligned), int(keep), mod[0], mod[1], mod[2], *head_out, _stream())

    # ---------------------------------------------------------------- linear
    def linear(self, x: torch.Tensor, weight: torch.Tensor, out: torch.Tensor,
               bias: Optional[torch.Tensor] = None) -> None:
        """out[M, N] = x[M, K] . weight[N, K]^T (+ bias), float accumulation.

        bfloat16 with up to 64 rows: the weight-streaming MFMA kernel. bfloat16
        with more rows and a bfloat16 result: the library product (hipBLASLt
        through torch), as the reference calls cuBLAS for its prompt products
        (crates/cuda/src/gemm.rs:226-292). bfloat16 with more rows and a float
        result (the head's logits for more than 64 wanted rows): the library
        product again, bfloat16 operands and a float result.
        Everything else, all of float32 included: the plain FMA kernel.
        """
        if x.dtype == torch.bfloat16 and weight.dtype == torch.bfloat16:
            M, K = x.shape
            if M <= 64 and K % 8 == 0 and x.stride(0) % 8 == 0 and x.stride(1) == 1:
                return self.linear_skinny(x, weight, out, bias)
            if out.dtype == torch.bfloat16 and x.is_cuda:
                self._check_linear(x, weight, out, bias)
                if bias is None:
                    torch.mm(x, weight.t(), out=out)
                else:
                    torch.addmm(bias, x, weight.t(), out=out)
                return
            if out.dtype == torch.float32 and x.is_cuda:
                # the library's product with a float result: one pass over the weights (a head of 151936 x
                # 4096 at 128 rows: 285 us against 530 for two passes of the weight-streaming kernel)
                self._check_linear(x, weight, out, bias)
                torch.mm(x, weight.t(), out_dtype=torch.float32, out=out)
                if bias is not None:
                    out.add_(bias)
                return
        self.linear_plain(x, weight, out, bias)

    @staticmethod
    def _check_linear(x, weight, out, bias):
        _dev(x, weight, out, bias)
        M, K = x.shape
        N = weight.shape[0]
        if weight.shape != (N, K) or out.shape != (M, N) or x.dtype != weight.dtype:
            raise ValueError(f"linear: x {tuple(x.shape)} {x.dtype}, weight {tuple(weight.shape)} "
                             f"{weight.dtype}, out {tuple(out.shape)}")
        if x.stride(1) != 1 or out.stride(1) != 1 or not weight.is_contiguous():
            raise ValueError("linear: rows must be contiguous")
        if bias is not None and (bias.shape != (N,) or bias.dtype != weight.dtype):
            raise ValueError("linear: bias must be [N] in the weight's dtype")
        return M, N, K

    def linear_plain(self, x, weight, out, bias=None) -> None:
        M, N, K = self._check_linear(x, weight, out, bias)
        library.call("ra_gemm_plain", x.data_ptr(), weight.data_ptr(), _ptr(bias), out.data_ptr(),
                     _tag(x, "linear input"), _tag(out, "linear output"), M, N, K, x.stride(0),
                     out.stride(0), _stream())

    def linear_skinny(self, x, weight, out, bias=None, accumulate: bool = False, row_sums=None,
                      emit=None, wide: Optional[bool] = None, finish=None, alpha: float = 1.0):
        """The weight-streaming product; with ``accumulate`` the float32 ``out`` is added to (with more rows
        than the weight-streaming kernels take, by the library's product).

        An RMSNorm can ride on the products around it, y = rstd[m] * ((x .* w) . W^T):
        ``row_sums`` = (ss float32 [parts, M], eps, width) scales result row m by
        rsqrt(sum_p ss[p, m] / width + eps); ``emit`` = (w [N], x_out bfloat16 [M, N],
        ss_out float32 [at least skinny_row_parts(M, N), M]), with ``accumulate`` only, also writes
        bf16(out * w) and each workgroup's sums of squares of its columns of ``out``: into the first
        rows of ss_out, as many as the kernel that ran has workgroups a row; that number comes back.
        ``finish`` = (w [N], x_out bfloat16 [M, N], eps), with ``accumulate`` and 65 to 128 rows, asks for the
        finished norm of the new ``out`` instead, x_out = bf16(rmsnorm(out, eps) * w): True comes back where
        the product that ran wrote it (``can_finish_norm``), False where it only added.
        ``alpha`` (with ``accumulate`` alone): out += alpha * (x . W^T)."""
        M, N, K = self._check_linear(x, weight, out, bias)
        if alpha != 1.0:
            if not accumulate or bias is not None or row_sums is not None or emit is not None or finish is not None \
                    or x.dtype != torch.bfloat16 or out.dtype != torch.float32:
                raise ValueError("linear_skinny: a factor rides on a plain accumulating bfloat16 product only")
            lib = library.load()
            if M > 64 and not bool(lib.ra_gemm_wide_preferred(2, M, N, K)):
                torch.addmm(out, x, weight.t(), alpha=float(alpha), out_dtype=torch.float32, out=out)
                return None
            if wide is None:
                wide = bool(lib.ra_gemm_wide_preferred(2, M, N, K))
            if not wide:
                library.call("ra_gemm_skinny_scaled", x.data_ptr(), weight.data_ptr(), out.data_ptr(), M, N, K,
                             x.stride(0), out.stride(0), float(alpha), _stream())
                return None
            need = int(lib.ra_gemm_wide_scratch(2, M, N, K, 0))
            scratch = torch.empty(need, dtype=torch.float32, device=x.device) if need else None
            library.call("ra_gemm_wide_scaled", x.data_ptr(), weight.data_ptr(), out.data_ptr(), M, N, K, x.stride(0),
                         out.stride(0), _ptr(scratch), need, float(alpha), _stream())
            return None
        if x.dtype != torch.bfloat16:
            raise TypeError("linear_skinny: bfloat16 only")
        if accumulate and out.dtype != torch.float32:
            raise TypeError("linear_skinny: accumulation is into a float32 matrix")
        if finish is not None:
            if not accumulate or row_sums is not None or emit is not None:
                raise ValueError("linear_skinny: a finished norm rides on a plain accumulating product only")
            if self.can_finish_norm(M, N, K):
                w, xo, eps = finish
                _dev(w, xo)
                if w.shape != (N,) or not w.is_contiguous() or xo.dtype != torch.bfloat16 or xo.shape != (M, N) \
                        or xo.stride(1) != 1:
                    raise ValueError(f"linear_skinny: norm weight {tuple(w.shape)}, finished rows {tuple(xo.shape)} "
                                     f"{xo.dtype}; expected [{N}] and bfloat16 [{M}, {N}]")
                need = int(library.load().ra_gemm_wide_scratch(2, M, N, K, 1))
                scratch = torch.empty(need, dtype=torch.float32, device=x.device)
                library.call("ra_gemm_wide_normed", x.data_ptr(), weight.data_ptr(), _ptr(bias), out.data_ptr(),
                             _tag(out, "linear output"), 2, M, N, K, x.stride(0), out.stride(0), scratch.data_ptr(),
                             need, None, 0, 0.0, 0, w.data_ptr(), _tag(w, "norm weight"), xo.data_ptr(),
                             xo.stride(0), None, float(eps), _stream())
                return True
            self.linear_skinny(x, weight, out, bias, accumulate=True, wide=wide)
            return False
        if accumulate and M > 64 and bias is None and row_sums is None and emit is None and wide is None \
                and not bool(library.load().ra_gemm_wide_preferred(2, M, N, K)):
            # more rows than the weight-streaming kernels take: the library's product, adding in place
            torch.addmm(out, x, weight.t(), out_dtype=torch.float32, out=out)
            return None
        if row_sums is None and emit is None:
            self._few_rows("linear output", x, weight, bias, out, 2 if accumulate else 0, M, N, K, wide)
            return None
        return self._skinny_normed(x, weight, bias, out, 2 if accumulate else 0, M, N, K, row_sums, emit)

    # Rows up to which an RMSNorm rides on the products around it (``row_sums`` / ``emit``) rather
    # than running as a kernel of its own: all that the weight-streaming products take. Up to 16
    # rows the kernel whose waves split K carries it, above that the other one, which has the
    # registers to spare (the first, at 32 and 64 rows, got slower than with a norm kernel).
    NORM_ON_PRODUCTS_ROWS = 64
    NORM_SKINNY_ROWS = 16
    # Rows up to which the adding kernel of a product cut into K ranges can finish the norm that follows
    # (a whole row a workgroup): the decode steps above the weight-streaming products' rows, whose other
    # products are the library's and can apply no row factor.
    NORM_FINISHED_ROWS = 128

    def can_finish_norm(self, M: int, N: int, K: int) -> bool:
        """True where ``linear_skinny(..., accumulate=True, finish=)`` writes the finished norm: the rows
        between the two limits, a product that the kernel with K ranges takes at these rows, rows of up to
        16384 columns in steps of 8."""
        return self.NORM_ON_PRODUCTS_ROWS < M <= self.NORM_FINISHED_ROWS and N % 8 == 0 and N <= 16384 \
            and K % 8 == 0 and bool(library.load().ra_gemm_wide_preferred(2, M, N, K))

    def _few_rows(self, what, x, weight, bias, out, epilogue, M, N, K, wide: Optional[bool] = None) -> None:
        """The weight-streaming product for up to 64 rows, by one of two kernels: the one whose
        waves split K (best up to 16 rows) or the one whose waves share the activations (it may
        need scratch for partial sums). ``wide`` forces the choice; the library knows where each
        is faster."""
        lib = library.load()
        if wide is None:
            wide = bool(lib.ra_gemm_wide_preferred(epilogue, M, N, K))
        if not wide:
            library.call("ra_gemm_skinny", x.data_ptr(), weight.data_ptr(), _ptr(bias), out.data_ptr(),
                         _tag(out, what), epilogue, M, N, K, x.stride(0), out.stride(0), _stream())
            return
        need = int(lib.ra_gemm_wide_scratch(epilogue, M, N, K, 0))
        scratch = torch.empty(need, dtype=torch.float32, device=x.device) if need else None
        library.call("ra_gemm_wide", x.data_ptr(), weight.data_ptr(), _ptr(bias), out.data_ptr(),
                     _tag(out, what), epilogue, M, N, K, x.stride(0), out.stride(0), _ptr(scratch), need,
                     _stream())

    def skinny_row_parts(self, M: int, N: int) -> int:
        """Partial sums a row that ``linear_skinny(..., emit=)`` writes for an [M, N] result at most:
        which of the two kernels runs, and with it the number, depends on the product's K as well."""
        lib = library.load()
        return max(int(lib.ra_gemm_skinny_row_parts(int(M), int(N))), int(lib.ra_gemm_wide_row_parts(int(N))))

    def _emits_from_skinny(self, epilogue: int, M: int, N: int, K: int) -> bool:
        """Whether an emitting product goes to the kernel whose waves split K: up to 16 rows always; up to
        32 where the other kernel would have to cut K into ranges and add them with a second launch for a
        small product (an output projection of 4096 x 4096 at 32 rows: 10 us against 16; the decode step of
        32 requests 6.19 -> 6.01 ms). With more rows the step gains nothing from it (33 and 64 requests:
        within 0.5 %), and the consumer has 16 times the partial sums to add."""
        if M <= self.NORM_SKINNY_ROWS:
            return True
        lib = library.load()
        return M <= 32 and not bool(lib.ra_gemm_wide_preferred(epilogue, M, N, K)) \
            and int(lib.ra_gemm_skinny_row_parts(M, N)) * 16 == N

    def _skinny_normed(self, x, weight, bias, out, epilogue, M, N, K, row_sums, emit) -> None:
        ss = eps = width = None
        parts = 0
        if row_sums is not None:
            ss, eps, width = row_sums
            _dev(ss)
            if ss.dtype != torch.float32 or ss.dim() != 2 or ss.shape[1] != M or not ss.is_contiguous():
                raise ValueError(f"linear_skinny: row sums {tuple(ss.shape)} {ss.dtype}, expected float32 [parts, {M}]")
            parts = ss.shape[0]
        w = xo = so = None
        parts_out = None
        if emit is not None:
            if epilogue != 2:
                raise ValueError("linear_skinny: only an accumulating product emits for a norm")
            w, xo, so = emit
            _dev(w, xo, so)
            lib = library.load()
            parts_out = int(lib.ra_gemm_skinny_row_parts(M, N)) if self._emits_from_skinny(epilogue, M, N, K) \
                else int(lib.ra_gemm_wide_row_parts(N))
            if w.shape != (N,) or not w.is_contiguous():
                raise ValueError(f"linear_skinny: norm weight {tuple(w.shape)}, expected [{N}]")
            if xo.dtype != torch.bfloat16 or xo.shape != (M, N) or xo.stride(1) != 1:
                raise ValueError(f"linear_skinny: scaled copy {tuple(xo.shape)} {xo.dtype}, expected bfloat16 [{M}, {N}]")
            if so.dtype != torch.float32 or so.dim() != 2 or so.shape[0] < parts_out or so.shape[1] != M or not so.is_contiguous():
                raise ValueError(f"linear_skinny: emitted sums {tuple(so.shape)}, expected float32 [{parts_out} or more, {M}]")
        norm_args = (_ptr(ss), parts, float(eps or 0.0), int(width or 0), _ptr(w),
                     _tag(w, "norm weight") if w is not None else 0, _ptr(xo),
                     xo.stride(0) if xo is not None else 0, _ptr(so))
        # the gated product of a wide feed-forward goes to the other kernel at every row count; it
        # takes row sums (any number of parts) and never emits
        gated_wide = epilogue == 1 and emit is None and bool(library.load().ra_gemm_wide_preferred(epilogue, M, N, K))
        to_skinny = self._emits_from_skinny(epilogue, M, N, K) if emit is not None else M <= self.NORM_SKINNY_ROWS
        if to_skinny and not gated_wide:
            library.call("ra_gemm_skinny_normed", x.data_ptr(), weight.data_ptr(), _ptr(bias), out.data_ptr(),
                         _tag(out, "linear output"), epilogue, M, N, K, x.stride(0), out.stride(0), *norm_args,
                         _stream())
            return parts_out
        need = int(library.load().ra_gemm_wide_scratch(epilogue, M, N, K, 1 if emit is not None else 0))
        scratch = torch.empty(need, dtype=torch.float32, device=x.device) if need else None
        library.call("ra_gemm_wide_normed", x.data_ptr(), weight.data_ptr(), _ptr(bias), out.data_ptr(),
                     _tag(out, "linear output"), epilogue, M, N, K, x.stride(0), out.stride(0), _ptr(scratch),
                     need, *norm_args, -1.0, _stream())
        return parts_out

    def can_accumulate(self, x: torch.Tensor, weight: torch.Tensor) -> bool:
        """True if ``linear_skinny(..., accumulate=True)`` takes this product (out += x . W^T):
        the residual add of an output projection then costs no kernel and no round trip."""
        if not (x.is_cuda and x.dtype == torch.bfloat16 and weight.dtype == torch.bfloat16
                and x.shape[1] % 8 == 0 and x.stride(0) % 8 == 0 and x.stride(1) == 1):
            return False
        M, K = x.shape
        # above 64 rows where the kernel that cuts K into ranges beats the library's product and an add,
        # or where the library's own product adds into the float matrix
        return M <= 64 or self.LIBRARY_ACCUMULATES_FROM <= M <= self.LIBRARY_ACCUMULATES_ROWS \
            or bool(library.load().ra_gemm_wide_preferred(2, M, weight.shape[0], K))

    # Rows up to which the library's product adds into the float residual stream itself (bfloat16 operands, a
    # float matrix read and written): up to here it takes as long as the product with a bfloat16 result
    # (2048 rows, 4096 x 4096: 67 against 69 us; 4096 x 12288: 187 against 191), and the norm kernel behind it
    # reads one matrix less (3072 rows: 95 against 85 and 248 against 275 us); from 4096 rows on it is the slower one
    # (4096: 116 against 95 and 314 against 279 us; 8192: 218 against 179, 620 against 539).
    # Below 129 rows (decode steps of 65 to 128 requests) it is a wash (a step of 96 requests 11.78 against
    # 11.69 ms with the norm kernel's add, of 128 requests 14.28 against 14.36): those steps stay as they were.
    LIBRARY_ACCUMULATES_FROM = 129
    LIBRARY_ACCUMULATES_ROWS = 3072

    GATE_GROUP = 8        # rows of gate, then rows of up, in the weight of gated_linear

    def gated_linear(self, x: torch.Tensor, weight: torch.Tensor, out: torch.Tensor, row_sums=None,
                     wide: Optional[bool] = None) -> None:
        """out[M, I] = silu(x . Wg^T) * (x . Wu^T) for ``weight`` [2I, K] whose rows alternate in
        runs of GATE_GROUP: 8 gate rows, the 8 up rows of the same features, and so on.

        bfloat16 with up to 64 rows: one kernel, the gate applied in the product's
        epilogue. Otherwise the product into a [M, 2I] buffer, then the gate kernel."""
        _dev(x, weight, out)
        M, K = x.shape
        I = out.shape[1]
        if weight.shape != (2 * I, K) or out.shape != (M, I) or I % self.GATE_GROUP != 0:
            raise ValueError(f"gated_linear: x {tuple(x.shape)}, weight {tuple(weight.shape)}, out {tuple(out.shape)}")
        if x.dtype == torch.bfloat16 and weight.dtype == torch.bfloat16 and out.dtype == torch.bfloat16 \
                and M <= 64 and K % 8 == 0 and x.stride(0) % 8 == 0 and x.stride(1) == 1 \
                and weight.is_contiguous() and out.stride(1) == 1:
            if row_sums is None:
                self._few_rows("linear output", x, weight, None, out, 1, M, 2 * I, K, wide)
            else:
                self._skinny_normed(x, weight, None, out, 1, M, 2 * I, K, row_sums, None)
            return
        if row_sums is not None:
            raise ValueError("gated_linear: row sums ride on the weight-streaming product only (bfloat16, <= 64 rows)")
        gu = torch.empty((M, 2 * I), dtype=out.dtype, device=x.device)
        self.linear(x, weight, gu)
        self.silu_mul(gu, out, self.GATE_GROUP)

    # ------------------------------------------------- around the stream
    def pair_hash_add(self, resid: torch.Tensor, table: torch.Tensor, batch, last_token: torch.Tensor,
                      buckets: int, mul_prev: int, mul_cur: int) -> None:
        """resid[t] += table[(prev * mul_prev + id * mul_cur) mod buckets], or the table's last row (number
        ``buckets``) for a request's first token. The token before a portion's first is read from
        ``last_token[state slot]`` (int32, one word a request slot), which then takes the portion's last token."""
        _dev(resid, table, last_token)
        T, h = resid.shape
        if T != batch.num_tokens or resid.dtype != torch.float32 or not resid.is_contiguous():
            raise TypeError("pair_hash_add: the residual stream is contiguous float32, one row a token of the step")
        if table.shape != (buckets + 1, h) or not table.is_contiguous():
            raise ValueError(f"pair_hash_add: table {tuple(table.shape)}, expected [{buckets + 1}, {h}]")
        _int32(last_token, "pair_hash_add state")
        slots_needed = int(last_token.numel())
        if slots_needed <= 0:
            raise ValueError("pair_hash_add: no state words")
        _int32(batch.token_ids, "token ids", T)
        _int32(batch.positions, "positions", T)
        _int32(batch.seq_of_token, "request of each token", T)
        _int32(batch.cu_tokens, "first token of each request", batch.num_seqs + 1)
        _int32(batch.state_slots, "state slots", batch.num_seqs)
        library.call("ra_pair_hash_add", resid.data_ptr(), table.data_ptr(), _tag(table, "pair table"),
                     batch.token_ids.data_ptr(), batch.positions.data_ptr(), batch.seq_of_token.data_ptr(),
                     batch.cu_tokens.data_ptr(), batch.state_slots.data_ptr(), last_token.data_ptr(), int(buckets),
                     int(mul_prev), int(mul_cur), T, h, _stream())

    def stream_add(self, resid: torch.Tensor, delta: Optional[torch.Tensor] = None,
                   other: Optional[torch.Tensor] = None, vec: Optional[torch.Tensor] = None,
                   delta_scale: float = 1.0) -> None:
        """resid += delta_scale * delta + other + vec: ``delta`` [T, width] in either dtype, ``other`` [T, width]
        float32, ``vec`` [width] in either dtype; each may be None."""
        _dev(resid, delta, other, vec)
        T, h = resid.shape
        if resid.dtype != torch.float32 or not resid.is_contiguous():
            raise TypeError("stream_add: the residual stream is contiguous float32")
        if delta is not None and (delta.shape != resid.shape or not delta.is_contiguous()):
            raise ValueError("stream_add: delta must match the residual's shape")
        if other is not None and (other.shape != resid.shape or other.dtype != torch.float32 or not other.is_contiguous()):
            raise ValueError("stream_add: the second addend is a float32 matrix of the residual's shape")
        if vec is not None and (vec.shape != (h,) or not vec.is_contiguous()):
            raise ValueError(f"stream_add: vector {tuple(vec.shape)}, expected [{h}]")
        if delta is None and other is None and vec is None:
            return
        library.call("ra_stream_add", resid.data_ptr(), _ptr(delta), _tag(delta, "stream_add delta") if delta is not None else 0,
                     _ptr(other), _ptr(vec), _tag(vec, "stream_add vector") if vec is not None else 0, T, h,
                     float(delta_scale), _stream())

    def tanh_cap(self, logits: torch.Tensor, cap: float) -> None:
        """logits <- cap * tanh(logits / cap), in place."""
        _dev(logits)
        if logits.dtype != torch.float32 or logits.dim() != 2 or logits.stride(1) != 1:
            raise TypeError("tanh_cap: logits are float32 rows")
        if logits.shape[0] == 0:
            return
        library.call("ra_tanh_cap", logits.data_ptr(), logits.shape[0], logits.shape[1], logits.stride(0),
                     float(cap), _stream())

    # ------------------------------------------------------ latent attention
    def latent_prep(self, proj: torch.Tensor, q_off: int, dkv_off: int, c_weight: torch.Tensor, eps: float,
                    positions: torch.Tensor, inv_freq: torch.Tensor, rot_dims: int, rot_width: int, rank: int,
                    num_heads: int, head_dim: int, q_lat: torch.Tensor, slots: torch.Tensor,
                    kcache: torch.Tensor, vcache: torch.Tensor, rope_style: int = 0, amp: float = 1.0) -> None:
        """Norm of the latent, rotation of the shared key part and of the queries' rotated parts, cache write.

        ``proj`` [T, *] holds the query heads ([head_dim | rot_width] each) from column ``q_off`` and
        [latent (rank) | key part (rot_width)] from ``dkv_off``. The cache row of a token,
        [rms(latent) * c_weight | rotated key part | zeros], goes to ``kcache`` / ``vcache`` (one KV head of
        size Dp = q_lat.shape[2]) at ``slots``; ``q_lat`` [T, heads, Dp] gets its columns from ``rank`` on. Pairs are half-split
        (``rope_style`` 0) or neighbours (1); sine and cosine are multiplied by ``amp``."""
        _dev(proj, c_weight, positions, inv_freq, q_lat, slots, kcache, vcache)
        T = proj.shape[0]
        if proj.dim() != 2 or proj.stride(1) != 1:
            raise ValueError("latent_prep: projection rows must be contiguous")
        if q_lat.dim() != 3 or q_lat.shape[:2] != (T, num_heads) or not q_lat.is_contiguous() or q_lat.dtype != proj.dtype:
            raise ValueError(f"latent_prep: q_lat {tuple(q_lat.shape)}, expected [{T}, {num_heads}, Dp] in the activations' dtype")
        Dp = q_lat.shape[2]
        self._check_cache("latent_prep", kcache, vcache, 1, Dp)
        if kcache.dtype != proj.dtype or vcache.dtype != proj.dtype:
            raise TypeError("latent_prep: the cache has the activations' dtype")
        if c_weight.shape != (rank,) or not c_weight.is_contiguous():
            raise ValueError(f"latent_prep: norm weight {tuple(c_weight.shape)}, expected [{rank}]")
        _int32(positions, "positions", T)
        _int32(slots, "cache slots", T)
        if inv_freq.dtype != torch.float32 or inv_freq.numel() < max(1, rot_dims // 2):
            raise ValueError("latent_prep: inv_freq is float32 with rot_dims/2 entries")
        library.call("ra_latent_prep", proj.data_ptr(), _tag(proj, "latent_prep"), proj.stride(0), int(q_off),
                     int(dkv_off), c_weight.data_ptr(), _tag(c_weight, "latent norm weight"), float(eps),
                     positions.data_ptr(), inv_freq.data_ptr(), int(rot_dims), int(rope_style), float(amp), int(rot_width), int(rank),
                     int(num_heads), int(head_dim), q_lat.data_ptr(), Dp, slots.data_ptr(), kcache.data_ptr(),
                     vcache.data_ptr(), kcache.shape[2] * 16, T, _stream())

    def head_linear(self, x: torch.Tensor, x_head: int, weight: torch.Tensor, out: torch.Tensor, o_head: int,
                    gate: Optional[torch.Tensor] = None, gate_per_head: bool = False) -> None:
        """Products head by head: out[t, h * o_head + n] = sum_k x[t, h * x_head + k] * weight[h, n, k], times
        sigmoid(gate[t, h * N + n]) where a gate is given. ``x``, ``out`` and ``gate`` are 2-D with unit
        column stride (they may be column ranges of wider buffers); ``weight`` is [heads, N, K] contiguous.
        bfloat16 with K and the strides of ``x`` in steps of 8: matrix cores; else a plain kernel."""
        _dev(x, weight, out, gate)
        H, N, K = weight.shape
        T = x.shape[0]
        if not weight.is_contiguous() or x.dtype != weight.dtype or out.dtype != weight.dtype:
            raise ValueError("head_linear: weight [heads, N, K] contiguous, all in one dtype")
        for t, what in ((x, "x"), (out, "out"), (gate, "gate")):
            if t is not None and (t.dim() != 2 or t.shape[0] != T or t.stride(1) != 1 or t.dtype != weight.dtype):
                raise ValueError(f"head_linear: {what} must be [T, *] rows of the weight's dtype with unit column stride")
        if x.shape[1] < (H - 1) * x_head + K or out.shape[1] < (H - 1) * o_head + N or o_head < N:
            raise ValueError(f"head_linear: x {tuple(x.shape)} / out {tuple(out.shape)} do not hold {H} heads of {K} / {N}")
        if gate is not None and gate.shape[1] < (H if gate_per_head else H * N):
            raise ValueError(f"head_linear: gate {tuple(gate.shape)}, expected [T, {H if gate_per_head else H * N}]")
        library.call("ra_head_linear", x.data_ptr(), x.stride(0), int(x_head), weight.data_ptr(), out.data_ptr(),
                     out.stride(0), int(o_head), _ptr(gate), gate.stride(0) if gate is not None else 0,
                     1 if gate_per_head else 0, _tag(x, "head_linear"), T, H, N, K, _stream())

    # ------------------------------------------------------ recurrent mixers
    _SCAN_KINDS = {"matrix_memory": 0, "delta_rule": 1, "wkv": 2, "decay_memory": 3, "gated_linear": 4}

    def scan_state_floats(self, kind: str, heads: int, key_dim: int, value_dim: int) -> int:
        """Floats of a request's state slot that the scan kernel of ``kind`` ("matrix_memory", "delta_rule", "wkv")
        keeps for ``heads`` heads of [key_dim, value_dim], in the kernel's own layout."""
        n = int(library.load().ra_scan_state_floats(self._SCAN_KINDS[kind], int(heads), int(key_dim), int(value_dim)))
        if n < 0:
            raise ValueError(f"{kind}: heads of {key_dim} x {value_dim} are not taken (keys up to 512)")
        return n

    @staticmethod
    def _check_scan(what: str, state: torch.Tensor, batch, T: int) -> None:
        if state.dtype != torch.float32 or state.dim() != 2 or not state.is_contiguous():
            raise TypeError(f"{what}: the state is contiguous float32 [slots, floats]")
        if T != batch.num_tokens:
            raise ValueError(f"{what}: {T} rows for a step of {batch.num_tokens} tokens")
        _int32(batch.cu_tokens, "first token of each request", batch.num_seqs + 1)
        _int32(batch.state_slots, "state slots", batch.num_seqs)
        _int32(batch.fresh, "first-step flags", batch.num_seqs)
        _int32(batch.seq_of_token, "request of each token", T)

    def matrix_memory_scan(self, proj: torch.Tensor, q_off: int, k_off: int, v_off: int, gates: torch.Tensor,
                           gate_bias: torch.Tensor, state: torch.Tensor, batch, heads: int, key_dim: int,
                           value_dim: int, gate_cap: float, q_scale: float, denom_eps: float,
                           out: torch.Tensor) -> None:
        """The matrix memory over the step's tokens, request by request in order, from and into ``state``
        [slots, floats]. ``proj`` [T, *] holds q and k (heads x key_dim) and v (heads x value_dim) from the
        given columns; ``gates`` float32 [T, 2 heads] holds the input and forget gates' pre-activations;
        ``out`` float32 [T, heads * value_dim] gets the read-out before its norm."""
        _dev(proj, gates, gate_bias, state, out)
        T = proj.shape[0]
        self._check_scan("matrix_memory_scan", state, batch, T)
        if proj.dim() != 2 or proj.stride(1) != 1 or max(q_off, k_off) + heads * key_dim > proj.shape[1] \
                or v_off + heads * value_dim > proj.shape[1]:
            raise ValueError(f"matrix_memory_scan: rows of {tuple(proj.shape)} do not hold q, k, v at {q_off}, {k_off}, {v_off}")
        if gates.shape != (T, 2 * heads) or gates.dtype != torch.float32 or not gates.is_contiguous() \
                or gate_bias.shape != (2 * heads,) or gate_bias.dtype != torch.float32 or not gate_bias.is_contiguous():
            raise ValueError("matrix_memory_scan: gates float32 [T, 2 heads], their bias float32 [2 heads]")
        if out.shape != (T, heads * value_dim) or out.dtype != torch.float32 or not out.is_contiguous():
            raise ValueError("matrix_memory_scan: out is contiguous float32 [T, heads * value_dim]")
        factors = torch.empty((T, 3 * heads), dtype=torch.float32, device=proj.device)     # decay, input, threshold
        library.call("ra_matrix_memory_scan", proj.data_ptr(), _tag(proj, "matrix_memory_scan"), proj.stride(0),
                     int(q_off), int(k_off), int(v_off), gates.data_ptr(), factors.data_ptr(), gate_bias.data_ptr(),
                     state.data_ptr(),
                     state.stride(0), batch.cu_tokens.data_ptr(), batch.state_slots.data_ptr(), batch.fresh.data_ptr(),
                     batch.num_seqs, T, int(getattr(batch, "max_q_len", 0) or 0), int(heads), int(key_dim),
                     int(value_dim), float(gate_cap), float(q_scale), float(denom_eps), out.data_ptr(), _stream())

    def delta_rule_prepare(self, proj: torch.Tensor, filt: torch.Tensor, state: torch.Tensor, tail_off: int, batch,
                           key_heads: int, key_dim: int, heads: int, value_dim: int, taps: int, unit_eps: float,
                           q_scale: float, qkv: torch.Tensor) -> None:
        """The delta rule's inputs: the causal filter over time (``filt`` float32 [channels, taps]; rows before
        the step's portion come from the ``taps - 1`` rows kept at ``tail_off`` in the request's state, which
        then move on), silu, unit norms of the q and k heads. ``proj`` [T, >= channels] holds q | k | v from
        column 0; ``qkv`` float32 [T, channels] gets the results."""
        _dev(proj, filt, state, qkv)
        T = proj.shape[0]
        C = 2 * key_heads * key_dim + heads * value_dim
        self._check_scan("delta_rule_prepare", state, batch, T)
        if proj.dim() != 2 or proj.stride(1) != 1 or proj.shape[1] < C:
            raise ValueError(f"delta_rule_prepare: rows of {tuple(proj.shape)} do not hold {C} channels")
        if filt.shape != (C, taps) or filt.dtype != torch.float32 or not filt.is_contiguous():
            raise ValueError(f"delta_rule_prepare: filter {tuple(filt.shape)} {filt.dtype}, expected float32 [{C}, {taps}]")
        if qkv.shape != (T, C) or qkv.dtype != torch.float32 or not qkv.is_contiguous():
            raise ValueError(f"delta_rule_prepare: qkv is contiguous float32 [T, {C}]")
        if state.shape[1] < tail_off + (taps - 1) * C:
            raise ValueError("delta_rule_prepare: the state slot does not hold the filter's tail")
        library.call("ra_delta_rule_prepare", proj.data_ptr(), _tag(proj, "delta_rule_prepare"), proj.stride(0),
                     filt.data_ptr(), state.data_ptr(), state.stride(0), int(tail_off), batch.seq_of_token.data_ptr(),
                     batch.cu_tokens.data_ptr(), batch.state_slots.data_ptr(), batch.fresh.data_ptr(), batch.num_seqs,
                     T, int(key_heads), int(key_dim), int(heads), int(value_dim), int(taps), float(unit_eps),
                     float(q_scale), qkv.data_ptr(), _stream())

    def delta_rule_scan(self, qkv: torch.Tensor, gates: torch.Tensor, a_log: torch.Tensor, dt_bias: torch.Tensor,
                        state: torch.Tensor, batch, heads: int, key_heads: int, key_dim: int, value_dim: int,
                        out: torch.Tensor) -> None:
        """The gated delta rule over the step's tokens from and into ``state``. ``qkv`` float32 [T, q | k | v]
        as ``delta_rule_prepare`` left it; ``gates`` float32 [T, 2 heads] holds the pre-activations of beta
        and of the decay and is overwritten with both; ``out`` float32 [T, heads * value_dim]."""
        _dev(qkv, gates, a_log, dt_bias, state, out)
        T = qkv.shape[0]
        C = 2 * key_heads * key_dim + heads * value_dim
        self._check_scan("delta_rule_scan", state, batch, T)
        if qkv.shape != (T, C) or qkv.dtype != torch.float32 or not qkv.is_contiguous():
            raise ValueError(f"delta_rule_scan: qkv is contiguous float32 [T, {C}]")
        if gates.shape != (T, 2 * heads) or gates.dtype != torch.float32 or not gates.is_contiguous():
            raise ValueError("delta_rule_scan: gates float32 [T, 2 heads]")
        for v, what in ((a_log, "A_log"), (dt_bias, "dt_bias")):
            if v.shape != (heads,) or v.dtype != torch.float32 or not v.is_contiguous():
                raise ValueError(f"delta_rule_scan: {what} is float32 [heads]")
        if out.shape != (T, heads * value_dim) or out.dtype != torch.float32 or not out.is_contiguous():
            raise ValueError("delta_rule_scan: out is contiguous float32 [T, heads * value_dim]")
        library.call("ra_delta_rule_scan", qkv.data_ptr(), qkv.stride(0), gates.data_ptr(), a_log.data_ptr(),
                     dt_bias.data_ptr(), state.data_ptr(), state.stride(0), batch.cu_tokens.data_ptr(),
                     batch.state_slots.data_ptr(), batch.fresh.data_ptr(), batch.num_seqs, T,
                     int(getattr(batch, "max_q_len", 0) or 0), int(heads), int(key_heads), int(key_dim), int(value_dim),
                     out.data_ptr(), _stream())

    def wkv_scan(self, proj: torch.Tensor, r_off: int, k_off: int, v_off: int, decay: torch.Tensor, w0: torch.Tensor,
                 u: torch.Tensor, state: torch.Tensor, batch, heads: int, dim: int, out: torch.Tensor) -> None:
        """A per-head matrix state with a decay a key channel and token, from and into ``state`` [slots, floats]:
        o = (S + diag(u) k v^T)^T r, then S <- diag(w) S + k v^T with w = exp(-exp(decay + w0)). ``proj`` [T, *]
        holds r, k, v (heads x dim each) from the given columns; ``decay`` float32 [T, heads * dim] the decays'
        pre-activations; ``w0`` and ``u`` float32 [heads * dim]; ``out`` float32 [T, heads * dim]."""
        _dev(proj, decay, w0, u, state, out)
        T = proj.shape[0]
        n = heads * dim
        self._check_scan("wkv_scan", state, batch, T)
        if proj.dim() != 2 or proj.stride(1) != 1 or max(r_off, k_off, v_off) + n > proj.shape[1]:
            raise ValueError(f"wkv_scan: rows of {tuple(proj.shape)} do not hold r, k, v at {r_off}, {k_off}, {v_off}")
        if decay.dim() != 2 or decay.shape[0] != T or decay.shape[1] < n or decay.dtype != torch.float32 \
                or decay.stride(1) != 1:
            raise ValueError(f"wkv_scan: decay pre-activations are float32 [T, {n}]")
        for v, what in ((w0, "w0"), (u, "u")):
            if v.shape != (n,) or v.dtype != torch.float32 or not v.is_contiguous():
                raise ValueError(f"wkv_scan: {what} is float32 [{n}]")
        if out.shape != (T, n) or out.dtype != torch.float32 or not out.is_contiguous():
            raise ValueError("wkv_scan: out is contiguous float32 [T, heads * dim]")
        library.call("ra_wkv_scan", proj.data_ptr(), _tag(proj, "wkv_scan"), proj.stride(0), int(r_off), int(k_off),
                     int(v_off), decay.data_ptr(), decay.stride(0), w0.data_ptr(), u.data_ptr(), state.data_ptr(),
                     state.stride(0), batch.cu_tokens.data_ptr(), batch.state_slots.data_ptr(), batch.fresh.data_ptr(),
                     batch.num_seqs, T, int(getattr(batch, "max_q_len", 0) or 0), int(heads), int(dim), out.data_ptr(),
                     _stream())

    # ------------------------------------------- the token before, gated adds
    def token_shift(self, h: torch.Tensor, mu: torch.Tensor, state: torch.Tensor, keep_off: int, batch,
                    out: torch.Tensor) -> None:
        """out[t, j * width + e] = h[t, e] + (prev(t)[e] - h[t, e]) * mu[j, e]: every row mixed with the row of
        the token before it, once for each row of ``mu`` [n_mix, width]. The row before a portion's first comes
        from ``state`` [slots, floats] at ``keep_off`` (zeros at a request's start), which then takes the
        portion's last row; the kept row is float and holds the activations' values exactly."""
        _dev(h, mu, state, out)
        T, width = h.shape
        if mu.dim() != 2 or mu.shape[1] != width or not mu.is_contiguous():
            raise ValueError(f"token_shift: factors {tuple(mu.shape)}, expected [mixes, {width}]")
        n_mix = mu.shape[0]
        if h.stride(1) != 1 or out.shape != (T, n_mix * width) or out.stride(1) != 1 or out.dtype != h.dtype:
            raise ValueError(f"token_shift: out {tuple(out.shape)}, expected [{T}, {n_mix * width}] in the input's dtype")
        if state.shape[1] < keep_off + width:
            raise ValueError("token_shift: the state slot does not hold the kept row")
        self._check_scan("token_shift", state, batch, T)
        single = 1 if int(getattr(batch, "max_q_len", 0) or 0) == 1 else 0
        library.call("ra_token_shift", h.data_ptr(), h.stride(0), mu.data_ptr(), _tag(mu, "token_shift factors"), n_mix,
                     state.data_ptr(), state.stride(0), int(keep_off), batch.seq_of_token.data_ptr(),
                     batch.cu_tokens.data_ptr(), batch.state_slots.data_ptr(), batch.fresh.data_ptr(), out.data_ptr(),
                     out.stride(0), _tag(h, "token_shift"), batch.num_seqs, T, width, single, _stream())

    def gated_stream_add(self, resid: torch.Tensor, gates: torch.Tensor, a: torch.Tensor,
                         b: Optional[torch.Tensor] = None) -> None:
        """resid += sigmoid(gates[:, :width]) * a + sigmoid(gates[:, width:2 width]) * b, element by element, in
        float; ``gates`` holds the pre-activations, ``b`` may be None."""
        _dev(resid, gates, a, b)
        T, width = resid.shape
        if resid.dtype != torch.float32 or not resid.is_contiguous():
            raise TypeError("gated_stream_add: the residual stream is contiguous float32")
        need = (2 if b is not None else 1) * width
        if gates.dim() != 2 or gates.shape[0] != T or gates.shape[1] < need or gates.stride(1) != 1:
            raise ValueError(f"gated_stream_add: gates {tuple(gates.shape)}, expected [{T}, >= {need}]")
        for t in (a, b):
            if t is not None and (t.shape != (T, width) or not t.is_contiguous()):
                raise ValueError("gated_stream_add: addends are contiguous [T, width]")
        library.call("ra_gated_stream_add", resid.data_ptr(), gates.data_ptr(), gates.stride(0), _tag(gates, "gates"),
                     a.data_ptr(), _tag(a, "addend"), _ptr(b), _tag(b, "addend") if b is not None else 0, T, width,
                     _stream())

    def rows_rmsnorm(self, x: torch.Tensor, weight: torch.Tensor, eps: float, out: torch.Tensor) -> None:
        """out = x / sqrt(mean(x^2) + eps) * weight over rows of activations (either may be a column range of a
        wider buffer); the sums are float."""
        _dev(x, weight, out)
        T, width = x.shape
        if out.shape != (T, width) or out.dtype != x.dtype or x.stride(1) != 1 or out.stride(1) != 1:
            raise ValueError(f"rows_rmsnorm: x {tuple(x.shape)} against out {tuple(out.shape)}")
        if weight.shape != (width,) or not weight.is_contiguous():
            raise ValueError(f"rows_rmsnorm: weight {tuple(weight.shape)}, expected [{width}]")
        library.call("ra_rows_rmsnorm", x.data_ptr(), x.stride(0), weight.data_ptr(), _tag(weight, "norm weight"),
                     out.data_ptr(), out.stride(0), _tag(x, "rows_rmsnorm"), T, width, float(eps), _stream())

    def tanh_rows(self, x: torch.Tensor) -> None:
        """x <- tanh(x), in place."""
        _dev(x)
        if not x.is_contiguous():
            raise ValueError("tanh_rows: a contiguous tensor")
        library.call("ra_tanh_rows", x.data_ptr(), _tag(x, "tanh_rows"), x.numel(), _stream())

    def head_norm_gate(self, read: torch.Tensor, weight: Optional[torch.Tensor], per_head: bool, gate: torch.Tensor, kind: str,
                       eps: float, heads: int, value_dim: int, out: torch.Tensor) -> None:
        """out[t, h] = read[t, h] / rms(read[t, h]) * weight * act(gate[t, h]) head by head: ``read`` float32
        [T, heads * value_dim], ``weight`` float32 [heads * value_dim] (``per_head``) or [value_dim] for all
        heads or None, ``gate`` [T, >= heads * value_dim] rows of the activations' dtype, ``kind`` "sigmoid" or "silu"."""
        _dev(read, weight, gate, out)
        T = read.shape[0]
        n = heads * value_dim
        if read.shape != (T, n) or read.dtype != torch.float32 or not read.is_contiguous():
            raise ValueError(f"head_norm_gate: read is contiguous float32 [T, {n}]")
        if weight is not None and (weight.dtype != torch.float32 or not weight.is_contiguous()
                                   or weight.shape != ((n,) if per_head else (value_dim,))):
            raise ValueError(f"head_norm_gate: weight {tuple(weight.shape)} {weight.dtype}")
        if gate.dim() != 2 or gate.shape[0] != T or gate.shape[1] < n or gate.stride(1) != 1 or gate.dtype != out.dtype:
            raise ValueError(f"head_norm_gate: gate {tuple(gate.shape)}, expected rows of at least {n} in the output's dtype")
        if out.shape != (T, n) or not out.is_contiguous():
            raise ValueError(f"head_norm_gate: out is contiguous [T, {n}]")
        if kind not in ("sigmoid", "silu"):
            raise ValueError(f"head_norm_gate: gate kind {kind!r}")
        library.call("ra_head_norm_gate", read.data_ptr(), _ptr(weight), 1 if per_head else 0, gate.data_ptr(),
                     gate.stride(0), _tag(out, "head_norm_gate"), 1 if kind == "silu" else 0, float(eps), T, int(heads),
                     int(value_dim), out.data_ptr(), _stream())

    # ------------------------------------------------ sublayers that read the stream, results behind a norm
    def stream_cast(self, resid: torch.Tensor, out: torch.Tensor) -> None:
        """out = resid in the activations' type: the float stream as a product's operand."""
        _dev(resid, out)
        if resid.dtype != torch.float32 or not resid.is_contiguous() or out.shape != resid.shape or not out.is_contiguous():
            raise ValueError("stream_cast: a contiguous float32 stream and a contiguous copy of its shape")
        library.call("ra_stream_cast", resid.data_ptr(), out.data_ptr(), _tag(out, "stream_cast"), resid.numel(), _stream())

    def sum_norm_add(self, xs, scales, weight: Optional[torch.Tensor], eps: float,
                     resid: Optional[torch.Tensor] = None, copy: Optional[torch.Tensor] = None) -> None:
        """y = sum_i scales[i] * xs[i] row by row in float; with ``weight`` (float32, [width] or one number)
        y <- y / rms(y) * weight; ``resid += y`` where the float stream is given; ``copy`` (any of the two
        types) gets the new stream, or without ``resid`` the result."""
        import ctypes
        n = len(xs)
        if not 1 <= n <= 4 or len(scales) != n:
            raise ValueError(f"sum_norm_add: {n} inputs with {len(scales)} factors (1 to 4 of each)")
        _dev(*xs, weight, resid, copy)
        T, h = xs[0].shape
        for x in xs:
            if x.shape != (T, h) or x.dtype != xs[0].dtype or not x.is_contiguous():
                raise ValueError("sum_norm_add: the inputs are contiguous [T, width] of one dtype")
        if weight is not None and (weight.dtype != torch.float32 or weight.numel() not in (1, h) or not weight.is_contiguous()):
            raise ValueError(f"sum_norm_add: the weight is float32, one number or [{h}]")
        if resid is None and copy is None:
            raise ValueError("sum_norm_add: the result goes into the stream or into a copy")
        for name, t, dt in (("resid", resid, torch.float32), ("copy", copy, None)):
            if t is not None and (t.shape != (T, h) or not t.is_contiguous() or (dt is not None and t.dtype != dt)):
                raise ValueError(f"sum_norm_add: {name} is contiguous [T, width]")
        px = (ctypes.c_void_p * n)(*[x.data_ptr() for x in xs])
        ps = (ctypes.c_float * n)(*[float(v) for v in scales])
        library.call("ra_sum_norm_add", px, ps, n, _tag(xs[0], "sum_norm_add"), _ptr(weight),
                     0 if weight is None or weight.numel() == 1 else 1, 0 if weight is None else 1, float(eps), T, h,
                     _ptr(resid), _ptr(copy), _tag(copy, "sum_norm_add copy") if copy is not None else 0, _stream())

    def span_rmsnorm(self, x: torch.Tensor, spans, eps: float) -> None:
        """Runs of columns of every row of ``x``, in place: ``spans`` = up to two (first column, width, weight
        float32 [width], count); a run is divided by sqrt(sum of squares / count + eps) and multiplied by its weight."""
        import ctypes
        n = len(spans)
        if not 1 <= n <= 2:
            raise ValueError("span_rmsnorm: one or two runs")
        _dev(x, *[s[2] for s in spans])
        if x.dim() != 2 or x.stride(1) != 1:
            raise ValueError("span_rmsnorm: rows with contiguous columns")
        for c0, w, wt, cnt in spans:
            if wt.dtype != torch.float32 or wt.shape != (w,) or not wt.is_contiguous() or c0 < 0 or c0 + w > x.shape[1] or cnt <= 0:
                raise ValueError(f"span_rmsnorm: run at {c0} of {w} with weight {tuple(wt.shape)} {wt.dtype}")
        ints = lambda k: (ctypes.c_int * n)(*[int(s[k]) for s in spans])
        pw = (ctypes.c_void_p * n)(*[s[2].data_ptr() for s in spans])
        library.call("ra_span_rmsnorm", x.data_ptr(), _tag(x, "span_rmsnorm"), x.stride(0), x.shape[0], n, ints(0),
                     ints(1), ints(3), pw, float(eps), _stream())

    def turn_heads(self, x: torch.Tensor, heads: int, head_stride: int, width: int, style: int,
                   positions: Optional[torch.Tensor], inv_freq: Optional[torch.Tensor], sign: float = 1.0,
                   gate: Optional[torch.Tensor] = None, gate_stride: int = 0) -> None:
        """In place on ``x`` (rows of ``heads`` heads ``head_stride`` apart; a column range of a wider buffer
        will do): the first ``width`` entries of every head turn by sign * position, pair m being (m, m + width / 2)
        (``style`` 0) or (2m, 2m + 1) (1), by position * inv_freq[m]; with ``gate`` (heads ``gate_stride`` apart)
        every entry of a head is then multiplied by the sigmoid of the gate's entry at the same place."""
        _dev(x, positions, inv_freq, gate)
        T = x.shape[0]
        if x.dim() != 2 or x.stride(1) != 1 or x.shape[1] < heads * head_stride:
            raise ValueError(f"turn_heads: rows of {heads} heads of {head_stride}")
        if width:
            _int32(positions, "positions", T)
            if inv_freq.dtype != torch.float32 or inv_freq.numel() < width // 2 or not inv_freq.is_contiguous():
                raise ValueError("turn_heads: inv_freq is float32 with width / 2 entries")
        if gate is not None and (gate.dim() != 2 or gate.shape[0] != T or gate.stride(1) != 1 or gate.dtype != x.dtype
                                 or gate.shape[1] < (heads - 1) * gate_stride + head_stride):
            raise ValueError("turn_heads: the gate's rows do not cover the heads")
        library.call("ra_turn_heads", x.data_ptr(), _tag(x, "turn_heads"), x.stride(0), T, int(heads), int(head_stride),
                     int(width), int(style), _ptr(positions), _ptr(inv_freq), float(sign), _ptr(gate),
                     gate.stride(0) if gate is not None else 0, int(gate_stride), _stream())

    # Portions from this many tokens on are taken in chunks of 16 tokens (keys up to CHUNK_KEYS), shorter ones token by
    # token; either form goes on from the state that the other left.
    CHUNK_FROM = 17
    CHUNK_KEYS = 256

    @staticmethod
    def _check_linear_scan(what: str, proj, q_off, k_off, v_off, heads, key_dim, value_dim, out) -> None:
        T = proj.shape[0]
        if proj.dim() != 2 or proj.stride(1) != 1 or max(q_off, k_off) + heads * key_dim > proj.shape[1] \
                or v_off + heads * value_dim > proj.shape[1] or min(q_off, k_off, v_off) < 0:
            raise ValueError(f"{what}: the projection rows do not hold q, k and v at the given offsets")
        if out.shape != (T, heads * value_dim) or out.dtype != torch.float32 or not out.is_contiguous():
            raise ValueError(f"{what}: out is contiguous float32 [T, {heads * value_dim}]")

    @staticmethod
    def _chunk_scratch(T, n_seqs, heads, key_dim, value_dim, device) -> torch.Tensor:
        n = int(library.load().ra_chunk_scratch_floats(T, n_seqs, int(heads), int(key_dim), int(value_dim)))
        if n < 0:
            raise ValueError(f"heads of {key_dim} x {value_dim} are not taken in chunks (keys up to 256)")
        return torch.empty(n, dtype=torch.float32, device=device)

    def decay_scan(self, proj: torch.Tensor, q_off: int, k_off: int, v_off: int, decays: torch.Tensor,
                   state: torch.Tensor, batch, heads: int, key_dim: int, value_dim: int, out: torch.Tensor,
                   act: str = "silu", inv_freq: Optional[torch.Tensor] = None, rot_dims: int = 0,
                   q_scale: float = 1.0, k_scale: float = 1.0, chunks: Optional[bool] = None) -> None:
        """S <- decays[h] S + k v^T, o = S^T q head by head; the state [slots, floats] is float32, ``out`` float32
        [T, heads * value_dim]. q, k and v are ``proj``'s columns at the given offsets: with ``act`` "silu" their silu;
        with "none" as they are, q and k turned by their position over their first ``rot_dims`` elements (pairs
        (i, i + rot_dims / 2), angle position * inv_freq[i]) and times ``q_scale`` and ``k_scale``. Everything behind
        the projection is float. ``chunks`` forces the form (None: by the step's longest portion)."""
        _dev(proj, decays, state, out, inv_freq)
        T = proj.shape[0]
        self._check_scan("decay_scan", state, batch, T)
        if decays.dtype != torch.float32 or decays.shape != (heads,) or not decays.is_contiguous():
            raise ValueError(f"decay_scan: one float32 factor a head ({heads})")
        self._check_linear_scan("decay_scan", proj, q_off, k_off, v_off, heads, key_dim, value_dim, out)
        if act not in ("silu", "none"):
            raise ValueError(f"decay_scan: activation {act!r}; built: silu, none")
        if act == "silu" and (rot_dims or q_scale != 1.0 or k_scale != 1.0):
            raise ValueError("decay_scan: with silu q and k neither turn nor carry a factor")
        if rot_dims < 0 or rot_dims % 2 or rot_dims > key_dim or \
                (rot_dims and (inv_freq is None or inv_freq.dtype != torch.float32 or inv_freq.numel() < rot_dims // 2
                               or not inv_freq.is_contiguous())):
            raise ValueError(f"decay_scan: {rot_dims} turned elements of {key_dim}, float32 frequencies of their pairs")
        if rot_dims:
            _int32(batch.positions, "positions", T)
        tag, longest = _tag(proj, "decay_scan"), int(batch.max_q_len)
        if chunks is None:
            chunks = longest >= self.CHUNK_FROM and key_dim <= self.CHUNK_KEYS
        tail = (state.data_ptr(), state.stride(0), batch.cu_tokens.data_ptr(), batch.state_slots.data_ptr(),
                batch.fresh.data_ptr(), batch.num_seqs, T)
        turned = (batch.positions.data_ptr() if rot_dims else None, _ptr(inv_freq) if rot_dims else None, int(rot_dims))
        if chunks:
            scratch = self._chunk_scratch(T, batch.num_seqs, heads, key_dim, value_dim, proj.device)
            library.call("ra_decay_chunks", proj.data_ptr(), tag, proj.stride(0), int(q_off), int(k_off), int(v_off),
                         1 if act == "silu" else 0, decays.data_ptr(), *turned, float(q_scale), float(k_scale), *tail,
                         int(heads), int(key_dim), int(value_dim), scratch.data_ptr(), scratch.numel(), out.data_ptr(),
                         _stream())
        elif act == "silu":
            library.call("ra_decay_scan", proj.data_ptr(), tag, proj.stride(0), int(q_off), int(k_off), int(v_off),
                         decays.data_ptr(), *tail, longest, int(heads), int(key_dim), int(value_dim), out.data_ptr(),
                         _stream())
        else:
            library.call("ra_retention_scan", proj.data_ptr(), tag, proj.stride(0), int(q_off), int(k_off), int(v_off),
                         decays.data_ptr(), *turned, float(q_scale), float(k_scale), *tail, longest, int(heads),
                         int(key_dim), int(value_dim), out.data_ptr(), _stream())

    def gated_linear_scan(self, proj: torch.Tensor, q_off: int, k_off: int, v_off: int, z: torch.Tensor,
                          bias: torch.Tensor, tau: float, state: torch.Tensor, batch, heads: int, key_dim: int,
                          value_dim: int, out: torch.Tensor, q_scale: float = 1.0, chunks: Optional[bool] = None) -> None:
        """S <- diag(alpha) S + k v^T, o = S^T q head by head with alpha = sigmoid(z + bias)^(1 / tau), one factor a head
        and key channel (``z`` float32 [T, heads * key_dim], ``bias`` float32 [heads * key_dim]); q times ``q_scale``.
        State, ``out`` and ``chunks`` as for :meth:`decay_scan`."""
        _dev(proj, z, bias, state, out)
        T, n = proj.shape[0], heads * key_dim
        self._check_scan("gated_linear_scan", state, batch, T)
        self._check_linear_scan("gated_linear_scan", proj, q_off, k_off, v_off, heads, key_dim, value_dim, out)
        if z.dim() != 2 or z.shape[0] != T or z.shape[1] < n or z.dtype != torch.float32 or z.stride(1) != 1 \
                or bias.shape != (n,) or bias.dtype != torch.float32 or not bias.is_contiguous():
            raise ValueError(f"gated_linear_scan: pre-activations float32 [T, {n}], their bias float32 [{n}]")
        if not tau > 0.0:
            raise ValueError("gated_linear_scan: tau is positive")
        tag, longest = _tag(proj, "gated_linear_scan"), int(batch.max_q_len)
        if chunks is None:
            chunks = longest >= self.CHUNK_FROM and key_dim <= self.CHUNK_KEYS
        head = (proj.data_ptr(), tag, proj.stride(0), int(q_off), int(k_off), int(v_off), z.data_ptr(), z.stride(0),
                bias.data_ptr(), float(tau))
        tail = (float(q_scale), state.data_ptr(), state.stride(0), batch.cu_tokens.data_ptr(),
                batch.state_slots.data_ptr(), batch.fresh.data_ptr(), batch.num_seqs, T)
        sizes = (int(heads), int(key_dim), int(value_dim))
        if chunks:
            scratch = self._chunk_scratch(T, batch.num_seqs, heads, key_dim, value_dim, proj.device)
            library.call("ra_gla_chunks", *head, *tail, *sizes, scratch.data_ptr(), scratch.numel(), out.data_ptr(), _stream())
        else:
            library.call("ra_gla_scan", *head, *tail, longest, *sizes, out.data_ptr(), _stream())

    # -------------------------------------------------------------- several residual streams
    def hyper_step(self, streams: torch.Tensor, base: Optional[torch.Tensor], y: Optional[torch.Tensor],
                   mix: Optional[torch.Tensor], w_out: Optional[torch.Tensor], w_in: Optional[torch.Tensor],
                   weight: Optional[torch.Tensor], eps: float, out: Optional[torch.Tensor],
                   rows: Optional[torch.Tensor] = None, store: bool = True) -> None:
        """``streams`` float32 [T, n, width]: X_t <- sum_s mix[s, t] X_s + w_out[t] y (``y`` None: as they are),
        u = sum_t w_in[t] X_t (None: ones), ``out`` = u / sqrt(mean u^2 + eps) * weight (``weight`` None: u itself).
        ``base`` [T, width]: every stream is still this row. ``store``: the new streams are kept; with ``rows`` only
        those rows are computed, into a compact ``out``, and nothing is kept."""
        _dev(streams, base, y, mix, w_out, w_in, weight, out, rows)
        if streams.dim() != 3 or streams.dtype != torch.float32 or not streams.is_contiguous():
            raise TypeError("hyper_step: the streams are contiguous float32 [T, n, width]")
        T, n, h = streams.shape
        for t, shape, what in ((base, (T, h), "base"), (mix, (n, n), "mix"), (w_out, (n,), "out factors"),
                               (w_in, (n,), "in factors"), (weight, (h,), "norm weight")):
            if t is not None and (t.dtype != torch.float32 or t.shape != shape or not t.is_contiguous()):
                raise ValueError(f"hyper_step: {what} {tuple(t.shape)} {t.dtype}, expected contiguous float32 {list(shape)}")
        if y is not None and (y.shape != (T, h) or not y.is_contiguous() or mix is None or w_out is None):
            raise ValueError("hyper_step: y is contiguous [T, width] and enters by mix and w_out")
        n_rows = T
        if rows is not None:
            n_rows = rows.numel()
            _int32(rows, "hyper_step rows", n_rows)
            store = False
        if out is not None and (out.shape != (n_rows, h) or not out.is_contiguous()):
            raise ValueError(f"hyper_step: out {tuple(out.shape)}, expected contiguous [{n_rows}, {h}]")
        library.call("ra_hyper_step", streams.data_ptr(), _ptr(base), _ptr(y), _tag(y, "hyper_step y") if y is not None else 0,
                     _ptr(mix), _ptr(w_out), _ptr(w_in), _ptr(weight), float(eps), _ptr(rows), n_rows, n, h,
                     1 if store else 0, _ptr(out), _tag(out, "hyper_step out") if out is not None else 0, _stream())

    def moe_table_route(self, token_ids: torch.Tensor, table: torch.Tensor, ids: torch.Tensor,
                        weights: torch.Tensor) -> None:
        """ids[t, j] = table[token_ids[t], j], weights[t, j] = 1 / top: experts looked up by token id."""
        _dev(token_ids, table, ids, weights)
        T, top = ids.shape
        _int32(token_ids, "token ids", T)
        if table.dtype != torch.int32 or table.dim() != 2 or table.shape[1] != top or not table.is_contiguous():
            raise ValueError(f"moe_table_route: an int32 table [vocabulary, {top}]")
        self._check_choice("moe_table_route", ids, weights, T, top)
        library.call("ra_moe_table_route", token_ids.data_ptr(), table.data_ptr(), top, ids.data_ptr(),
                     weights.data_ptr(), T, _stream())

    def normed_mean(self, xs, weights, eps: float, out: Optional[torch.Tensor] = None,
                    resid: Optional[torch.Tensor] = None, scale: float = 1.0) -> None:
        """y = mean_i xs[i] / rms(xs[i]) * weights[i] row by row (float); written to ``out`` (the inputs' dtype)
        or ``resid += scale * y`` (the float stream): exactly one of the two is given."""
        import ctypes
        n = len(xs)
        if not 1 <= n <= 4 or len(weights) != n:
            raise ValueError(f"normed_mean: {n} inputs with {len(weights)} weights (1 to 4 of each)")
        _dev(*xs, *weights, out, resid)
        T, h = xs[0].shape
        for x, w in zip(xs, weights):
            if x.shape != (T, h) or x.dtype != xs[0].dtype or not x.is_contiguous():
                raise ValueError("normed_mean: the inputs are contiguous [T, width] of one dtype")
            if w.shape != (h,) or w.dtype != torch.float32 or not w.is_contiguous():
                raise ValueError(f"normed_mean: weights are float32 [{h}]")
        if (out is None) == (resid is None):
            raise ValueError("normed_mean: the result goes into the stream or into out")
        if out is not None and (out.shape != (T, h) or out.dtype != xs[0].dtype or not out.is_contiguous()):
            raise ValueError("normed_mean: out is contiguous [T, width] in the inputs' dtype")
        if resid is not None and (resid.shape != (T, h) or resid.dtype != torch.float32 or not resid.is_contiguous()):
            raise ValueError("normed_mean: the residual stream is contiguous float32 [T, width]")
        px = (ctypes.c_void_p * n)(*[x.data_ptr() for x in xs])
        pw = (ctypes.c_void_p * n)(*[w.data_ptr() for w in weights])
        library.call("ra_normed_mean", px, pw, n, _tag(xs[0], "normed_mean"), float(eps), T, h, _ptr(out), _ptr(resid),
                     float(scale), _stream())

    # ---------------------------------------------------- mixture of experts
    def moe_route(self, x: torch.Tensor, router: torch.Tensor, top: int, ids: torch.Tensor,
                  weights: torch.Tensor, scoring: str = "softmax_chosen", scale: float = 1.0, groups: int = 1,
                  groups_kept: int = 1, group_top: int = 2, correction: Optional[torch.Tensor] = None,
                  norm_eps: float = 0.0, outputs: Optional[int] = None) -> torch.Tensor:
        """Router logits x . router^T accumulated and kept in float (``router`` [experts, width] in the
        activations' dtype: a bfloat16 product's terms are exact in float), the ``top`` largest a token in
        falling order into ``ids`` [T, top] (int32), the softmax over those alone into ``weights`` [T, top]
        (float32). ``scoring`` "sigmoid": scores are the logits' sigmoids; with ``groups`` > 1 only experts of
        the ``groups_kept`` best groups of neighbours (a group's score: the sum of its ``group_top`` largest
        scores) can be chosen; the weights are the chosen scores times ``scale``. ``scoring`` "softmax": scores
        are the softmax over all outputs, the choice is by score + ``correction`` (float32 [outputs] or None)
        inside the best groups (a group's score: its largest choice score), the weights the chosen scores over
        their sum + ``norm_eps``. ``outputs``: the router's first rows that are routed over (default: all);
        further rows are logits for the caller, who gets the float32 logits [T, rows] back."""
        _dev(x, router, ids, weights)
        T, width = x.shape
        E = router.shape[0]
        if router.shape != (E, width) or router.dtype != x.dtype or not router.is_contiguous():
            raise ValueError(f"moe_route: router {tuple(router.shape)} {router.dtype}, expected [experts, {width}] "
                             "in the activations' dtype")
        if ids.shape != (T, top) or ids.dtype != torch.int32 or not ids.is_contiguous() \
                or weights.shape != (T, top) or weights.dtype != torch.float32 or not weights.is_contiguous():
            raise ValueError(f"moe_route: ids int32 and weights float32, both [{T}, {top}]")
        logits = torch.empty((T, E), dtype=torch.float32, device=x.device)
        self.linear(x, router, logits)
        if outputs is not None:
            if not 0 < outputs <= E:
                raise ValueError(f"moe_route: {outputs} routed outputs of {E} router rows")
            E = int(outputs)
        if scoring == "softmax":
            if correction is not None:
                _dev(correction)
                if correction.shape != (E,) or correction.dtype != torch.float32 or not correction.is_contiguous():
                    raise ValueError(f"moe_route: correction is float32 [{E}]")
            library.call("ra_moe_route_softmax", logits.data_ptr(), logits.stride(0), E, int(top), int(groups),
                         int(groups_kept), _ptr(correction), float(norm_eps), ids.data_ptr(), weights.data_ptr(), T,
                         _stream())
            return logits
        if scoring == "sigmoid":
            library.call("ra_moe_route_sigmoid", logits.data_ptr(), logits.stride(0), E, int(top), int(groups),
                         int(groups_kept), int(group_top), float(scale), ids.data_ptr(), weights.data_ptr(), T,
                         _stream())
            return logits
        if scoring != "softmax_chosen":
            raise ValueError(f"moe_route: scoring {scoring!r}")
        library.call("ra_moe_topk", logits.data_ptr(), logits.stride(0), E, int(top), ids.data_ptr(),
                     weights.data_ptr(), T, _stream())
        return logits

    def moe_silu_gate_scale(self, gu: torch.Tensor, act: torch.Tensor, ids: torch.Tensor, weights: torch.Tensor,
                            experts: int, ff: int, shared: int = 0, shared_logit: Optional[torch.Tensor] = None) -> None:
        """``gu`` [T, 2 (experts ff + shared)]: [gate | up] of each expert, a shared expert's behind them.
        act[t, e ff + j] = weight(t, e) silu(gate) up for the chosen experts, 0 for the others; the shared
        expert's columns behind them with weight 1, or with sigmoid(``shared_logit``[t]) (float32, one number a
        token; it may be a column of a wider matrix). A chosen id of ``experts`` or more names no matrices."""
        _dev(gu, act, ids, weights)
        T = gu.shape[0]
        n = experts * ff + shared
        if gu.shape != (T, 2 * n) or act.shape != (T, n) or act.dtype != gu.dtype or not gu.is_contiguous() \
                or not act.is_contiguous():
            raise ValueError(f"moe_silu_gate_scale: gu {tuple(gu.shape)} / act {tuple(act.shape)}, expected "
                             f"[T, {2 * n}] and [T, {n}]")
        self._check_choice("moe_silu_gate_scale", ids, weights, T, ids.shape[1])
        ld = 0
        if shared_logit is not None:
            _dev(shared_logit)
            if shared_logit.dtype != torch.float32 or shared_logit.shape[0] != T or shared_logit.numel() != T:
                raise ValueError("moe_silu_gate_scale: the shared expert's logits are float32, one a token")
            ld = shared_logit.stride(0)
        library.call("ra_moe_silu_gate_scale_shared", gu.data_ptr(), act.data_ptr(), _tag(gu, "moe_silu_gate_scale"),
                     ids.data_ptr(), weights.data_ptr(), ids.shape[1], int(experts), int(ff), int(shared),
                     _ptr(shared_logit), int(ld), T, _stream())

    def moe_identity_add(self, y: torch.Tensor, x: torch.Tensor, ids: torch.Tensor, weights: torch.Tensor,
                         experts: int) -> None:
        """y[t] += (sum of weights[t, j] over choices with ids[t, j] >= experts) * x[t]: chosen ids past the
        experts stand for the identity."""
        _dev(y, x, ids, weights)
        T, width = y.shape
        if x.shape != (T, width) or x.dtype != y.dtype or x.stride(1) != 1 or y.stride(1) != 1:
            raise ValueError(f"moe_identity_add: y {tuple(y.shape)} against x {tuple(x.shape)}")
        self._check_choice("moe_identity_add", ids, weights, T, ids.shape[1])
        library.call("ra_moe_identity_add", y.data_ptr(), y.stride(0), x.data_ptr(), x.stride(0), _tag(y, "moe_identity_add"),
                     ids.data_ptr(), weights.data_ptr(), ids.shape[1], int(experts), T, width, _stream())

    def moe_relu2_scale(self, up: torch.Tensor, act: torch.Tensor, ids: torch.Tensor, weights: torch.Tensor,
                        experts: int, ff: int) -> None:
        """act[t, e * ff + j] = weight(t, e) * relu(up[t, e * ff + j])^2 for the chosen experts, 0 for the rest."""
        _dev(up, act, ids, weights)
        T = up.shape[0]
        top = ids.shape[1]
        if up.shape != (T, experts * ff) or act.shape != up.shape or act.dtype != up.dtype \
                or not up.is_contiguous() or not act.is_contiguous():
            raise ValueError(f"moe_relu2_scale: up {tuple(up.shape)} / act {tuple(act.shape)}, expected [T, {experts * ff}]")
        if ids.shape != (T, top) or ids.dtype != torch.int32 or weights.shape != (T, top) \
                or weights.dtype != torch.float32 or not ids.is_contiguous() or not weights.is_contiguous():
            raise ValueError("moe_relu2_scale: ids int32 and weights float32, both [T, top]")
        library.call("ra_moe_relu2_scale", up.data_ptr(), act.data_ptr(), _tag(up, "moe_relu2_scale"), ids.data_ptr(),
                     weights.data_ptr(), top, int(experts), int(ff), T, _stream())

    # Steps of so few tokens that their choices name at most this share of the experts read only the chosen
    # experts' rows (two kernels, a wave a row) instead of running every expert through the matrix cores
    MOE_CHOSEN_SHARE = 0.5
    MOE_CHOSEN_TOKENS = 8

    def moe_reads_chosen(self, n_tokens: int, top: int, experts: int) -> bool:
        """Whether a step of ``n_tokens`` should read only its chosen experts (``moe_up_chosen`` /
        ``moe_down_chosen``): its token-expert pairs are few against the experts there are."""
        return n_tokens <= self.MOE_CHOSEN_TOKENS and n_tokens * top <= self.MOE_CHOSEN_SHARE * experts

    def moe_up_chosen(self, x: torch.Tensor, w_up: torch.Tensor, ids: torch.Tensor, weights: torch.Tensor,
                      act: torch.Tensor, ff: int) -> None:
        """act[t * top + j] = weights[t, j] * relu(w_up[ids[t, j] * ff : ... + ff] . x[t])^2 for the chosen
        experts only; ``w_up`` is [experts * ff, width], ``act`` [T * top, ff]."""
        _dev(x, w_up, ids, weights, act)
        T, width = x.shape
        top = ids.shape[1]
        E = w_up.shape[0] // ff
        if w_up.shape != (E * ff, width) or not w_up.is_contiguous() or x.dtype != w_up.dtype or x.stride(1) != 1:
            raise ValueError(f"moe_up_chosen: x {tuple(x.shape)}, w_up {tuple(w_up.shape)} for experts of {ff}")
        if act.shape != (T * top, ff) or act.dtype != x.dtype or not act.is_contiguous():
            raise ValueError(f"moe_up_chosen: act {tuple(act.shape)}, expected [{T * top}, {ff}]")
        self._check_choice("moe_up_chosen", ids, weights, T, top)
        library.call("ra_moe_up_chosen", x.data_ptr(), x.stride(0), w_up.data_ptr(), ids.data_ptr(),
                     weights.data_ptr(), act.data_ptr(), _tag(x, "moe_up_chosen"), T, top, E, int(ff), width, _stream())

    def moe_down_chosen(self, act: torch.Tensor, w_down: torch.Tensor, ids: torch.Tensor, ff: int,
                        resid: Optional[torch.Tensor] = None, out: Optional[torch.Tensor] = None) -> None:
        """y[t] = sum_j w_down[:, ids[t, j] * ff : ... + ff] . act[t * top + j], added into the float ``resid``
        or written to ``out`` (exactly one is given); ``w_down`` is [width, experts * ff]."""
        _dev(act, w_down, ids, resid, out)
        T, top = ids.shape
        width = w_down.shape[0]
        E = w_down.shape[1] // ff
        if w_down.shape != (width, E * ff) or not w_down.is_contiguous() or act.dtype != w_down.dtype \
                or act.shape != (T * top, ff) or not act.is_contiguous():
            raise ValueError(f"moe_down_chosen: act {tuple(act.shape)}, w_down {tuple(w_down.shape)} for experts of {ff}")
        if ids.dtype != torch.int32 or not ids.is_contiguous():
            raise ValueError("moe_down_chosen: ids are contiguous int32 [T, top]")
        if (resid is None) == (out is None):
            raise ValueError("moe_down_chosen: the result goes into the stream or into out")
        if resid is not None and (resid.shape != (T, width) or resid.dtype != torch.float32 or not resid.is_contiguous()):
            raise ValueError("moe_down_chosen: the residual stream is contiguous float32 [T, width]")
        if out is not None and (out.shape != (T, width) or out.dtype != act.dtype or not out.is_contiguous()):
            raise ValueError("moe_down_chosen: out is contiguous [T, width] in the activations' dtype")
        library.call("ra_moe_down_chosen", act.data_ptr(), w_down.data_ptr(), ids.data_ptr(), _ptr(resid), _ptr(out),
                     _tag(act, "moe_down_chosen"), T, top, E, int(ff), width, _stream())

    def moe_gate_up_chosen(self, x: torch.Tensor, w_gate_up: torch.Tensor, ids: torch.Tensor, weights: torch.Tensor,
                           act: torch.Tensor, experts: int, ff: int, shared: int,
                           shared_logit: Optional[torch.Tensor] = None) -> None:
        """Gated experts, the chosen ones only: act[t, j * ff : ...] = weights[t, j] * silu(W_gate x[t]) * (W_up x[t])
        of expert ids[t, j] (zeros for an id of ``experts`` or more), and behind the ``top`` choices the shared
        expert's, times sigmoid(shared_logit[t]) where that is given. ``w_gate_up`` is [2 (experts ff + shared),
        width] with [gate; up] an expert, the shared expert's last; ``act`` [T, top * ff + shared]."""
        _dev(x, w_gate_up, ids, weights, act)
        T, width = x.shape
        top = ids.shape[1]
        if w_gate_up.shape != (2 * (experts * ff + shared), width) or not w_gate_up.is_contiguous() \
                or x.dtype != w_gate_up.dtype or x.stride(1) != 1:
            raise ValueError(f"moe_gate_up_chosen: x {tuple(x.shape)}, w_gate_up {tuple(w_gate_up.shape)} for "
                             f"{experts} experts of {ff} and a shared one of {shared}")
        if act.shape != (T, top * ff + shared) or act.dtype != x.dtype or not act.is_contiguous():
            raise ValueError(f"moe_gate_up_chosen: act {tuple(act.shape)}, expected [{T}, {top * ff + shared}]")
        self._check_choice("moe_gate_up_chosen", ids, weights, T, top)
        ld = 0
        if shared_logit is not None:
            _dev(shared_logit)
            if shared_logit.dtype != torch.float32 or shared_logit.shape[0] != T or shared_logit.numel() != T:
                raise ValueError("moe_gate_up_chosen: the shared expert's logits are float32, one a token")
            ld = shared_logit.stride(0)
        library.call("ra_moe_gate_up_chosen", x.data_ptr(), x.stride(0), w_gate_up.data_ptr(), ids.data_ptr(),
                     weights.data_ptr(), _ptr(shared_logit), int(ld), act.data_ptr(), _tag(x, "moe_gate_up_chosen"), T,
                     top, int(experts), int(ff), int(shared), width, _stream())

    def moe_down_gated_chosen(self, act: torch.Tensor, w_down: torch.Tensor, ids: torch.Tensor, weights: torch.Tensor,
                              x: torch.Tensor, out: torch.Tensor, experts: int, ff: int, shared: int) -> None:
        """out[t] = sum_j w_down[:, ids[t, j] * ff : ...] . act[t, j * ff : ...] + the shared expert's columns times
        its part of act + (the weights of chosen ids of ``experts`` or more) * x[t]; ``w_down`` is
        [width, experts * ff + shared], ``act`` as ``moe_gate_up_chosen`` leaves it."""
        _dev(act, w_down, ids, weights, x, out)
        T, top = ids.shape
        width = w_down.shape[0]
        if w_down.shape != (width, experts * ff + shared) or not w_down.is_contiguous() or act.dtype != w_down.dtype \
                or act.shape != (T, top * ff + shared) or not act.is_contiguous():
            raise ValueError(f"moe_down_gated_chosen: act {tuple(act.shape)}, w_down {tuple(w_down.shape)} for "
                             f"{experts} experts of {ff} and a shared one of {shared}")
        self._check_choice("moe_down_gated_chosen", ids, weights, T, top)
        if x.shape != (T, width) or x.dtype != act.dtype or x.stride(1) != 1:
            raise ValueError(f"moe_down_gated_chosen: x {tuple(x.shape)}, expected [{T}, {width}]")
        if out.shape != (T, width) or out.dtype != act.dtype or not out.is_contiguous():
            raise ValueError("moe_down_gated_chosen: out is contiguous [T, width] in the activations' dtype")
        library.call("ra_moe_down_gated_chosen", act.data_ptr(), w_down.data_ptr(), ids.data_ptr(), weights.data_ptr(),
                     x.data_ptr(), x.stride(0), out.data_ptr(), _tag(act, "moe_down_gated_chosen"), T, top,
                     int(experts), int(ff), int(shared), width, _stream())

    @staticmethod
    def _check_choice(what: str, ids, weights, T: int, top: int) -> None:
        if ids.shape != (T, top) or ids.dtype != torch.int32 or not ids.is_contiguous() \
                or weights.shape != (T, top) or weights.dtype != torch.float32 or not weights.is_contiguous():
            raise ValueError(f"{what}: ids int32 and weights float32, both [{T}, {top}]")

    # -------------------------------------------------------------- sampling
    def sample(self, logits: torch.Tensor, temperature: torch.Tensor, seeds: torch.Tensor,
               positions: torch.Tensor, tokens: torch.Tensor) -> None:
        _dev(logits, temperature, seeds, positions, tokens)
        n, V = logits.shape
        if logits.dtype != torch.float32 or logits.stride(1) != 1:
            raise TypeError("sample: logits are float32 rows")
        if temperature.dtype != torch.float32 or seeds.dtype != torch.int64:
            raise TypeError("sample: temperature float32, seeds int64")
        _int32(positions, "sample positions", n)
        _int32(tokens, "sampled tokens", n)
        if temperature.numel() < n or seeds.numel() < n:
            raise ValueError("sample: one temperature and seed per row")
        slices = library.load().ra_sample_slices(V)
        val = torch.empty((n, slices), dtype=torch.float32, device=logits.device)
        idx = torch.empty((n, slices), dtype=torch.int32, device=logits.device)
        library.call("ra_sample", logits.data_ptr(), n, V, logits.stride(0), temperature.data_ptr(),
                     seeds.data_ptr(), positions.data_ptr(), val.data_ptr(), idx.data_ptr(),
                     tokens.data_ptr(), _stream())

    def filter_logits(self, logits: torch.Tensor, params, histories) -> None:
        """Logit bias, penalties and top-k / top-p / min-p of every row's SamplingParams, in
        place (removed tokens become -inf); ``histories[i]`` are row i's tokens so far."""
        import numpy as np
        _dev(logits)
        n, V = logits.shape
        if logits.dtype != torch.float32 or logits.stride(1) != 1:
            raise TypeError("filter_logits: logits are float32 rows")
        rec = np.zeros((n, 12), dtype=np.float32)
        irec = rec.view(np.int32)
        window, off = [], 0
        for i, (p, hist) in enumerate(zip(params, histories)):
            rec[i, 0] = max(0.0, float(p.temperature))
            rec[i, 1] = float(p.top_p or 0.0)
            rec[i, 2] = float(p.min_p or 0.0)
            rec[i, 3] = float(p.repeat_penalty or 0.0)
            rec[i, 4] = max(0.0, float(p.frequency_penalty or 0.0))
            rec[i, 5] = max(0.0, float(p.presence_penalty or 0.0))
            irec[i, 6] = int(p.top_k or 0)
            win = list(hist[-p.repeat_last_n:]) if (p.penalties and p.repeat_last_n > 0) else []
            irec[i, 7], irec[i, 8] = off, len(win)
            window += win
            off += len(win)
            bias = getattr(p, "logit_bias", ())
            if bias:
                pairs = np.zeros((len(bias), 2), dtype=np.int32)
                pairs[:, 0] = [int(t) for t, _ in bias]
                pairs[:, 1] = np.asarray([float(b) for _, b in bias], dtype=np.float32).view(np.int32)
                irec[i, 9], irec[i, 10] = off, len(bias)
                window += pairs.reshape(-1).tolist()
                off += 2 * len(bias)
        rows_t = torch.from_numpy(rec).to(logits.device)
        win_t = torch.tensor(window or [0], dtype=torch.int32).to(logits.device)
        library.call("ra_filter_logits", logits.data_ptr(), n, V, logits.stride(0), rows_t.data_ptr(),
                     win_t.data_ptr(), _stream())

    # ------------------------------------------------------------ measurement
    def measure_peaks(self, device="cuda:0", read_bytes: int = 4 << 30) -> dict:
        """What the machine gives at best: GB/s of a plain read of ``read_bytes`` of device memory
        (more than the chip's caches hold) and TFLOP/s of bfloat16 matrix-core products on
        registers, in both instruction shapes. For pricing measured kernels beside the published peaks; not on the product path."""
        import ctypes
        buf = torch.empty(read_bytes // 4, dtype=torch.int32, device=device).random_()
        sink = torch.zeros(1, dtype=torch.int32, device=device)
        e0, e1 = torch.cuda.Event(enable_timing=True), torch.cuda.Event(enable_timing=True)

        def timed(fn, reps):
            fn()
            torch.cuda.synchronize(device)
            best = float("inf")
            for _ in range(reps):
                e0.record()
                fn()
                e1.record()
                torch.cuda.synchronize(device)
                best = min(best, e0.elapsed_time(e1) * 1e-3)
            return best

        with torch.cuda.device(device):
            t_read = timed(lambda: library.call("ra_stream_read", buf.data_ptr(), read_bytes, sink.data_ptr(), _stream()), 5)
            out = {"hbm_read_GBps": read_bytes / t_read / 1e9}
            for shape, name in ((32, "mfma_bf16_32x32x16_TFLOPs"), (16, "mfma_bf16_16x16x32_TFLOPs")):
                flops = ctypes.c_double(0.0)
                t = timed(lambda: library.call("ra_mfma_loop", shape, 10000, 16, sink.data_ptr(),
                                               ctypes.byref(flops), _stream()), 3)
                out[name] = flops.value / t / 1e12
        del buf
        return out
