"""The kernels' further options that came with Dokanex, each against a plain PyTorch form of the same operation: the three
attention kernels with chunks counted from position 0, a sink a head and a gate a head (single tokens through parts of keys,
portions in query tiles whole and cut by keys, the float kernel; alone and together, with and without a cap on the scores, and
sinks and gates with sliding windows), the head kernel on rows wider than their heads and on queries alone, and the latent's
rotation of neighbouring pairs with a factor on sine and cosine."""
import math

import pytest
import torch

from kernel_double import KernelDouble
from reinfer_amd import kernels
from reinfer_amd.cache.layout import unpack_k, unpack_v
from test_gpu_kernels import DEC_BATCHES, DT, PRE_BATCHES, FakeBatch, close, kt, vt

pytestmark = pytest.mark.gpu
DEV = "cuda:0"


# ------------------------------------------------------------------ attention: chunks, sinks, gates
def first_key(p, window, chunked):
    return 0 if not window else (p // window * window if chunked else max(0, p - window + 1))


def make_case(dtype, Hq, Hkv, d, q_lens, starts, window, chunked, seed, bs=16):
    """Queries, sinks, gates, caches and tables as the engine leaves them: blocks that the first query's window or chunk does
    not reach have been given back, their table entries read 0, and block 0 and every slot never written hold NaN."""
    g = torch.Generator().manual_seed(seed)
    ctx = [s + q for s, q in zip(starts, q_lens)]
    need = [-(-c // bs) for c in ctx]
    total = sum(need) + 4
    perm = [b for b in torch.randperm(total, generator=g).tolist() if b != 0]
    tables = torch.zeros(len(q_lens), max(need), dtype=torch.int32)
    kc = torch.full((total, Hkv, bs, d), float("nan"))
    vc = kc.clone()
    p = 0
    for i in range(len(q_lens)):
        for b in range(first_key(starts[i], window, chunked) // bs, need[i]):
            blk = perm[p]
            p += 1
            tables[i, b] = blk
            fill = min(bs, ctx[i] - b * bs)
            kc[blk, :, :fill] = torch.randn(Hkv, fill, d, generator=g)
            vc[blk, :, :fill] = torch.randn(Hkv, fill, d, generator=g)
    T = sum(q_lens)
    q = torch.randn(T, Hq, d, generator=g)
    sink = 3.0 * torch.randn(Hq, generator=g) + 1.0
    wide = torch.randn(T, Hq + 16, generator=g)
    c = lambda x: x.to(DT[dtype]).to(DEV)
    return c(q), c(kc), c(vc), tables.to(DEV), sink.to(DEV), c(wide)[:, 8:8 + Hq]


def attention_reference(q, kc, vc, tables, q_lens, starts, Hq, Hkv, d, scale, window, chunked, cap=0.0, sink=None, gate=None):
    bs = kc.shape[2]
    kc, vc, q, tables = kc.double().cpu(), vc.double().cpu(), q.double().cpu(), tables.cpu()
    out, t0 = [], 0
    for i, (ql, st) in enumerate(zip(q_lens, starts)):
        for j in range(ql):
            p = st + j
            keys = torch.arange(first_key(p, window, chunked), p + 1)
            blk = tables[i, keys // bs].long()
            K, V = kc[blk, :, keys % bs, :], vc[blk, :, keys % bs, :]
            row = []
            for a in range(Hq):
                s = (K[:, a // (Hq // Hkv)] @ q[t0 + j, a]) * scale
                if cap:
                    s = cap * torch.tanh(s / cap)
                if sink is not None:
                    s = torch.cat([s, sink[a:a + 1].double().cpu()])
                o = torch.softmax(s, 0)[:keys.numel()] @ V[:, a // (Hq // Hkv)]
                if gate is not None:
                    o = o * torch.sigmoid(gate[t0 + j, a].double().cpu())
                row.append(o)
            out.append(torch.cat(row))
        t0 += ql
    return torch.stack(out)


# window, chunked, cap, sink, gate
OPTIONS = [(16, True, 0.0, True, True), (37, True, 2.0, True, True), (64, True, 0.0, False, False), (150, True, 0.5, True, False),
           (5, True, 0.0, False, True), (0, False, 0.0, True, True), (19, False, 0.0, True, True), (1, True, 0.0, True, False),
           (1024, True, 2.0, True, True)]


def options(o, sink, gate):
    window, chunked, cap, with_sink, with_gate = o
    return window, chunked, cap, (sink if with_sink else None), (gate if with_gate else None)


def call_args(ops, o, sink, gate, q, Hq):
    """The keyword arguments of a kernel's own method."""
    window, chunked, cap, sink, gate = options(o, sink, gate)
    return {"mod": ops._score_mod(cap, None, Hq, q.device), "aligned": chunked and window > 0,
            "head_out": ops._head_out(sink, gate, q, Hq)}


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("Hq,Hkv,d", [(4, 2, 16), (6, 3, 96), (8, 1, 272)])
def test_attention_plain(dtype, Hq, Hkv, d):
    ops = kernels.current()
    for bi, (q_lens, starts) in enumerate([([1, 1, 1], [31, 32, 300]), ([2, 17, 1, 40], [0, 30, 99, 1])]):
        for o in OPTIONS:
            q, kc, vc, tables, sink, gate = make_case(dtype, Hq, Hkv, d, q_lens, starts, o[0], o[1], bi)
            T, scale = sum(q_lens), 1.0 / math.sqrt(d)
            out = torch.empty(T, Hq * d, device=DEV, dtype=DT[dtype])
            ops.attention_plain(q.view(T, Hq * d), Hq * d, out, kt(kc), vt(vc), FakeBatch(q_lens, starts, tables), Hq, Hkv, d,
                                scale, o[0], 0, **call_args(ops, o, sink, gate, q.view(T, Hq * d), Hq))
            w, ch, cap, s, gt = options(o, sink, gate)
            ref = attention_reference(q, kc, vc, tables, q_lens, starts, Hq, Hkv, d, scale, w, ch, cap, s, gt)
            close(out, ref, 2e-5 if dtype == "float32" else 2 ** -7)


@pytest.mark.parametrize("Hq,Hkv,d", [(4, 2, 16), (6, 2, 64), (8, 1, 128), (3, 3, 48), (10, 2, 80), (9, 3, 112), (2, 1, 256)])
def test_attention_decode(Hq, Hkv, d):
    ops = kernels.current()
    for bi, (q_lens, starts) in enumerate(DEC_BATCHES[:6]):
        for o in OPTIONS:
            q, kc, vc, tables, sink, gate = make_case("bfloat16", Hq, Hkv, d, q_lens, starts, o[0], o[1], 10 + bi)
            T, scale = sum(q_lens), 1.0 / math.sqrt(d)
            w, ch, cap, s, gt = options(o, sink, gate)
            ref = attention_reference(q, kc, vc, tables, q_lens, starts, Hq, Hkv, d, scale, w, ch, cap, s, gt)
            for chunk, waves in ((None, None), (128, 4), (512, 12)):
                out = torch.full((T, Hq * d), float("nan"), device=DEV, dtype=torch.bfloat16)
                ops.attention_decode(q.view(T, Hq * d), Hq * d, out, kt(kc), vt(vc), FakeBatch(q_lens, starts, tables), Hq, Hkv, d,
                                     scale, o[0], 0, chunk=chunk, waves=waves, **call_args(ops, o, sink, gate, q.view(T, Hq * d), Hq))
                close(out, ref, 2 ** -7)


def test_attention_decode_merges_many_parts_of_keys_with_sinks_and_gates():
    """More parts than the merging kernel asks for ahead, and heads of each of its sizes."""
    ops = kernels.current()
    for Hq, Hkv, d in ((4, 2, 64), (3, 1, 128), (2, 1, 256)):
        q_lens, starts = [1, 1, 1], [2900, 40, 1500]
        for window, chunked in ((0, False), (2048, True)):
            q, kc, vc, tables, sink, gate = make_case("bfloat16", Hq, Hkv, d, q_lens, starts, window, chunked, 3)
            o, scale = (window, chunked, 0.0, True, True), 1.0 / math.sqrt(d)
            ref = attention_reference(q, kc, vc, tables, q_lens, starts, Hq, Hkv, d, scale, window, chunked, 0.0, sink, gate)
            for chunk in (128, 256):
                out = torch.full((3, Hq * d), float("nan"), device=DEV, dtype=torch.bfloat16)
                ops.attention_decode(q.view(3, Hq * d), Hq * d, out, kt(kc), vt(vc), FakeBatch(q_lens, starts, tables), Hq, Hkv, d,
                                     scale, window, 0, chunk=chunk, waves=4, **call_args(ops, o, sink, gate, q.view(3, Hq * d), Hq))
                close(out, ref, 2 ** -7)


@pytest.mark.parametrize("Hq,Hkv,d", [(4, 2, 16), (6, 2, 64), (8, 1, 128), (3, 3, 48), (10, 2, 80), (9, 3, 112), (2, 1, 256)])
def test_attention_prefill(Hq, Hkv, d):
    ops = kernels.current()
    tile = kernels.library.load().ra_attention_prefill_tile(Hq, Hkv, d)
    for bi, (q_lens, starts) in enumerate(PRE_BATCHES[1:]):
        info, t = [], 0
        for i, (ql, st) in enumerate(zip(q_lens, starts)):
            for q0 in range(0, ql, tile):
                info += [i, t + q0, min(tile, ql - q0), st + q0]
            t += ql
        i32 = lambda v: torch.tensor(v, dtype=torch.int32, device=DEV)
        # every other tile cut by keys into parts of two rounds of 64, added by the second kernel
        items, merge, n_slots = [], [], 0
        for k in range(len(info) // 4):
            i, row, n, pos = info[4 * k:4 * k + 4]
            parts = -(-(-(-(pos + n) // 64)) // 2)
            if k % 2 == 1 or parts < 2:
                items.append(((i, row, n, pos), (0, 1 << 30, -1)))
                continue
            merge += [row, n, n_slots, parts]
            for c in range(parts):
                items.append(((i, row, n, pos), (c * 128, (c + 1) * 128 if c + 1 < parts else 1 << 30, n_slots + c)))
            n_slots += parts
        for o in OPTIONS:
            q, kc, vc, tables, sink, gate = make_case("bfloat16", Hq, Hkv, d, q_lens, starts, o[0], o[1], 20 + bi)
            batch, T, scale = FakeBatch(q_lens, starts, tables), sum(q_lens), 1.0 / math.sqrt(d)
            w, ch, cap, s, gt = options(o, sink, gate)
            ref = attention_reference(q, kc, vc, tables, q_lens, starts, Hq, Hkv, d, scale, w, ch, cap, s, gt)
            more = call_args(ops, o, sink, gate, q.view(T, Hq * d), Hq)
            out = torch.full((T, Hq * d), float("nan"), device=DEV, dtype=torch.bfloat16)
            ops.attention_prefill(q.view(T, Hq * d), Hq * d, out, kt(kc), vt(vc), batch, Hq, Hkv, d, scale, o[0], 0, i32(info),
                                  len(info) // 4, **more)
            close(out, ref, 2 ** -7)
            if merge:
                out2 = torch.full((T, Hq * d), float("nan"), device=DEV, dtype=torch.bfloat16)
                ops.attention_prefill(q.view(T, Hq * d), Hq * d, out2, kt(kc), vt(vc), batch, Hq, Hkv, d, scale, o[0], 0,
                                      i32([v for it in items for v in it[0]]), len(items), i32([v for it in items for v in it[1]]),
                                      i32(merge), len(merge) // 4, n_slots, **more)
                close(out2, ref, 2 ** -7)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_attention_dispatch_passes_chunks_sinks_and_gates_on(dtype):
    """Mixed steps (single tokens beside portions, one deep in its prompt) through ``attention``: whatever kernels it picks and
    however it lists and cuts the tiles, all three are in the result."""
    ops = kernels.current()
    for Hq, Hkv, d, chunk in ((6, 3, 96, 50), (8, 2, 64, 300), (20, 1, 32, 50)):
        q_lens, starts = [1, 70, 1, 3, 200, 1, 1, 1, 1, 1, 1], [260, 0, 17, 40, 900, 5, 90, 300, 33, 64, 128]
        q, kc, vc, tables, sink, gate = make_case(dtype, Hq, Hkv, d, q_lens, starts, chunk, True, 5)
        T, scale = sum(q_lens), 1.0 / math.sqrt(d)
        rows = torch.zeros(T, Hq * d + -(-Hq // 16) * 16, device=DEV, dtype=DT[dtype])               # gates behind the heads
        rows[:, :Hq * d], rows[:, Hq * d:Hq * d + Hq] = q.view(T, Hq * d), gate
        out = torch.full((T, Hq * d), float("nan"), device=DEV, dtype=DT[dtype])
        ops.attention(rows, rows.stride(0), out, kt(kc), vt(vc), FakeBatch(q_lens, starts, tables), Hq, Hkv, d, scale, chunk, 0,
                      softcap=3.0, aligned=True, sink=sink, gate=rows[:, Hq * d:])
        ref = attention_reference(q, kc, vc, tables, q_lens, starts, Hq, Hkv, d, scale, chunk, True, 3.0, sink, gate)
        close(out, ref, 2 ** -7 if dtype == "bfloat16" else 2e-5)
        for other in (attention_reference(q, kc, vc, tables, q_lens, starts, Hq, Hkv, d, scale, chunk, True, 3.0, None, gate),
                      attention_reference(q, kc, vc, tables, q_lens, starts, Hq, Hkv, d, scale, chunk, True, 3.0, sink, None)):
            assert float((other - ref).abs().max()) > 0.1 * float(ref.abs().max())     # neither is small here


def test_attention_refuses_what_it_does_not_take():
    ops = kernels.current()
    q, kc, vc, tables, sink, gate = make_case("float32", 4, 2, 16, [1], [3], 0, False, 1)
    call = lambda **kw: ops.attention(q.view(1, 64), 64, torch.empty(1, 64, device=DEV), kt(kc), vt(vc),
                                      FakeBatch([1], [3], tables), 4, 2, 16, 0.2, 8, 0, **kw)
    for bad in ({"aligned": True, "keep": 2}, {"sink": sink[:3]}, {"sink": sink.double()}, {"gate": gate[:, :3]},
                {"gate": gate.to(torch.bfloat16)}):
        with pytest.raises(ValueError):
            call(**bad)


# ------------------------------------------------------------------ the head kernel
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("Hq,Hkv,d,rot,style", [(4, 2, 16, 16, 0), (6, 3, 64, 64, 0), (8, 1, 128, 128, 0), (5, 5, 48, 0, 0),
                                                (2, 1, 256, 256, 0), (3, 3, 96, 32, 1)])
@pytest.mark.parametrize("T", [11, 45, 203])
def test_head_kernel_on_wider_rows_and_on_queries_alone(dtype, Hq, Hkv, d, rot, style, T):
    """Rows with other columns behind the heads give what rows of the heads alone give and leave those columns as they are;
    rows of queries alone give the same queries."""
    ops = kernels.current()
    torch.manual_seed(d + T)
    width = (Hq + 2 * Hkv) * d
    rows = torch.randn(T, width + 16, device=DEV).to(DT[dtype])
    src = rows.clone()
    alone = src[:, :width].contiguous()
    q_only = torch.cat([src[:, :Hq * d], src[:, width:]], dim=1).contiguous()
    w = torch.rand(d, device=DEV) + 0.5
    slots = torch.tensor([-1 if t == 5 else 32 + t for t in range(T)], dtype=torch.int32, device=DEV)
    pos = ((torch.arange(T, dtype=torch.int32) * 5) % 128).to(DEV)
    inv = (10000.0 ** (-torch.arange(0, max(rot, 2), 2).double() / max(rot, 2))).float().to(DEV)
    caches = [[torch.zeros((T // 16 + 4, Hkv, 1, 16 * d), device=DEV, dtype=DT[dtype]) for _ in "kv"] for _ in range(2)]
    call = lambda x, kc, vc, G: ops.qk_norm_rope_cache(x, w, w, 1e-6, pos, inv, rot, style, slots, kc, vc, Hq, G, d)
    call(alone, *caches[0], Hkv)
    call(rows, *caches[1], Hkv)
    call(q_only, None, None, 0)
    assert torch.equal(rows[:, width:], src[:, width:]) and torch.equal(q_only[:, Hq * d:], src[:, width:])
    assert torch.equal(rows[:, :Hq * d], alone[:, :Hq * d]) and torch.equal(q_only[:, :Hq * d], alone[:, :Hq * d])
    assert all(torch.equal(a, b) for a, b in zip(*caches))
    x = src[:, :Hq * d].float().view(T, Hq, d)
    assert not torch.equal(alone[:, :Hq * d], src[:, :Hq * d]) and float(x.abs().max()) > 0


# ------------------------------------------------------------------ the latent's rotation
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("H,D,R,rank,rot,style,amp", [(3, 20, 12, 40, 12, 1, 1.2), (2, 16, 8, 24, 6, 1, 1.0), (5, 0, 32, 17, 32, 0, 1.4),
                                                      (4, 48, 16, 112, 16, 1, 0.1 * math.log(8.0) + 1.0), (2, 8, 0, 16, 0, 0, 1.0)])
def test_latent_prep_turns_neighbours_and_takes_a_factor(dtype, H, D, R, rank, rot, style, amp):
    ops = kernels.current()
    torch.manual_seed(rank)
    T = 21
    pad8 = lambda n: -(-n // 8) * 8
    dkv_off = pad8(H * (D + R))
    proj = torch.randn(T, dkv_off + pad8(rank + R), device=DEV).to(DT[dtype])
    w = (torch.rand(rank, device=DEV) + 0.5).to(DT[dtype])
    Dp = -(-(rank + R) // 16) * 16
    pos = (torch.arange(T, dtype=torch.int32) * 37).to(DEV)
    inv = (500.0 ** (-torch.arange(0, max(rot, 2), 2).double() / max(rot, 2))).float().to(DEV)
    slots = torch.tensor([-1 if t == 3 else 16 + t for t in range(T)], dtype=torch.int32, device=DEV)

    def run(k, dev):
        to = lambda x: x.to(dev)
        q_lat = torch.zeros(T, H, Dp, dtype=DT[dtype], device=dev)
        kc, vc = (torch.zeros(4, 1, 1, 16 * Dp, dtype=DT[dtype], device=dev) for _ in "kv")
        k.latent_prep(to(proj), 0, dkv_off, to(w), 1e-5, to(pos), to(inv), rot, R, rank, H, D, q_lat, to(slots), kc, vc,
                      rope_style=style, amp=amp)
        return q_lat[:, :, rank:], unpack_k(kc, Dp), unpack_v(vc, Dp)
    for got, want in zip(run(ops, DEV), run(KernelDouble(), "cpu")):
        if got.numel():
            close(got, want, 1e-5 if dtype == "float32" else 2 ** -7)
