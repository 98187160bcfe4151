"""The kernels that came with Sagalorn, each against a plain PyTorch form of the same operation: the three attention kernels
with a window that keeps the first keys (single tokens through chunks of keys, portions in query tiles whole and cut by
keys, the float kernel; with and without a change of the scores), the head kernel where the values are the keys, retention
and gated linear attention token by token and in chunks (key sizes on either side of every switch, both forms taking turns
on one state, factors of 0 and 1, gates that close within a chunk), the norm and gate of narrow heads with and without a
weight, and the step of several residual streams. Several requests of unequal length in one call, calls that go on from the
state the calls before left, a request that starts afresh in a slot that was used, and padding rows (state slot -1) that must
leave every state alone."""
import pytest
import torch

from kernel_double import KernelDouble
from reinfer_amd import kernels
from reinfer_amd.cache.layout import unpack_k, unpack_v
from test_gpu_detatar_kernels import CALLS, close, make_batch
from test_gpu_kernels import DEC_BATCHES, DT, PRE_BATCHES, FakeBatch, kt, vt

pytestmark = pytest.mark.gpu
DEV = "cuda:0"


# ------------------------------------------------------------------ a window that keeps the first keys
def make_kept_case(dtype, Hq, Hkv, d, q_lens, starts, window, keep, seed, bs=16):
    """Queries, caches and tables as the engine leaves them: blocks that neither the window of a request's first query nor
    the kept keys need have been given back, their table entries read 0, and block 0 and every slot never written hold NaN."""
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
        for b in range(need[i]):
            if window > 0 and (b + 1) * bs - 1 < starts[i] - window + 1 and b * bs >= keep:
                continue
            blk = perm[p]
            p += 1
            tables[i, b] = blk
            fill = min(bs, ctx[i] - b * bs)
            kc[blk, :, :fill] = torch.randn(Hkv, fill, d, generator=g)
            vc[blk, :, :fill] = torch.randn(Hkv, fill, d, generator=g)
    q = torch.randn(sum(q_lens), Hq, d, generator=g)
    return q.to(DT[dtype]).to(DEV), kc.to(DT[dtype]).to(DEV), vc.to(DT[dtype]).to(DEV), tables.to(DEV)


def kept_reference(q, kc, vc, tables, q_lens, starts, Hq, Hkv, d, scale, window, keep, cap=0.0):
    bs = kc.shape[2]
    kc, vc, q, tables = kc.double().cpu(), vc.double().cpu(), q.double().cpu(), tables.cpu()
    out, t0 = [], 0
    for i, (ql, st) in enumerate(zip(q_lens, starts)):
        for j in range(ql):
            p = st + j
            keys = torch.tensor([x for x in range(p + 1) if window == 0 or p - x < window or x < keep])
            blk = tables[i, keys // bs].long()
            K, V = kc[blk, :, keys % bs, :], vc[blk, :, keys % bs, :]
            row = []
            for a in range(Hq):
                s = (K[:, a // (Hq // Hkv)] @ q[t0 + j, a]) * scale
                if cap:
                    s = cap * torch.tanh(s / cap)
                row.append(torch.softmax(s, 0) @ V[:, a // (Hq // Hkv)])
            out.append(torch.cat(row))
        t0 += ql
    return torch.stack(out)


# window, kept: within a tile, a tile exactly, over tiles and rounds of 64, overlapping the window, no window
MASKS = [(19, 1), (19, 16), (150, 5), (16, 70), (1, 130), (33, 17), (0, 9), (200, 64)]


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("Hq,Hkv,d", [(4, 2, 16), (6, 3, 96), (8, 1, 128)])
def test_attention_plain_keeps_the_first_keys(dtype, Hq, Hkv, d):
    ops = kernels.current()
    for bi, (q_lens, starts) in enumerate([([1, 1, 1], [31, 32, 300]), ([2, 17, 1, 40], [0, 30, 99, 1])]):
        for window, keep in MASKS:
            q, kc, vc, tables = make_kept_case(dtype, Hq, Hkv, d, q_lens, starts, window, keep, bi)
            batch, T = FakeBatch(q_lens, starts, tables), sum(q_lens)
            out = torch.empty(T, Hq * d, device=DEV, dtype=DT[dtype])
            ops.attention_plain(q.view(T, Hq * d), Hq * d, out, kt(kc), vt(vc), batch, Hq, Hkv, d, 0.2, window, 0, keep=keep)
            ref = kept_reference(q, kc, vc, tables, q_lens, starts, Hq, Hkv, d, 0.2, window, keep)
            close(out, ref, 2e-5 if dtype == "float32" else 2 ** -7, (bi, window, keep))


@pytest.mark.parametrize("Hq,Hkv,d", [(4, 2, 16), (6, 2, 64), (8, 1, 128), (3, 3, 48), (2, 1, 256)])
def test_attention_decode_keeps_the_first_keys(Hq, Hkv, d):
    ops = kernels.current()
    for bi, (q_lens, starts) in enumerate(DEC_BATCHES[:6]):
        for window, keep in MASKS:
            q, kc, vc, tables = make_kept_case("bfloat16", Hq, Hkv, d, q_lens, starts, window, keep, 10 + bi)
            batch, T = FakeBatch(q_lens, starts, tables), sum(q_lens)
            ref = kept_reference(q, kc, vc, tables, q_lens, starts, Hq, Hkv, d, 0.2, window, keep)
            for chunk, waves in ((None, None), (128, 4), (512, 12)):
                out = torch.full((T, Hq * d), float("nan"), device=DEV, dtype=torch.bfloat16)
                ops.attention_decode(q.view(T, Hq * d), Hq * d, out, kt(kc), vt(vc), batch, Hq, Hkv, d, 0.2, window, 0,
                                     chunk=chunk, waves=waves, keep=keep)
                close(out, ref, 2 ** -7, (bi, window, keep, chunk))
        q, kc, vc, tables = make_kept_case("bfloat16", Hq, Hkv, d, q_lens, starts, 19, 20, 30 + bi)
        out = torch.full((T, Hq * d), float("nan"), device=DEV, dtype=torch.bfloat16)
        ops.attention_decode(q.view(T, Hq * d), Hq * d, out, kt(kc), vt(vc), FakeBatch(q_lens, starts, tables), Hq, Hkv, d,
                             0.2, 19, 0, keep=20, mod=ops._score_mod(0.5, None, Hq, q.device))
        close(out, kept_reference(q, kc, vc, tables, q_lens, starts, Hq, Hkv, d, 0.2, 19, 20, cap=0.5), 2 ** -7, (bi, "capped"))


@pytest.mark.parametrize("Hq,Hkv,d", [(4, 2, 16), (6, 2, 64), (8, 1, 128), (3, 3, 48), (2, 1, 256)])
def test_attention_prefill_keeps_the_first_keys(Hq, Hkv, d):
    ops = kernels.current()
    tile = kernels.library.load().ra_attention_prefill_tile(Hq, Hkv, d)
    for bi, (q_lens, starts) in enumerate(PRE_BATCHES[1:]):
        info, t = [], 0
        for i, (ql, st) in enumerate(zip(q_lens, starts)):
            for q0 in range(0, ql, tile):
                info += [i, t + q0, min(tile, ql - q0), st + q0]
            t += ql
        tiles = torch.tensor(info, dtype=torch.int32, device=DEV)
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
        i32 = lambda v: torch.tensor(v, dtype=torch.int32, device=DEV)
        for window, keep in MASKS:
            q, kc, vc, tables = make_kept_case("bfloat16", Hq, Hkv, d, q_lens, starts, window, keep, 20 + bi)
            batch, T = FakeBatch(q_lens, starts, tables), sum(q_lens)
            ref = kept_reference(q, kc, vc, tables, q_lens, starts, Hq, Hkv, d, 0.2, window, keep)
            out = torch.full((T, Hq * d), float("nan"), device=DEV, dtype=torch.bfloat16)
            ops.attention_prefill(q.view(T, Hq * d), Hq * d, out, kt(kc), vt(vc), batch, Hq, Hkv, d, 0.2, window, 0, tiles,
                                  len(info) // 4, keep=keep)
            close(out, ref, 2 ** -7, (bi, window, keep))
            if merge:
                out2 = torch.full((T, Hq * d), float("nan"), device=DEV, dtype=torch.bfloat16)
                ops.attention_prefill(q.view(T, Hq * d), Hq * d, out2, kt(kc), vt(vc), batch, Hq, Hkv, d, 0.2, window, 0,
                                      i32([v for it in items for v in it[0]]), len(items), i32([v for it in items for v in it[1]]),
                                      i32(merge), len(merge) // 4, n_slots, keep=keep)
                close(out2, ref, 2 ** -7, (bi, window, keep, "cut"))


def test_attention_dispatch_passes_the_kept_keys_on():
    """A mixed step (single tokens beside portions) through ``attention``: whatever kernels it picks, the kept keys are in
    the result."""
    ops = kernels.current()
    Hq, Hkv, d = 6, 3, 96
    q_lens, starts = [1, 70, 1, 3, 200, 1, 1, 1, 1, 1, 1], [260, 0, 17, 40, 100, 5, 90, 300, 33, 64, 128]
    for dtype in ("bfloat16", "float32"):
        q, kc, vc, tables = make_kept_case(dtype, Hq, Hkv, d, q_lens, starts, 50, 7, 5)
        T = sum(q_lens)
        out = torch.full((T, Hq * d), float("nan"), device=DEV, dtype=DT[dtype])
        ops.attention(q.view(T, Hq * d), Hq * d, out, kt(kc), vt(vc), FakeBatch(q_lens, starts, tables), Hq, Hkv, d, 0.2, 50,
                      0, keep=7)
        ref = kept_reference(q, kc, vc, tables, q_lens, starts, Hq, Hkv, d, 0.2, 50, 7)
        close(out, ref, 2 ** -7 if dtype == "bfloat16" else 2e-5, dtype)
        less = kept_reference(q, kc, vc, tables, q_lens, starts, Hq, Hkv, d, 0.2, 50, 6)
        assert float((less - ref).abs().max()) > 0.1          # one kept key fewer is not small here


# ------------------------------------------------------------------ values that are the keys
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("Hq,Hkv,d,rot", [(4, 2, 16, 16), (6, 3, 64, 64), (8, 1, 128, 128), (5, 5, 48, 0), (2, 1, 256, 256),
                                          (3, 3, 96, 32)])
@pytest.mark.parametrize("T", [11, 45, 203])
def test_values_are_the_keys_before_norm_and_rotation(dtype, Hq, Hkv, d, rot, T):
    ops = kernels.current()
    torch.manual_seed(d + T)
    qkv = torch.randn(T, (Hq + Hkv) * d, device=DEV).to(DT[dtype])
    src = qkv.clone()
    qw, kw = (torch.rand(d, device=DEV) + 0.5).to(DT[dtype]), (torch.rand(d, device=DEV) + 0.5).to(DT[dtype])
    slots_l = [32 + t for t in range(T)]
    slots_l[5] = -1
    pos = ((torch.arange(T, dtype=torch.int32) * 5) % 128).to(DEV)
    nblk = T // 16 + 4
    kc = torch.full((nblk, Hkv, 1, 16 * d), float("nan"), device=DEV, dtype=DT[dtype])
    vc = torch.full_like(kc, float("nan"))
    inv = (10000.0 ** (-torch.arange(0, max(rot, 2), 2).double() / max(rot, 2))).float().to(DEV)
    ops.qk_norm_rope_cache(qkv, qw, kw, 1e-6, pos, inv, rot, 0, torch.tensor(slots_l, dtype=torch.int32, device=DEV), kc, vc,
                           Hq, Hkv, d, values_are_keys=True)
    # the same keys through rows that hold them twice
    three = torch.cat([src, src[:, Hq * d:]], dim=1).contiguous()
    kc2, vc2 = torch.full_like(kc, float("nan")), torch.full_like(kc, float("nan"))
    ops.qk_norm_rope_cache(three, qw, kw, 1e-6, pos, inv, rot, 0, torch.tensor(slots_l, dtype=torch.int32, device=DEV), kc2, vc2,
                           Hq, Hkv, d)
    assert torch.equal(qkv[:, :Hq * d], three[:, :Hq * d]) and torch.equal(qkv[:, Hq * d:], src[:, Hq * d:])
    assert torch.equal(torch.nan_to_num(kc), torch.nan_to_num(kc2)) and torch.equal(torch.nan_to_num(vc), torch.nan_to_num(vc2))
    k, v = unpack_k(kc, d), unpack_v(vc, d)
    for t, s in enumerate(slots_l):
        if s >= 0:
            assert torch.equal(v[s // 16, :, s % 16], src[t, Hq * d:].view(Hkv, d))
            assert not torch.equal(k[s // 16, :, s % 16], v[s // 16, :, s % 16])


# ------------------------------------------------------------------ linear attention
# key sizes: one lane run and more, rows that are whole 16-byte pieces and not, both sides of 32, 64, 128, 256
SHAPES = [(2, 32, 32), (3, 20, 12), (1, 136, 8), (4, 64, 32), (1, 8, 40), (5, 12, 12), (2, 4, 6), (1, 40, 8), (2, 128, 64),
          (2, 96, 17), (1, 256, 16), (1, 300, 16), (9, 16, 16)]
FORMS = ["tokens", "chunks", "turns"]


def form_of(form, call, dk):
    if dk > 256:
        return None                          # chunks take keys up to 256: the dispatch's own choice
    return {"tokens": False, "chunks": True, "turns": call % 2 == 0}[form]


def with_positions(batch, starts, device):
    pos = [s + j for s, q in zip(starts, batch.q_lens) for j in range(q)]
    batch.positions = torch.tensor(pos, dtype=torch.int32, device=device)
    return batch


@pytest.mark.parametrize("form", FORMS)
@pytest.mark.parametrize("H,dk,dv", SHAPES)
@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
def test_retention(H, dk, dv, dtype, form):
    ops, ref = kernels.current(), KernelDouble()
    g = torch.Generator().manual_seed(H * 1000 + dk)
    nk, nv = H * dk, H * dv
    lead = 8 if dk % 8 == 0 else 2                         # aligned rows where the shape allows the vector forms
    width = -(-(lead + 2 * nk + nv + 9) // 8) * 8
    q_off, k_off, v_off = lead, lead + nk, lead + 2 * nk
    decays = torch.rand(H, generator=g) * 0.6 + 0.399
    decays[0] = 1.0
    decays[-1] = 0.0 if H > 2 else decays[-1]
    for rot in sorted({0, dk - dk % 2, dk // 2 - (dk // 2) % 2, 16 if dk >= 16 else 2}):
        inv = (1000.0 ** (-torch.arange(0, max(rot, 2), 2).double() / max(rot, 2))).float()
        st_gpu = torch.full((4, ops.scan_state_floats("decay_memory", H, dk, dv) + 3), float("nan"), device=DEV)
        st_ref = torch.full((4, ref.scan_state_floats("decay_memory", H, dk, dv) + 3), float("nan"))
        for i, (q_lens, slots, fresh) in enumerate(CALLS):
            T = sum(q_lens)
            starts = [0 if f else 17 * (i + 1) + s for f, s in zip(fresh, range(len(q_lens)))]
            proj = (torch.randn(T, width, generator=g) * 0.9).to(dtype)
            out_ref, out = torch.empty(T, nv), torch.empty(T, nv, device=DEV)
            more = dict(act="none", rot_dims=rot, q_scale=1.5, k_scale=0.3)
            ref.decay_scan(proj, q_off, k_off, v_off, decays, st_ref,
                           with_positions(make_batch(q_lens, slots, fresh, "cpu"), starts, "cpu"), H, dk, dv, out_ref,
                           inv_freq=inv, **more)
            before = st_gpu.clone()
            ops.decay_scan(proj.to(DEV), q_off, k_off, v_off, decays.to(DEV), st_gpu,
                           with_positions(make_batch(q_lens, slots, fresh, DEV), starts, DEV), H, dk, dv, out,
                           inv_freq=inv.to(DEV), chunks=form_of(form, i, dk), **more)
            close(out, out_ref, 2e-5, (rot, f"call {i}"))
            untouched = [s for s in range(4) if s not in slots]
            assert torch.equal(torch.nan_to_num(st_gpu[untouched], nan=7.0), torch.nan_to_num(before[untouched], nan=7.0))
            assert torch.isnan(st_gpu[:, -3:]).all()


@pytest.mark.parametrize("H,dk,dv", [(3, 20, 12), (4, 64, 32), (2, 128, 64), (1, 136, 8)])
@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
def test_the_fading_memory_with_silu_in_chunks(H, dk, dv, dtype):
    ops, ref = kernels.current(), KernelDouble()
    g = torch.Generator().manual_seed(dk)
    nk, nv = H * dk, H * dv
    decays = torch.rand(H, generator=g) * 0.6 + 0.399
    st_gpu = torch.full((4, ops.scan_state_floats("decay_memory", H, dk, dv)), float("nan"), device=DEV)
    st_ref = torch.full((4, ref.scan_state_floats("decay_memory", H, dk, dv)), float("nan"))
    for i, (q_lens, slots, fresh) in enumerate(CALLS):
        T = sum(q_lens)
        proj = (torch.randn(T, 2 * nk + nv, generator=g) * 0.9).to(dtype)
        out_ref, out = torch.empty(T, nv), torch.empty(T, nv, device=DEV)
        ref.decay_scan(proj, 0, nk, 2 * nk, decays, st_ref, make_batch(q_lens, slots, fresh, "cpu"), H, dk, dv, out_ref)
        ops.decay_scan(proj.to(DEV), 0, nk, 2 * nk, decays.to(DEV), st_gpu, make_batch(q_lens, slots, fresh, DEV), H, dk, dv,
                       out, chunks=i != 1)
        close(out, out_ref, 2e-5, f"call {i}")


@pytest.mark.parametrize("form", FORMS)
@pytest.mark.parametrize("H,dk,dv", SHAPES)
@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
def test_gated_linear_attention(H, dk, dv, dtype, form):
    """Gates of every kind side by side: open, half open, nearly closed (a chunk's product below 2^-60, and far below what a
    float holds) and closed."""
    ops, ref = kernels.current(), KernelDouble()
    g = torch.Generator().manual_seed(H * 1000 + dk)
    nk, nv = H * dk, H * dv
    lead = 8 if dk % 8 == 0 else 2
    width = -(-(lead + 2 * nk + nv + 9) // 8) * 8
    q_off, k_off, v_off = lead, lead + nk, lead + 2 * nk
    for tau, kinds in ((16.0, (0.0, 3.0)), (1.0, (0.0, -6.0, -40.0, 4.0)), (2.5, (-200.0, 1.0))):
        bias = torch.randn(nk, generator=g)
        for j, shift in enumerate(kinds):
            bias[j::len(kinds)] += shift
        st_gpu = torch.full((4, ops.scan_state_floats("gated_linear", H, dk, dv) + 3), float("nan"), device=DEV)
        st_ref = torch.full((4, ref.scan_state_floats("gated_linear", H, dk, dv) + 3), float("nan"))
        for i, (q_lens, slots, fresh) in enumerate(CALLS):
            T = sum(q_lens)
            proj = (torch.randn(T, width, generator=g) * 0.9).to(dtype)
            z = torch.randn(T, nk + 5, generator=g) * 1.5                   # rows wider than needed
            out_ref, out = torch.empty(T, nv), torch.empty(T, nv, device=DEV)
            ref.gated_linear_scan(proj, q_off, k_off, v_off, z, bias, tau, st_ref, make_batch(q_lens, slots, fresh, "cpu"), H,
                                  dk, dv, out_ref, q_scale=0.4)
            before = st_gpu.clone()
            ops.gated_linear_scan(proj.to(DEV), q_off, k_off, v_off, z.to(DEV), bias.to(DEV), tau, st_gpu,
                                  make_batch(q_lens, slots, fresh, DEV), H, dk, dv, out, q_scale=0.4,
                                  chunks=form_of(form, i, dk))
            close(out, out_ref, 2e-5, (tau, f"call {i}"))
            untouched = [s for s in range(4) if s not in slots]
            assert torch.equal(torch.nan_to_num(st_gpu[untouched], nan=7.0), torch.nan_to_num(before[untouched], nan=7.0))
            assert torch.isnan(st_gpu[:, -3:]).all()


def test_linear_attention_over_a_long_portion():
    """A thousand tokens in one portion: the chunks against the scan, a slow head, rotation at positions up to 30,000."""
    ops = kernels.current()
    g = torch.Generator().manual_seed(3)
    H, dk, dv, T = 4, 64, 48, 1003
    nk, nv = H * dk, H * dv
    proj = torch.randn(T, 2 * nk + nv, generator=g).to(torch.bfloat16).to(DEV)
    decays = torch.tensor([0.9999, 0.99, 0.5, 0.0], device=DEV)
    inv = (10000.0 ** (-torch.arange(0, dk, 2).double() / dk)).float().to(DEV)
    z = torch.randn(T, nk, generator=g).to(DEV) + 3.0
    bias = torch.randn(nk, generator=g).to(DEV)
    batch = with_positions(make_batch([T], [0], [1], DEV), [29000], DEV)
    outs = {}
    for chunks in (False, True):
        st = torch.full((1, ops.scan_state_floats("decay_memory", H, dk, dv)), float("nan"), device=DEV)
        a, b = torch.empty(T, nv, device=DEV), torch.empty(T, nv, device=DEV)
        ops.decay_scan(proj, 0, nk, 2 * nk, decays, st, batch, H, dk, dv, a, act="none", inv_freq=inv, rot_dims=dk,
                       k_scale=dk ** -0.5, chunks=chunks)
        st2 = torch.full((1, ops.scan_state_floats("gated_linear", H, dk, dv)), float("nan"), device=DEV)
        ops.gated_linear_scan(proj, 0, nk, 2 * nk, z, bias, 16.0, st2, batch, H, dk, dv, b, chunks=chunks)
        outs[chunks] = (a, b, st, st2)
    for x, y, what in zip(outs[True], outs[False], ("retention", "gla", "retention state", "gla state")):
        close(x, y, 2e-5, what)


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("H,dv", [(3, 8), (5, 16), (2, 64), (7, 128), (1, 256), (3, 512), (4, 12), (3, 40), (2, 96)])
def test_norm_and_gate_of_narrow_heads_with_and_without_a_weight(dtype, H, dv):
    ops, ref = kernels.current(), KernelDouble()
    g = torch.Generator().manual_seed(dv)
    T, n = 11, H * dv
    read = torch.randn(T, n, generator=g) * 3
    gate = torch.randn(T, n + 16, generator=g).to(dtype)
    for kind in ("sigmoid", "silu"):
        for weight, per_head in ((None, False), (torch.rand(dv, generator=g) + 0.5, False), (torch.rand(n, generator=g) + 0.5, True)):
            want, got = torch.empty(T, n, dtype=dtype), torch.empty(T, n, dtype=dtype, device=DEV)
            ref.head_norm_gate(read, weight, per_head, gate, kind, 1e-5, H, dv, want)
            ops.head_norm_gate(read.to(DEV), weight.to(DEV) if weight is not None else None, per_head, gate.to(DEV), kind,
                               1e-5, H, dv, got)
            close(got, want, 2e-6 if dtype == torch.float32 else 2 ** -8, (kind, per_head))


# ------------------------------------------------------------------ several residual streams
@pytest.mark.parametrize("n", [1, 2, 3, 4, 5, 6, 7, 8])
@pytest.mark.parametrize("h", [36, 42, 256, 2048, 4096, 8192, 9000])
def test_hyper_step(n, h):
    ops, ref = kernels.current(), KernelDouble()
    g = torch.Generator().manual_seed(n * 10000 + h)
    for T in ((5, 600) if h <= 256 or (h == 2048 and n == 4) else (5,)):
        X = torch.randn(T, n, h, generator=g)
        base = torch.randn(T, h, generator=g)
        mix, w_out, w_in = torch.randn(n, n, generator=g), torch.randn(n, generator=g), torch.randn(n, generator=g)
        weight = torch.rand(h, generator=g) + 0.5
        rows = torch.tensor([T - 1, 0, 3], dtype=torch.int32)
        dv = lambda t: t.to(DEV) if t is not None else None
        for y_dtype, o_dtype in ((torch.float32, torch.float32), (torch.bfloat16, torch.bfloat16), (torch.float32, torch.bfloat16)):
            y = torch.randn(T, h, generator=g).to(y_dtype)
            for b, yy, wi, wt, rr, store in ((None, y, w_in, weight, None, True), (base, None, w_in, weight, None, False),
                                             (base, y, w_in, weight, None, True), (None, y, None, weight, rows, False),
                                             (base, y, None, weight, rows, False), (None, y, None, None, None, False)):
                x_ref, x_gpu = X.clone(), X.to(DEV)
                if b is not None:
                    x_gpu.fill_(float("nan"))                     # nothing is read from the streams yet
                m = T if rr is None else 3
                want, got = torch.empty(m, h, dtype=o_dtype), torch.empty(m, h, dtype=o_dtype, device=DEV)
                mx, wo = (mix, w_out) if yy is not None else (None, None)
                ref.hyper_step(x_ref, b, yy, mx, wo, wi, wt, 1e-5, want, rows=rr, store=store)
                before = x_gpu.clone()
                ops.hyper_step(x_gpu, dv(b), dv(yy), dv(mx), dv(wo), dv(wi), dv(wt), 1e-5, got, rows=dv(rr), store=store)
                close(got, want, 5e-6 if o_dtype == torch.float32 else 2 ** -8, (T, y_dtype, b is not None, rr is not None))
                if store:
                    close(x_gpu, x_ref, 5e-6, (T, "streams"))
                else:
                    assert torch.equal(torch.nan_to_num(x_gpu, nan=3.0), torch.nan_to_num(before, nan=3.0))


def test_hyper_step_refuses_what_it_does_not_take():
    ops = kernels.current()
    X, out = torch.zeros(2, 3, 8, device=DEV), torch.zeros(2, 8, device=DEV)
    with pytest.raises(ValueError):
        ops.hyper_step(X, None, out, None, None, None, None, 0.0, out)           # a result without its mix
    with pytest.raises(ValueError):
        ops.hyper_step(X, None, None, None, None, torch.zeros(2, device=DEV), None, 0.0, out)
    with pytest.raises(TypeError):
        ops.hyper_step(X.view(2, 24), None, None, None, None, None, None, 0.0, out)
