"""Dokanex through the engine against the plain implementation: configuration, whole prompts, prompts against token-by-token
decoding, portions down to two tokens, unequal requests in one batch with blocks that are given back and used again, the first
tokens, long decoding, keys far back, at block borders and on either side of a chunk's edge (in layers with keys of their own
and in readers of another layer's with a chunk size of their own), sinks that take all the weight, and greedy generation
through the entry point and the scheduler. Without a GPU the engine's bookkeeping runs on the CPU stand-in for the kernels
(float32); the ``gpu`` tests run the same checks on the real kernels in float32 and bfloat16.
"""
import json
import os

import pytest
import torch

import plain_dokanex as plain
from dokanex_helpers import (CONFIGS, DK_A, TORCH, attn, draw_weights, latent, make_folder, read_folder, sharp,
                             write_folder)
from helpers import random_tokens, rel_err, run_plan
from kernel_double import KernelDouble
from reinfer_amd import LLMEngine, SamplingParams, kernels
from reinfer_amd.config import ConfigError, DokanexConfig, config_from_dict, load_config
from reinfer_amd.config.schema import PositionSpec, YarnSpec
from reinfer_amd.engine import ModelRunner
from reinfer_amd.parts import KVNeed, covering, lookup

# float32: both sides add a few hundred float or double terms in another order over half a dozen layers: 3e-5 of the largest
# logit. bfloat16: one rounding is 2^-9; about a dozen storage roundings a layer, in quadrature over six layers: 1.7e-2 of the
# stream; 5e-2 is three deviations.
TOL = {"float32": 3e-5, "bfloat16": 5e-2}
# What a sublayer reads, makes its queries, keys, values, latents and gates of and returns is off by about this much of itself:
# one rounding to bfloat16, or the rounding of a sum of a few dozen float terms.
ROUNDING = {"float32": 2.0 ** -21, "bfloat16": 2.0 ** -9}


def moved_by_rounding(raw, w, toks, dtype, ref, draws=4):
    """How far the logits at each position move (of the largest logit) when each of these is off by ``ROUNDING``, the largest
    of a few random draws: sharp scores, and heads divided by a small root mean square, amplify what they are made of."""
    g = torch.Generator().manual_seed(1234)
    eps = ROUNDING[dtype]
    noise = lambda x: x * (1.0 + eps * torch.randn(x.shape, generator=g, dtype=torch.float64))
    ref = ref.double()
    moved = [(plain.forward(raw, w, toks, noise=noise) - ref).abs().max(-1).values for _ in range(draws)]
    return torch.stack(moved).max(0).values / ref.abs().max()


def assert_close(got, ref, dtype, what, moved=None):
    """Position by position: no logit further from the reference than the bound, but for one position in fifty (at least
    one), which may be off by up to five times that. The bound is ``TOL`` (of the largest logit) or, where the model's own
    sensitivity there is given (``moved``), four times that if it is more."""
    got, ref = got.double().cpu(), ref.double().cpu()
    assert got.shape == ref.shape and torch.isfinite(got).all(), what
    bound = torch.full((ref.shape[0],), TOL[dtype], dtype=torch.float64)
    if moved is not None:
        bound = torch.maximum(bound, 4.0 * moved)
    per = (got - ref).abs().max(dim=-1).values / ref.abs().max() / bound
    over = int((per > 1.0).sum())
    assert over <= max(1, per.numel() // 50) and float(per.max()) < 5.0, (what, over, float(per.max()))


# ------------------------------------------------------------------ configuration
def test_configuration_round_trip_and_spec():
    for which, (raw, _) in CONFIGS.items():
        cfg = config_from_dict(raw)
        assert isinstance(cfg, DokanexConfig)
        assert config_from_dict(cfg.to_dict()) == cfg, which
    spec = config_from_dict(DK_A).to_spec()
    assert [b.kind for b in spec.blocks] == ["prenorm"] * 4
    assert [b.mixer.kind for b in spec.blocks] == ["gqa_attention", "latent_attention"] * 2
    assert [(e.block, e.cache_from) for e in spec.run_order] == [(0, None), (1, None), (2, 0), (3, None)]
    assert spec.tie_embeddings and spec.embed_scale == 4.0 and spec.logit_softcap == 12.0
    a, l, r = (spec.blocks[i].mixer for i in range(3))
    assert (a.num_heads, a.num_kv_heads, a.head_dim, a.value_dim, a.window, a.softcap) == (4, 2, 24, 16, 21, 4.0)
    assert a.chunked and a.sink and a.head_gate and a.qk_norm and not a.qk_norm_weights and not a.kv_shared
    assert a.position.kind == "none" and a.scale == 1.5 * 24 ** -0.5
    assert r.kv_shared and r.window == 42 and r.softcap == 6.0
    p = l.params
    assert (l.num_heads, l.head_dim, p.rot_width, p.value_dim, p.q_rank, p.rank) == (3, 20, 12, 24, 28, 40) and not p.gated
    assert l.position == PositionSpec("rope_interleaved", rotary_dim=12, theta=500.0, scaling=YarnSpec(4.0, 40, 8.0, 1.0))
    assert spec.blocks[0].ffn.intermediate == 96 and spec.blocks[1].ffn is None
    # whatever may be absent is absent
    d = config_from_dict(CONFIGS["D"][0]).to_spec()
    assert d.embed_scale == 1.0 and d.logit_softcap == 0.0
    assert d.blocks[0].mixer.window == 0 and not d.blocks[0].mixer.chunked and d.blocks[0].mixer.softcap == 0.0
    assert d.blocks[1].mixer.position.rotary_dim == 6 and d.blocks[1].mixer.position.scaling is None
    assert d.blocks[2].mixer.position.kind == "none"
    # a layer may leave out its score scale
    raw = json.loads(json.dumps(DK_A))
    del raw["layers"][0]["mixer"]["scale"], raw["layers"][1]["mixer"]["scale"]
    s = config_from_dict(raw).to_spec()
    assert s.blocks[0].mixer.scale == 24 ** -0.5 and s.blocks[1].mixer.scale == 32 ** -0.5


def test_configuration_errors_name_the_key():
    def broken(path, value):
        raw = json.loads(json.dumps(DK_A))
        node = raw
        for k in path[:-1]:
            node = node[k]
        if value is None:
            del node[path[-1]]
        else:
            node[path[-1]] = value
        return raw
    at = ["layers", 0, "mixer"]
    la = ["layers", 1, "mixer"]
    for path, value, key in ((["width"], None, "width"), (["norm", "eps"], None, "norm.eps"),
                             (["logit_softcap"], -1.0, "logit_softcap"), (at + ["kv_heads"], 3, "layers[0].mixer.kv_heads"),
                             (at + ["mask", "size"], 0, "layers[0].mixer.mask.size"),
                             (at + ["softcap"], -2.0, "layers[0].mixer.softcap"),
                             (["layers", 2, "mixer", "kv_from"], 1, "layers[2].mixer.kv_from"),
                             (["layers", 2, "mixer", "kv_from"], 2, "layers[2].mixer.kv_from"),
                             (["layers", 2, "mixer", "dim"], 32, "layers[2].mixer.kv_from"),
                             (la + ["q_rank"], None, "layers[1].mixer.q_rank"), (la + ["kv_rank"], 0, "layers[1].mixer.kv_rank"),
                             (la + ["rot", "dims"], 14, "layers[1].mixer.rot.dims"),
                             (la + ["rot", "dims"], 3, "layers[1].mixer.rot.dims"),
                             (la + ["rot", "base"], -1.0, "layers[1].mixer.rot.base"),
                             (la + ["rot", "scaling", "slow"], None, "layers[1].mixer.rot.scaling.slow"),
                             (la + ["rot", "scaling", "factor"], 0.0, "layers[1].mixer.rot.scaling.factor"),
                             (["layers", 0, "type"], "conv", "layers[0].type"),
                             (["layers", 0, "mlp", "kind"], "moe", "layers[0].mlp.kind"),
                             (["layers", 0, "mlp", "ff"], None, "layers[0].mlp.ff")):
        with pytest.raises(ConfigError) as e:
            config_from_dict(broken(path, value))
        assert e.value.key == key, (path, e.value.key)


def test_the_position_part_has_the_scaled_frequencies():
    for rot in ({"dims": 12, "base": 500.0, "scaling": {"factor": 4.0, "original": 40, "fast": 8.0, "slow": 1.0}},
                {"dims": 10, "base": 2e5, "scaling": {"factor": 10.0, "original": 1500, "fast": 24.0, "slow": 1.0}},
                {"dims": 32, "base": 200.0, "scaling": {"factor": 8.0, "original": 1000, "fast": 2.0, "slow": 2.0}},
                {"dims": 6, "base": 50.0}):
        want, amp = plain.yarn(rot)
        sc = YarnSpec(**rot["scaling"]) if "scaling" in rot else None
        part = lookup("position", "rope_interleaved")(PositionSpec("rope_interleaved", rot["dims"], rot["base"], scaling=sc),
                                                      torch.device("cpu"))
        assert torch.allclose(part.inv_freq.double(), torch.tensor(want, dtype=torch.float64), rtol=1e-7, atol=0)
        assert part.amplitude == pytest.approx(amp, rel=1e-12)
        assert sc is None or (part.inv_freq.double() < torch.tensor([rot["base"] ** (-2 * i / rot["dims"]) * 1.0000001
                                                                     for i in range(rot["dims"] // 2)])).all()


def test_pages_cover_what_every_reader_sees():
    need = lambda w, c=True, keep=0: KVNeed(1, 16, w, keep, c and w > 0)
    assert covering(need(16), need(16)) == need(16)
    assert covering(need(16), need(48)) == need(48) and covering(need(48), need(16)) == need(48)
    assert covering(need(16), need(40)) == need(40, False)            # no multiple: the last 40 tokens hold both chunks
    assert covering(need(16), need(0)) == need(0) and covering(need(0), need(16)) == need(0)
    assert covering(need(16), need(9, False)) == need(16, False)
    assert covering(need(9, False, 3), need(16, False, 1)) == need(16, False, 3)


def test_the_folder_gives_caches_and_groups(tmp_path):
    folder = make_folder(tmp_path, "C", "float32")
    _, w = read_folder(folder)
    assert {"embed", "final.norm", "l0.mix.q", "l0.mix.k", "l0.mix.sink", "l0.mix.g", "l2.mix.dq", "l2.mix.dq.norm", "l2.mix.uq",
            "l2.mix.dkv", "l2.mix.dkv.norm", "l2.mix.uk", "l2.mix.uv", "l0.norm2", "l0.mlp.gate"} <= set(w)
    assert not any(n.startswith(("head", "l1.mix.k", "l1.mix.v", "l1.norm2", "l2.mix.g", "l0.mix.q.norm")) for n in w)
    assert w["l0.mix.sink"].shape == (8,) and w["l0.mix.g"].shape == (8, 96) and w["l3.mix.o"].shape == (96, 6 * 48)
    assert isinstance(load_config(folder), DokanexConfig)
    with kernels.use(KernelDouble()):
        runner = ModelRunner.from_folder(folder, dtype="float32", device="cpu", max_tokens=64)
    # layer 0 sees chunks of 16, its readers chunks of 48 and 40: the last 48 tokens are kept; layer 3 keeps its own chunks,
    # of 40, for a reader of 24: no multiple
    assert sorted((g.window, g.chunked, g.entries) for g in runner.groups) == [(0, False, (2,)), (40, False, (3,)), (48, False, (0,))]
    assert [c.writes for c in runner.caches] == [True, False, True, True, False, False]
    folder = make_folder(tmp_path, "A", "float32")
    with kernels.use(KernelDouble()):
        runner = ModelRunner.from_folder(folder, dtype="float32", device="cpu", max_tokens=64)
    assert sorted((g.window, g.chunked, g.entries) for g in runner.groups) == [(0, False, (1, 3)), (42, True, (0,))]


# ------------------------------------------------------------------ the checks, on either device
def reference(folder, toks, dtype, cache={}):
    """(logits, how far rounding may move each position)"""
    key = (folder, tuple(toks), dtype)
    if key not in cache:
        raw, w = read_folder(folder)
        ref = plain.forward(raw, w, toks).float()
        cache[key] = ref, moved_by_rounding(raw, w, toks, dtype, ref)
    return cache[key]


def runner_for(folder, device, dtype, **limits):
    return ModelRunner.from_folder(folder, dtype=dtype, device=device, **limits)


def vocab(which):
    return CONFIGS[which][0]["vocab"]


def poison_all(runner):
    """Every block starts out as NaN and becomes NaN again when it is given back."""
    for c in runner.paged_caches():
        for t in c.tensors.values():
            t.fill_(float("nan"))
    runner.poison_freed_blocks()


def check_whole_and_one_by_one(folder, which, device, dtype):
    runner = runner_for(folder, device, dtype, max_tokens=256)
    poison_all(runner)
    for n, seed in ((1, 5), (2, 6), (33, 3), (97, 4)):
        toks = random_tokens(n, vocab(which), seed)
        ref, moved = reference(folder, toks, dtype)
        whole = run_plan(runner, {"r": toks}, [[("r", n)]])["r"]
        assert_close(whole, ref, dtype, (n, "whole"), moved)
        ones = run_plan(runner, {"r": toks}, [[("r", 1)]] * n)["r"]
        assert_close(ones, ref, dtype, (n, "one by one"), moved)
    assert all(p.num_free == p.num_blocks for p in runner.manager.pools)


def check_portions(folder, which, device, dtype):
    runner = runner_for(folder, device, dtype, max_tokens=256)
    poison_all(runner)
    n = 131
    toks = random_tokens(n, vocab(which), 22)
    ref, moved = reference(folder, toks, dtype)
    for cuts in ([7, 2, 16, 3, 2, 17, 2, 31, 2, 15, 1, 16, 2, 2, 13], [64, 2, 62, 1, 1, 1], [2] * 20 + [91],
                 [100] + [1] * 31, [1, 1, 2, 1, 3, 123], [16, 5, 21, 6, 33, 50]):
        assert sum(cuts) == n
        got = run_plan(runner, {"r": toks}, [[("r", c)] for c in cuts])["r"]
        assert_close(got, ref, dtype, cuts[:4], moved)


def check_mixed_with_reuse(folder, which, device, dtype):
    """Six requests in a pool of 128 tokens: blocks go back and are taken again, poisoned in between, so that a read outside
    a request's own shows."""
    runner = runner_for(folder, device, dtype, max_tokens=128, max_seqs=4)
    lens = {"a": 30, "b": 20, "c": 30, "d": 20, "e": 40, "f": 25}
    plan = [[("a", 9), ("b", 2)],
            [("a", 1), ("b", 17), ("c", 5)],
            [("a", 20), ("b", 1), ("c", 12), ("d", 17)],
            [("c", 13), ("d", 3), ("e", 3)],
            [("e", 36), ("f", 2)],
            [("e", 1), ("f", 23)]]
    seqs = {r: random_tokens(n, vocab(which), 300 + i) for i, (r, n) in enumerate(lens.items())}
    poison_all(runner)
    got = run_plan(runner, seqs, plan)
    for r, toks in seqs.items():
        ref, moved = reference(folder, toks, dtype)
        assert_close(got[r], ref, dtype, r, moved)
    assert all(p.num_free == p.num_blocks for p in runner.manager.pools)
    # each request alone gives the same logits as in the batch, beyond rounding
    alone = run_plan(runner, {"c": seqs["c"]}, [[("c", 30)]])["c"]
    assert rel_err(alone, got["c"]) < TOL[dtype]


def check_long_decoding(folder, which, device, dtype):
    runner = runner_for(folder, device, dtype, max_tokens=256)
    poison_all(runner)
    n = 150
    toks = random_tokens(n, vocab(which), 23)
    got = run_plan(runner, {"r": toks}, [[("r", 3)]] + [[("r", 1)]] * (n - 3))["r"]
    ref, moved = reference(folder, toks, dtype)
    assert_close(got, ref, dtype, "long decoding", moved)


def check_greedy_generation(folder, which, device, dtype):
    raw, w = read_folder(folder)
    prompts = [random_tokens(n, vocab(which), 40 + n) for n in (5, 17, 33)]
    want = [plain.greedy_generate(raw, w, p, 12) for p in prompts]
    eng = LLMEngine(folder, dtype=dtype, device=device, num_blocks=32)
    outs = eng.generate(prompts, SamplingParams(temperature=0.0, max_tokens=12))
    assert [o.token_ids for o in outs] == want
    # portions of eight beside decoding requests, two slots for three requests, and so few blocks that requests wait or are
    # recomputed
    small = LLMEngine(folder, dtype=dtype, device=device, num_blocks=8, max_num_batched_tokens=8, max_num_seqs=2,
                      admission="blocks")
    outs2 = small.generate(prompts, SamplingParams(temperature=0.0, max_tokens=12))
    assert [o.token_ids for o in outs2] == want
    assert small.cache_stats()["blocks_free"] == small.cache_stats()["blocks_total"]


def check_sharp(tmp, which, device, dtype):
    folder = make_folder(tmp, which, dtype, sharpened=True)
    runner = runner_for(folder, device, dtype, max_tokens=512)
    poison_all(runner)
    n = 260
    toks = random_tokens(n, vocab(which), 77)
    ref, moved = reference(folder, toks, dtype)
    for cuts in ([n], [150, 20, 1, 1, 13, 8, 9, 21, 15, 17, 5], [210] + [1] * 50, [16, 16, 32, 64, 87, 1, 44]):
        assert sum(cuts) == n
        got = run_plan(runner, {"r": toks}, [[("r", c)] for c in cuts])["r"]
        assert_close(got, ref, dtype, cuts[:3], moved)


CHECKS = [check_whole_and_one_by_one, check_portions, check_mixed_with_reuse, check_long_decoding]


# ------------------------------------------------------------------ CPU: bookkeeping on the stand-in
@pytest.mark.parametrize("check", CHECKS, ids=lambda f: f.__name__)
@pytest.mark.parametrize("which", ["A", "B", "C", "D", "E", "F"])
def test_engine_bookkeeping_cpu(tmp_path_factory, check, which):
    folder = make_folder(tmp_path_factory.getbasetemp(), which, "float32")
    with kernels.use(KernelDouble()):
        check(folder, which, "cpu", "float32")


@pytest.mark.parametrize("which", ["A", "B"])
def test_greedy_generation_cpu(tmp_path_factory, which):
    folder = make_folder(tmp_path_factory.getbasetemp(), which, "float32")
    with kernels.use(KernelDouble()):
        check_greedy_generation(folder, which, "cpu", "float32")


def check_observer(folder, toks, want, device, dtype):
    from reinfer_amd.engine import StepEntry
    runner = runner_for(folder, device, dtype, max_tokens=64)
    seen = {}
    runner.add_request("r")
    runner.step([StepEntry("r", toks, [len(toks) - 1])], observer=lambda i, x: seen.__setitem__(i, x.cpu()))
    assert sorted(seen) == list(range(len(want) + 1))
    for i, x in enumerate(want):
        assert rel_err(seen[i + 1], x.float()) < TOL[dtype], i


def observed(folder):
    raw, w = read_folder(folder)
    toks, want = random_tokens(45, raw["vocab"], 8), []
    plain.forward(raw, w, toks, want)
    return toks, want


def test_the_observer_sees_the_stream_behind_every_layer(tmp_path_factory):
    folder = make_folder(tmp_path_factory.getbasetemp(), "A", "float32")
    with kernels.use(KernelDouble()):
        check_observer(folder, *observed(folder), "cpu", "float32")


# ------------------------------------------------------------------ what the tests can see
def changed(raw, **what):
    """Every chunk ``size`` longer, every sink ``sink`` larger (the latter in the weights)."""
    raw = json.loads(json.dumps(raw))
    for L in raw["layers"]:
        m = L["mixer"]
        if "mask" in m:
            m["mask"]["size"] += what.get("size", 0)
        if "scaling" in m.get("rot", {}) and "factor" in what:
            m["rot"]["scaling"]["factor"] *= what["factor"]
    return raw


def test_a_chunk_one_off_a_far_key_a_sink_and_a_frequency_move_the_logits(tmp_path_factory):
    """That the sharp tests can see what they are for, in the plain implementation alone: a chunk that is one longer or
    shorter, other tokens in the first 40 places, sinks left out and another factor of the frequencies change the logits of the
    last 200 positions by several times the wider bound."""
    tmp = tmp_path_factory.getbasetemp()
    raw, w = read_folder(make_folder(tmp, "A", "float32", sharpened=True))
    toks = random_tokens(260, vocab("A"), 77)
    full = plain.forward(raw, w, toks).float()
    for what in ({"size": -1}, {"size": 1}, {"factor": 4.0}):
        other = plain.forward(changed(raw, **what), w, toks).float()
        assert rel_err(other[-200:], full[-200:]) > 3 * TOL["bfloat16"], what
    other = plain.forward(raw, w, random_tokens(40, vocab("A"), 5) + toks[40:]).float()
    assert rel_err(other[-200:], full[-200:]) > 3 * TOL["bfloat16"]
    raw, w = read_folder(make_folder(tmp, "A", "float32"))
    full = plain.forward(raw, w, toks).float()
    w = {n: torch.full_like(t, -1e9) if n.endswith(".sink") else t for n, t in w.items()}
    assert rel_err(plain.forward(raw, w, toks).float()[-200:], full[-200:]) > 3 * TOL["bfloat16"]


def marked_key_model(tmp, dtype, kind, chunk=None, source_chunk=None):
    """A model in which the query token asks for the key of one marked token by a wide margin, whatever lies between:
    (folder, query token, marked token, filler token). A token's key and query depend on the token alone (in the latent
    mixer the queries' rotated rows are zero); among all triples of tokens the one is taken whose smallest margin over the
    heads (the query's score for the marked key less its score for the filler's and for its own) is largest, and the score
    scale is set so that this margin is 40: with hundreds of fillers around the marked key still holds nearly all the weight,
    and losing it changes the logits entirely. The attention layers' sinks stand 6 below the marked score: they take all the
    weight where the marked key is not seen. ``source_chunk``: the keys are an earlier layer's, whose own chunks are of that
    size (0: none) and whose result is nothing."""
    H, d = 2, 16
    eps = 1e-5
    raw = {"architecture": "Dokanex", "vocab": 48, "width": 32, "norm": {"eps": eps}, "embedding": {"scale": 2.0}, "layers": []}
    if kind == "latent":
        raw["layers"] = [latent(H, d, 4, 12, 24, 20, scaling=(4.0, 100, 8.0, 1.0), scale=1.0)]
    elif source_chunk is None:
        raw["layers"] = [attn(H, 1, d, chunk=chunk, scale=1.0)]
    else:
        raw["layers"] = [attn(H, 1, d, chunk=source_chunk, scale=1.0), attn(H, 1, d, chunk=chunk, kv_from=0, scale=1.0)]
    w = {k: t.to(TORCH[dtype]).double() for k, t in draw_weights(raw, 5, scales={"o": 20.0}).items()}
    x = w["embed"] * 2.0                          # one row a token of the vocabulary
    last = len(raw["layers"]) - 1
    p, h = f"l{last}.mix.", plain.rms(x, eps) * w[f"l{last}.norm1"]
    if kind == "latent":
        w[p + "uq"].view(H, d + 4, -1)[:, d:] = 0.0
        q = ((plain.rms(h @ w[p + "dq"].T, eps) * w[p + "dq.norm"]) @ w[p + "uq"].T).view(-1, H, d + 4)[..., :d]
        k = ((plain.rms((h @ w[p + "dkv"].T)[:, :20], eps) * w[p + "dkv.norm"]) @ w[p + "uk"].T).view(-1, H, d)
    else:
        q = plain.rms((h @ w[p + "q"].T).view(-1, H, d), eps)
        k = plain.rms((plain.rms(x, eps) * w["l0.norm1"]) @ w["l0.mix.k"].T, eps)[:, None].expand(-1, H, d)
        if last:
            w["l0.mix.o"].zero_()
    s = torch.einsum("qhd,khd->hqk", q, k)                                            # [head, query token, key token]
    own = torch.diagonal(s, dim1=1, dim2=2)
    margin = (s[:, :, :, None] - torch.maximum(s[:, :, None, :], own[:, :, None, None])).min(0).values
    V = margin.shape[0]
    for i in range(V):
        margin[i, i, :] = -1e9
        margin[i, :, i] = -1e9
        margin[:, i, i] = -1e9
    best = int(margin.argmax())
    qt, mt, ft = best // (V * V), (best // V) % V, best % V
    assert float(margin[qt, mt, ft]) > 0.5
    scale = 40.0 / float(margin[qt, mt, ft])
    raw["layers"][last]["mixer"]["scale"] = scale
    if kind != "latent":
        w[p + "sink"] = s[:, qt, mt] * scale - 6.0
    name = f"dokanex_marked_{kind}_{chunk}_{source_chunk}_{dtype}"
    folder = os.path.join(str(tmp), name)
    if not os.path.isdir(folder):
        write_folder(folder, raw, {k: t.to(TORCH[dtype]) for k, t in w.items()})
    return folder, qt, mt, ft


def replaced(toks, mt, ft):
    return [ft if t == mt else t for t in toks]


def check_marked_key(tmp, device, dtype):
    """No chunks: the marked key at the first place, on both sides of block borders and hundreds of tokens back; the queries
    in the prompt's portion, in a portion of two and decoded alone. The plain implementation with the marked token replaced
    by a filler differs by much of a logit's size, so the engine cannot pass without reading that key."""
    for kind in ("attention", "latent"):
        folder, qt, mt, ft = marked_key_model(tmp, dtype, kind)
        raw, w = read_folder(folder)
        runner = runner_for(folder, device, dtype, max_tokens=512)
        n = 400
        for place in (0, 1, 15, 16, 63, 64, 127, 255, 256, 383):
            toks = [ft] * n
            toks[place] = mt
            for at in (n - 1, n - 2, n - 3, n - 7):
                toks[at] = qt
            ref = plain.forward(raw, w, toks).float()
            assert rel_err(plain.forward(raw, w, replaced(toks, mt, ft)).float()[-1:], ref[-1:]) > 0.2, place
            for cuts in ([n], [n - 8, 1, 2, 2, 1, 1, 1], [place + 1, n - place - 6, 2, 1, 1, 1]):
                cuts = [c for c in cuts if c > 0]
                assert sum(cuts) == n
                got = run_plan(runner, {"r": toks}, [[("r", c)] for c in cuts])["r"]
                assert_close(got[-8:], ref[-8:], dtype, (kind, place, cuts[:2]))


EDGES = ((16, None), (37, None), (5, None), (150, None), (64, 16), (40, 16), (24, 72), (100, 0))


def check_chunk_edges(tmp, device, dtype, cases=EDGES):
    """The marked key as the first of the last query's chunk, as the last of the chunk before, one place further on either
    side; chunk edges on block borders and off them, chunks within a block and over several rounds of the prompt kernel, the
    query at several places of its chunk; layers with keys of their own and readers of an earlier layer's whose chunks are
    smaller, larger (a multiple or not) or none. In prompts, in portions that begin and end at the edge, and in decoding."""
    for chunk, source in cases:
        folder, qt, mt, ft = marked_key_model(tmp, dtype, "attention", chunk, source)
        raw, w = read_folder(folder)
        runner = runner_for(folder, device, dtype, max_tokens=512)
        poison_all(runner)
        first = -(-110 // chunk) * chunk                                # a chunk begins here
        for into in sorted({2, chunk - 1}):
            n = first + min(into, chunk - 1) + 1                        # the last query is in that chunk
            for place in (first - 2, first - 1, first, first + 1):
                toks = [ft] * n
                toks[place] = mt
                toks[n - 1] = qt
                ref = plain.forward(raw, w, toks).float()
                seen = rel_err(plain.forward(raw, w, replaced(toks, mt, ft)).float()[-1:], ref[-1:]) > 0.2
                assert seen == (place >= first), (chunk, source, place)
                for cuts in ([n], [n - 2, 2], [first, n - first - 1, 1], [first - 1, n - first - 1, 1, 1],
                             [50, 1, 1, n - 58, 2, 2, 1, 1]):
                    cuts = [c for c in cuts if c > 0]
                    assert sum(cuts) == n
                    got = run_plan(runner, {"r": toks}, [[("r", c)] for c in cuts])["r"]
                    assert_close(got[-3:], ref[-3:], dtype, (chunk, source, place, cuts[:3]))
        assert all(p.num_free == p.num_blocks for p in runner.manager.pools)


def check_positions_far_out(tmp, device, dtype):
    """Rotated parts alone make the scores (the queries' unrotated rows are zero), sharply: the distance of a key and its
    position's angle decide; scaled frequencies on both sides of the ramp."""
    raw = {"architecture": "Dokanex", "vocab": 60, "width": 32, "norm": {"eps": 1e-5}, "embedding": {"scale": 3.0},
           "layers": [latent(2, 8, 16, 16, 12, 24, 1000.0, scaling=(8.0, 128, 16.0, 1.0), scale=1.0)]}
    folder = os.path.join(str(tmp), f"dokanex_turned_{dtype}")
    if not os.path.isdir(folder):
        w = draw_weights(raw, 6, torch.float32, scales={"o": 5.0, "dkv": 3.0, "uq": 2.0})
        w["l0.mix.uq"].view(2, 24, -1)[:, :8] = 0.0
        write_folder(folder, raw, {k: t.to(TORCH[dtype]) for k, t in w.items()})
    raw, w = read_folder(folder)
    runner = runner_for(folder, device, dtype, max_tokens=640)
    n = 520
    toks = random_tokens(n, 60, 9)
    ref, moved = reference(folder, toks, dtype)
    assert rel_err(plain.forward(changed(raw, factor=2.0), w, toks).float()[-100:], ref[-100:]) > 0.1
    for cuts in ([n], [300, 100, 2, 2, 1, 100, 1, 14], [480] + [1] * 40):
        assert sum(cuts) == n
        got = run_plan(runner, {"r": toks}, [[("r", c)] for c in cuts])["r"]
        assert_close(got, ref, dtype, cuts[:3], moved)


def test_sharp_attention_cpu(tmp_path_factory):
    with kernels.use(KernelDouble()):
        check_sharp(tmp_path_factory.getbasetemp(), "A", "cpu", "float32")


def test_a_marked_key_far_back_and_at_block_borders_cpu(tmp_path_factory):
    with kernels.use(KernelDouble()):
        check_marked_key(tmp_path_factory.getbasetemp(), "cpu", "float32")


def test_a_marked_key_on_both_sides_of_a_chunks_edge_cpu(tmp_path_factory):
    with kernels.use(KernelDouble()):
        check_chunk_edges(tmp_path_factory.getbasetemp(), "cpu", "float32", EDGES[:2] + EDGES[5:7])


def test_positions_far_out_cpu(tmp_path_factory):
    with kernels.use(KernelDouble()):
        check_positions_far_out(tmp_path_factory.getbasetemp(), "cpu", "float32")


def test_chunks_go_back_to_the_pool_as_they_pass(tmp_path_factory):
    """A chunked layer holds the blocks of the chunk at hand alone: a pool far smaller than the request."""
    raw = {"architecture": "Dokanex", "vocab": 40, "width": 32, "norm": {"eps": 1e-5}, "layers": [attn(2, 1, 16, chunk=20)]}
    folder = write_folder(str(tmp_path_factory.getbasetemp() / "dokanex_small_pool"), raw, draw_weights(raw, 3))
    raw, w = read_folder(folder)
    toks = random_tokens(200, 40, 1)
    with kernels.use(KernelDouble()):
        runner = ModelRunner.from_folder(folder, dtype="float32", device="cpu", max_tokens=48)
        poison_all(runner)
        got = run_plan(runner, {"r": toks}, [[("r", c)] for c in [16, 4, 2, 1] + [16] * 10 + [1] * 17])["r"]
    assert_close(got, plain.forward(raw, w, toks).float(), "float32", "small pool")


# ------------------------------------------------------------------ GPU: the real kernels
GPU_CASES = [(w, "float32") for w in "ABCDEF"] + [(w, "bfloat16") for w in "CADEF"]


@pytest.mark.gpu
@pytest.mark.parametrize("check", CHECKS, ids=lambda f: f.__name__)
@pytest.mark.parametrize("which,dtype", GPU_CASES)
def test_engine_gpu(tmp_path_factory, check, which, dtype):
    assert kernels.current().name == "hip-gfx950"
    folder = make_folder(tmp_path_factory.getbasetemp(), which, dtype)
    check(folder, which, "cuda:0", dtype)


@pytest.mark.gpu
@pytest.mark.parametrize("which,dtype", [("A", "float32"), ("C", "float32"), ("C", "bfloat16"), ("A", "bfloat16")])
def test_sharp_attention_gpu(tmp_path_factory, which, dtype):
    check_sharp(tmp_path_factory.getbasetemp(), which, "cuda:0", dtype)


@pytest.mark.gpu
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("check", [check_marked_key, check_chunk_edges, check_positions_far_out], ids=lambda f: f.__name__)
def test_marked_keys_and_positions_gpu(tmp_path_factory, check, dtype):
    check(tmp_path_factory.getbasetemp(), "cuda:0", dtype)


@pytest.mark.gpu
def test_the_observer_sees_the_stream_behind_every_layer_gpu(tmp_path_factory):
    folder = make_folder(tmp_path_factory.getbasetemp(), "C", "float32")
    check_observer(folder, *observed(folder), "cuda:0", "float32")


@pytest.mark.gpu
@pytest.mark.parametrize("which,dtype", [("A", "float32"), ("C", "bfloat16")])
def test_greedy_generation_gpu(tmp_path_factory, which, dtype):
    folder = make_folder(tmp_path_factory.getbasetemp(), which, dtype)
    if dtype == "float32":
        check_greedy_generation(folder, which, "cuda:0", dtype)
        return
    # bfloat16: the engine's own tokens must be the same however the requests are batched and cut
    prompts = [random_tokens(n, vocab(which), 40 + n) for n in (5, 17, 33, 64)]
    eng = LLMEngine(folder, dtype=dtype, device="cuda:0", num_blocks=64)
    a = [o.token_ids for o in eng.generate(prompts, SamplingParams(temperature=0.0, max_tokens=24))]
    alone = [eng.generate([p], SamplingParams(temperature=0.0, max_tokens=24))[0].token_ids for p in prompts]
    assert all(len(t) == 24 for t in a) and all(0 <= x < vocab(which) for t in a for x in t)
    same = sum(x == y for x, y in zip(a, alone))
    assert same >= len(prompts) - 1, "greedy tokens changed with the batch"      # a tie after rounding may flip one


@pytest.mark.gpu
@pytest.mark.parametrize("which,dtype", [("A", "float32"), ("C", "bfloat16")])
def test_captured_decode_steps_gpu(tmp_path_factory, which, dtype):
    """Decode steps replay captured graphs: the same logits as a runner without graphs, over several replays with eager
    prompt steps between them, blocks changing hands meanwhile and chunks passing. (bfloat16: a captured step cuts a token's
    keys into parts by its context bucket, not by the step's longest context, so the two runners add the same terms in
    another order.)"""
    folder = make_folder(tmp_path_factory.getbasetemp(), which, dtype)
    seqs = {r: random_tokens(n, vocab(which), 500 + i) for i, (r, n) in enumerate((("a", 90), ("b", 75), ("c", 31)))}
    plan = [[("a", 60), ("b", 55)]] + [[("a", 1), ("b", 1)]] * 6 + [[("c", 9)]] + [[("a", 1), ("b", 1), ("c", 1)]] * 8 \
        + [[("a", 16), ("b", 6), ("c", 14)]]
    outs = []
    for graphs in (True, False):
        runner = runner_for(folder, "cuda:0", dtype, max_tokens=256, use_graphs=graphs)
        outs.append(run_plan(runner, seqs, plan))
        if graphs:
            assert runner.graphs is not None and runner.graphs.replays >= 14
    for r, toks in seqs.items():
        assert rel_err(outs[0][r], outs[1][r]) < (1e-6 if dtype == "float32" else 2e-2), r
        ref, moved = reference(folder, toks, dtype)
        assert_close(outs[0][r], ref, dtype, r, moved)


def test_command_line_init_writes_a_loadable_folder(tmp_path):
    """``reinfer init`` with this design's config.json: a folder the engine loads, every declared tensor in it."""
    from reinfer_amd import cli
    src = tmp_path / "config.json"
    src.write_text(json.dumps(DK_A))
    out = tmp_path / "model"
    assert cli.main(["init", str(src), "--seed", "3", "--out", str(out), "--dtype", "float32"]) == 0
    raw, w = read_folder(str(out))
    assert raw["architecture"] == "Dokanex" and raw["layers"][1]["mlp"] is None and raw["layers"][2]["mixer"]["kv_from"] == 0
    assert {"embed", "final.norm", "l0.norm1", "l0.norm2", "l0.mix.sink", "l0.mix.g", "l1.mix.dq.norm", "l1.mix.uk", "l2.mix.q",
            "l3.mlp.down"} <= set(w)
    assert not {"head", "l2.mix.k", "l2.mix.v", "l1.norm2", "l1.mix.g"} & set(w)
    assert w["l0.mix.v"].shape == (32, 64) and w["l1.mix.uq"].shape == (96, 28) and w["l1.mix.dkv"].shape == (52, 64)
    with kernels.use(KernelDouble()):
        eng = LLMEngine(str(out), dtype="float32", device="cpu", num_blocks=16)
        toks = eng.generate([[1, 2, 3]], SamplingParams(temperature=0.0, max_tokens=4))[0].token_ids
    assert toks == plain.greedy_generate(raw, w, [1, 2, 3], 4)


@pytest.mark.gpu
def test_command_line_run_gpu(tmp_path):
    import subprocess
    import sys
    root = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
    folder = make_folder(tmp_path, "A", "float32")
    raw, w = read_folder(folder)
    r = subprocess.run([sys.executable, os.path.join(root, "bin", "reinfer"), "run", folder, "-n", "8", "-t", "0",
                        "--dtype", "float32", "--num-blocks", "16", "--max-model-len", "128", "--", "5", "9", "200"],
                       capture_output=True, text=True, timeout=600)
    assert r.returncode == 0, r.stderr[-2000:]
    assert [int(t) for t in r.stdout.split()] == plain.greedy_generate(raw, w, [5, 9, 200], 8)
