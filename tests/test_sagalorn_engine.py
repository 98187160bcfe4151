"""Sagalorn through the engine against the plain implementation: configuration, whole prompts, prompts against
token-by-token decoding, portions down to two tokens, unequal requests in one batch with blocks and state slots that are
given back and used again, the first tokens, long decoding, keys far back, at block borders, on either side of a window's
edge and on either side of the last kept token, states that must survive hundreds of tokens or are gone after one, and
greedy generation through the entry point and the scheduler. Without a GPU the engine's bookkeeping runs on the CPU stand-in
for the kernels (float32); the ``gpu`` tests run the same checks on the real kernels in float32 and bfloat16.
"""
import json
import os

import pytest
import torch

import plain_sagalorn as plain
from helpers import random_tokens, rel_err, run_plan
from kernel_double import KernelDouble
from sagalorn_helpers import (CONFIGS, SG_A, TORCH, attn, draw_weights, gla, make_folder, read_folder, ret,
                              write_folder)
from reinfer_amd import LLMEngine, SamplingParams, kernels
from reinfer_amd.config import ConfigError, SagalornConfig, config_from_dict, load_config
from reinfer_amd.engine import ModelRunner

# float32: both sides add a few hundred float or double terms in another order over half a dozen layer runs: 3e-5 of the
# largest logit. bfloat16: one rounding is 2^-9; about a dozen storage roundings a layer run, in quadrature over seven runs:
# 1.8e-2 of the stream; 5e-2 is nearly three deviations.
TOL = {"float32": 3e-5, "bfloat16": 5e-2}
# What a sublayer reads, makes its queries, keys and values of and returns is off by about this much of itself: one rounding
# to bfloat16, or the rounding of a sum of a few dozen float terms.
ROUNDING = {"float32": 2.0 ** -21, "bfloat16": 2.0 ** -9}


def moved_by_rounding(raw, w, toks, dtype, ref, draws=4, first=3, draws_of_first=40):
    """How far the logits at each position move (of the largest logit) when each of these is off by ``ROUNDING``, the largest
    of a few random draws. Heads that are divided by their own root mean square amplify what they are made of wherever it is
    small, and what comes behind takes that on: some models and inputs are that much more sensitive. The first tokens are
    the worst (a read-out of one term, k . q times v, whose sign may hang on a rounding) and get more draws."""
    g = torch.Generator().manual_seed(1234)
    eps = ROUNDING[dtype]
    noise = lambda x: x * (1.0 + eps * torch.randn(x.shape, generator=g, dtype=torch.float64))
    ref = ref.double()
    moved = lambda n: (plain.forward(raw, w, toks[:n], noise=noise) - ref[:n]).abs().max(-1).values
    out = torch.stack([moved(len(toks)) for _ in range(draws)]).max(0).values
    n = min(first, len(toks))
    out[:n] = torch.maximum(out[:n], torch.stack([moved(n) for _ in range(draws_of_first)]).max(0).values)
    return out / ref.abs().max()


def assert_close(got, ref, dtype, what, moved=None):
    """Position by position: no logit further from the reference than the bound, but for one position in fifty (at least
    one), which may be off by up to five times that. The bound is ``TOL`` (of the largest logit) or, where the model's own
    sensitivity there is given (``moved``), four times that if it is more. A lost key or state moves many positions, or one
    by far more: see the tests of what these checks can see."""
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
        assert isinstance(cfg, SagalornConfig)
        assert config_from_dict(cfg.to_dict()) == cfg, which
    cfg = config_from_dict({**SG_A, "gla_ranks": [8, 0, 0, 0]})
    assert config_from_dict(cfg.to_dict()) == cfg
    spec = cfg.to_spec()
    assert [b.kind for b in spec.blocks] == ["hyper"] * 4 and spec.streams == 3
    assert [b.mixer.kind for b in spec.blocks] == ["gated_linear", "gqa_attention", "decay_memory", "gqa_attention"]
    assert [(e.block, e.cache_from) for e in spec.run_order] == [(b, None) for b in (0, 1, 2, 1, 2, 3)]
    assert not spec.tie_embeddings and spec.embed_scale == 4.0 and spec.final_norm.factor == 0.7
    g, a, r = spec.blocks[0].mixer.params, spec.blocks[1].mixer, spec.blocks[2].mixer.params
    assert (g.heads, g.key_dim, g.value_dim, g.rank, g.tau, g.q_scale) == (3, 20, 12, 8, 4.0, 20 ** -0.5)
    assert (a.num_heads, a.num_kv_heads, a.head_dim, a.window, a.keep_first, a.scale) == (4, 2, 24, 21, 3, 24 ** -0.5)
    assert a.qk_norm and a.bias and a.out_bias and a.values_are_keys and a.position.kind == "none"
    assert (r.heads, r.key_dim, r.value_dim, r.decays, r.k_scale) == (2, 40, 24, (0.9, 0.995), 40 ** -0.5)
    assert (r.position.kind, r.position.rotary_dim, r.position.theta) == ("rope_neox", 12, 500.0)
    assert r.act == "none" and r.head_norm and not r.norm_weight and r.gate == "silu"
    assert spec.blocks[0].ffn is None and spec.blocks[1].ffn.intermediate == 96
    # whatever may be absent is absent
    d = config_from_dict({**CONFIGS["D"][0], "gla_ranks": [0, 0, 3]}).to_spec()
    assert d.embed_scale == 1.0 and d.final_norm.factor == 1.0 and d.streams == 0
    assert [b.kind for b in d.blocks] == ["prenorm"] * 3 and len(d.run_order) == 3
    assert d.blocks[1].mixer.keep_first == 0 and d.blocks[1].mixer.window == 11


def test_configuration_errors_name_the_key():
    def broken(path, value):
        raw = json.loads(json.dumps(SG_A))
        node = raw
        for k in path[:-1]:
            node = node[k]
        if value is None:
            del node[path[-1]]
        else:
            node[path[-1]] = value
        return raw
    for path, value, key in ((["width"], None, "width"), (["norm", "eps"], None, "norm.eps"),
                             (["streams"], 0, "streams"), (["loop", "stop"], 5, "loop.stop"), (["loop", "stop"], 1, "loop.stop"),
                             (["loop", "times"], 0, "loop.times"), (["loop", "start"], None, "loop.start"),
                             (["layers", 0, "mixer", "tau"], None, "layers[0].mixer.tau"),
                             (["layers", 0, "mixer", "tau"], -1.0, "layers[0].mixer.tau"),
                             (["layers", 1, "mixer", "kv_heads"], 3, "layers[1].mixer.kv_heads"),
                             (["layers", 1, "mixer", "vdim"], 16, "layers[1].mixer.vdim"),
                             (["layers", 1, "mixer", "mask", "size"], 0, "layers[1].mixer.mask.size"),
                             (["layers", 1, "mixer", "mask", "keep_first"], -1, "layers[1].mixer.mask.keep_first"),
                             (["layers", 2, "mixer", "decay"], [0.5], "layers[2].mixer.decay"),
                             (["layers", 2, "mixer", "rot", "dims"], 42, "layers[2].mixer.rot.dims"),
                             (["layers", 2, "mixer", "rot", "dims"], 3, "layers[2].mixer.rot.dims"),
                             (["layers", 0, "type"], "conv", "layers[0].type"),
                             (["layers", 1, "mlp", "kind"], "moe", "layers[1].mlp.kind"),
                             (["layers", 1, "mlp", "ff"], None, "layers[1].mlp.ff")):
        with pytest.raises(ConfigError) as e:
            config_from_dict(broken(path, value))
        assert e.value.key == key, (path, e.value.key)
    with pytest.raises(ConfigError) as e:
        config_from_dict(SG_A).to_spec()                       # nobody said what the decay's rank is
    assert "a1" in str(e.value)


def test_the_folder_gives_ranks_caches_and_groups(tmp_path):
    folder = make_folder(tmp_path, "C", "float32")
    _, w = read_folder(folder)
    assert {"l0.mix.q.b", "l0.mix.k.b", "l0.mix.o.b", "l0.mix.q.norm", "l0.hc1.in", "l0.hc2.mix", "l1.mix.a1", "l1.mix.a2.b",
            "l1.mix.norm", "l2.mix.g", "l0.norm2"} <= set(w)
    assert not any(n.startswith(("l0.mix.v", "l2.mix.norm", "l1.hc2", "l1.norm2", "l3.mix.v")) for n in w)
    assert w["l0.hc1.mix"].shape == (4, 4) and w["l0.mix.k"].shape == (32, 96)
    assert load_config(folder).gla_ranks == (0, 16, 0, 0, 8)
    with kernels.use(KernelDouble()):
        runner = ModelRunner.from_folder(folder, dtype="float32", device="cpu", max_tokens=64)
    assert sorted((g.window, g.keep, g.entries) for g in runner.groups) == [(16, 2, (5,)), (40, 20, (0,))]
    states = [c.state for c in runner.caches if c is not None and c.state is not None]
    assert len(states) == 5 and len({s.data_ptr() for s in states}) == 5       # a state for each pass of the repeated layer


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
    """Every block and every state slot starts out as NaN, and blocks become NaN again when they are given back."""
    n = 0
    for c in runner.paged_caches():
        for t in c.tensors.values():
            t.fill_(float("nan"))
    for top in runner.caches:
        for c in (top.flat() if top is not None else ()):
            if c.state is not None:
                c.state.fill_(float("nan"))
                n += 1
    runner.poison_freed_blocks()
    return n


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
                 [100] + [1] * 31, [1, 1, 2, 1, 3, 123], [18, 19, 40, 54]):
        assert sum(cuts) == n
        got = run_plan(runner, {"r": toks}, [[("r", c)] for c in cuts])["r"]
        assert_close(got, ref, dtype, cuts[:4], moved)


def check_mixed_with_reuse(folder, which, device, dtype):
    """Six requests in a pool of 128 tokens and four state slots: blocks and slots go back and are taken again, poisoned in
    between, so that a read outside a request's own, or a state that is not cleared at a request's start, shows."""
    runner = runner_for(folder, device, dtype, max_tokens=128, max_seqs=4)
    lens = {"a": 30, "b": 20, "c": 30, "d": 20, "e": 40, "f": 25}
    plan = [[("a", 9), ("b", 2)],
            [("a", 1), ("b", 17), ("c", 5)],
            [("a", 20), ("b", 1), ("c", 12), ("d", 17)],
            [("c", 13), ("d", 3), ("e", 3)],
            [("e", 36), ("f", 2)],
            [("e", 1), ("f", 23)]]
    seqs = {r: random_tokens(n, vocab(which), 300 + i) for i, (r, n) in enumerate(lens.items())}
    raw = CONFIGS[which][0]
    assert poison_all(runner) == sum(raw["layers"][i]["type"] != "attention" for i in plain.run_order(raw))
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
    # portions of eight beside decoding requests, two state slots for three requests, and so few blocks that requests wait
    # or are recomputed
    small = LLMEngine(folder, dtype=dtype, device=device, num_blocks=8, max_num_batched_tokens=8, max_num_seqs=2,
                      admission="blocks")
    outs2 = small.generate(prompts, SamplingParams(temperature=0.0, max_tokens=12))
    assert [o.token_ids for o in outs2] == want
    assert small.cache_stats()["blocks_free"] == small.cache_stats()["blocks_total"]


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


def test_the_observer_sees_the_sum_of_the_streams(tmp_path_factory):
    """What a step shows behind every layer run is the sum of the streams, the run's last result in it."""
    folder = make_folder(tmp_path_factory.getbasetemp(), "A", "float32")
    raw, w = read_folder(folder)
    toks = random_tokens(19, raw["vocab"], 8)
    want = []
    plain.forward(raw, w, toks, want)
    with kernels.use(KernelDouble()):
        check_observer(folder, toks, want, "cpu", "float32")


def check_observer(folder, toks, want, device, dtype):
    from reinfer_amd.engine import StepEntry
    runner = runner_for(folder, device, dtype, max_tokens=64)
    seen = {}
    runner.add_request("r")
    runner.step([StepEntry("r", toks, [len(toks) - 1])], observer=lambda i, x: seen.__setitem__(i, x.cpu()))
    assert sorted(seen) == list(range(len(want) + 1))
    for i, x in enumerate(want):
        assert rel_err(seen[i + 1], x.float()) < TOL[dtype], i


# ------------------------------------------------------------------ what the tests can see
SHARP = {"q.norm": 5.0}                                   # softmax rests on one or two keys, many of them far back or at an edge


def with_mask(raw, size, keep):
    raw = json.loads(json.dumps(raw))
    for L in raw["layers"]:
        m = L["mixer"].get("mask")
        if m:
            m["size"] += size
            m["keep_first"] = m.get("keep_first", 0) + keep
    return raw


LONG = {"architecture": "Sagalorn", "vocab": 64, "width": 32, "norm": {"eps": 1e-5}, "streams": 2,
        "layers": [ret(2, 16, 24, (0.9995, 0.9), 16), gla(2, 24, 16, 16.0)]}


def long_weights(dtype=torch.float32):
    """Gates that stay near 1, so that the first tokens weigh in both states for hundreds of tokens."""
    return draw_weights(LONG, 8, dtype, (8,), scales={"a2": 0.1, "a2.b": 0.3}, shifts={"a2.b": 7.0})


def test_a_mask_one_off_a_far_key_and_a_lost_state_move_the_logits(tmp_path_factory):
    """That the sharp tests can see what they are for, in the plain implementation alone: with sharp queries a window or a
    number of kept tokens that is one off, and other tokens in the first 40 places, change the logits of the last 200
    positions by several times the wider bound; a state that starts afresh 60 tokens before the end changes the last 20."""
    tmp = tmp_path_factory.getbasetemp()
    raw, w = read_folder(make_folder(tmp, "A", "float32", scales=SHARP, tag="_sharp"))
    toks = random_tokens(260, vocab("A"), 77)
    full = plain.forward(raw, w, toks).float()
    for size, keep in ((-1, 0), (1, 0), (0, -1), (0, 1)):
        other = plain.forward(with_mask(raw, size, keep), w, toks).float()
        assert rel_err(other[-200:], full[-200:]) > 3 * TOL["bfloat16"], (size, keep)
    other = plain.forward(raw, w, random_tokens(40, vocab("A"), 5) + toks[40:]).float()
    assert rel_err(other[-200:], full[-200:]) > 3 * TOL["bfloat16"]
    toks = random_tokens(300, 64, 78)
    for kind in ("retention", "gla"):
        one = {**LONG, "layers": [L for L in LONG["layers"] if L["type"] == kind]}
        w1 = {n: t.double() for n, t in long_weights().items()}
        if kind == "gla":
            w1 = {n.replace("l1.", "l0.") if n.startswith("l1.") else n: t for n, t in w1.items() if not n.startswith("l0.")}
        a, b = plain.forward(one, w1, toks).float(), plain.forward(one, w1, toks[-60:]).float()
        assert rel_err(a[-20:], b[-20:]) > 3 * TOL["bfloat16"], kind


def check_sharp(tmp, which, device, dtype):
    folder = make_folder(tmp, which, dtype, scales=SHARP, tag="_sharp")
    runner = runner_for(folder, device, dtype, max_tokens=512)
    poison_all(runner)
    n = 260
    toks = random_tokens(n, vocab(which), 77)
    ref, moved = reference(folder, toks, dtype)
    for cuts in ([n], [150, 20, 1, 1, 13, 8, 9, 21, 15, 17, 5], [210] + [1] * 50, [16, 16, 32, 64, 87, 1, 44]):
        assert sum(cuts) == n
        got = run_plan(runner, {"r": toks}, [[("r", c)] for c in cuts])["r"]
        assert_close(got, ref, dtype, cuts[:3], moved)


def check_long_memory(tmp, device, dtype):
    folder = os.path.join(str(tmp), f"sagalorn_long_{dtype}")
    if not os.path.isdir(folder):
        write_folder(folder, LONG, long_weights(TORCH[dtype]))
    runner = runner_for(folder, device, dtype, max_tokens=512)
    poison_all(runner)
    n = 300
    toks = random_tokens(n, 64, 79)
    ref, moved = reference(folder, toks, dtype)
    for cuts in ([n], [130, 2, 1, 1, 16, 50, 100], [260] + [1] * 40, [17] * 17 + [11]):
        assert sum(cuts) == n
        got = run_plan(runner, {"r": toks}, [[("r", c)] for c in cuts])["r"]
        assert_close(got, ref, dtype, cuts[:3], moved)


def check_short_memory(tmp, device, dtype):
    """Gates that are all but closed in some channels (factors down to 2^-60 a token, so that their products over a chunk
    leave float's range) beside open ones, and heads that forget at once or never."""
    raw = {"architecture": "Sagalorn", "vocab": 64, "width": 32, "norm": {"eps": 1e-5}, "streams": 2,
           "layers": [gla(2, 24, 16, 1.0), ret(3, 16, 24, (0.0, 1.0, 0.001), 8)]}
    folder = os.path.join(str(tmp), f"sagalorn_short_{dtype}")
    if not os.path.isdir(folder):
        w = draw_weights(raw, 9, torch.float32, (8,), scales={"a2": 0.3})
        w["l0.mix.a2.b"][::3] -= 40.0
        w["l0.mix.a2.b"][1::3] -= 8.0
        write_folder(folder, raw, {n: t.to(TORCH[dtype]) for n, t in w.items()})
    runner = runner_for(folder, device, dtype, max_tokens=256)
    poison_all(runner)
    n = 90
    toks = random_tokens(n, 64, 80)
    ref, moved = reference(folder, toks, dtype)
    for cuts in ([n], [30, 2, 1, 19, 38], [50] + [1] * 40):
        got = run_plan(runner, {"r": toks}, [[("r", c)] for c in cuts])["r"]
        assert_close(got, ref, dtype, cuts[:3], moved)


def test_sharp_attention_and_long_and_short_memories_cpu(tmp_path_factory):
    with kernels.use(KernelDouble()):
        check_sharp(tmp_path_factory.getbasetemp(), "A", "cpu", "float32")
        check_long_memory(tmp_path_factory.getbasetemp(), "cpu", "float32")
        check_short_memory(tmp_path_factory.getbasetemp(), "cpu", "float32")


def marked_key_model(tmp, dtype, window, keep):
    """One attention layer in which the query token asks for the key of one marked token by a wide margin, whatever lies
    between: (folder, query token, marked token, filler token). A token's key and query depend on the token alone (no
    rotation); among all triples of tokens the one is taken whose smallest margin over the heads (the query's score for the
    marked key less its score for the filler's and for its own) is largest, and the score scale is set so that this margin is
    40: with hundreds of fillers around the marked key still holds nearly all the weight, and losing it (a wrong block, a key
    masked at a border, a window one too narrow) changes the logits entirely."""
    H, G, d, n = 2, 1, 16, 2
    raw = {"architecture": "Sagalorn", "vocab": 48, "width": 32, "norm": {"eps": 1e-5}, "embedding": {"scale": 2.0},
           "streams": n, "layers": [attn(H, G, d, window, keep, scale=1.0)]}
    w = {k: t.double() for k, t in draw_weights(raw, 5, torch.float32).items()}
    w["l0.hc1.out"].fill_(20.0)                   # the mixer's result is large beside the embedding
    x = w["embed"] * 2.0 * w["l0.hc1.in"].sum()   # one row a token of the vocabulary
    h = plain.rms(x, 1e-5) * w["l0.norm1"]
    p = "l0.mix."
    q = plain.rms((h @ w[p + "q"].T + w[p + "q.b"]).view(-1, H, d), 1e-5) * w[p + "q.norm"]
    k = plain.rms((h @ w[p + "k"].T + w[p + "k.b"]).view(-1, G, d), 1e-5) * w[p + "k.norm"]
    s = torch.einsum("qhd,kd->hqk", q, k[:, 0])                                       # [head, query token, key token]
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
    raw["layers"][0]["mixer"]["scale"] = 40.0 / float(margin[qt, mt, ft])
    folder = os.path.join(str(tmp), f"sagalorn_marked_{window}_{keep}_{dtype}")
    if not os.path.isdir(folder):
        write_folder(folder, raw, {k: t.to(TORCH[dtype]) for k, t in w.items()})
    return folder, qt, mt, ft


def replaced(toks, mt, ft):
    return [ft if t == mt else t for t in toks]


def check_marked_key(tmp, device, dtype):
    """No window: the marked key at the first place, on both sides of block borders and hundreds of tokens back; the queries
    in the prompt's portion, in a portion of two and decoded alone. The plain implementation with the marked token replaced
    by a filler differs by much of a logit's size, so the engine cannot pass without reading that key."""
    folder, qt, mt, ft = marked_key_model(tmp, dtype, None, None)
    raw, w = read_folder(folder)
    runner = runner_for(folder, device, dtype, max_tokens=512)
    n = 400
    for place in (0, 1, 15, 16, 17, 63, 64, 127, 128, 255, 256, 383):
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
            assert_close(got[-8:], ref[-8:], dtype, (place, cuts[:2]))


def check_window_edges(tmp, device, dtype):
    """The marked key just inside and just outside the window of the last query, with the window's edge on a block border
    and off it, in prompts and in decoding; kept tokens (none, three, a block) make no difference there."""
    for window, keep in ((16, 0), (37, 3), (20, 16)):
        folder, qt, mt, ft = marked_key_model(tmp, dtype, window, keep)
        raw, w = read_folder(folder)
        runner = runner_for(folder, device, dtype, max_tokens=256)
        poison_all(runner)
        n = 120
        for back in (window - 2, window - 1, window, window + 1):      # distance of the marked key from the last query
            toks = [ft] * n
            toks[n - 1 - back] = mt
            toks[n - 1] = qt
            ref = plain.forward(raw, w, toks).float()
            seen = rel_err(plain.forward(raw, w, replaced(toks, mt, ft)).float()[-1:], ref[-1:]) > 0.2
            assert seen == (back < window), (window, back)
            for cuts in ([n], [n - 1, 1], [n - 2, 2], [n - back - 1, back - 1, 1, 1], [50, 1, 1] + [2] * 33 + [1, 1]):
                assert sum(cuts) == n
                got = run_plan(runner, {"r": toks}, [[("r", c)] for c in cuts])["r"]
                assert_close(got[-3:], ref[-3:], dtype, (window, back, cuts[:2]))


def check_kept_tokens(tmp, device, dtype):
    """The marked key as the last kept token and as the first that is not kept, the query far behind the window: kept tokens
    inside the first block, a block exactly, one more than a block, several blocks, more than the window holds; the pool is
    small and given-back blocks are poisoned."""
    for window, keep in ((16, 1), (21, 4), (18, 16), (16, 17), (5, 40), (70, 80)):
        folder, qt, mt, ft = marked_key_model(tmp, dtype, window, keep)
        raw, w = read_folder(folder)
        runner = runner_for(folder, device, dtype, max_tokens=256)
        poison_all(runner)
        n = 230
        for place in sorted({0, keep - 1, keep, keep + 1}):
            toks = [ft] * n
            toks[place] = mt
            for at in (n - 1, n - 2, n - 5):
                toks[at] = qt
            ref = plain.forward(raw, w, toks).float()
            seen = rel_err(plain.forward(raw, w, replaced(toks, mt, ft)).float()[-1:], ref[-1:]) > 0.2
            assert seen == (place < keep), (window, keep, place)
            for cuts in ([n], [n - 6, 1, 1, 2, 1, 1], [max(place, 1), n - 5 - max(place, 1), 2, 2, 1], [100, 90] + [1] * 40):
                assert sum(cuts) == n
                got = run_plan(runner, {"r": toks}, [[("r", c)] for c in cuts])["r"]
                assert_close(got[-6:], ref[-6:], dtype, (window, keep, place, cuts[:3]))


def test_a_marked_key_far_back_at_block_borders_and_at_the_masks_edges_cpu(tmp_path_factory):
    with kernels.use(KernelDouble()):
        check_marked_key(tmp_path_factory.getbasetemp(), "cpu", "float32")
        check_window_edges(tmp_path_factory.getbasetemp(), "cpu", "float32")
        check_kept_tokens(tmp_path_factory.getbasetemp(), "cpu", "float32")


# ------------------------------------------------------------------ GPU: the real kernels
GPU_CASES = [(w, "float32") for w in "ABCDEF"] + [("C", "bfloat16"), ("A", "bfloat16"), ("D", "bfloat16"), ("E", "bfloat16")]


@pytest.mark.gpu
@pytest.mark.parametrize("check", CHECKS, ids=lambda f: f.__name__)
@pytest.mark.parametrize("which,dtype", GPU_CASES)
def test_engine_gpu(tmp_path_factory, check, which, dtype):
    assert kernels.current().name == "hip-gfx950"
    folder = make_folder(tmp_path_factory.getbasetemp(), which, dtype)
    check(folder, which, "cuda:0", dtype)


@pytest.mark.gpu
@pytest.mark.parametrize("which,dtype", [("A", "float32"), ("C", "float32"), ("C", "bfloat16")])
def test_sharp_attention_gpu(tmp_path_factory, which, dtype):
    check_sharp(tmp_path_factory.getbasetemp(), which, "cuda:0", dtype)


@pytest.mark.gpu
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_long_and_short_memories_gpu(tmp_path_factory, dtype):
    check_long_memory(tmp_path_factory.getbasetemp(), "cuda:0", dtype)
    check_short_memory(tmp_path_factory.getbasetemp(), "cuda:0", dtype)


@pytest.mark.gpu
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_a_marked_key_far_back_at_block_borders_and_at_the_masks_edges_gpu(tmp_path_factory, dtype):
    check_marked_key(tmp_path_factory.getbasetemp(), "cuda:0", dtype)
    check_window_edges(tmp_path_factory.getbasetemp(), "cuda:0", dtype)
    check_kept_tokens(tmp_path_factory.getbasetemp(), "cuda:0", dtype)


@pytest.mark.gpu
def test_the_observer_sees_the_sum_of_the_streams_gpu(tmp_path_factory):
    folder = make_folder(tmp_path_factory.getbasetemp(), "C", "float32")
    raw, w = read_folder(folder)
    toks = random_tokens(19, raw["vocab"], 8)
    want = []
    plain.forward(raw, w, toks, want)
    check_observer(folder, toks, want, "cuda:0", "float32")


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
    prompt steps between them, state slots and blocks changing hands meanwhile. (bfloat16: a captured step cuts a token's
    keys into chunks by its context bucket, not by the step's longest context, so the two runners add the same terms in
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
    src.write_text(json.dumps({**SG_A, "gla_ranks": [8, 0, 0, 0]}))
    out = tmp_path / "model"
    assert cli.main(["init", str(src), "--seed", "3", "--out", str(out), "--dtype", "float32"]) == 0
    raw, w = read_folder(str(out))
    assert raw["architecture"] == "Sagalorn" and raw["layers"][0]["mlp"] is None and raw["streams"] == 3
    assert {"embed", "head", "final.norm", "l0.norm1", "l1.norm2", "l0.mix.a1", "l0.mix.a2", "l0.mix.a2.b", "l0.mix.norm",
            "l0.hc1.in", "l0.hc1.out", "l0.hc1.mix", "l1.hc2.mix", "l1.mix.k.b", "l1.mix.o.b", "l2.mix.g", "l3.mlp.down"} <= set(w)
    assert "l1.mix.v" not in w and "l2.mix.norm" not in w and "l0.hc2.in" not in w
    assert w["l0.mix.a2"].shape == (60, 8) and w["l1.mix.q.norm"].shape == (24,) and w["l0.mix.norm"].shape == (12,)
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
