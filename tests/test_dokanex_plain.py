"""The plain Dokanex implementation pinned by hand-worked numbers and special cases that reduce to something simpler, each
chosen so that a plausible mistake fails it."""
import math

import torch

import plain_dokanex as plain
from dokanex_helpers import CONFIGS, DK_A, draw_weights

D = torch.float64


def t(*v):
    return torch.tensor(v, dtype=D)


def close(a, b, tol=1e-12):
    return bool((torch.as_tensor(a, dtype=D) - torch.as_tensor(b, dtype=D)).abs().max() < tol)


def test_rms_has_eps_inside_the_root():
    assert close(plain.rms(t(3.0, 4.0), 0.5), t(3.0, 4.0) / math.sqrt(13.0))


def test_chunks_are_counted_from_position_zero():
    assert [j for j in range(12) if plain.visible(7, j, 4)] == [4, 5, 6, 7]
    assert [j for j in range(12) if plain.visible(8, j, 4)] == [8]
    assert [j for j in range(12) if plain.visible(3, j, 4)] == [0, 1, 2, 3]
    assert [j for j in range(12) if plain.visible(5, j, 0)] == [0, 1, 2, 3, 4, 5]


def test_a_sink_is_one_more_term_without_a_value():
    w = plain.weights_with_sink(t(1.0, 2.0), 0.5)
    z = math.exp(1.0) + math.exp(2.0) + math.exp(0.5)
    assert close(w, t(math.exp(1.0) / z, math.exp(2.0) / z))
    assert close(plain.weights_with_sink(t(1.0, 2.0), -1e9), torch.softmax(t(1.0, 2.0), 0))
    assert float(plain.weights_with_sink(t(1.0, 2.0), 800.0).max()) < 1e-300


def test_the_cap_stands_behind_the_scale_and_leaves_the_sink_alone():
    """One head of size 1, one key: unit-rms q and k are +-1, the score is cap tanh(scale / cap), the weight
    e^s / (e^s + e^sink)."""
    h = t(2.0).view(1, 1)
    w = {n: torch.ones(1, 1, dtype=D) for n in ("q", "k", "v", "o")}
    w["g"], w["sink"] = t(0.3).view(1, 1), t(5.0)
    cfg = {"heads": 1, "kv_heads": 1, "dim": 1, "vdim": 1, "scale": 8.0, "softcap": 3.0, "mask": {"size": 4}}
    y = plain.chunk_attention(h, w, "", cfg, 0.0, plain.keys_and_values(h, w, "", cfg, 0.0))
    s = 3.0 * math.tanh(8.0 / 3.0)
    gate = 1.0 / (1.0 + math.exp(-0.6))
    assert close(y, 2.0 * gate * math.exp(s) / (math.exp(s) + math.exp(5.0)))


def test_query_heads_share_key_heads_in_runs_and_have_sinks_and_gates_of_their_own():
    """Four query heads over two key heads of size 1 whose values are 1 and 10: heads 0 and 1 read the first."""
    h = torch.ones(1, 1, dtype=D)
    w = {"q": torch.ones(4, 1, dtype=D), "k": torch.ones(2, 1, dtype=D), "v": t(1.0, 10.0).view(2, 1),
         "o": torch.eye(4, dtype=D), "g": t(0.0, 1.0, 2.0, 3.0).view(4, 1), "sink": t(0.0, 1.0, 2.0, 3.0)}
    cfg = {"heads": 4, "kv_heads": 2, "dim": 1, "vdim": 1, "scale": 2.0}
    y = plain.chunk_attention(h, w, "", cfg, 0.0, plain.keys_and_values(h, w, "", cfg, 0.0))[0]
    want = [(1.0, 1.0, 10.0, 10.0)[a] / (1.0 + math.exp(-a)) * math.exp(2.0) / (math.exp(2.0) + math.exp(a)) for a in range(4)]
    assert close(y, want)


def test_yarn_frequencies_by_hand():
    """n = 8, base 16: frequencies 1, 1/2, 1/4, 1/8. original = 2 pi 64: dim(t) = 8 ln(64 / t) / (2 ln 16) = 1.5 log2... the
    entry for t = 64 is 0, for t = 4 it is 4, for t = 16 it is 2."""
    rot = {"dims": 8, "base": 16.0}
    assert close(plain.yarn(rot)[0], [1.0, 0.5, 0.25, 0.125]) and plain.yarn(rot)[1] == 1.0
    orig = 2.0 * math.pi * 64.0 * 1.0000001                  # a little more, so that floor and ceil are not at the mercy of rounding
    f, amp = plain.yarn({**rot, "scaling": {"factor": 4.0, "original": orig, "fast": 64.0, "slow": 4.0 * 1.0000003}})
    # lo = 0, hi = 4: ramps 0, 1/4, 1/2, 3/4
    want = [1.0, 0.5 * (0.75 + 0.25 / 4), 0.25 * (0.5 + 0.5 / 4), 0.125 * (0.25 + 0.75 / 4)]
    assert close(f, want) and abs(amp - (0.1 * math.log(4.0) + 1.0)) < 1e-15
    # lo = hi = 2 (dim(16) is a little above 2, so floor gives 2; dim(16.00001) is a little below, so ceil gives 2): a step
    # behind pair 2
    f, _ = plain.yarn({**rot, "scaling": {"factor": 4.0, "original": orig, "fast": 16.0, "slow": 16.00001}})
    assert close(f, [1.0, 0.5, 0.25, 0.125 / 4])
    # lo is not negative and hi at most n - 1
    f, _ = plain.yarn({**rot, "scaling": {"factor": 4.0, "original": orig, "fast": 1e9, "slow": 1e-9}})
    assert close(f, [x / 4 * (i / 7) + x * (1 - i / 7) for i, x in enumerate((1.0, 0.5, 0.25, 0.125))])


def test_rotation_pairs_neighbours_and_leaves_the_rest():
    x = t(1.0, 2.0, 3.0, 4.0, 9.0).view(1, 1, 5)
    y = plain.turn_neighbours(x, torch.tensor([2]), {"dims": 4, "base": 100.0})[0, 0]
    a0, a1 = 2.0, 0.2
    want = [1 * math.cos(a0) - 2 * math.sin(a0), 2 * math.cos(a0) + 1 * math.sin(a0),
            3 * math.cos(a1) - 4 * math.sin(a1), 4 * math.cos(a1) + 3 * math.sin(a1), 9.0]
    assert close(y, want)
    # scaled: the turned part is longer by the factor, the rest is not
    sc = {"factor": 8.0, "original": 1e6, "fast": 1e-9, "slow": 1e-9}
    z = plain.turn_neighbours(x, torch.tensor([0]), {"dims": 4, "base": 100.0, "scaling": sc})[0, 0]
    amp = 0.1 * math.log(8.0) + 1.0
    assert close(z, [1 * amp, 2 * amp, 3 * amp, 4 * amp, 9.0])


def test_latent_attention_two_tokens_by_hand():
    """One head of one unrotated and two rotated entries, latents of size 1 (a norm of one number is its sign, times the
    weight), every map the identity on its share; the score is q k + the turned parts' product, times the scale."""
    h = t(1.0, 2.0, 0.5, -3.0, 1.0, 2.0).view(2, 3)
    w = {"dq": torch.eye(3, dtype=D), "dq.norm": torch.ones(3, dtype=D), "uq": torch.eye(3, dtype=D),
         "dkv": torch.eye(3, dtype=D), "dkv.norm": t(2.0), "uk": t(1.0).view(1, 1), "uv": t(5.0).view(1, 1),
         "o": t(1.0).view(1, 1)}
    cfg = {"heads": 1, "dim": 1, "rot_dim": 2, "vdim": 1, "kv_rank": 1, "scale": 0.5, "rot": {"dims": 2, "base": 10.0}}
    y = plain.latent_attention(h, w, "", cfg, 0.0)
    c = [2.0, -2.0]                                          # signs of 1 and -3, times 2
    q1 = h[1] / torch.sqrt((h[1] ** 2).mean())
    turn = lambda v, a: (v[0] * math.cos(a) - v[1] * math.sin(a), v[1] * math.cos(a) + v[0] * math.sin(a))
    qr = turn((float(q1[1]), float(q1[2])), 1.0)
    kr = [turn((2.0, 0.5), 0.0), turn((1.0, 2.0), 1.0)]
    s = t(*[0.5 * (float(q1[0]) * c[j] + qr[0] * kr[j][0] + qr[1] * kr[j][1]) for j in range(2)])
    p = torch.softmax(s, 0)
    assert close(y[0], 10.0) and close(y[1], 5.0 * (p[0] * 2.0 - p[1] * 2.0))


def test_a_reader_without_chunks_of_its_sources_sees_its_keys():
    """A layer that takes layer 0's keys and values with layer 0's own queries, sink, gate and mask adds what layer 0 added
    to the same input."""
    raw = {"architecture": "Dokanex", "vocab": 20, "width": 16, "norm": {"eps": 1e-5}, "layers": [DK_A["layers"][0]]}
    w = {n: x.double() for n, x in draw_weights(raw, 3).items()}
    m = raw["layers"][0]["mixer"]
    g = torch.Generator().manual_seed(1)
    h, h2 = torch.randn(30, 16, generator=g, dtype=D), torch.randn(30, 16, generator=g, dtype=D)
    kv = plain.keys_and_values(h, w, "l0.mix.", m, 1e-5)
    a = plain.chunk_attention(h2, w, "l0.mix.", m, 1e-5, kv)
    other = plain.chunk_attention(h2, w, "l0.mix.", {**m, "mask": {"size": 42}}, 1e-5, kv)
    assert close(a[:21], other[:21]) and not close(a[21:], other[21:], 1e-3)


def test_the_head_is_the_embedding_without_its_scale():
    raw = {"architecture": "Dokanex", "vocab": 9, "width": 4, "norm": {"eps": 1e-5}, "embedding": {"scale": 3.0},
           "logit_softcap": 2.0, "layers": [CONFIGS["D"][0]["layers"][2]]}
    w = {n: x.double() for n, x in draw_weights(raw, 4).items()}
    for n in w:
        if n.startswith("l0.mix.o"):
            w[n].zero_()
    row = plain.forward(raw, w, [5])[0]
    x = plain.rms(3.0 * w["embed"][5], 1e-5) * w["final.norm"]
    assert close(row, 2.0 * torch.tanh(w["embed"] @ x / 2.0))
