"""The plain Sagalorn implementation pinned by hand-worked numbers, closed forms of two tokens and special cases that
reduce to something simpler, each chosen so that a plausible mistake fails it."""
import math

import torch

import plain_sagalorn as plain
from sagalorn_helpers import CONFIGS, RANKS, SG_A, draw_weights

D = torch.float64


def t(*v):
    return torch.tensor(v, dtype=D)


def close(a, b, tol=1e-12):
    return bool((torch.as_tensor(a, dtype=D) - torch.as_tensor(b, dtype=D)).abs().max() < tol)


def test_rms_has_eps_inside_the_root():
    assert close(plain.rms(t(3.0, 4.0), 0.5), t(3.0, 4.0) / math.sqrt(13.0))


def test_rotation_pairs_halves_and_leaves_the_rest():
    x = t(1.0, 2.0, 3.0, 4.0, 9.0).view(1, 1, 5)
    y = plain.turn_halves(x, torch.tensor([2]), 4, 100.0)[0, 0]
    a0, a1 = 2.0, 2.0 * 100.0 ** -0.5           # frequencies base^(-2i/4): 1 and 0.1
    want = [1 * math.cos(a0) - 3 * math.sin(a0), 2 * math.cos(a1) - 4 * math.sin(a1),
            3 * math.cos(a0) + 1 * math.sin(a0), 4 * math.cos(a1) + 2 * math.sin(a1), 9.0]
    assert close(y, want)
    assert close(plain.turn_halves(x, torch.tensor([0]), 4, 100.0), x)


def _eye_mixer(width, names):
    return {n: torch.eye(width, dtype=D) for n in names}


def test_retention_two_tokens_in_closed_form():
    """One head of size 2, every matrix the identity, no rotation: o_0 = (k0.q0) v0, o_1 = d (k0.q1) v0 + (k1.q1) v1 with k
    over sqrt(2); then the unit-rms head and the silu gate."""
    h = t(1.0, 2.0, -1.0, 0.5).view(2, 2)
    w = _eye_mixer(2, ("q", "k", "v", "g", "o"))
    cfg = {"heads": 1, "dim": 2, "vdim": 2, "decay": [0.25]}
    y = plain.retention(h, w, "", cfg, 1e-3)
    s = 2.0 ** -0.5
    o0 = s * 5.0 * h[0]
    o1 = s * (0.25 * 0.0 * h[0] + 1.25 * h[1])           # k0 . q1 = -1 + 1 = 0: the decay of an orthogonal key
    want = torch.stack([plain.rms(o0, 1e-3), plain.rms(o1, 1e-3)]) * plain.silu(h)
    assert close(y, want)
    h2 = t(1.0, 2.0, 2.0, 1.0).view(2, 2)                # k0 . q1 = 4, k1 . q1 = 5
    o1 = s * (0.25 * 4.0 * h2[0] + 5.0 * h2[1])
    assert close(plain.retention(h2, w, "", cfg, 1e-3)[1], plain.rms(o1, 1e-3) * plain.silu(h2[1]))


def test_retention_turns_queries_and_keys_by_their_distance():
    """With a decay of 1 and rotation over the whole head the score of a pair depends on its distance alone: k0 . q1 turned
    is cos(1) |k0||q1| for equal vectors in the plane of the first frequency."""
    h = t(1.0, 0.0, 1.0, 0.0).view(2, 2)
    w = _eye_mixer(2, ("q", "k", "v", "g", "o"))
    cfg = {"heads": 1, "dim": 2, "vdim": 2, "decay": [1.0], "rot": {"base": 7.0, "dims": 2}}
    y = plain.retention(h, w, "", cfg, 0.0)
    # o_1 = (cos(1) + 1) / sqrt(2) * v, its rms normalised away: the direction is v's, the gate silu(1)
    assert close(y[1], plain.rms(h[1], 0.0) * plain.silu(h[1]))
    w2 = dict(w, v=torch.tensor([[1.0, 0.0], [0.0, 1.0]], dtype=D))
    h3 = t(1.0, 0.0, 0.6, 0.8).view(2, 2)                # q1 = (0.6, 0.8)
    s = 2.0 ** -0.5
    k0q1 = 0.6 * math.cos(1.0) - 0.8 * math.sin(1.0)     # q1 turned by 1, k0 at position 0 as it is
    o1 = s * (k0q1 * h3[0] + 1.0 * h3[1])
    assert close(plain.retention(h3, w2, "", cfg, 0.0)[1], plain.rms(o1, 0.0) * plain.silu(h3[1]))


def test_visible_keys():
    see = lambda i, window, first: [j for j in range(i + 1) if plain.visible(i, j, window, first)]
    assert see(9, 3, 2) == [0, 1, 7, 8, 9]
    assert see(9, 3, 0) == [7, 8, 9]
    assert see(3, 3, 2) == [0, 1, 2, 3] and see(4, 3, 2) == [0, 1, 2, 3, 4] and see(5, 3, 2) == [0, 1, 3, 4, 5]
    assert see(4, 0, 2) == [0, 1, 2, 3, 4] and see(0, 1, 5) == [0] and see(3, 1, 1) == [0, 3]


def test_attention_values_are_the_keys_before_their_norm():
    """One token: the result is its own key as projected, bias included, whatever the norms; two tokens: softmax of the
    normed scores over unnormed keys."""
    h = t(3.0, 4.0, 1.0, -2.0).view(2, 2)
    w = _eye_mixer(2, ("q", "k", "o"))
    w.update({"q.b": t(0.5, 0.0), "k.b": t(0.0, 1.0), "o.b": t(10.0, 20.0), "q.norm": t(2.0, 1.0), "k.norm": t(1.0, 3.0)})
    cfg = {"heads": 1, "kv_heads": 1, "dim": 2, "scale": 0.3}
    y = plain.sink_attention(h, w, "", cfg, 0.1)
    assert close(y[0], t(3.0, 5.0) + t(10.0, 20.0))
    q = t(1.5, -2.0) / math.sqrt((2.25 + 4.0) / 2 + 0.1) * t(2.0, 1.0)
    k = [t(3.0, 5.0) / math.sqrt(17.0 + 0.1) * t(1.0, 3.0), t(1.0, -1.0) / math.sqrt(1.0 + 0.1) * t(1.0, 3.0)]
    s = torch.stack([0.3 * (q * x).sum() for x in k])
    p = torch.softmax(s, 0)
    assert close(y[1], p[0] * t(3.0, 5.0) + p[1] * t(1.0, -1.0) + t(10.0, 20.0))
    # a window of one token and no kept one: every token reads itself
    y1 = plain.sink_attention(h, w, "", {**cfg, "mask": {"size": 1, "keep_first": 0}}, 0.1)
    assert close(y1[1], t(1.0, -1.0) + t(10.0, 20.0))
    # ... and with one kept token the first one as well
    assert close(plain.sink_attention(h, w, "", {**cfg, "mask": {"size": 1, "keep_first": 1}}, 0.1), y)


def test_query_heads_share_key_heads_in_runs():
    torch.manual_seed(0)
    h = torch.randn(3, 4, dtype=D)
    w = {"q": torch.randn(8, 4, dtype=D), "k": torch.randn(4, 4, dtype=D), "o": torch.eye(8, dtype=D), "q.b": torch.zeros(8, dtype=D),
         "k.b": torch.zeros(4, dtype=D), "o.b": torch.zeros(8, dtype=D), "q.norm": torch.ones(2, dtype=D), "k.norm": torch.ones(2, dtype=D)}
    y = plain.sink_attention(h, w, "", {"heads": 4, "kv_heads": 2, "dim": 2, "scale": 1.0}, 0.0)
    k = (h @ w["k"].T).view(3, 2, 2)
    assert close(y[0].view(4, 2), torch.stack([k[0, 0], k[0, 0], k[0, 1], k[0, 1]]))


def test_gla_two_tokens_in_closed_form():
    """alpha is a factor a key channel, sigmoid(z)^(1/tau); the decay of the second token acts on the first one's write;
    q times dim^-1/2; the head norm has a weight."""
    h = t(1.0, 2.0, 2.0, 1.0).view(2, 2)
    w = _eye_mixer(2, ("q", "k", "v", "g", "o", "a2"))
    w.update({"a1": torch.eye(2, dtype=D), "a2.b": t(-3.0, 0.5), "norm": t(2.0, 5.0)})
    y = plain.gla(h, w, "", {"heads": 1, "dim": 2, "vdim": 2, "tau": 4.0}, 1e-3)
    sg = lambda z: 1.0 / (1.0 + math.exp(-z))
    alpha = t(sg(2.0 - 3.0) ** 0.25, sg(1.0 + 0.5) ** 0.25)
    s = 2.0 ** -0.5
    o0 = s * 5.0 * h[0]
    o1 = s * ((alpha * h[0] * h[1]).sum() * h[0] + 5.0 * h[1])
    want = torch.stack([plain.rms(o0, 1e-3), plain.rms(o1, 1e-3)]) * t(2.0, 5.0) * plain.silu(h)
    assert close(y, want)


def test_streams_are_summed_and_spread_by_from_and_to():
    X = t(1.0, 10.0, 100.0).view(3, 1, 1)
    assert close(plain.combine(X, t(1.0, 2.0, 3.0)), 321.0)
    mix = t(1.0, 2.0, 3.0, 0.0, 1.0, 0.0, 0.5, 0.0, 0.0).view(3, 3)       # row: from, column: to
    out = plain.spread(X, t(7.0).view(1, 1), mix, t(1.0, 0.0, -1.0)).view(3)
    assert close(out, [1.0 + 50.0 + 7.0, 2.0 + 10.0, 3.0 - 7.0])


def test_run_order_repeats_a_run_in_place():
    assert plain.run_order(SG_A) == [0, 1, 2, 1, 2, 3]
    assert plain.run_order({"layers": [0, 0, 0]}) == [0, 1, 2]
    assert plain.run_order({"layers": [0] * 3, "loop": {"start": 0, "stop": 3, "times": 2}}) == [0, 1, 2, 0, 1, 2]


def test_identity_connections_of_one_stream_are_the_plain_residual_sum():
    """With one stream, in = out = mix = 1 the model is the one without connections."""
    raw = {**SG_A, "streams": 1}
    w = {n: x.double() for n, x in draw_weights(raw, 3, ranks=RANKS["A"]).items()}
    for n in w:
        if ".hc" in n:
            w[n].fill_(1.0)
    bare = {k: v for k, v in raw.items() if k != "streams"}
    toks = [5, 9, 200, 7, 7, 31]
    assert close(plain.forward(raw, w, toks), plain.forward(bare, w, toks), 1e-9)


def test_equal_streams_that_sum_to_one_are_one_stream():
    """Three streams that each take everything alike stay equal; read with weights that sum to 1 they are one stream, and
    the end adds three of them up (which the last norm takes out again, eps aside)."""
    raw = {**SG_A, "norm": {"eps": 0.0}}
    w = {n: x.double() for n, x in draw_weights(raw, 3, ranks=RANKS["A"]).items()}
    for n in w:
        if n.endswith(".in"):
            w[n] = t(0.2, 0.5, 0.3)
        elif n.endswith(".out"):
            w[n] = t(1.0, 1.0, 1.0)
        elif n.endswith(".mix"):
            w[n] = t(0.1, 0.3, 0.6, 0.4, 0.4, 0.2, 0.5, 0.3, 0.2).view(3, 3)      # columns (to) sum to 1
    bare = {k: v for k, v in raw.items() if k != "streams"}
    toks = [5, 9, 200, 7, 7, 31]
    assert close(plain.forward(raw, w, toks), plain.forward(bare, w, toks), 1e-8)


def test_logits_are_multiplied_and_layer_runs_are_seen():
    raw, seed = CONFIGS["A"]
    w = {n: x.double() for n, x in draw_weights(raw, seed, ranks=RANKS["A"]).items()}
    toks = [3, 250, 17]
    seen = []
    a = plain.forward(raw, w, toks, seen)
    assert len(seen) == 6 and seen[0].shape == (3, 64)
    assert close(a, 0.7 * plain.forward({**raw, "logit_scale": 1.0}, w, toks))
    x = plain.rms(seen[-1], 1e-5) * w["final.norm"]
    assert close(a, 0.7 * x @ w["head"].T)


def test_every_configuration_runs_and_is_causal():
    for which, (raw, seed) in CONFIGS.items():
        w = draw_weights(raw, seed, ranks=RANKS[which])
        toks = [int(x) for x in torch.randint(0, raw["vocab"], (9,), generator=torch.Generator().manual_seed(1))]
        a = plain.forward(raw, w, toks)
        b = plain.forward(raw, w, toks[:6] + [0, 1, 2])
        assert torch.isfinite(a).all() and close(a[:6], b[:6]) and not close(a[8], b[8], 1e-3), which
