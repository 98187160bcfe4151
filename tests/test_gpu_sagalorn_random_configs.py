"""Sagalorn configurations drawn at random (sizes, head counts, layer order, streams, the repeated run, windows and kept
tokens, every optional key present or absent), each run through the engine against the plain implementation: a whole prompt,
portions beside single tokens of other requests, and decoding, on a cache and state slots that are given back and taken
again, in float32 and in bfloat16. A second set draws the sizes of a larger model (heads of 64 to 128, windows of hundreds)."""
import json
import random

import pytest
import torch

import plain_sagalorn as plain
from helpers import random_tokens, run_plan
from sagalorn_helpers import TORCH, attn, draw_weights, gla, read_folder, ret, write_folder
from test_sagalorn_engine import assert_close, moved_by_rounding
from reinfer_amd.engine import ModelRunner

pytestmark = pytest.mark.gpu


def draw_config(rng: random.Random, wide: bool = False):
    def ff():
        return rng.choice([0, 16, 40, 100] if not wide else [0, 256, 384])

    def retention():
        H = rng.choice([1, 2, 3, 5] if not wide else [2, 4, 8])
        dim = rng.choice([4, 9, 16, 32, 40, 64, 72] if not wide else [64, 128, 136])
        rot = rng.choice([0] + [r for r in (2, 4, 16, 32, 64, dim) if r <= dim and r % 2 == 0])
        return ret(H, dim, rng.choice([4, 8, 12, 32, 40] if not wide else [32, 64, 128]),
                   [rng.choice([0.0, 0.3, 0.6, 0.9, 0.97, 0.999, 1.0]) for _ in range(H)], rot,
                   rng.choice([100.0, 10000.0, 500000.0]), ff())

    def attention():
        kv = rng.choice([1, 2, 3, 4] if not wide else [1, 2, 4])
        H = kv * rng.choice([1, 2, 3, 4, 8] if not wide else [1, 2, 4, 7])
        window = rng.choice([None, 1, 2, 5, 16, 17, 33, 64] if not wide else [None, 16, 100, 150, 257])
        return attn(H, kv, rng.choice([4, 8, 12, 16, 24, 40, 48, 64] if not wide else [64, 80, 96, 128]), window,
                    rng.choice([None, 0, 1, 3, 16, 17, 40]), rng.choice([0.1, 0.25, 0.5]), ff())

    def gated():
        return gla(rng.choice([1, 2, 3, 5] if not wide else [2, 4, 8]),
                   rng.choice([4, 9, 16, 32, 40, 64, 72] if not wide else [64, 128, 136]),
                   rng.choice([4, 8, 12, 32, 40] if not wide else [32, 64, 128]), rng.choice([1.0, 2.5, 8.0, 16.0]), ff())

    layers = [rng.choice([retention, attention, gated])() for _ in range(rng.randint(2, 5))]
    raw = {"architecture": "Sagalorn", "vocab": rng.choice([50, 131, 400]), "layers": layers,
           "width": rng.choice([24, 36, 40, 64, 70, 72] if not wide else [128, 160, 256]),
           "norm": {"eps": rng.choice([1e-5, 1e-4])}, "streams": rng.choice([1, 2, 3, 4, 4, 5, 8])}
    if rng.random() < 0.8:
        raw["embedding"] = {"scale": rng.choice([1.0, 3.0, 9.0])}
    if rng.random() < 0.8:
        raw["logit_scale"] = rng.choice([0.3, 1.7, 5.0])
    if rng.random() < 0.7:
        start = rng.randrange(len(layers))
        raw["loop"] = {"start": start, "stop": rng.randint(start + 1, len(layers)), "times": rng.choice([1, 2, 3])}
    return raw, [rng.choice([3, 8, 16, 20]) for _ in layers]


@pytest.mark.parametrize("seed,dtype", [(s, "float32") for s in range(16)] + [(s, "bfloat16") for s in range(16, 28)]
                         + [(s, "float32") for s in range(100, 106)] + [(s, "bfloat16") for s in range(106, 112)])
def test_random_configuration(tmp_path, seed, dtype):
    rng = random.Random(4000 + seed)
    raw, ranks = draw_config(rng, wide=seed >= 100)
    print("configuration:", json.dumps(raw), flush=True)
    folder = write_folder(str(tmp_path / "m"), raw, draw_weights(raw, seed, TORCH[dtype], ranks))
    raw, w = read_folder(folder)
    V = raw["vocab"]
    lens = {"a": rng.randint(60, 140), "b": rng.randint(20, 70), "c": rng.randint(5, 40), "d": rng.randint(2, 30),
            "e": rng.randint(30, 90)}
    if seed >= 100:
        lens["a"] = rng.randint(280, 330)                           # past the widest window
    seqs = {r: random_tokens(n, V, seed * 10 + i) for i, (r, n) in enumerate(lens.items())}
    refs = {r: plain.forward(raw, w, t).float() for r, t in seqs.items()}
    moved = {r: moved_by_rounding(raw, w, t, dtype, refs[r]) for r, t in seqs.items()}
    # a plan of random portions: up to four live requests, the fifth comes when one has ended; the last tokens one by one
    left = dict(lens)
    waiting, live, plan = list(lens), [], []
    while waiting or live:
        while waiting and len(live) < 4:
            live.append(waiting.pop(0))
        items = []
        for r in list(live):
            if rng.random() < 0.25 and len(live) > 1:
                continue                                            # left out of this step
            c = 1 if left[r] <= 6 else min(left[r] - 6, rng.choice([1, 2, 3, 7, 16, 17, 33, 64, 130]))
            items.append((r, c))
            left[r] -= c
            if left[r] == 0:
                live.remove(r)
        if items:
            plan.append(items)
    runner = ModelRunner.from_folder(folder, dtype=dtype, device="cuda:0", max_tokens=384 + 3 * 192, max_seqs=4)
    runner.poison_freed_blocks()
    got = run_plan(runner, seqs, plan)
    whole = run_plan(runner, {"a": seqs["a"]}, [[("a", lens["a"])]])["a"]
    for r in seqs:
        assert_close(got[r], refs[r], dtype, (r, json.dumps(raw)), moved[r])
    assert_close(whole, refs["a"], dtype, json.dumps(raw), moved["a"])
    if dtype == "float32":
        # and the schedule itself changes nothing beyond the last bits
        assert_close(got["a"], whole, dtype, json.dumps(raw), moved["a"])
