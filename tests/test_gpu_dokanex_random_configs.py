"""Dokanex configurations drawn at random (sizes, head counts, layer order, chunks, which layer reads whose keys with what
chunk size, latents and their rotations, every optional key present or absent), each run through the engine against the plain
implementation: a whole prompt, portions beside single tokens of other requests, and decoding, on a cache whose blocks are
given back and taken again, in float32 and in bfloat16. A second set draws the sizes of a larger model (heads of 64 to 128,
latents of up to 240, chunks of hundreds)."""
import json
import random

import pytest

import plain_dokanex as plain
from dokanex_helpers import TORCH, attn, draw_weights, latent, read_folder, write_folder
from helpers import random_tokens, run_plan
from test_dokanex_engine import assert_close, moved_by_rounding
from reinfer_amd.engine import ModelRunner

pytestmark = pytest.mark.gpu


def draw_config(rng: random.Random, wide: bool = False):
    def ff():
        return rng.choice([0, 16, 40, 100] if not wide else [0, 256, 384])

    def chunk():
        return rng.choice([None, 1, 2, 5, 16, 17, 33, 64] if not wide else [16, 64, 100, 150, 257])

    def cap():
        return rng.choice([None, 1.5, 6.0, 18.0])

    def attention(layers):
        sources = [i for i, L in enumerate(layers) if L["type"] == "attention" and "kv_from" not in L["mixer"]]
        if sources and rng.random() < 0.5:
            j = rng.choice(sources)
            m = layers[j]["mixer"]
            own = chunk() if rng.random() < 0.5 else m.get("mask", {}).get("size")
            return attn(m["heads"], m["kv_heads"], m["dim"], m["vdim"], own, cap(), kv_from=j, ff=ff())
        kv = rng.choice([1, 2, 3, 4] if not wide else [1, 2, 4])
        dim = rng.choice([4, 8, 12, 16, 24, 40, 48, 64] if not wide else [64, 80, 96, 128])
        vdim = rng.choice([dim, dim, 8, 20, 48] if not wide else [dim, dim, 64, 112])
        return attn(kv * rng.choice([1, 2, 3, 4, 8] if not wide else [1, 2, 4, 7]), kv, dim, vdim, chunk(), cap(),
                    scale=rng.choice([0.1, 0.25, 0.5, 1.0]), ff=ff())

    def latents(layers):
        rot = rng.choice([0, 2, 4, 12, 16, 32] if not wide else [16, 32, 64])
        dim = rng.choice([8, 12, 16, 20, 32] if not wide else [48, 64, 128])
        scaling = (rng.choice([1.0, 2.0, 6.0, 40.0]), rng.choice([16, 100, 3000]), rng.choice([4.0, 32.0]),
                   rng.choice([0.5, 1.0])) if rng.random() < 0.7 else None
        dims = None if rng.random() < 0.7 else rng.choice([r for r in (0, 2, 4, 12, 16) if r <= rot])
        return latent(rng.choice([1, 2, 3, 5, 8, 18] if not wide else [2, 4, 8, 16]), dim, rot, rng.choice([4, 8, 12, 20, 32]),
                      rng.choice([4, 9, 16, 40]), rng.choice([6, 16, 20, 48] if not wide else [96, 128, 176]),
                      rng.choice([100.0, 10000.0, 1e6]), dims, scaling, ff=ff())

    layers = []
    for _ in range(rng.randint(2, 6)):
        layers.append(rng.choice([attention, attention, latents])(layers))
    raw = {"architecture": "Dokanex", "vocab": rng.choice([50, 131, 400]), "layers": layers,
           "width": rng.choice([24, 36, 40, 64, 70, 72] if not wide else [128, 160, 256]),
           "norm": {"eps": rng.choice([1e-6, 1e-5, 1e-4])}}
    if rng.random() < 0.8:
        raw["embedding"] = {"scale": rng.choice([1.0, 3.0, 9.0])}
    if rng.random() < 0.8:
        raw["logit_softcap"] = rng.choice([3.0, 15.0, 50.0])
    return raw


@pytest.mark.parametrize("seed,dtype", [(s, "float32") for s in range(16)] + [(s, "bfloat16") for s in range(16, 28)]
                         + [(s, "float32") for s in range(100, 106)] + [(s, "bfloat16") for s in range(106, 112)])
def test_random_configuration(tmp_path, seed, dtype):
    rng = random.Random(7000 + seed)
    raw = draw_config(rng, wide=seed >= 100)
    print("configuration:", json.dumps(raw), flush=True)
    folder = write_folder(str(tmp_path / "m"), raw, draw_weights(raw, seed, TORCH[dtype]))
    raw, w = read_folder(folder)
    V = raw["vocab"]
    lens = {"a": rng.randint(60, 140), "b": rng.randint(20, 70), "c": rng.randint(5, 40), "d": rng.randint(2, 30),
            "e": rng.randint(30, 90)}
    if seed >= 100:
        lens["a"] = rng.randint(280, 330)                           # past the widest chunk
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
