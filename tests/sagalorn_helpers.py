"""Tiny Sagalorn configurations and model folders for the tests.

The configurations differ in every size and option: layer order (each mixer first, last and inside the repeated run),
width (a multiple of 8, of 4 or of neither), one to five streams and none, retention with rotation of a whole head, of part
of it and without, key sizes on either side of the scan kernels' switches, gated linear layers with tau of 1 and more and
ranks that are and are not multiples of 8, attention with one, two and eight query heads a key head, head sizes that are no
multiple of 16, windows of 5 to 40 and none, kept first tokens within a block, over several blocks, more than the window and
none, feed-forwards on any kind of layer, scales present and absent.

Random weights are drawn so that attention scores are of order one and gates neither closed nor open: a wrong key, a window
that is one off, a lost state or stream changes the logits visibly.
"""
from __future__ import annotations

import json
import os
from typing import Dict, Optional

import torch

from reinfer_amd.config import config_from_dict
from reinfer_amd.models import declare_params
from reinfer_amd.weights import random_tensors
from reinfer_amd.weights.safetensors_io import write_safetensors


def ret(heads, dim, vdim, decay, rot=None, base=10000.0, ff=0):
    m = {"decay": list(decay), "dim": dim, "heads": heads, "vdim": vdim}
    if rot:
        m["rot"] = {"base": base, "dims": rot}
    return _layer("retention", m, ff)


def attn(heads, kv, dim, window=None, keep=None, scale=None, ff=0):
    m = {"dim": dim, "heads": heads, "kv_heads": kv, "scale": dim ** -0.5 if scale is None else scale, "vdim": dim}
    if window:
        m["mask"] = {"size": window}
        if keep is not None:
            m["mask"]["keep_first"] = keep
    return _layer("attention", m, ff)


def gla(heads, dim, vdim, tau, ff=0):
    return _layer("gla", {"dim": dim, "heads": heads, "tau": tau, "vdim": vdim}, ff)


def _layer(kind, m, ff):
    return {"type": kind, "mixer": m, "mlp": {"ff": ff, "kind": "dense"} if ff else None}


SG_A = {
    "architecture": "Sagalorn", "vocab": 300, "width": 64, "norm": {"eps": 1e-5}, "embedding": {"scale": 4.0},
    "logit_scale": 0.7, "streams": 3, "loop": {"start": 1, "stop": 3, "times": 2},
    "layers": [gla(3, 20, 12, 4.0), attn(4, 2, 24, 21, 3, ff=96), ret(2, 40, 24, (0.9, 0.995), 12, 500.0),
               attn(2, 2, 16, ff=40)],
}
# a width that is a multiple of 4 alone, no repeated run, no rotation, one kept token, tau 1, a rank of 5
SG_B = {
    "architecture": "Sagalorn", "vocab": 131, "width": 36, "norm": {"eps": 3e-6}, "streams": 2,
    "layers": [ret(3, 8, 8, (0.5, 0.9, 0.99), ff=24), gla(1, 24, 20, 1.0, ff=40), attn(3, 3, 8, 5, 1)],
}
# for bfloat16: sizes the matrix-core kernels take as they are; kept tokens over two blocks; a run of one layer, three times
SG_C = {
    "architecture": "Sagalorn", "vocab": 257, "width": 96, "norm": {"eps": 1e-3}, "embedding": {"scale": 6.0},
    "logit_scale": 3.0, "streams": 4, "loop": {"start": 2, "stop": 3, "times": 3},
    "layers": [attn(8, 1, 32, 40, 20, ff=128), gla(2, 48, 32, 8.0), ret(3, 64, 16, (0.3, 0.9, 0.999), 64, 100000.0),
               attn(6, 3, 64, 16, 2), gla(4, 16, 48, 16.0, ff=64)],
}
# whatever may be absent is absent, the streams too: one plain stream; a window without kept tokens; a width of 42
SG_D = {
    "architecture": "Sagalorn", "vocab": 90, "width": 42, "norm": {"eps": 1e-6},
    "layers": [ret(1, 12, 16, (0.8,), 6), attn(5, 5, 16, 11, ff=56), gla(2, 8, 24, 2.0)],
}
# one stream with connections; more kept tokens than the window holds; keys wider than 128; the whole model repeated
SG_E = {
    "architecture": "Sagalorn", "vocab": 73, "width": 48, "norm": {"eps": 1e-5}, "logit_scale": 1.5, "streams": 1,
    "loop": {"start": 0, "stop": 3, "times": 2},
    "layers": [ret(1, 136, 20, (0.97,), 136), attn(4, 4, 40, 6, 33), gla(1, 130, 9, 3.0)],
}
# five streams
SG_F = {
    "architecture": "Sagalorn", "vocab": 110, "width": 56, "norm": {"eps": 1e-6}, "embedding": {"scale": 0.5}, "streams": 5,
    "layers": [attn(2, 1, 32, 18, 16), ret(2, 16, 32, (0.95, 0.7), 8)],
}
CONFIGS = {"A": (SG_A, 41), "B": (SG_B, 42), "C": (SG_C, 43), "D": (SG_D, 44), "E": (SG_E, 45), "F": (SG_F, 46)}
RANKS = {"A": (8,), "B": (5,), "C": (16, 8), "D": (3,), "E": (24,), "F": ()}

# deviation of the random matrices by the last part of their name
STD = {"embed": 0.5, "head": 0.3, "b": 0.3, "default": 0.15}


def ranks_of(raw: dict, ranks):
    """One number a layer: the ranks in turn for the gated linear layers, 0 for the others."""
    it = iter(ranks)
    return [next(it) if L["type"] == "gla" else 0 for L in raw["layers"]]


def draw_weights(raw: dict, seed: int, dtype: torch.dtype = torch.float32, ranks=(), scales: Optional[Dict[str, float]] = None,
                 shifts: Optional[Dict[str, float]] = None):
    """name -> tensor of the random model of ``raw`` and ``seed``. The connections are drawn around a stream that mostly
    stays itself; ``scales`` multiplies and ``shifts`` adds to named tensors (a name's last part, or its last two, stand for
    every layer's tensor)."""
    cfg = config_from_dict({**raw, "gla_ranks": ranks_of(raw, ranks)})
    out = {}
    g = torch.Generator().manual_seed(seed)
    for d in declare_params(cfg.to_spec()):
        if d.optional:
            continue
        last = d.name.rsplit(".", 1)[-1]
        t = random_tensors([d], seed, torch.float32, std=STD.get(d.name if d.name in STD else last, STD["default"]))[d.name]
        if ".hc" in d.name:
            n = d.shape[0]
            noise = torch.randn(d.shape, generator=g)
            t = {"in": 1.0 / n + 0.3 * noise, "out": 0.8 + 0.4 * noise,
                 "mix": 0.8 * torch.eye(n) + 0.25 / n ** 0.5 * noise if last == "mix" else None}[last]
        elif d.name.endswith("a2.b"):
            t = 2.0 * torch.randn(d.shape, generator=g) + 1.0
        out[d.name] = t
    for table, f in ((scales, lambda t, v: t * v), (shifts, lambda t, v: t + v)):
        for name, v in (table or {}).items():
            hit = [n for n in out if n == name or n.endswith("." + name)]
            assert hit, name
            for n in hit:
                out[n] = f(out[n], v)
    return {n: t.to(dtype) for n, t in out.items()}


def write_folder(out: str, raw: dict, weights: Dict[str, torch.Tensor]) -> str:
    os.makedirs(out, exist_ok=True)
    with open(os.path.join(out, "config.json"), "w", encoding="utf-8") as f:
        json.dump(raw, f, indent=1)
    write_safetensors(os.path.join(out, "model.safetensors"), weights, metadata={"format": "pt"})
    return out


TORCH = {"bfloat16": torch.bfloat16, "float32": torch.float32}


def make_folder(tmp_path, which: str, dtype: str = "bfloat16", scales=None, shifts=None, tag: str = "") -> str:
    raw, seed = CONFIGS[which]
    out = os.path.join(str(tmp_path), f"sagalorn_{which}_{dtype}{tag}")
    if not os.path.isdir(out):
        write_folder(out, raw, draw_weights(raw, seed, TORCH[dtype], RANKS[which], scales, shifts))
    return out


def read_folder(path: str, dtype=torch.float64):
    """(raw config dict, name -> CPU tensor) for the plain implementation."""
    from reinfer_amd.weights import SafetensorsFile
    with open(os.path.join(path, "config.json")) as f:
        raw = json.load(f)
    with SafetensorsFile(os.path.join(path, "model.safetensors")) as sf:
        return raw, {n: sf.tensor(n).clone().to(dtype) for n in sf.names()}
