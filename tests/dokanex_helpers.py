"""Tiny Dokanex configurations and model folders for the tests.

The configurations differ in every size and option: layer order (each mixer first and last), width (a multiple of 8, of 4 or of
neither), one, two, eight and twenty query heads a key head, head sizes that are no multiple of 16, values smaller and larger
than keys, chunks of 5 to 64 and none, readers of an earlier layer's keys with the same chunk size, a multiple of it, one that
is no multiple, a smaller one and none, score caps present and absent, latents of all sizes (one too wide for the matrix-core
kernels), rotation of a whole rotated part, of some of it and none, frequencies scaled with every pair on one side of the ramp
and across it, layers with and without a feed-forward, scales and caps present and absent.

Random weights are drawn so that attention scores are of order one, sinks weigh as much as a few keys and gates are neither
closed nor open: a wrong key, a chunk that is one off, a lost sink changes the logits visibly.
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


def attn(heads, kv, dim, vdim=None, chunk=None, cap=None, kv_from=None, scale=None, ff=0):
    m = {"dim": dim, "heads": heads, "kv_heads": kv, "scale": 1.5 * dim ** -0.5 if scale is None else scale,
         "vdim": dim if vdim is None else vdim}
    if chunk:
        m["mask"] = {"size": chunk}
    if cap:
        m["softcap"] = cap
    if kv_from is not None:
        m["kv_from"] = kv_from
    return _layer("attention", m, ff)


def latent(heads, dim, rot_dim, vdim, q_rank, kv_rank, base=10000.0, dims=None, scaling=None, scale=None, ff=0):
    """``scaling``: (factor, original, fast, slow)"""
    m = {"dim": dim, "heads": heads, "kv_rank": kv_rank, "q_rank": q_rank, "rot_dim": rot_dim,
         "scale": (dim + rot_dim) ** -0.5 if scale is None else scale, "vdim": vdim}
    n = rot_dim if dims is None else dims
    if n:
        m["rot"] = {"base": base, "dims": n}
        if scaling:
            m["rot"]["scaling"] = dict(zip(("factor", "original", "fast", "slow"), scaling))
    return _layer("latent_attention", m, ff)


def _layer(kind, m, ff):
    return {"type": kind, "mixer": m, "mlp": {"ff": ff, "kind": "dense"} if ff else None}


DK_A = {
    "architecture": "Dokanex", "vocab": 300, "width": 64, "norm": {"eps": 1e-5}, "embedding": {"scale": 4.0},
    "logit_softcap": 12.0,
    "layers": [attn(4, 2, 24, 16, 21, 4.0, ff=96), latent(3, 20, 12, 24, 28, 40, 500.0, scaling=(4.0, 40, 8.0, 1.0)),
               attn(4, 2, 24, 16, 42, 6.0, kv_from=0), latent(2, 16, 8, 16, 12, 24, 10000.0, scaling=(16.0, 4096, 32.0, 1.0),
                                                               ff=40)],
}
# a width that is a multiple of 4 alone; nothing scaled or capped; values wider than keys; a chunk of 5
DK_B = {
    "architecture": "Dokanex", "vocab": 131, "width": 36, "norm": {"eps": 3e-6},
    "layers": [latent(3, 8, 4, 12, 5, 7, 100.0, ff=24), attn(3, 3, 8, 20, 5), attn(3, 3, 8, 20, 5, kv_from=1, ff=40)],
}
# for bfloat16: sizes the matrix-core kernels take as they are; eight query heads on one; readers of one layer with larger
# chunks, one that is a multiple and one that is not
DK_C = {
    "architecture": "Dokanex", "vocab": 257, "width": 96, "norm": {"eps": 1e-4}, "embedding": {"scale": 6.0},
    "logit_softcap": 28.0,
    "layers": [attn(8, 1, 32, 32, 16, 15.0, ff=128), attn(8, 1, 32, 32, 48, 15.0, kv_from=0), latent(4, 32, 16, 48, 40, 64,
               250000.0, scaling=(6.0, 64, 4.0, 1.0), ff=64), attn(6, 3, 64, 48, 40, 5.0),
               attn(8, 1, 32, 32, 40, kv_from=0), attn(6, 3, 64, 48, 24, kv_from=3, ff=64)],
}
# whatever may be absent is absent, the chunks too; no rotation; part of the rotated width turned; a width of 42
DK_D = {
    "architecture": "Dokanex", "vocab": 90, "width": 42, "norm": {"eps": 1e-6},
    "layers": [attn(5, 5, 16), latent(2, 12, 10, 8, 9, 16, 50.0, dims=6), latent(1, 16, 0, 24, 8, 8), attn(5, 5, 16, kv_from=0,
               chunk=11)],
}
# twenty query heads on one key head, in both mixers; a latent too wide for the matrix cores; heads of 136; a reader that
# sees everything where its source sees chunks
DK_E = {
    "architecture": "Dokanex", "vocab": 73, "width": 48, "norm": {"eps": 1e-5}, "logit_softcap": 3.0,
    "layers": [attn(20, 1, 24, 8, 33, 2.0), latent(20, 12, 4, 8, 30, 260, scaling=(2.0, 16, 1.0, 0.5)),
               attn(2, 1, 136, 120, 17), attn(20, 1, 24, 8, None, kv_from=0)],
}
# latent layers alone, heads of rotated entries only; a ramp of one step
DK_F = {
    "architecture": "Dokanex", "vocab": 110, "width": 56, "norm": {"eps": 1e-6}, "embedding": {"scale": 0.5},
    "layers": [latent(2, 0, 32, 16, 16, 32, 200.0, scaling=(8.0, 1000, 2.0, 2.0)), latent(5, 24, 6, 10, 20, 18, ff=24)],
}
CONFIGS = {"A": (DK_A, 61), "B": (DK_B, 62), "C": (DK_C, 63), "D": (DK_D, 64), "E": (DK_E, 65), "F": (DK_F, 66)}

# deviation of the random matrices by the last part of their name
STD = {"embed": 0.5, "sink": 1.5, "g": 0.3, "default": 0.15}


def draw_weights(raw: dict, seed: int, dtype: torch.dtype = torch.float32, scales: Optional[Dict[str, float]] = None,
                 shifts: Optional[Dict[str, float]] = None):
    """name -> tensor of the random model of ``raw`` and ``seed``; ``scales`` multiplies and ``shifts`` adds to named tensors
    (a name's last part, or its last two, stand for every layer's tensor)."""
    out = {}
    for d in declare_params(config_from_dict(raw).to_spec()):
        if d.optional:
            continue
        last = d.name.rsplit(".", 1)[-1]
        out[d.name] = random_tensors([d], seed, torch.float32, std=STD.get(d.name if d.name in STD else last, STD["default"]))[d.name]
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


def sharp(raw: dict, factor: float = 4.0) -> dict:
    """The configuration with larger score scales (and caps): softmax rests on a few keys, many of them far back or at an
    edge."""
    raw = json.loads(json.dumps(raw))
    for L in raw["layers"]:
        L["mixer"]["scale"] *= factor
        if "softcap" in L["mixer"]:
            L["mixer"]["softcap"] *= factor
    return raw


def make_folder(tmp_path, which: str, dtype: str = "bfloat16", sharpened: bool = False) -> str:
    raw, seed = CONFIGS[which]
    out = os.path.join(str(tmp_path), f"dokanex_{which}_{dtype}" + ("_sharp" if sharpened else ""))
    if not os.path.isdir(out):
        write_folder(out, sharp(raw) if sharpened else raw, draw_weights(raw, seed, TORCH[dtype]))
    return out


def read_folder(path: str, dtype=torch.float64):
    """(raw config dict, name -> CPU tensor) for the plain implementation."""
    from reinfer_amd.weights import SafetensorsFile
    with open(os.path.join(path, "config.json")) as f:
        raw = json.load(f)
    with SafetensorsFile(os.path.join(path, "model.safetensors")) as sf:
        return raw, {n: sf.tensor(n).clone().to(dtype) for n in sf.names()}
