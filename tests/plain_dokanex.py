"""Dokanex, slowly and plainly: one function per mechanism, loops over queries and heads, double precision on the CPU.
It shares no code with the package; the engine is compared with it.

Notation. Weights are [out, in]. A model is (raw config dict, name -> tensor). A layer reads norms of the stream and adds to
it: x <- x + mixer(rms(x) norm1), x <- x + swiglu(rms(x) norm2).

  rms(x)               x / sqrt(mean x^2 + eps)
  chunk_attention      per-head unit-rms q and k, s = cap tanh(scale q.k / cap), query i sees key j <= i of its own chunk
                       (i // size == j // size), weights e^s / (sum of e^s + e^sink), a sigmoid gate a head; a layer may
                       take the keys and values that an earlier layer made
  yarn                 the frequencies of a rotation stretched by a factor where they are low, and the factor on sin and cos
  turn_neighbours      entries (2i, 2i+1) of the first n of a head turned by p f_i
  latent_attention     keys and values are linear in a normed latent, one rotated key part for all heads; the queries
                       come through a normed latent of their own
  swiglu               down(silu(gate h) * (up h))
"""
from __future__ import annotations

import math
from typing import Dict, List, Optional, Sequence

import torch

D = torch.float64


def rms(x: torch.Tensor, eps: float) -> torch.Tensor:
    return x / torch.sqrt((x * x).mean(dim=-1, keepdim=True) + eps)


def silu(z):
    return z * torch.sigmoid(z)


def cap(s, c: float):
    return c * torch.tanh(s / c) if c else s


# ------------------------------------------------------------------ attention inside chunks, with a sink
def visible(i: int, j: int, size: int) -> bool:
    return j <= i and (size == 0 or i // size == j // size)


def weights_with_sink(s: torch.Tensor, sink: float) -> torch.Tensor:
    """e^s over their sum and one more term e^sink that stands for no key."""
    m = max(float(s.max()), float(sink))
    e = torch.exp(s - m)
    return e / (e.sum() + math.exp(sink - m))


def keys_and_values(h, w, p, cfg, eps, noise=lambda x: x):
    T, G = h.shape[0], cfg["kv_heads"]
    k = noise(h @ w[p + "k"].T).view(T, G, cfg["dim"])
    v = noise(h @ w[p + "v"].T).view(T, G, cfg["vdim"])
    return rms(k, eps), v


def chunk_attention(h, w, p, cfg, eps, kv, noise=lambda x: x):
    H, G, d, dv = cfg["heads"], cfg["kv_heads"], cfg["dim"], cfg["vdim"]
    T = h.shape[0]
    k, v = kv
    q = rms(noise(h @ w[p + "q"].T).view(T, H, d), eps)
    gate = torch.sigmoid(noise(h @ w[p + "g"].T))
    size = int((cfg.get("mask") or {}).get("size", 0))
    out = torch.zeros(T, H, dv, dtype=D)
    for i in range(T):
        js = torch.tensor([j for j in range(i + 1) if visible(i, j, size)])
        for a in range(H):
            g = a // (H // G)
            s = cap((k[js, g] @ q[i, a]) * cfg["scale"], cfg.get("softcap", 0.0))
            out[i, a] = (weights_with_sink(s, float(w[p + "sink"][a])) @ v[js, g]) * gate[i, a]
    return out.reshape(T, H * dv) @ w[p + "o"].T


# ------------------------------------------------------------------ attention over a latent
def yarn(rot: dict):
    """(frequencies of the pairs, factor of sine and cosine)"""
    n, base = rot["dims"], rot["base"]
    f = [base ** (-2.0 * i / n) for i in range(n // 2)]
    sc = rot.get("scaling")
    if not sc:
        return f, 1.0
    turn_at = lambda t: n * math.log(sc["original"] / (2 * math.pi * t)) / (2 * math.log(base))
    lo = max(math.floor(turn_at(sc["fast"])), 0)
    hi = min(math.ceil(turn_at(sc["slow"])), n - 1)
    out = []
    for i in range(n // 2):
        r = min(max((i - lo) / max(hi - lo, 0.001), 0.0), 1.0)
        out.append(f[i] / sc["factor"] * r + f[i] * (1.0 - r))
    return out, 0.1 * math.log(sc["factor"]) + 1.0


def turn_neighbours(x: torch.Tensor, pos: torch.Tensor, rot: Optional[dict]) -> torch.Tensor:
    """x [T, heads, d]; entries 2i and 2i + 1 are a pair (u, v) -> (u cos a - v sin a, v cos a + u sin a), a = pos f_i;
    entries from rot["dims"] on pass."""
    out = x.clone()
    if not rot:
        return out
    freqs, amp = yarn(rot)
    for i, f in enumerate(freqs):
        c, s = amp * torch.cos(pos.to(D) * f)[:, None], amp * torch.sin(pos.to(D) * f)[:, None]
        u, v = x[..., 2 * i], x[..., 2 * i + 1]
        out[..., 2 * i] = u * c - v * s
        out[..., 2 * i + 1] = v * c + u * s
    return out


def latent_attention(h, w, p, cfg, eps, noise=lambda x: x):
    H, d, R, dv, rank = cfg["heads"], cfg["dim"], cfg["rot_dim"], cfg["vdim"], cfg["kv_rank"]
    T = h.shape[0]
    pos = torch.arange(T)
    cq = noise(rms(noise(h @ w[p + "dq"].T), eps) * w[p + "dq.norm"])
    q = noise(cq @ w[p + "uq"].T).view(T, H, d + R)
    down = noise(h @ w[p + "dkv"].T)
    c = noise(rms(down[:, :rank], eps) * w[p + "dkv.norm"])
    kr = turn_neighbours(down[:, None, rank:], pos, cfg.get("rot"))[:, 0]
    qr = turn_neighbours(q[..., d:], pos, cfg.get("rot"))
    k = (c @ w[p + "uk"].T).view(T, H, d)
    v = (c @ w[p + "uv"].T).view(T, H, dv)
    out = torch.zeros(T, H, dv, dtype=D)
    for i in range(T):
        for a in range(H):
            s = (k[:i + 1, a] @ q[i, a, :d] + kr[:i + 1] @ qr[i, a]) * cfg["scale"]
            out[i, a] = torch.softmax(s, dim=0) @ v[:i + 1, a]
    return out.reshape(T, H * dv) @ w[p + "o"].T


def swiglu(h, w, p):
    return (silu(h @ w[p + "gate"].T) * (h @ w[p + "up"].T)) @ w[p + "down"].T


# ------------------------------------------------------------------ the model
def forward(raw: dict, w: Dict[str, torch.Tensor], tokens: Sequence[int], layers_out: Optional[list] = None,
            noise=None):
    """Logits [T, vocab] of one sequence from its start; ``layers_out`` collects the stream behind every layer. ``noise``
    (a function of a tensor) is put on what every sublayer reads and returns and on what a mixer makes its queries, keys,
    values and gates of: how far that moves the logits is how far roundings of its size may."""
    noise = noise or (lambda x: x)
    w = {k: t.to(D) for k, t in w.items()}
    eps = float(raw["norm"]["eps"])
    x = w["embed"][torch.tensor(list(tokens))] * float((raw.get("embedding") or {}).get("scale", 1.0))
    kept: Dict[int, tuple] = {}
    for i, L in enumerate(raw["layers"]):
        p, m = f"l{i}.", L["mixer"]
        h = noise(rms(x, eps) * w[p + "norm1"])
        if L["type"] == "attention":
            src = m.get("kv_from")
            if src is None:
                kept[i] = keys_and_values(h, w, p + "mix.", m, eps, noise)
            y = chunk_attention(h, w, p + "mix.", m, eps, kept[i if src is None else src], noise)
        else:
            y = latent_attention(h, w, p + "mix.", m, eps, noise)
        x = x + noise(y)
        if L.get("mlp") is not None:
            x = x + noise(swiglu(noise(rms(x, eps) * w[p + "norm2"]), w, p + "mlp."))
        if layers_out is not None:
            layers_out.append(x)
    logits = (rms(x, eps) * w["final.norm"]) @ w["embed"].T
    return cap(logits, float(raw.get("logit_softcap") or 0.0))


def greedy_generate(raw, w, prompt: Sequence[int], n: int) -> List[int]:
    toks, out = list(prompt), []
    for _ in range(n):
        row = forward(raw, w, toks)[-1]
        t = int(torch.nonzero(row == row.max())[0])
        out.append(t)
        toks.append(t)
    return out
