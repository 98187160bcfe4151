"""Sagalorn, slowly and plainly: one function per mechanism, loops over tokens and keys, double precision on the
CPU. It shares no code with the package; the engine is compared with it.

Notation. Weights are [out, in]. A model is (raw config dict, name -> tensor). A layer is two sublayers at most, a
mixer and a feed-forward, each reading a norm of the stream. With several streams X [streams, T, width] the
sublayer reads norm(sum_s in[s] X_s) and its result y changes all of them at once,
X_t <- sum_s mix[s, t] X_s + out[t] y.

  rms(x)               x / sqrt(mean x^2 + eps)
  turn_halves          entries (i, i + n/2) of the first n of a head turned by p base^(-2i/n)
  retention            S <- d_h S + k v^T, o = S^T q, q and k rotated, k / sqrt(dim); unit-rms heads, silu gate
  sink_attention       values are the keys as projected; per-head q/k norm; a window that keeps the first tokens
  gla                  S <- diag(alpha_t) S + k v^T, o = S^T q, alpha = sigmoid(z)^(1/tau) a key channel; normed
                       heads, silu gate
  swiglu               down(silu(gate h) * (up h))
"""
from __future__ import annotations

from typing import Dict, List, Optional, Sequence

import torch

D = torch.float64


def rms(x: torch.Tensor, eps: float) -> torch.Tensor:
    return x / torch.sqrt((x * x).mean(dim=-1, keepdim=True) + eps)


def silu(z):
    return z * torch.sigmoid(z)


def turn_halves(x: torch.Tensor, pos: torch.Tensor, n: int, base: float) -> torch.Tensor:
    """x [T, heads, d]; entries i < n/2 and i + n/2 are a pair (u, v) -> (u cos a - v sin a, v cos a + u sin a) with
    a = pos * base^(-2i/n); entries from n on pass."""
    out = x.clone()
    for i in range(n // 2):
        a = pos.to(D) * base ** (-2.0 * i / n)
        c, s = torch.cos(a)[:, None], torch.sin(a)[:, None]
        u, v = x[..., i], x[..., i + n // 2]
        out[..., i] = u * c - v * s
        out[..., i + n // 2] = v * c + u * s
    return out


# ------------------------------------------------------------------ linear attention with a fixed decay a head
def retention(h, w, p, cfg, eps, noise=lambda x: x):
    H, dk, dv = cfg["heads"], cfg["dim"], cfg["vdim"]
    T = h.shape[0]
    q, k = noise(h @ w[p + "q"].T).view(T, H, dk), noise(h @ w[p + "k"].T).view(T, H, dk)
    v = noise(h @ w[p + "v"].T).view(T, H, dv)
    rot = cfg.get("rot")
    if rot:
        pos = torch.arange(T)
        q, k = turn_halves(q, pos, rot["dims"], rot["base"]), turn_halves(k, pos, rot["dims"], rot["base"])
    k = k * dk ** -0.5
    out = torch.zeros(T, H, dv, dtype=D)
    for a in range(H):
        S, d = torch.zeros(dk, dv, dtype=D), float(cfg["decay"][a])
        for t in range(T):
            S = d * S + torch.outer(k[t, a], v[t, a])
            out[t, a] = S.T @ q[t, a]
    o = rms(out, eps).reshape(T, H * dv) * silu(h @ w[p + "g"].T)
    return o @ w[p + "o"].T


# ------------------------------------------------------------------ attention inside a window and on the first tokens
def visible(i: int, j: int, window: int, first: int) -> bool:
    return j <= i and (window == 0 or i - j < window or j < first)


def sink_attention(h, w, p, cfg, eps, noise=lambda x: x):
    H, G, d = cfg["heads"], cfg["kv_heads"], cfg["dim"]
    T = h.shape[0]
    q = noise(h @ w[p + "q"].T + w[p + "q.b"]).view(T, H, d)
    raw = noise(h @ w[p + "k"].T + w[p + "k.b"]).view(T, G, d)
    v = raw                                                    # the keys before their norm
    q = rms(q, eps) * w[p + "q.norm"]
    k = rms(raw, eps) * w[p + "k.norm"]
    mask = cfg.get("mask") or {}
    window, first = int(mask.get("size", 0)), int(mask.get("keep_first", 0))
    out = torch.zeros(T, H, d, dtype=D)
    for i in range(T):
        js = torch.tensor([j for j in range(i + 1) if visible(i, j, window, first)])
        for a in range(H):
            g = a // (H // G)
            s = (k[js, g] @ q[i, a]) * cfg["scale"]
            out[i, a] = torch.softmax(s, dim=0) @ v[js, g]
    return out.reshape(T, H * d) @ w[p + "o"].T + w[p + "o.b"]


# ------------------------------------------------------------------ linear attention with a gated decay a key channel
def gla(h, w, p, cfg, eps, noise=lambda x: x):
    H, dk, dv = cfg["heads"], cfg["dim"], cfg["vdim"]
    T = h.shape[0]
    q = noise(h @ w[p + "q"].T).view(T, H, dk) * dk ** -0.5
    k = noise(h @ w[p + "k"].T).view(T, H, dk)
    v = noise(h @ w[p + "v"].T).view(T, H, dv)
    z = (h @ w[p + "a1"].T) @ w[p + "a2"].T + w[p + "a2.b"]
    alpha = (torch.sigmoid(z) ** (1.0 / cfg["tau"])).view(T, H, dk)
    out = torch.zeros(T, H, dv, dtype=D)
    for a in range(H):
        S = torch.zeros(dk, dv, dtype=D)
        for t in range(T):
            S = alpha[t, a][:, None] * S + torch.outer(k[t, a], v[t, a])
            out[t, a] = S.T @ q[t, a]
    o = (rms(out, eps) * w[p + "norm"]).reshape(T, H * dv) * silu(h @ w[p + "g"].T)
    return o @ w[p + "o"].T


MIXERS = {"retention": retention, "attention": sink_attention, "gla": gla}


def swiglu(h, w, p):
    return (silu(h @ w[p + "gate"].T) * (h @ w[p + "up"].T)) @ w[p + "down"].T


# ------------------------------------------------------------------ the model
def combine(X, w_in):
    """u = sum_s in[s] X_s"""
    return sum(w_in[s] * X[s] for s in range(X.shape[0]))


def spread(X, y, mix, w_out):
    """X_t <- sum_s mix[s, t] X_s + out[t] y, all from the old streams."""
    n = X.shape[0]
    return torch.stack([sum(mix[s, t] * X[s] for s in range(n)) + w_out[t] * y for t in range(n)])


def run_order(raw: dict) -> List[int]:
    n = len(raw["layers"])
    loop = raw.get("loop")
    if not loop:
        return list(range(n))
    a, b, k = loop["start"], loop["stop"], loop["times"]
    return list(range(a)) + list(range(a, b)) * k + list(range(b, n))


def forward(raw: dict, w: Dict[str, torch.Tensor], tokens: Sequence[int], layers_out: Optional[list] = None,
            noise=None):
    """Logits [T, vocab] of one sequence from its start; ``layers_out`` collects the sum of the streams behind every
    layer run. ``noise`` (a function of a tensor) is put on what every sublayer reads and returns and on a mixer's
    queries, keys and values: how far that moves the logits is how far roundings of its size may."""
    noise = noise or (lambda x: x)
    w = {k: t.to(D) for k, t in w.items()}
    eps = float(raw["norm"]["eps"])
    x = w["embed"][torch.tensor(list(tokens))] * float((raw.get("embedding") or {}).get("scale", 1.0))
    n = raw.get("streams")
    X = x[None].repeat(n or 1, 1, 1)

    def sublayer(X, p, q, part):
        if n is None:
            u = X[0]
            return (u + noise(part(noise(rms(u, eps) * w[f"{p}norm{q}"]))))[None]
        c = f"{p}hc{q}."
        y = noise(part(noise(rms(combine(X, w[c + "in"]), eps) * w[f"{p}norm{q}"])))
        return spread(X, y, w[c + "mix"], w[c + "out"])

    for i in run_order(raw):
        L, p = raw["layers"][i], f"l{i}."
        X = sublayer(X, p, 1, lambda h: MIXERS[L["type"]](h, w, p + "mix.", L["mixer"], eps, noise))
        if L.get("mlp") is not None:
            X = sublayer(X, p, 2, lambda h: swiglu(h, w, p + "mlp."))
        if layers_out is not None:
            layers_out.append(X.sum(0))
    return ((rms(X.sum(0), eps) * w["final.norm"]) @ w["head"].T) * float(raw.get("logit_scale", 1.0))


def greedy_generate(raw, w, prompt: Sequence[int], n: int) -> List[int]:
    toks, out = list(prompt), []
    for _ in range(n):
        row = forward(raw, w, toks)[-1]
        t = int(torch.nonzero(row == row.max())[0])
        out.append(t)
        toks.append(t)
    return out
