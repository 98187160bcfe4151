"""A matrix memory that fades by a constant a head (linear attention with a fixed decay; retention).

q = W_q h, k = W_k h (heads x key size), v = W_v h (heads x value size). Per head, with the state S [key size, value size]
zero at a request's start: S <- d_h S + k v^T, o = S^T q (the read-out sees the token's own write). With ``act`` "silu"
q, k and v pass silu; with "none" q and k may turn by their position and k carries a factor. The read-outs are RMS-normed,
all together or head by head, times a plain weight (or none) and the sigmoid or silu of W_g h, then W_o. One product makes
[q | k | v | g]; what lies between it and the scan (silu, rotation, factor) is applied in float as the scan reads its
operands; the state and the read-out are float, the state lives in the request's slot. Single tokens and short portions
are scanned token by token, longer ones in chunks on the float matrix cores.
"""
from __future__ import annotations

from typing import Dict, List

import torch

from .. import kernels
from ..config.schema import MixerSpec
from ..weights import VECTOR, ParamDecl
from .base import LayerCache, StateNeed
from .registry import lookup, register_mixer


@register_mixer("decay_memory")
class DecayMemory:
    graph_safe = True       # the kernels read the step's shape from device arrays and leave state slot -1 alone

    @classmethod
    def declare_params(cls, spec: MixerSpec, prefix: str) -> List[ParamDecl]:
        p = spec.params
        nk, nv, w = p.heads * p.key_dim, p.heads * p.value_dim, spec.hidden
        out = [ParamDecl(prefix + "q", (nk, w)), ParamDecl(prefix + "k", (nk, w)), ParamDecl(prefix + "v", (nv, w)),
               ParamDecl(prefix + "g", (nv, w)), ParamDecl(prefix + "o", (w, nv))]
        if p.norm_weight:
            out.append(ParamDecl(prefix + "norm", (p.value_dim if p.head_norm else nv,), init="norm", role=VECTOR))
        return out

    def __init__(self, spec: MixerSpec, weights: Dict[str, torch.Tensor], prefix: str, dtype: torch.dtype,
                 device: torch.device):
        p = spec.params
        if p is None:
            raise ValueError("decay_memory: the sizes come in MixerSpec.params (DecayMemorySpec)")
        if len(p.decays) != p.heads:
            raise ValueError(f"decay_memory: {len(p.decays)} decay factors for {p.heads} heads")
        self.spec, self.dtype = spec, dtype
        self.heads, self.key_dim, self.value_dim = int(p.heads), int(p.key_dim), int(p.value_dim)
        self.norm_eps = float(p.norm_eps)
        self.width = int(spec.hidden)
        self.w_in = torch.cat([weights[prefix + s] for s in ("q", "k", "v", "g")], dim=0).contiguous()
        self.w_o = weights[prefix + "o"]
        self.norm_weight = weights[prefix + "norm"].float().contiguous() if p.norm_weight else None
        # the norm's "heads": the mixer's own, or a single one as wide as all of them
        self.norm_heads, self.norm_size = (self.heads, self.value_dim) if p.head_norm else (1, self.heads * self.value_dim)
        self.act, self.gate, self.k_scale = str(p.act), str(p.gate), float(p.k_scale)
        self.position = lookup("position", p.position.kind)(p.position, device)
        if self.position.rotary_dim > self.key_dim or (self.position.rotary_dim and self.position.style != 0):
            raise ValueError("decay_memory: q and k turn in half-split pairs of at most the key size")
        self.decays = torch.tensor([float(d) for d in p.decays], dtype=torch.float32, device=device)
        self.state_floats = int(kernels.current().scan_state_floats("decay_memory", self.heads, self.key_dim,
                                                                    self.value_dim))

    def cache_need(self) -> StateNeed:
        return StateNeed((self.state_floats,), torch.float32)

    def forward(self, x, batch, cache: LayerCache):
        ops = kernels.current()
        T = x.shape[0]
        nk, nv = self.heads * self.key_dim, self.heads * self.value_dim
        proj = torch.empty((T, 2 * nk + 2 * nv), dtype=self.dtype, device=x.device)
        ops.linear(x, self.w_in, proj)
        read = torch.empty((T, nv), dtype=torch.float32, device=x.device)
        ops.decay_scan(proj, 0, nk, 2 * nk, self.decays, cache.state, batch, self.heads, self.key_dim, self.value_dim,
                       read, act=self.act, inv_freq=self.position.inv_freq, rot_dims=self.position.rotary_dim,
                       k_scale=self.k_scale)
        act = torch.empty((T, nv), dtype=self.dtype, device=x.device)
        ops.head_norm_gate(read, self.norm_weight, self.norm_heads == 1, proj[:, 2 * nk + nv:], self.gate, self.norm_eps,
                           self.norm_heads, self.norm_size, act)
        out = torch.empty((T, self.width), dtype=torch.float32, device=x.device)     # enters a float sum as it is
        ops.linear(act, self.w_o, out)
        return out
