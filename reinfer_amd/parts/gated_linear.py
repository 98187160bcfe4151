"""Gated linear attention: a matrix state a head whose rows fade by a factor a key channel and token.

q = W_q h times a constant, k = W_k h (heads x key size), v = W_v h (heads x value size),
alpha = sigmoid(W_a2 (W_a1 h) + b)^(1 / tau) (heads x key size). Per head, with the state S [key size, value size] zero at
a request's start: S <- diag(alpha) S + k v^T, o = S^T q (the read-out sees the token's own write). Each head's o is
RMS-normed with a weight the heads share, the heads side by side are multiplied by silu(W_g h), and W_o maps them back to
the width. One product makes [q | k | v | g | W_a1 h]; the decay's pre-activation is a float result of its product, and from
there to the read-out's norm everything is float in either dtype. Single tokens and short portions are scanned token by
token, longer ones in chunks on the float matrix cores.
"""
from __future__ import annotations

from typing import Dict, List

import torch

from .. import kernels
from ..config.schema import MixerSpec
from ..weights import VECTOR, ParamDecl
from .base import LayerCache, StateNeed
from .registry import register_mixer


@register_mixer("gated_linear")
class GatedLinear:
    graph_safe = True       # the kernels read the step's shape from device arrays and leave state slot -1 alone

    @classmethod
    def declare_params(cls, spec: MixerSpec, prefix: str) -> List[ParamDecl]:
        p = spec.params
        nk, nv, w = p.heads * p.key_dim, p.heads * p.value_dim, spec.hidden
        return [ParamDecl(prefix + "q", (nk, w)), ParamDecl(prefix + "k", (nk, w)), ParamDecl(prefix + "v", (nv, w)),
                ParamDecl(prefix + "g", (nv, w)), ParamDecl(prefix + "o", (w, nv)),
                ParamDecl(prefix + "norm", (p.value_dim,), init="norm", role=VECTOR),
                ParamDecl(prefix + "a1", (p.rank, w)), ParamDecl(prefix + "a2", (nk, p.rank)),
                ParamDecl(prefix + "a2.b", (nk,), init="zeros", role=VECTOR)]

    def __init__(self, spec: MixerSpec, weights: Dict[str, torch.Tensor], prefix: str, dtype: torch.dtype,
                 device: torch.device):
        p = spec.params
        if p is None:
            raise ValueError("gated_linear: the sizes come in MixerSpec.params (GatedLinearSpec)")
        self.spec, self.dtype = spec, dtype
        self.heads, self.key_dim, self.value_dim, self.rank = int(p.heads), int(p.key_dim), int(p.value_dim), int(p.rank)
        self.tau, self.q_scale, self.norm_eps = float(p.tau), float(p.q_scale), float(p.norm_eps)
        self.width = int(spec.hidden)
        # the next product reads the low-rank input out of this product's rows: it starts and the rows end on a multiple
        # of 8 (16 bytes), with rows of zeros before and behind it where the sizes want them
        parts = [weights[prefix + s] for s in ("q", "k", "v", "g")]
        rows = 2 * self.heads * (self.key_dim + self.value_dim)
        self.low_at = -(-rows // 8) * 8
        zeros = lambda n: torch.zeros((n, self.width), dtype=parts[0].dtype, device=parts[0].device)
        parts += [zeros(self.low_at - rows), weights[prefix + "a1"], zeros(-self.rank % 8)]
        self.w_in = torch.cat(parts, dim=0).contiguous()
        self.w_a2 = weights[prefix + "a2"]
        self.b_a2 = weights[prefix + "a2.b"].float().contiguous()
        self.w_o = weights[prefix + "o"]
        self.norm_weight = weights[prefix + "norm"].float().contiguous()
        self.state_floats = int(kernels.current().scan_state_floats("gated_linear", self.heads, self.key_dim,
                                                                    self.value_dim))

    def cache_need(self) -> StateNeed:
        return StateNeed((self.state_floats,), torch.float32)

    def forward(self, x, batch, cache: LayerCache):
        ops = kernels.current()
        T = x.shape[0]
        nk, nv = self.heads * self.key_dim, self.heads * self.value_dim
        proj = torch.empty((T, self.w_in.shape[0]), dtype=self.dtype, device=x.device)
        ops.linear(x, self.w_in, proj)
        z = torch.empty((T, nk), dtype=torch.float32, device=x.device)      # pre-activation, kept in float
        ops.linear(proj[:, self.low_at:self.low_at + self.rank], self.w_a2, z)
        read = torch.empty((T, nv), dtype=torch.float32, device=x.device)
        ops.gated_linear_scan(proj, 0, nk, 2 * nk, z, self.b_a2, self.tau, cache.state, batch, self.heads, self.key_dim,
                              self.value_dim, read, q_scale=self.q_scale)
        act = torch.empty((T, nv), dtype=self.dtype, device=x.device)
        ops.head_norm_gate(read, self.norm_weight, False, proj[:, 2 * nk + nv:2 * nk + 2 * nv], "silu", self.norm_eps, self.heads,
                           self.value_dim, act)
        out = torch.empty((T, self.width), dtype=torch.float32, device=x.device)     # enters a float sum as it is
        ops.linear(act, self.w_o, out)
        return out
