"""Layers over several residual streams (hyper-connections).

The stream is ``streams`` copies X_1 .. X_n, all equal to the embedding at the start. A sublayer (the mixer, then the
feed-forward where there is one) reads h = norm(sum_s in[s] X_s), and its result y changes all of them at once,

    X_t <- sum_s mix[s, t] X_s + out[t] y        (mix is indexed [from, to])

Streams, sums and norms are float. A sublayer's y stays pending (:class:`StreamMix`) until the next one's input is formed:
one kernel a sublayer reads the streams and y, stores the new streams and writes h. At the model's start the copies are not
made: the first two sublayers read the embedding in their place.
"""
from __future__ import annotations

from typing import Dict, List, Optional

import torch

from ..config.schema import BlockSpec
from ..weights import VECTOR, ParamDecl
from .base import LayerCache, StreamMix
from .registry import lookup, register_block


@register_block("hyper")
class HyperBlock:
    @classmethod
    def declare_params(cls, spec: BlockSpec) -> List[ParamDecl]:
        p, n = spec.prefix, int(spec.params.streams)
        out = lookup("norm", spec.mixer_norm.kind).declare_params(spec.mixer_norm, p + spec.mixer_norm_name)
        out += lookup("mixer", spec.mixer.kind).declare_params(spec.mixer, p + spec.mixer_prefix)
        if spec.ffn is not None:
            out += lookup("norm", spec.ffn_norm.kind).declare_params(spec.ffn_norm, p + spec.ffn_norm_name)
            out += lookup("feed_forward", spec.ffn.kind).declare_params(spec.ffn, p + spec.ffn_prefix)
        for name in spec.params.names[:2 if spec.ffn is not None else 1]:
            out += [ParamDecl(f"{p}{name}.in", (n,), role=VECTOR), ParamDecl(f"{p}{name}.out", (n,), role=VECTOR),
                    ParamDecl(f"{p}{name}.mix", (n, n), role=VECTOR)]
        return out

    def __init__(self, spec: BlockSpec, weights: Dict[str, torch.Tensor], dtype: torch.dtype, device: torch.device):
        missing = [n for n in ("mixer", "mixer_norm") if getattr(spec, n) is None]
        if spec.ffn is not None and spec.ffn_norm is None:
            missing.append("ffn_norm")
        if missing:
            raise ValueError(f"a hyper block is made of a mixer with a norm before it and at most a feed-forward with a "
                             f"norm before it; block {spec.prefix!r} names no {', '.join(missing)}")
        p = spec.prefix
        self.spec, self.dtype = spec, dtype
        self.mixer_norm = lookup("norm", spec.mixer_norm.kind)(spec.mixer_norm, weights, p + spec.mixer_norm_name, dtype,
                                                               device)
        self.mixer = lookup("mixer", spec.mixer.kind)(spec.mixer, weights, p + spec.mixer_prefix, dtype, device)
        self.ffn_norm = self.ffn = None
        if spec.ffn is not None:
            self.ffn_norm = lookup("norm", spec.ffn_norm.kind)(spec.ffn_norm, weights, p + spec.ffn_norm_name, dtype, device)
            self.ffn = lookup("feed_forward", spec.ffn.kind)(spec.ffn, weights, p + spec.ffn_prefix, dtype, device)
        for n in (self.mixer_norm, self.ffn_norm):
            if n is not None and getattr(n, "groups", 1) != 1:
                raise ValueError("a hyper block norms the sum of its streams over the whole width")
        # (in, out, mix) of each sublayer, float
        self.connections = [tuple(weights[f"{p}{name}.{s}"].float().contiguous() for s in ("in", "out", "mix"))
                            for name in spec.params.names[:2 if self.ffn is not None else 1]]

    @property
    def graph_safe(self) -> bool:
        return bool(getattr(self.mixer, "graph_safe", False)
                    and (self.ffn is None or getattr(self.ffn, "graph_safe", False)))

    def cache_need(self):
        return self.mixer.cache_need() if hasattr(self.mixer, "cache_need") else None

    def parts(self):
        return tuple(p for p in (self.mixer_norm, self.mixer, self.ffn_norm, self.ffn) if p is not None)

    def _sublayer(self, ops, streams, pending: StreamMix, norm, connection, part) -> StreamMix:
        w_in, w_out, mix = connection
        h = pending.norm_of(ops, streams, w_in, norm.float_weight, norm.eps, self.dtype)
        return StreamMix(base=pending.stored().base, y=part(h), mix=mix, w_out=w_out)

    def forward(self, streams: torch.Tensor, pending: StreamMix, batch, cache: Optional[LayerCache]) -> StreamMix:
        from .. import kernels
        ops = kernels.current()
        pending = self._sublayer(ops, streams, pending, self.mixer_norm, self.connections[0],
                                 lambda h: self.mixer.forward(h, batch, cache))
        if self.ffn is not None:
            pending = self._sublayer(ops, streams, pending, self.ffn_norm, self.connections[1],
                                     lambda h: self.ffn.forward(h, batch))
        return pending
