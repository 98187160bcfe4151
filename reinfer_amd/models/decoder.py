"""A decoder put together from a :class:`ModelSpec`: embedding, blocks in run
order, final norm, head. It knows no architecture by name; what differs between
architectures is in the spec and in the parts the spec names.
"""
from __future__ import annotations

from typing import Dict, List, Optional, Sequence

import torch

from .. import kernels
from ..config.schema import ModelSpec
from ..parts import KVNeed, LayerCache, StateNeed, StreamMix, lookup
from ..weights import MATRIX, ParamDecl


def declare_params(spec: ModelSpec) -> List[ParamDecl]:
    """Every tensor the model reads, each once, in a fixed order."""
    out = [ParamDecl(spec.embed_name, (spec.vocab_size, spec.hidden))]
    if spec.input_position is not None:
        part = lookup("position", spec.input_position.kind)
        if hasattr(part, "declare_input_params"):
            out += part.declare_input_params(spec.input_position, spec.input_position_prefix)
    for inp in spec.inputs:
        out += lookup("input", inp.kind).declare_params(inp, spec.hidden)
    for name, rows in spec.stream_vectors:
        out.append(ParamDecl(name, (rows, spec.hidden)))
    for b in spec.blocks:
        out += lookup("block", b.kind).declare_params(b)
    out += lookup("norm", spec.final_norm.kind).declare_params(spec.final_norm, spec.final_norm_name)
    # a tied model may still carry a head tensor in its file: it is not read
    out.append(ParamDecl(spec.head_name, (spec.vocab_size, spec.hidden), optional=spec.tie_embeddings))
    seen = set()
    for d in out:
        if d.name in seen:
            raise ValueError(f"tensor {d.name} is declared twice")
        seen.add(d.name)
    return out


class DecoderModel:
    def __init__(self, spec: ModelSpec, weights: Dict[str, torch.Tensor], dtype: torch.dtype,
                 device: torch.device):
        self.spec = spec
        self.dtype = dtype
        self.device = device
        self.embed = weights[spec.embed_name]
        # a position part at the embedding stage: built with the model's tensors, it adds its encoding of
        # the step's positions into the stream (``add_to_stream(resid, batch)``)
        self.input_position = None
        if spec.input_position is not None:
            part = lookup("position", spec.input_position.kind)
            if not hasattr(part, "add_to_stream"):
                raise ValueError(f"position part {spec.input_position.kind!r} cannot stand at the embedding: "
                                 "it has no add_to_stream(resid, batch)")
            self.input_position = part(spec.input_position, device, weights=weights,
                                       prefix=spec.input_position_prefix, dtype=dtype)
        # further parts that add to the embedding; one that keeps per-request state says so (``state_need()``)
        # and is handed that state by whoever runs the model (``input_states``, in the order of ``inputs``)
        self.inputs = [lookup("input", inp.kind)(inp, weights, spec.hidden, dtype, device) for inp in spec.inputs]
        # rows that run-order entries add to the stream, and whether any of them adds the embedding again
        self.stream_vectors = {name: weights[name] for name, _ in spec.stream_vectors}
        self.keeps_embedding = any(e.before is not None and e.before.embedding for e in spec.run_order)
        self.blocks = [lookup("block", b.kind)(b, weights, dtype, device) for b in spec.blocks]
        self.final_norm = lookup("norm", spec.final_norm.kind)(spec.final_norm, weights,
                                                               spec.final_norm_name, dtype, device)
        # tied: the embedding matrix is the head (crates/cpu/src/model.rs:218-225)
        self.head = self.embed if spec.tie_embeddings else weights[spec.head_name]
        self.run_order = spec.run_order

    def cache_needs(self) -> List[Optional[object]]:
        """What each run-order entry keeps: KVNeed, PagedNeed, StateNeed, or None. The block arrangement
        answers (``cache_need()``); one that does not is asked for a ``mixer`` attribute's answer."""
        needs: List[Optional[object]] = []
        for e in self.run_order:
            block = self.blocks[e.block]
            if hasattr(block, "cache_need"):
                needs.append(block.cache_need())
                continue
            mixer = getattr(block, "mixer", None)
            needs.append(mixer.cache_need() if mixer is not None and hasattr(mixer, "cache_need") else None)
        return needs

    def parts(self):
        """Every part of the model once: blocks, what they say they are made of, the norms and position part
        at either end."""
        seen, out = set(), []
        def add(p):
            if p is not None and id(p) not in seen:
                seen.add(id(p))
                out.append(p)
        add(self.input_position)
        for p in self.inputs:
            add(p)
        for b in self.blocks:
            add(b)
            for p in (b.parts() if hasattr(b, "parts") else (getattr(b, "mixer", None), getattr(b, "ffn", None))):
                add(p)
        add(self.final_norm)
        return out

    def plan_captured_step(self, batch, num_rows: int, ctx_cap: int) -> None:
        """A decode step that is captured once and replayed takes no host-side number from the step it
        replays for: whatever a part's kernels choose grids or buffers by on the host must be fixed for the
        bucket. Every part with a ``plan_captured_step(batch, num_rows, ctx_cap)`` is asked to write what it
        needs into ``batch.extra`` (``num_rows`` requests of one token each, contexts of at most ``ctx_cap``)."""
        for p in self.parts():
            hook = getattr(p, "plan_captured_step", None)
            if hook is not None:
                hook(batch, num_rows, ctx_cap)

    def input_needs(self) -> List[Optional[StateNeed]]:
        """Per-request state that each input part keeps (None: none), in the order of ``inputs``."""
        return [p.state_need() if hasattr(p, "state_need") else None for p in self.inputs]

    def forward_layers(self, batch, caches: Sequence[Optional[LayerCache]], observer=None, input_states=None):
        """Embedding and all blocks: (residual stream, last addend not yet added).

        ``observer(i, hidden)``, if given, is called with the float32 hidden state [T, hidden] behind
        the embedding (i = 0) and behind run-order entry i - 1 (the reference reads activations back
        layer by layer the same way, crates/cuda/src/engine.rs:3744-3765)."""
        ops = kernels.current()
        resid = torch.empty((batch.num_tokens, self.spec.hidden), dtype=torch.float32, device=self.device)
        if self.spec.embed_scale != 1.0:
            ops.embed(self.embed, batch.token_ids, resid, scale=float(self.spec.embed_scale))
        else:
            ops.embed(self.embed, batch.token_ids, resid)
        if self.input_position is not None:
            self.input_position.add_to_stream(resid, batch)
        for k, part in enumerate(self.inputs):
            part.add_to_stream(resid, batch, input_states[k] if input_states is not None else None)
        if observer is not None:
            observer(0, resid.clone())
        embedded = resid.clone() if self.keeps_embedding else None
        delta = None
        if self.spec.streams:
            # several streams: all equal to the embedding until the first sublayer's result has entered
            delta = StreamMix(base=resid)
            resid = torch.empty((batch.num_tokens, self.spec.streams, self.spec.hidden), dtype=torch.float32,
                                device=self.device)
        n = len(self.run_order)
        for i, e in enumerate(self.run_order):
            block = self.blocks[e.block]
            if e.before is not None:
                # what the run order adds ahead of this entry, together with the last block's pending addend
                if delta is not None and not isinstance(delta, torch.Tensor):
                    delta = None
                ops.stream_add(resid, delta, embedded if e.before.embedding else None,
                               self.stream_vectors[e.before.vector][e.before.row] if e.before.vector else None)
                delta = None
            # the block that runs next may offer buffers that let this block's last product prepare
            # its first norm
            tgt = None
            if i + 1 < n and getattr(block, "passes_emit", False):
                nxt = self.blocks[self.run_order[i + 1].block]
                if hasattr(nxt, "entry_target"):
                    tgt = nxt.entry_target(resid)
            if tgt is not None:
                delta = block.forward(resid, delta, batch, caches[i], emit=tgt)
            else:
                delta = block.forward(resid, delta, batch, caches[i])
            if observer is not None:
                # the block's last addend may not be in the stream yet
                if isinstance(delta, StreamMix):
                    observer(i + 1, delta.norm_of(ops, resid, None, None, 0.0, torch.float32, store=False))
                    continue
                observer(i + 1, resid + delta.float() if isinstance(delta, torch.Tensor) else resid.clone())
        return resid, delta

    def forward(self, batch, caches: Sequence[Optional[LayerCache]], observer=None, input_states=None) -> torch.Tensor:
        """Logits [len(batch.logit_rows), vocab] in float32 for the step's tokens.

        The head runs on the wanted rows only (the reference computes all rows of
        a prompt and keeps the last, crates/cuda/src/engine.rs:5685-5720)."""
        resid, delta = self.forward_layers(batch, caches, observer, input_states)
        if isinstance(delta, StreamMix):
            # the model's norm reads the sum of the streams
            xn = delta.norm_of(kernels.current(), resid, None, self.final_norm.float_weight, self.final_norm.eps, self.dtype,
                               rows=batch.logit_rows)
        else:
            if delta is not None and not isinstance(delta, torch.Tensor):
                delta = None               # a filled norm target: the sum is already in the stream
            xn = self.final_norm.add_norm(resid, delta, rows=batch.logit_rows)
        logits = torch.empty((batch.num_logit_rows, self.spec.vocab_size), dtype=torch.float32,
                             device=self.device)
        kernels.current().linear(xn, self.head, logits)
        if self.spec.logit_softcap > 0.0:
            kernels.current().tanh_cap(logits, self.spec.logit_softcap)
        return logits
