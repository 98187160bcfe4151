"""Dokanex: typed configuration from its config.json.

A decoder of pre-norm layers. A layer's mixer is attention inside chunks of the sequence ("attention": queries and keys
divided by their root mean square a head, capped scores, a sink a head in the softmax, a sigmoid gate a head; such a layer may
take the keys and values of an earlier one, ``kv_from``, with a chunk size of its own) or attention over a cached latent
("latent_attention": queries through a latent too, one rotated key part for all heads, neighbouring pairs turned, the
frequencies fitted to longer contexts). Its feed-forward is a silu-gated dense one or absent. The embedding is scaled on its
way in and is the head as well, without that scale; the logits are capped by a tanh.

config.json nests its keys: ``vocab``, ``width``, ``norm.eps``, ``embedding.scale``, ``logit_softcap`` and ``layers[i]`` with
``type``, ``mixer`` and ``mlp``. Tensor names: ``embed``, ``final.norm``, ``l<i>.norm1``, ``l<i>.norm2``, ``l<i>.mix.*``,
``l<i>.mlp.*``. What a model may leave out means "not there": no chunks (every earlier key), no cap, no rotation, frequencies
as they are, factors of 1, a scale of 1 / sqrt(size).
"""
from __future__ import annotations

from dataclasses import dataclass
from typing import Any, Dict, List, Mapping, Optional, Tuple, Union

from .puresun import _At, _section
from .schema import (BlockSpec, ConfigError, FeedForwardSpec, LatentAttentionSpec, MixerSpec, ModelSpec, NormSpec,
                     PositionSpec, RunEntry, YarnSpec, read_float, read_int)

ARCHITECTURE = "Dokanex"

# config.json gives no context limit; the engine's own (block tables and captured steps are sized by it)
DEFAULT_MAX_POSITIONS = 1 << 16


@dataclass(frozen=True)
class DokanexAttention:
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    scale: float
    chunk: int = 0              # 0: every earlier key
    softcap: float = 0.0        # 0: none
    kv_from: Optional[int] = None


@dataclass(frozen=True)
class DokanexLatent:
    heads: int
    dim: int                    # unrotated query/key entries a head
    rot_dim: int                # rotated ones
    vdim: int
    q_rank: int
    kv_rank: int
    scale: float
    rot_base: float = 10000.0
    rot_dims: int = 0           # 0: no rotation
    scaling: Optional[YarnSpec] = None


@dataclass(frozen=True)
class DokanexLayer:
    kind: str                                   # "attention" or "latent_attention"
    mixer: Union[DokanexAttention, DokanexLatent]
    ff: int = 0                                 # 0: no feed-forward


@dataclass(frozen=True)
class DokanexConfig:
    vocab: int
    width: int
    norm_eps: float
    embedding_scale: float
    logit_softcap: float
    layers: Tuple[DokanexLayer, ...]
    max_positions: int = DEFAULT_MAX_POSITIONS
    architecture: str = ARCHITECTURE

    # ---------------------------------------------------------------- reading
    @classmethod
    def from_dict(cls, cfg: Mapping[str, Any]) -> "DokanexConfig":
        vocab = read_int(cfg, "vocab", minimum=1)
        width = read_int(cfg, "width", minimum=1)
        eps = _At(_section(cfg, "norm"), "norm.").float("eps")
        if eps < 0.0:
            raise ConfigError("norm.eps", "must be >= 0")
        emb = _section(cfg, "embedding", required=False)
        emb_scale = _At(emb, "embedding.").float("scale", 1.0) if emb is not None else 1.0
        cap = read_float(cfg, "logit_softcap", 0.0)
        if cap < 0.0:
            raise ConfigError("logit_softcap", "must be >= 0 (absent: no cap)")
        raw_layers = cfg.get("layers", None)
        if not isinstance(raw_layers, list) or not raw_layers:
            raise ConfigError("layers", "expected a non-empty list of layers")
        layers = tuple(cls._read_layer(L, f"layers[{i}].") for i, L in enumerate(raw_layers))
        for i, L in enumerate(layers):
            src = L.mixer.kv_from if L.kind == "attention" else None
            if src is None:
                continue
            where = f"layers[{i}].mixer.kv_from"
            if not 0 <= src < i:
                raise ConfigError(where, f"layer {src} must come before layer {i}")
            S = layers[src]
            if S.kind != "attention" or S.mixer.kv_from is not None:
                raise ConfigError(where, f"layer {src} keeps no keys and values of its own for an attention layer to read")
            a, b = L.mixer, S.mixer
            if (a.kv_heads, a.dim, a.vdim) != (b.kv_heads, b.dim, b.vdim):
                raise ConfigError(where, f"layer {src} keeps other heads than layer {i} reads")
        return cls(vocab=vocab, width=width, norm_eps=eps, embedding_scale=emb_scale, logit_softcap=cap, layers=layers,
                   max_positions=read_int(cfg, "max_positions", DEFAULT_MAX_POSITIONS, minimum=1))

    @staticmethod
    def _read_attention(m: Mapping[str, Any], where: str) -> DokanexAttention:
        at = _At(m, where)
        heads, kv = at.int("heads", minimum=1), at.int("kv_heads", minimum=1)
        if heads % kv:
            raise ConfigError(where + "kv_heads", f"{heads} query heads do not divide into {kv} groups")
        dim = at.int("dim", minimum=1)
        mask = _section(m, "mask", where, required=False)
        chunk = _At(mask, where + "mask.").int("size", minimum=1) if mask is not None else 0
        cap = at.float("softcap", 0.0)
        if cap < 0.0:
            raise ConfigError(where + "softcap", "must be > 0 (absent: no cap)")
        src = at.int("kv_from", minimum=0) if m.get("kv_from", None) is not None else None
        return DokanexAttention(heads=heads, kv_heads=kv, dim=dim, vdim=at.int("vdim", dim, minimum=1),
                                scale=at.float("scale", float(dim) ** -0.5), chunk=chunk, softcap=cap, kv_from=src)

    @staticmethod
    def _read_latent(m: Mapping[str, Any], where: str) -> DokanexLatent:
        at = _At(m, where)
        heads, dim, rot_dim = at.int("heads", minimum=1), at.int("dim", minimum=0), at.int("rot_dim", 0, minimum=0)
        if dim + rot_dim == 0:
            raise ConfigError(where + "dim", "a head needs at least one query/key entry")
        rot = _section(m, "rot", where, required=False)
        base, dims, scaling = 10000.0, 0, None
        if rot is not None:
            rat = _At(rot, where + "rot.")
            base, dims = rat.float("base"), rat.int("dims", rot_dim, minimum=0)
            if base <= 0.0:
                raise ConfigError(where + "rot.base", "must be > 0")
            if dims % 2 or dims > rot_dim:
                raise ConfigError(where + "rot.dims", f"{dims} entries in pairs out of {rot_dim}")
            sc = _section(rot, "scaling", where + "rot.", required=False)
            if sc is not None:
                sat = _At(sc, where + "rot.scaling.")
                scaling = YarnSpec(factor=sat.float("factor"), original=sat.float("original"), fast=sat.float("fast"),
                                   slow=sat.float("slow"))
                for key in ("factor", "original", "fast", "slow"):
                    if not getattr(scaling, key) > 0.0:
                        raise ConfigError(where + "rot.scaling." + key, "must be > 0")
                if base == 1.0:
                    raise ConfigError(where + "rot.base", "frequencies that are all alike are not scaled by their turns")
        return DokanexLatent(heads=heads, dim=dim, rot_dim=rot_dim, vdim=at.int("vdim", minimum=1),
                             q_rank=at.int("q_rank", minimum=1), kv_rank=at.int("kv_rank", minimum=1),
                             scale=at.float("scale", float(dim + rot_dim) ** -0.5), rot_base=base, rot_dims=dims,
                             scaling=scaling if dims else None)

    @classmethod
    def _read_layer(cls, L: Any, where: str) -> DokanexLayer:
        if not isinstance(L, dict):
            raise ConfigError(where.rstrip("."), f"expected an object, got {L!r}")
        kind = L.get("type", None)
        readers = {"attention": cls._read_attention, "latent_attention": cls._read_latent}
        if kind not in readers:
            raise ConfigError(where + "type", f"unknown mixer {kind!r}; this design has 'attention' and 'latent_attention'")
        mixer = readers[kind](_section(L, "mixer", where), where + "mixer.")
        ff = 0
        f = L.get("mlp", None)
        if f is not None:
            if not isinstance(f, dict):
                raise ConfigError(where + "mlp", f"expected an object or null, got {f!r}")
            if f.get("kind", None) != "dense":
                raise ConfigError(where + "mlp.kind", f"unknown feed-forward {f.get('kind')!r}; this design has 'dense'")
            ff = _At(f, where + "mlp.").int("ff", minimum=1)
        return DokanexLayer(kind=kind, mixer=mixer, ff=ff)

    # ---------------------------------------------------------------- writing
    def to_dict(self) -> Dict[str, Any]:
        layers: List[Dict[str, Any]] = []
        for L in self.layers:
            m = L.mixer
            if L.kind == "attention":
                mixer: Dict[str, Any] = {"dim": m.dim, "heads": m.heads, "kv_heads": m.kv_heads, "scale": m.scale,
                                         "vdim": m.vdim}
                if m.chunk:
                    mixer["mask"] = {"size": m.chunk}
                if m.softcap:
                    mixer["softcap"] = m.softcap
                if m.kv_from is not None:
                    mixer["kv_from"] = m.kv_from
            else:
                mixer = {"dim": m.dim, "heads": m.heads, "kv_rank": m.kv_rank, "q_rank": m.q_rank, "rot_dim": m.rot_dim,
                         "scale": m.scale, "vdim": m.vdim}
                if m.rot_dims:
                    mixer["rot"] = {"base": m.rot_base, "dims": m.rot_dims}
                    if m.scaling is not None:
                        mixer["rot"]["scaling"] = dict(vars(m.scaling))
            layers.append({"mixer": mixer, "mlp": {"ff": L.ff, "kind": "dense"} if L.ff else None, "type": L.kind})
        d: Dict[str, Any] = {"architecture": ARCHITECTURE, "embedding": {"scale": self.embedding_scale}, "layers": layers,
                             "norm": {"eps": self.norm_eps}, "vocab": self.vocab, "width": self.width}
        if self.logit_softcap:
            d["logit_softcap"] = self.logit_softcap
        if self.max_positions != DEFAULT_MAX_POSITIONS:
            d["max_positions"] = self.max_positions
        return d

    # ---------------------------------------------------------------- the model
    def _mixer_spec(self, L: DokanexLayer) -> MixerSpec:
        m = L.mixer
        if L.kind == "attention":
            return MixerSpec(kind="gqa_attention", hidden=self.width, num_heads=m.heads, num_kv_heads=m.kv_heads,
                             head_dim=m.dim, value_dim=m.vdim, scale=m.scale, window=m.chunk, chunked=m.chunk > 0,
                             qk_norm=True, qk_norm_weights=False, qk_norm_eps=self.norm_eps, softcap=m.softcap, sink=True,
                             head_gate=True, kv_shared=m.kv_from is not None, extra=(("names", ("q", "k", "v", "o")),))
        position = PositionSpec("none")
        if m.rot_dims:
            position = PositionSpec("rope_interleaved", rotary_dim=m.rot_dims, theta=m.rot_base, scaling=m.scaling)
        return MixerSpec(kind="latent_attention", hidden=self.width, num_heads=m.heads, num_kv_heads=1, head_dim=m.dim,
                         scale=m.scale, position=position,
                         params=LatentAttentionSpec(rank=m.kv_rank, rot_width=m.rot_dim, value_dim=m.vdim,
                                                    norm_eps=self.norm_eps, gated=False, q_rank=m.q_rank))

    def to_spec(self) -> ModelSpec:
        norm = NormSpec("rmsnorm", self.width, self.norm_eps)
        blocks: List[BlockSpec] = []
        order: List[RunEntry] = []
        for i, L in enumerate(self.layers):
            ffn = None
            if L.ff:
                ffn = FeedForwardSpec(kind="swiglu", hidden=self.width, intermediate=L.ff,
                                      extra=(("names", ("gate", "up", "down")),))
            blocks.append(BlockSpec(kind="prenorm", mixer=self._mixer_spec(L), ffn=ffn, mixer_norm=norm,
                                    ffn_norm=norm if ffn is not None else None, prefix=f"l{i}.", mixer_prefix="mix.",
                                    ffn_prefix="mlp.", mixer_norm_name="norm1", ffn_norm_name="norm2"))
            order.append(RunEntry(i, cache_from=L.mixer.kv_from if L.kind == "attention" else None))
        return ModelSpec(
            architecture=ARCHITECTURE, vocab_size=self.vocab, hidden=self.width, max_positions=self.max_positions,
            blocks=tuple(blocks), run_order=tuple(order), final_norm=norm, tie_embeddings=True, embed_name="embed",
            final_norm_name="final.norm", head_name="head", embed_scale=self.embedding_scale,
            logit_softcap=self.logit_softcap)
