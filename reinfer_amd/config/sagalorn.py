"""Sagalorn: typed configuration from its config.json.

A decoder of pre-norm layers over several residual streams (hyper-connections): a sublayer reads a weighted sum of the
streams and its result changes all of them at once. A layer's mixer is retention (linear attention with a fixed decay a
head, queries and keys turned by their position, a silu gate), attention inside a sliding window that keeps the first
tokens in sight (values are the keys as projected, per-head query/key norms, biases, no rotation), or gated linear
attention (a decay a key channel that depends on the input). Its feed-forward is a silu-gated dense one or absent. A run of
layers may be repeated with the same weights, each pass with caches and states of its own. The embedding is scaled on its
way in, the head is a tensor of its own, the logits are multiplied by a constant.

config.json nests its keys: ``vocab``, ``width``, ``norm.eps``, ``embedding.scale``, ``logit_scale``, ``streams``,
``loop.{start, stop, times}`` and ``layers[i]`` with ``type``, ``mixer`` and ``mlp``. Tensor names: ``embed``, ``head``,
``final.norm``, ``l<i>.norm1``, ``l<i>.norm2``, ``l<i>.mix.*``, ``l<i>.mlp.*``, ``l<i>.hc1.{in, out, mix}``, ``l<i>.hc2.*``.
What a model may leave out means "not there": no window, no kept tokens, no rotation, one plain stream without
connections, no repeated run, factors of 1. The rank of a gated linear layer's decay is given by its tensors alone.
"""
from __future__ import annotations

from dataclasses import dataclass
from typing import Any, Dict, List, Mapping, Optional, Tuple, Union

from .puresun import _At, _section
from .schema import (BlockSpec, ConfigError, DecayMemorySpec, FeedForwardSpec, GatedLinearSpec, HyperSpec, MixerSpec,
                     ModelSpec, NormSpec, PositionSpec, RunEntry, read_float, read_int)

ARCHITECTURE = "Sagalorn"

# config.json gives no context limit; the engine's own (block tables and captured steps are sized by it)
DEFAULT_MAX_POSITIONS = 1 << 16


@dataclass(frozen=True)
class SagalornRetention:
    heads: int
    dim: int
    vdim: int
    decay: Tuple[float, ...]
    rot_base: float = 10000.0
    rot_dims: int = 0           # 0: no rotation


@dataclass(frozen=True)
class SagalornAttention:
    heads: int
    kv_heads: int
    dim: int
    scale: float
    window: int = 0             # 0: every earlier key
    keep_first: int = 0


@dataclass(frozen=True)
class SagalornGLA:
    heads: int
    dim: int
    vdim: int
    tau: float


@dataclass(frozen=True)
class SagalornLayer:
    kind: str                                   # "retention", "attention" or "gla"
    mixer: Union[SagalornRetention, SagalornAttention, SagalornGLA]
    ff: int = 0                                 # 0: no feed-forward


@dataclass(frozen=True)
class SagalornConfig:
    vocab: int
    width: int
    norm_eps: float
    embedding_scale: float
    logit_scale: float
    streams: int                                # 0: one plain stream
    loop: Optional[Tuple[int, int, int]]        # start, stop, times
    layers: Tuple[SagalornLayer, ...]
    gla_ranks: Tuple[int, ...] = ()             # a layer each, 0 where it has no such decay
    max_positions: int = DEFAULT_MAX_POSITIONS
    architecture: str = ARCHITECTURE

    # ---------------------------------------------------------------- reading
    @classmethod
    def from_dict(cls, cfg: Mapping[str, Any]) -> "SagalornConfig":
        vocab = read_int(cfg, "vocab", minimum=1)
        width = read_int(cfg, "width", minimum=1)
        eps = _At(_section(cfg, "norm"), "norm.").float("eps")
        if eps < 0.0:
            raise ConfigError("norm.eps", "must be >= 0")
        emb = _section(cfg, "embedding", required=False)
        emb_scale = _At(emb, "embedding.").float("scale", 1.0) if emb is not None else 1.0
        raw_layers = cfg.get("layers", None)
        if not isinstance(raw_layers, list) or not raw_layers:
            raise ConfigError("layers", "expected a non-empty list of layers")
        layers = tuple(cls._read_layer(L, f"layers[{i}].") for i, L in enumerate(raw_layers))
        loop = None
        section = _section(cfg, "loop", required=False)
        if section is not None:
            at = _At(section, "loop.")
            start, stop, times = at.int("start", minimum=0), at.int("stop", minimum=0), at.int("times", minimum=1)
            if not start < stop <= len(layers):
                raise ConfigError("loop.stop", f"layers {start} to {stop - 1} of {len(layers)} are no run of layers")
            loop = (start, stop, times)
        ranks = cfg.get("gla_ranks", None)
        if ranks is not None and (not isinstance(ranks, list) or len(ranks) != len(layers)
                                  or any(isinstance(r, bool) or not isinstance(r, int) or r < 0 for r in ranks)):
            raise ConfigError("gla_ranks", f"expected {len(layers)} numbers, one a layer")
        return cls(vocab=vocab, width=width, norm_eps=eps, embedding_scale=emb_scale,
                   logit_scale=read_float(cfg, "logit_scale", 1.0), streams=read_int(cfg, "streams", 0, minimum=1),
                   loop=loop, layers=layers, gla_ranks=tuple(ranks) if ranks is not None else (),
                   max_positions=read_int(cfg, "max_positions", DEFAULT_MAX_POSITIONS, minimum=1))

    @staticmethod
    def _read_retention(m: Mapping[str, Any], where: str) -> SagalornRetention:
        at = _At(m, where)
        heads, dim = at.int("heads", minimum=1), at.int("dim", minimum=1)
        decay = m.get("decay", None)
        if not isinstance(decay, list) or len(decay) != heads or \
                any(isinstance(d, bool) or not isinstance(d, (int, float)) for d in decay):
            raise ConfigError(where + "decay", f"expected {heads} numbers, one a head")
        rot = _section(m, "rot", where, required=False)
        base, dims = 10000.0, 0
        if rot is not None:
            rat = _At(rot, where + "rot.")
            base, dims = rat.float("base"), rat.int("dims", minimum=0)
            if base <= 0.0:
                raise ConfigError(where + "rot.base", "must be > 0")
            if dims % 2 or dims > dim:
                raise ConfigError(where + "rot.dims", f"{dims} entries in pairs out of {dim}")
        return SagalornRetention(heads=heads, dim=dim, vdim=at.int("vdim", minimum=1),
                                 decay=tuple(float(d) for d in decay), rot_base=base, rot_dims=dims)

    @staticmethod
    def _read_attention(m: Mapping[str, Any], where: str) -> SagalornAttention:
        at = _At(m, where)
        heads, kv = at.int("heads", minimum=1), at.int("kv_heads", minimum=1)
        if heads % kv:
            raise ConfigError(where + "kv_heads", f"{heads} query heads do not divide into {kv} groups")
        dim = at.int("dim", minimum=1)
        if at.int("vdim", dim, minimum=1) != dim:
            raise ConfigError(where + "vdim", f"the values are the keys: their size is {dim}")
        mask = _section(m, "mask", where, required=False)
        window = keep = 0
        if mask is not None:
            mat = _At(mask, where + "mask.")
            window, keep = mat.int("size", minimum=1), mat.int("keep_first", 0, minimum=0)
        return SagalornAttention(heads=heads, kv_heads=kv, dim=dim, scale=at.float("scale", float(dim) ** -0.5),
                                 window=window, keep_first=keep)

    @staticmethod
    def _read_gla(m: Mapping[str, Any], where: str) -> SagalornGLA:
        at = _At(m, where)
        tau = at.float("tau")
        if not tau > 0.0:
            raise ConfigError(where + "tau", "must be > 0")
        return SagalornGLA(heads=at.int("heads", minimum=1), dim=at.int("dim", minimum=1), vdim=at.int("vdim", minimum=1),
                           tau=tau)

    @classmethod
    def _read_layer(cls, L: Any, where: str) -> SagalornLayer:
        if not isinstance(L, dict):
            raise ConfigError(where.rstrip("."), f"expected an object, got {L!r}")
        kind = L.get("type", None)
        readers = {"retention": cls._read_retention, "attention": cls._read_attention, "gla": cls._read_gla}
        if kind not in readers:
            raise ConfigError(where + "type", f"unknown mixer {kind!r}; this design has 'retention', 'attention' and 'gla'")
        mixer = readers[kind](_section(L, "mixer", where), where + "mixer.")
        ff = 0
        f = L.get("mlp", None)
        if f is not None:
            if not isinstance(f, dict):
                raise ConfigError(where + "mlp", f"expected an object or null, got {f!r}")
            if f.get("kind", None) != "dense":
                raise ConfigError(where + "mlp.kind", f"unknown feed-forward {f.get('kind')!r}; this design has 'dense'")
            ff = _At(f, where + "mlp.").int("ff", minimum=1)
        return SagalornLayer(kind=kind, mixer=mixer, ff=ff)

    # ---------------------------------------------------------------- writing
    def to_dict(self) -> Dict[str, Any]:
        layers: List[Dict[str, Any]] = []
        for L in self.layers:
            m = L.mixer
            if L.kind == "retention":
                mixer: Dict[str, Any] = {"decay": list(m.decay), "dim": m.dim, "heads": m.heads, "vdim": m.vdim}
                if m.rot_dims:
                    mixer["rot"] = {"base": m.rot_base, "dims": m.rot_dims}
            elif L.kind == "attention":
                mixer = {"dim": m.dim, "heads": m.heads, "kv_heads": m.kv_heads, "scale": m.scale, "vdim": m.dim}
                if m.window:
                    mixer["mask"] = {"keep_first": m.keep_first, "size": m.window}
            else:
                mixer = {"dim": m.dim, "heads": m.heads, "tau": m.tau, "vdim": m.vdim}
            layers.append({"mixer": mixer, "mlp": {"ff": L.ff, "kind": "dense"} if L.ff else None, "type": L.kind})
        d: Dict[str, Any] = {"architecture": ARCHITECTURE, "embedding": {"scale": self.embedding_scale}, "layers": layers,
                             "logit_scale": self.logit_scale, "norm": {"eps": self.norm_eps}, "vocab": self.vocab,
                             "width": self.width}
        if self.streams:
            d["streams"] = self.streams
        if self.loop is not None:
            d["loop"] = dict(zip(("start", "stop", "times"), self.loop))
        if any(self.gla_ranks):
            d["gla_ranks"] = list(self.gla_ranks)
        if self.max_positions != DEFAULT_MAX_POSITIONS:
            d["max_positions"] = self.max_positions
        return d

    # ---------------------------------------------------------------- the model
    def with_tensor_shapes(self, shapes: Mapping[str, Tuple[int, ...]]) -> "SagalornConfig":
        """The configuration with the sizes that only the tensors give: the rank of a gated linear layer's decay, the rows
        of ``l<i>.mix.a1``."""
        ranks = []
        for i, L in enumerate(self.layers):
            shape = shapes.get(f"l{i}.mix.a1") if L.kind == "gla" else None
            ranks.append(int(shape[0]) if shape is not None else 0)
        return SagalornConfig(**{**self.__dict__, "gla_ranks": tuple(ranks)})

    def _rank(self, i: int) -> int:
        r = self.gla_ranks[i] if i < len(self.gla_ranks) else 0
        if r <= 0:
            raise ConfigError(f"layers[{i}].mixer", "the rank of the decay is the number of rows of the layer's mix.a1 "
                                                    "tensor: read it with with_tensor_shapes(), or give gla_ranks")
        return r

    def _mixer_spec(self, i: int, L: SagalornLayer) -> MixerSpec:
        m = L.mixer
        if L.kind == "retention":
            return MixerSpec(kind="decay_memory", hidden=self.width,
                             params=DecayMemorySpec(
                                 heads=m.heads, key_dim=m.dim, value_dim=m.vdim, decays=m.decay, norm_eps=self.norm_eps,
                                 act="none", k_scale=float(m.dim) ** -0.5, head_norm=True, norm_weight=False, gate="silu",
                                 position=PositionSpec("rope_neox", rotary_dim=m.rot_dims, theta=m.rot_base)
                                 if m.rot_dims else PositionSpec("none")))
        if L.kind == "gla":
            return MixerSpec(kind="gated_linear", hidden=self.width,
                             params=GatedLinearSpec(heads=m.heads, key_dim=m.dim, value_dim=m.vdim, rank=self._rank(i),
                                                    tau=m.tau, norm_eps=self.norm_eps, q_scale=float(m.dim) ** -0.5))
        return MixerSpec(kind="gqa_attention", hidden=self.width, num_heads=m.heads, num_kv_heads=m.kv_heads,
                         head_dim=m.dim, scale=m.scale, window=m.window, keep_first=m.keep_first, qk_norm=True,
                         qk_norm_eps=self.norm_eps, bias=True, out_bias=True, values_are_keys=True,
                         extra=(("names", ("q", "k", "v", "o")), ("bias_suffix", ".b"),
                                ("norm_names", ("q.norm", "k.norm"))))

    def run_order(self) -> List[int]:
        n = len(self.layers)
        if self.loop is None:
            return list(range(n))
        start, stop, times = self.loop
        return list(range(start)) + list(range(start, stop)) * times + list(range(stop, n))

    def to_spec(self) -> ModelSpec:
        norm = NormSpec("rmsnorm", self.width, self.norm_eps)
        blocks: List[BlockSpec] = []
        for i, L in enumerate(self.layers):
            ffn = None
            if L.ff:
                ffn = FeedForwardSpec(kind="swiglu", hidden=self.width, intermediate=L.ff,
                                      extra=(("names", ("gate", "up", "down")),))
            blocks.append(BlockSpec(kind="hyper" if self.streams else "prenorm", mixer=self._mixer_spec(i, L), ffn=ffn,
                                    mixer_norm=norm, ffn_norm=norm if ffn is not None else None, prefix=f"l{i}.",
                                    mixer_prefix="mix.", ffn_prefix="mlp.", mixer_norm_name="norm1",
                                    ffn_norm_name="norm2", params=HyperSpec(self.streams) if self.streams else None))
        return ModelSpec(
            architecture=ARCHITECTURE, vocab_size=self.vocab, hidden=self.width, max_positions=self.max_positions,
            blocks=tuple(blocks), run_order=tuple(RunEntry(i) for i in self.run_order()),
            # the constant on the logits stands behind a linear map of the last norm: it goes into that norm's weight
            final_norm=NormSpec("rmsnorm", self.width, self.norm_eps, factor=self.logit_scale), tie_embeddings=False,
            embed_name="embed", final_norm_name="final.norm", head_name="head", embed_scale=self.embedding_scale,
            streams=self.streams)
