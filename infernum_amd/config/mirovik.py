"""Configuration of the Mirovik decoder, read from its own config.json keys.

The file names its design in ``architecture`` and describes every layer by itself:
  vocab, width, norm.eps, embedding.scale,
  loop             null | {start, stop, times}: layers start .. stop-1 run ``times`` times in a row,
  layers[i].type   the mixer: "parallel" | "mamba1",
  layers[i].mixer  parallel: {left: {heads, kv_heads, dim, vdim, scale, bias_max, buckets (only random weights need it)},
                   right: {heads, dim, vdim, decay [heads], rot: {base, dims}}, left_scale, right_scale};
                   mamba1: {inner, state, dt_rank, conv},
  layers[i].mlp    null | {kind: "dense", ff} | {kind: "moe", expert: {ff}, router: {experts, top}, shared: {ff}}.
Layers may differ in every size.  What a file does not mention is not there: no ``embedding``, the table's rows as they
are; no ``loop``, no repetition; no ``rot``, no rotation; no ``shared``, no shared expert.
"""
from __future__ import annotations

from dataclasses import dataclass
from typing import Any, List, Mapping, Optional, Tuple, Union

from .base import ConfigError, KeyReader

MIROVIK_MODEL_TYPE = "Mirovik"
MIXER_TYPES = ("parallel", "mamba1")
MLP_KINDS = ("dense", "moe")


def _need(r: Optional[KeyReader], where: str, key: str) -> KeyReader:
    if r is None:
        raise ConfigError(f"{where}: required key '{key}' is missing")
    return r


@dataclass(frozen=True)
class BiasedAttentionConfig:
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    scale: float
    bias_max: float             # the distance at which the bias table's last row begins, or would
    buckets: Optional[int] = None   # rows of the bias table; None: read off a file's tensor

    @staticmethod
    def from_reader(r: KeyReader) -> "BiasedAttentionConfig":
        heads, kv = r.integer("heads", minimum=1), r.integer("kv_heads", minimum=1)
        if heads % kv:
            raise ConfigError(f"{r.where}: heads {heads} is not a multiple of kv_heads {kv}")
        return BiasedAttentionConfig(heads, kv, r.integer("dim", minimum=1), r.integer("vdim", minimum=1),
                                     r.number("scale", positive=True), r.number("bias_max", positive=True),
                                     r.integer("buckets", None, minimum=2))

    def to_dict(self) -> dict:
        out = {"heads": self.heads, "kv_heads": self.kv_heads, "dim": self.dim, "vdim": self.vdim, "scale": self.scale,
               "bias_max": self.bias_max}
        if self.buckets is not None:
            out["buckets"] = self.buckets
        return out


@dataclass(frozen=True)
class RetentionConfig:
    heads: int
    dim: int
    vdim: int
    decay: Tuple[float, ...]
    rot_base: float = 10000.0
    rot_dims: int = 0

    @staticmethod
    def from_reader(r: KeyReader, raw: Mapping[str, Any]) -> "RetentionConfig":
        heads, dim = r.integer("heads", minimum=1), r.integer("dim", minimum=1)
        decay = raw.get("decay")
        if not isinstance(decay, list) or len(decay) != heads or \
                not all(isinstance(d, (int, float)) and not isinstance(d, bool) and 0 <= d <= 1 for d in decay):
            raise ConfigError(f"{r.where}: 'decay' must list a number between 0 and 1 for each of the {heads} heads, got {decay!r}")
        rot = r.obj("rot")
        base, dims = (rot.number("base", positive=True), rot.integer("dims", minimum=0)) if rot is not None else (10000.0, 0)
        if dims > dim or dims % 2:
            raise ConfigError(f"{r.where}: rot.dims must be even and at most {dim}, got {dims}")
        return RetentionConfig(heads, dim, r.integer("vdim", minimum=1), tuple(float(d) for d in decay), base, dims)

    def to_dict(self) -> dict:
        out = {"heads": self.heads, "dim": self.dim, "vdim": self.vdim, "decay": list(self.decay)}
        if self.rot_dims:
            out["rot"] = {"base": self.rot_base, "dims": self.rot_dims}
        return out


@dataclass(frozen=True)
class ParallelConfig:
    left: BiasedAttentionConfig
    right: RetentionConfig
    left_scale: float
    right_scale: float

    @staticmethod
    def from_reader(r: KeyReader, raw: Mapping[str, Any]) -> "ParallelConfig":
        return ParallelConfig(BiasedAttentionConfig.from_reader(_need(r.obj("left"), r.where, "left")),
                              RetentionConfig.from_reader(_need(r.obj("right"), r.where, "right"), raw["right"]),
                              r.number("left_scale", 1.0), r.number("right_scale", 1.0))

    def to_dict(self) -> dict:
        return {"left": self.left.to_dict(), "right": self.right.to_dict(), "left_scale": self.left_scale,
                "right_scale": self.right_scale}


@dataclass(frozen=True)
class MambaConfig:
    inner: int
    state: int
    dt_rank: int
    conv: int

    @staticmethod
    def from_reader(r: KeyReader, raw: Mapping[str, Any]) -> "MambaConfig":
        return MambaConfig(r.integer("inner", minimum=1), r.integer("state", minimum=1), r.integer("dt_rank", minimum=1),
                           r.integer("conv", minimum=1))

    def to_dict(self) -> dict:
        return {"inner": self.inner, "state": self.state, "dt_rank": self.dt_rank, "conv": self.conv}


_MIXERS = {"parallel": ParallelConfig, "mamba1": MambaConfig}


@dataclass(frozen=True)
class MlpConfig:
    kind: str
    ff: int                     # the dense middle, or an expert's
    experts: int = 0
    top: int = 0
    shared_ff: Optional[int] = None

    @staticmethod
    def from_reader(r: KeyReader) -> "MlpConfig":
        kind = r.string("kind", choices=MLP_KINDS)
        if kind == "dense":
            return MlpConfig(kind, r.integer("ff", minimum=1))
        router, expert = _need(r.obj("router"), r.where, "router"), _need(r.obj("expert"), r.where, "expert")
        shared = r.obj("shared")
        m = MlpConfig(kind, expert.integer("ff", minimum=1), router.integer("experts", minimum=1), router.integer("top", minimum=1),
                      shared.integer("ff", minimum=1) if shared is not None else None)
        if m.top > m.experts:
            raise ConfigError(f"{r.where}: {m.experts} experts cannot give a token {m.top}")
        return m

    def to_dict(self) -> dict:
        if self.kind == "dense":
            return {"kind": self.kind, "ff": self.ff}
        out = {"kind": self.kind, "expert": {"ff": self.ff}, "router": {"experts": self.experts, "top": self.top}}
        if self.shared_ff is not None:
            out["shared"] = {"ff": self.shared_ff}
        return out


@dataclass(frozen=True)
class LoopConfig:
    start: int
    stop: int
    times: int


@dataclass(frozen=True)
class MirovikLayerConfig:
    type: str
    mixer: Union[ParallelConfig, MambaConfig]
    mlp: Optional[MlpConfig]


@dataclass(frozen=True)
class MirovikConfig:
    vocab: int
    width: int
    norm_eps: float
    layers: Tuple[MirovikLayerConfig, ...]
    embedding_scale: float = 1.0
    loop: Optional[LoopConfig] = None
    model_type: str = MIROVIK_MODEL_TYPE

    # what the generation entry points ask of every configuration
    @property
    def vocab_size(self) -> int:
        return self.vocab

    @property
    def hidden_size(self) -> int:
        return self.width

    @property
    def num_hidden_layers(self) -> int:
        return len(self.layers)

    bos_token_id = None
    eos_token_id = None

    def layer_runs(self) -> List[Tuple[int, int]]:
        """(layer, pass of the loop that the run belongs to, 0 outside the loop) in the order the layers run."""
        n = len(self.layers)
        if self.loop is None:
            return [(i, 0) for i in range(n)]
        a, b = self.loop.start, self.loop.stop
        return [(i, 0) for i in range(a)] + [(i, t) for t in range(self.loop.times) for i in range(a, b)] + \
            [(i, 0) for i in range(b, n)]

    @staticmethod
    def from_dict(raw: Mapping[str, Any], where: str = "config.json") -> "MirovikConfig":
        r = KeyReader(raw, where)
        norm = _need(r.obj("norm"), where, "norm")
        emb = r.obj("embedding")
        listed = raw.get("layers")
        if not isinstance(listed, list) or not listed:
            raise ConfigError(f"{where}: 'layers' must be a list with at least one layer")
        layers = []
        for i, entry in enumerate(listed):
            lr = KeyReader(entry, f"{where}:layers[{i}]")
            kind = lr.string("type", choices=MIXER_TYPES)
            mixer = _MIXERS[kind].from_reader(_need(lr.obj("mixer"), lr.where, "mixer"), entry["mixer"])
            mlp = lr.obj("mlp")
            layers.append(MirovikLayerConfig(kind, mixer, MlpConfig.from_reader(mlp) if mlp is not None else None))
        loop, lp = None, r.obj("loop")
        if lp is not None:
            loop = LoopConfig(lp.integer("start", minimum=0), lp.integer("stop", minimum=0), lp.integer("times", minimum=1))
            if not loop.start <= loop.stop <= len(layers):
                raise ConfigError(f"{where}: loop {loop.start} .. {loop.stop} does not lie within the {len(layers)} layers")
        return MirovikConfig(vocab=r.integer("vocab", minimum=1), width=r.integer("width", minimum=1),
                             norm_eps=norm.number("eps", positive=True), layers=tuple(layers),
                             embedding_scale=emb.number("scale", 1.0) if emb is not None else 1.0, loop=loop)

    def to_dict(self) -> dict:
        out = {"architecture": self.model_type, "vocab": self.vocab, "width": self.width, "norm": {"eps": self.norm_eps},
               "embedding": {"scale": self.embedding_scale},
               "layers": [{"type": l.type, "mixer": l.mixer.to_dict(), "mlp": l.mlp.to_dict() if l.mlp else None}
                          for l in self.layers]}
        if self.loop is not None:
            out["loop"] = {"start": self.loop.start, "stop": self.loop.stop, "times": self.loop.times}
        return out
