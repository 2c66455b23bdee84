"""Configuration of the Pamazen decoder, read from its own config.json keys.

The file names its design in ``architecture`` and describes every layer by itself:
  vocab, width, norm.eps, streams, residual_mult, logit_softcap,
  layers[i].type   the mixer: "parallel" | "attention",
  layers[i].mixer  parallel: {left: {heads, kv_heads, dim, vdim, scale, softcap, mask: {size, keep_first}},
                   right: {heads, dim, rank (only random weights need it)}, left_scale, right_scale};
                   attention: {heads, kv_heads, dim, vdim, scale, v_mix, rot: {base, dims, scaling: {factor}}},
  layers[i].mlp    null | {kind: "moe", expert: {ff}, router: {experts, identity, top, groups: {count, keep}},
                   shared: {ff}}.
Layers may differ in every size.  What a file does not mention is not there: no ``mask``, every earlier key; no
``softcap`` or ``logit_softcap``, scores or logits as they are; no ``rot``, no rotation; no ``rot.scaling``, the plain
frequencies; no ``v_mix``, a layer's own values; no ``groups``, one group; no ``identity``, none; no ``shared``, none.
"""
from __future__ import annotations

from dataclasses import dataclass
from typing import Any, Mapping, Optional, Tuple, Union

from .base import ConfigError, KeyReader

PAMAZEN_MODEL_TYPE = "Pamazen"
MIXER_TYPES = ("parallel", "attention")
MLP_KINDS = ("moe",)


def _need(r: Optional[KeyReader], where: str, key: str) -> KeyReader:
    if r is None:
        raise ConfigError(f"{where}: required key '{key}' is missing")
    return r


def _heads(r: KeyReader) -> Tuple[int, int]:
    heads, kv = r.integer("heads", minimum=1), r.integer("kv_heads", minimum=1)
    if heads % kv:
        raise ConfigError(f"{r.where}: heads {heads} is not a multiple of kv_heads {kv}")
    return heads, kv


@dataclass(frozen=True)
class Rotation:
    base: float
    dims: int
    factor: float = 1.0         # every frequency is divided by it

    @staticmethod
    def from_reader(r: Optional[KeyReader], most: int) -> Optional["Rotation"]:
        if r is None:
            return None
        sc = r.obj("scaling")
        rot = Rotation(r.number("base", positive=True), r.integer("dims", minimum=0),
                       sc.number("factor", positive=True) if sc is not None else 1.0)
        if rot.dims > most or rot.dims % 2:
            raise ConfigError(f"{r.where}: dims must be even and at most {most}, got {rot.dims}")
        return rot if rot.dims > 0 else None

    def to_dict(self) -> dict:
        out = {"base": self.base, "dims": self.dims}
        if self.factor != 1.0:
            out["scaling"] = {"factor": self.factor}
        return out


@dataclass(frozen=True)
class AttentionConfig:
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    scale: float
    rot: Optional[Rotation]
    v_mix: bool                 # values mixed with those of the first layer that mixes

    @staticmethod
    def from_reader(r: KeyReader) -> "AttentionConfig":
        heads, kv = _heads(r)
        dim = r.integer("dim", minimum=1)
        return AttentionConfig(heads, kv, dim, r.integer("vdim", minimum=1), r.number("scale", positive=True),
                               Rotation.from_reader(r.obj("rot"), dim), bool(r.boolean("v_mix", False)))

    def to_dict(self) -> dict:
        out = {"heads": self.heads, "kv_heads": self.kv_heads, "dim": self.dim, "vdim": self.vdim, "scale": self.scale,
               "v_mix": self.v_mix}
        if self.rot is not None:
            out["rot"] = self.rot.to_dict()
        return out


@dataclass(frozen=True)
class WindowAttentionConfig:
    heads: int
    kv_heads: int
    dim: int                    # of queries, keys and values: the values are the keys
    scale: float
    softcap: Optional[float]
    window: Optional[int]
    keep_first: int             # positions at a request's start that stay visible beside the window

    @staticmethod
    def from_reader(r: KeyReader) -> "WindowAttentionConfig":
        heads, kv = _heads(r)
        dim = r.integer("dim", minimum=1)
        if r.integer("vdim", dim, minimum=1) != dim:
            raise ConfigError(f"{r.where}: the values are the keys, so vdim must be dim, {dim}")
        mask = r.obj("mask")
        return WindowAttentionConfig(heads, kv, dim, r.number("scale", positive=True),
                                     r.number("softcap", None, positive=True),
                                     mask.integer("size", None, minimum=1) if mask is not None else None,
                                     mask.integer("keep_first", 0, minimum=0) if mask is not None else 0)

    def to_dict(self) -> dict:
        out = {"heads": self.heads, "kv_heads": self.kv_heads, "dim": self.dim, "vdim": self.dim, "scale": self.scale}
        if self.softcap is not None:
            out["softcap"] = self.softcap
        if self.window is not None:
            out["mask"] = {"size": self.window, "keep_first": self.keep_first}
        return out


@dataclass(frozen=True)
class DeltaConfig:
    heads: int
    dim: int
    rank: Optional[int] = None  # the middle of the decays' two products; None: read off a file's tensors

    @staticmethod
    def from_reader(r: KeyReader) -> "DeltaConfig":
        return DeltaConfig(r.integer("heads", minimum=1), r.integer("dim", minimum=1), r.integer("rank", None, minimum=1))

    def to_dict(self) -> dict:
        out = {"heads": self.heads, "dim": self.dim}
        if self.rank is not None:
            out["rank"] = self.rank
        return out


@dataclass(frozen=True)
class ParallelConfig:
    left: WindowAttentionConfig
    right: DeltaConfig
    left_scale: float
    right_scale: float

    @staticmethod
    def from_reader(r: KeyReader) -> "ParallelConfig":
        return ParallelConfig(WindowAttentionConfig.from_reader(_need(r.obj("left"), r.where, "left")),
                              DeltaConfig.from_reader(_need(r.obj("right"), r.where, "right")),
                              r.number("left_scale", 1.0), r.number("right_scale", 1.0))

    def to_dict(self) -> dict:
        return {"left": self.left.to_dict(), "right": self.right.to_dict(), "left_scale": self.left_scale,
                "right_scale": self.right_scale}


_MIXERS = {"parallel": ParallelConfig, "attention": AttentionConfig}


@dataclass(frozen=True)
class MoeConfig:
    ff: int                     # an expert's middle
    experts: int
    top: int
    identity: int = 0           # experts whose result is their input, after the others
    groups: int = 1
    keep: int = 1
    shared_ff: Optional[int] = None

    @staticmethod
    def from_reader(r: KeyReader) -> "MoeConfig":
        r.string("kind", choices=MLP_KINDS)
        router, expert = _need(r.obj("router"), r.where, "router"), _need(r.obj("expert"), r.where, "expert")
        groups, shared = router.obj("groups"), r.obj("shared")
        m = MoeConfig(expert.integer("ff", minimum=1), router.integer("experts", minimum=1), router.integer("top", minimum=1),
                      router.integer("identity", 0, minimum=0), groups.integer("count", minimum=1) if groups else 1,
                      groups.integer("keep", minimum=1) if groups else 1,
                      shared.integer("ff", minimum=1) if shared is not None else None)
        total = m.experts + m.identity
        if total % m.groups or m.keep > m.groups or m.top > m.keep * (total // m.groups):
            raise ConfigError(f"{r.where}: {total} experts in {m.groups} groups, {m.keep} of them kept, cannot give a token {m.top}")
        return m

    def to_dict(self) -> dict:
        router = {"experts": self.experts, "identity": self.identity, "top": self.top}
        if self.groups > 1:
            router["groups"] = {"count": self.groups, "keep": self.keep}
        out = {"kind": "moe", "expert": {"ff": self.ff}, "router": router}
        if self.shared_ff is not None:
            out["shared"] = {"ff": self.shared_ff}
        return out


@dataclass(frozen=True)
class PamazenLayerConfig:
    type: str
    mixer: Union[ParallelConfig, AttentionConfig]
    mlp: Optional[MoeConfig]


@dataclass(frozen=True)
class PamazenConfig:
    vocab: int
    width: int
    norm_eps: float
    streams: int
    residual_mult: float
    layers: Tuple[PamazenLayerConfig, ...]
    logit_softcap: Optional[float] = None
    model_type: str = PAMAZEN_MODEL_TYPE

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

    @property
    def first_value_layer(self) -> Optional[int]:
        """The layer whose values later layers mix theirs with; None when no layer mixes."""
        for i, layer in enumerate(self.layers):
            if isinstance(layer.mixer, AttentionConfig) and layer.mixer.v_mix:
                return i
        return None

    @staticmethod
    def from_dict(raw: Mapping[str, Any], where: str = "config.json") -> "PamazenConfig":
        r = KeyReader(raw, where)
        norm = _need(r.obj("norm"), where, "norm")
        listed = raw.get("layers")
        if not isinstance(listed, list) or not listed:
            raise ConfigError(f"{where}: 'layers' must be a list with at least one layer")
        layers = []
        for i, entry in enumerate(listed):
            lr = KeyReader(entry, f"{where}:layers[{i}]")
            kind = lr.string("type", choices=MIXER_TYPES)
            mixer = _MIXERS[kind].from_reader(_need(lr.obj("mixer"), lr.where, "mixer"))
            mlp = lr.obj("mlp")
            layers.append(PamazenLayerConfig(kind, mixer, MoeConfig.from_reader(mlp) if mlp is not None else None))
        cfg = PamazenConfig(
            vocab=r.integer("vocab", minimum=1), width=r.integer("width", minimum=1), norm_eps=norm.number("eps", positive=True),
            streams=r.integer("streams", minimum=1), residual_mult=r.number("residual_mult", 1.0), layers=tuple(layers),
            logit_softcap=r.number("logit_softcap", None, positive=True))
        mixing = {l.mixer.kv_heads * l.mixer.vdim for l in cfg.layers if isinstance(l.mixer, AttentionConfig) and l.mixer.v_mix}
        if len(mixing) > 1:
            raise ConfigError(f"{where}: layers that mix values must have as many of them, got {sorted(mixing)}")
        return cfg

    def to_dict(self) -> dict:
        out = {"architecture": self.model_type, "vocab": self.vocab, "width": self.width, "norm": {"eps": self.norm_eps},
               "streams": self.streams, "residual_mult": self.residual_mult,
               "layers": [{"type": l.type, "mixer": l.mixer.to_dict(), "mlp": l.mlp.to_dict() if l.mlp else None}
                          for l in self.layers]}
        if self.logit_softcap is not None:
            out["logit_softcap"] = self.logit_softcap
        return out
