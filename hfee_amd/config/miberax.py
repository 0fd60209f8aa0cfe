"""MiberaxConfig: the Miberax decoder's configuration, read from config.json.

The file lists the layers one by one: each entry has the sizes and constants of its mixer (`type`: "parallel", two
mixers side by side: `left`, attention over chunks of positions, and `right`, the gated delta rule) and its feed-forward
(`mlp`: {"kind": "dense", "ff"}, {"kind": "moe", "expert": {"ff", "limit"}, "router": {"experts", "top", "scale",
"identity", "groups": {"count", "keep"}}, "shared": {"ff", "limit"}}, or null for a layer without one).  Beside the
list it gives the vocabulary, the width, and the norms' eps and groups.  What an entry does not name does not exist: a
left mixer without `rot` is not rotated, one without `mask` sees every earlier position, a router without `groups`
chooses among all, one without `identity` has matrices for every expert, experts without `shared` stand alone.
"""
from __future__ import annotations

from dataclasses import dataclass
from typing import Optional

from .base import ConfigError, KeyReader


def _positive(r: KeyReader, **values):
    for name, v in values.items():
        r.require(v is None or v > 0, f"{name} must be positive")


@dataclass(frozen=True)
class RotationConfig:
    base: float
    dims: int
    factor: Optional[float]         # every frequency is divided by it; None: as they are

    @staticmethod
    def read(data, where: str, head_dim: int) -> Optional["RotationConfig"]:
        if data is None:
            return None
        r = KeyReader(data, where)
        base, dims = r.float("base"), r.int("dims", head_dim)
        sc = r.object("scaling", None)
        factor = None
        if sc is not None:
            rs = KeyReader(sc, where + ".scaling")
            factor = rs.float("factor")
            _positive(rs, factor=factor)
            rs.finish()
        r.require(base is None or base > 0, "the rotation's base must be positive")
        r.require(dims is None or (dims > 0 and dims % 2 == 0), "the rotated dims must be even and positive")
        r.require(dims is None or head_dim is None or dims <= head_dim, f"{dims} rotated dims do not fit a head of {head_dim}")
        r.finish()
        return RotationConfig(base, dims, factor)

    def to_dict(self) -> dict:
        out = {"base": self.base, "dims": self.dims}
        if self.factor is not None:
            out["scaling"] = {"factor": self.factor}
        return out


def _heads(r: KeyReader):
    """(heads, kv_heads, dim, vdim) of a mixer."""
    heads, dim = r.int("heads"), r.int("dim")
    kv_heads, vdim = r.int("kv_heads", heads), r.int("vdim", dim)
    _positive(r, dim=dim, vdim=vdim)
    r.require(heads is None or kv_heads is None or (heads > 0 and kv_heads > 0 and heads % kv_heads == 0),
              f"{heads} heads are not a multiple of {kv_heads} kv_heads")
    return heads, kv_heads, dim, vdim


@dataclass(frozen=True)
class ChunkAttentionConfig:
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    scale: float
    chunk: int                      # 0: every earlier position
    rot: Optional[RotationConfig]

    @staticmethod
    def read(data: dict, where: str) -> "ChunkAttentionConfig":
        r = KeyReader(data, where)
        heads, kv_heads, dim, vdim = _heads(r)
        scale, rot, mask = r.float("scale"), r.object("rot", None), r.object("mask", None)
        r.finish()
        chunk = 0
        if mask is not None:
            rm = KeyReader(mask, where + ".mask")
            chunk = rm.int("size")
            _positive(rm, size=chunk)
            rm.finish()
        return ChunkAttentionConfig(heads, kv_heads, dim, vdim, scale, chunk, RotationConfig.read(rot, where + ".rot", dim))

    def to_dict(self) -> dict:
        out = {"heads": self.heads, "kv_heads": self.kv_heads, "dim": self.dim, "vdim": self.vdim, "scale": self.scale}
        if self.chunk:
            out["mask"] = {"size": self.chunk}
        if self.rot is not None:
            out["rot"] = self.rot.to_dict()
        return out


@dataclass(frozen=True)
class DeltaConfig:
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    conv: int                       # taps of the short convolutions

    @staticmethod
    def read(data: dict, where: str) -> "DeltaConfig":
        r = KeyReader(data, where)
        heads, kv_heads, dim, vdim = _heads(r)
        conv = r.int("conv")
        _positive(r, conv=conv)
        r.finish()
        return DeltaConfig(heads, kv_heads, dim, vdim, conv)

    def to_dict(self) -> dict:
        return {"heads": self.heads, "kv_heads": self.kv_heads, "dim": self.dim, "vdim": self.vdim, "conv": self.conv}


@dataclass(frozen=True)
class PairConfig:
    left: ChunkAttentionConfig
    right: DeltaConfig
    type: str = "parallel"

    @staticmethod
    def read(data: dict, where: str) -> "PairConfig":
        r = KeyReader(data, where)
        left, right = r.object("left"), r.object("right")
        r.finish()
        return PairConfig(ChunkAttentionConfig.read(left, where + ".left"), DeltaConfig.read(right, where + ".right"))

    def to_dict(self) -> dict:
        return {"left": self.left.to_dict(), "right": self.right.to_dict()}


MIXERS = {"parallel": PairConfig}


@dataclass(frozen=True)
class DenseConfig:
    ff: int

    def to_dict(self) -> dict:
        return {"kind": "dense", "ff": self.ff}


@dataclass(frozen=True)
class ExpertsConfig:
    ff: int
    limit: float
    experts: int
    top: int
    scale: float
    identity: int                   # router outputs behind the experts' that hand on their input
    groups: Optional[tuple]         # (count, keep) or None
    shared: Optional[tuple]         # (ff, limit) of the expert that every token uses, or None

    def to_dict(self) -> dict:
        router = {"experts": self.experts, "top": self.top, "scale": self.scale}
        if self.identity:
            router["identity"] = self.identity
        if self.groups is not None:
            router["groups"] = dict(zip(("count", "keep"), self.groups))
        out = {"kind": "moe", "expert": {"ff": self.ff, "limit": self.limit}, "router": router}
        if self.shared is not None:
            out["shared"] = {"ff": self.shared[0], "limit": self.shared[1]}
        return out


def _expert(data: dict, where: str) -> tuple:
    r = KeyReader(data, where)
    ff, limit = r.int("ff"), r.float("limit")
    _positive(r, ff=ff)
    r.require(limit is None or limit >= 0, "limit must not be negative")
    r.finish()
    return ff, limit


def _router(data: dict, where: str) -> tuple:
    """(experts, top, scale, identity, groups)"""
    r = KeyReader(data, where)
    experts, top, scale, identity = r.int("experts"), r.int("top"), r.float("scale", 1.0), r.int("identity", 0)
    groups = r.object("groups", None)
    _positive(r, experts=experts, top=top)
    r.require(identity is None or identity >= 0, "identity must not be negative")
    kept = outputs = (experts or 0) + (identity or 0)
    pair = None
    if groups is not None:
        rg = KeyReader(groups, where + ".groups")
        pair = rg.int("count"), rg.int("keep")
        rg.require(None in pair or 1 <= pair[1] <= pair[0], "of the groups at least one and at most all are kept")
        rg.require(None in pair or pair[0] < 1 or outputs % pair[0] == 0, f"{outputs} experts are not {pair[0]} equal groups")
        rg.finish()
        kept = outputs // pair[0] * pair[1]
    r.require(not experts or not top or top <= kept, f"a token cannot use {top} of {kept} experts")
    r.finish()
    return experts, top, scale, identity, pair


def read_mlp(data: dict, where: str):
    r = KeyReader(data, where)
    kind = r.str("kind")
    if kind == "dense":
        ff = r.int("ff")
        _positive(r, ff=ff)
        r.finish()
        return DenseConfig(ff)
    if kind == "moe":
        expert, router, shared = r.object("expert"), r.object("router"), r.object("shared", None)
        r.finish()
        return ExpertsConfig(*_expert(expert, where + ".expert"), *_router(router, where + ".router"),
                             None if shared is None else _expert(shared, where + ".shared"))
    r.finish()
    raise ConfigError(f"{where}: unknown feed-forward kind {kind!r} (known: dense, moe)")


@dataclass(frozen=True)
class LayerConfig:
    mixer: PairConfig
    mlp: object                     # DenseConfig, ExpertsConfig or None


@dataclass(frozen=True)
class MiberaxConfig:
    architecture: str
    vocab: int
    width: int
    norm_eps: float
    norm_groups: int
    layers: tuple                   # of LayerConfig
    max_positions: int
    eos_token_ids: tuple = ()
    bos_token_id: Optional[int] = None

    # the design names no longest context; the engine's tables are made for what a caller asks for, up to this
    DEFAULT_MAX_POSITIONS = 1 << 20

    @staticmethod
    def from_dict(data: dict, where: str = "config.json") -> "MiberaxConfig":
        r = KeyReader(data, where)
        arch = r.str("architecture", "Miberax")
        vocab, width = r.int("vocab"), r.int("width")
        norm = r.object("norm")
        layers = data.get("layers")
        r.require(isinstance(layers, list) and len(layers) > 0, "key 'layers' must be a non-empty list")
        _positive(r, vocab=vocab, width=width)
        max_positions = r.int("max_positions", MiberaxConfig.DEFAULT_MAX_POSITIONS)
        eos = r.int_or_list("eos_token_id", None)
        bos = r.int("bos_token_id", None)
        r.finish()
        rn = KeyReader(norm, where + ".norm")
        eps, groups = rn.float("eps"), rn.int("groups", 1)
        rn.require(eps is None or eps >= 0, "eps must not be negative")
        rn.require(groups is None or (groups >= 1 and width % groups == 0), f"a width of {width} is not {groups} equal groups")
        rn.finish()
        out = []
        for i, layer in enumerate(layers):
            at = f"{where}.layers[{i}]"
            rl = KeyReader(layer, at)
            kind = rl.str("type")
            mixer, mlp = rl.object("mixer"), rl.object("mlp", None)
            rl.require(kind is None or kind in MIXERS, f"unknown mixer type {kind!r} (known: {', '.join(sorted(MIXERS))})")
            rl.finish()
            out.append(LayerConfig(MIXERS[kind].read(mixer, at + ".mixer"), None if mlp is None else read_mlp(mlp, at + ".mlp")))
        return MiberaxConfig(arch, vocab, width, eps, groups, tuple(out), max_positions, tuple(eos), bos)

    def to_dict(self) -> dict:
        out = {"architecture": self.architecture, "vocab": self.vocab, "width": self.width,
               "norm": {"eps": self.norm_eps, "groups": self.norm_groups},
               "layers": [{"type": l.mixer.type, "mixer": l.mixer.to_dict(), "mlp": None if l.mlp is None else l.mlp.to_dict()}
                          for l in self.layers]}
        if self.max_positions != self.DEFAULT_MAX_POSITIONS:
            out["max_positions"] = self.max_positions
        if self.eos_token_ids:
            out["eos_token_id"] = list(self.eos_token_ids)
        if self.bos_token_id is not None:
            out["bos_token_id"] = self.bos_token_id
        return out
