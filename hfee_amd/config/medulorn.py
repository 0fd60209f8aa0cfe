"""MedulornConfig: the Medulorn decoder's configuration, read from config.json.

The file lists the layers one by one: each entry names its mixer (`type`: "attention" or "parallel", two mixers
side by side) with that mixer's sizes and constants (`mixer`), and its feed-forward (`mlp`: {"kind": "dense", "ff"},
{"kind": "moe", "expert": {"ff", "limit"}, "router": {"experts", "top"}, "shared": {"ff", "limit"}}, or null for a layer
without one).  Beside the list it gives the vocabulary, the width, the norms' eps, the number that the stream is
multiplied by before a sub-layer's result joins it (`postln_alpha`), the embedding's scale and the cap on the
logits.  What an entry does not name does not exist: a mixer without `rot` is not rotated, one without `mask` sees every
earlier position, a mask without `keep_first` keeps none of the first tokens, experts without `shared` stand alone.
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
    scaling: Optional[tuple]       # (factor, low, high, original) or None

    @staticmethod
    def read(data, where: str, head_dim: int) -> Optional["RotationConfig"]:
        if data is None:
            return None
        r = KeyReader(data, where)
        base, dims = r.float("base"), r.int("dims", head_dim)
        sc = r.object("scaling", None)
        scaling = None
        if sc is not None:
            rs = KeyReader(sc, where + ".scaling")
            scaling = (rs.float("factor"), rs.float("low"), rs.float("high"), rs.float("original"))
            rs.require(all(v is None or v > 0 for v in scaling), "factor, low, high and original must be positive")
            rs.require(None in scaling or scaling[1] < scaling[2], "low must lie below high")
            rs.finish()
        r.require(base is None or base > 1, "the rotation's base must exceed 1")
        r.require(dims is None or (dims > 0 and dims % 2 == 0), "the rotated dims must be even and positive")
        r.require(dims is None or head_dim is None or dims <= head_dim, f"{dims} rotated dims do not fit a head of {head_dim}")
        r.finish()
        return RotationConfig(base, dims, scaling)

    def to_dict(self) -> dict:
        out = {"base": self.base, "dims": self.dims}
        if self.scaling is not None:
            out["scaling"] = dict(zip(("factor", "low", "high", "original"), self.scaling))
        return out


def _heads(r: KeyReader):
    """(heads, kv_heads, dim, vdim) of an attention entry."""
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
    type: str = "attention"

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
class KeptWindowConfig:
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    scale: float
    window: int                     # 0: every earlier position
    keep_first: int
    rot: Optional[RotationConfig]

    @staticmethod
    def read(data: dict, where: str) -> "KeptWindowConfig":
        r = KeyReader(data, where)
        heads, kv_heads, dim, vdim = _heads(r)
        scale, rot, mask = r.float("scale"), r.object("rot", None), r.object("mask", None)
        r.finish()
        window = keep = 0
        if mask is not None:
            rm = KeyReader(mask, where + ".mask")
            window, keep = rm.int("size"), rm.int("keep_first", 0)
            _positive(rm, size=window)
            rm.require(keep is None or keep >= 0, "keep_first must not be negative")
            rm.finish()
        return KeptWindowConfig(heads, kv_heads, dim, vdim, scale, window, keep, RotationConfig.read(rot, where + ".rot", dim))

    def to_dict(self) -> dict:
        out = {"heads": self.heads, "kv_heads": self.kv_heads, "dim": self.dim, "vdim": self.vdim, "scale": self.scale}
        if self.window:
            out["mask"] = {"size": self.window}
            if self.keep_first:
                out["mask"]["keep_first"] = self.keep_first
        if self.rot is not None:
            out["rot"] = self.rot.to_dict()
        return out


@dataclass(frozen=True)
class LightningConfig:
    heads: int
    dim: int
    vdim: int
    decay: tuple                    # one number a head

    @staticmethod
    def read(data: dict, where: str) -> "LightningConfig":
        r = KeyReader(data, where)
        heads, dim = r.int("heads"), r.int("dim")
        vdim = r.int("vdim", dim)
        decay = data.get("decay")
        _positive(r, heads=heads, dim=dim, vdim=vdim)
        numbers = isinstance(decay, list) and all(isinstance(d, (int, float)) and not isinstance(d, bool) for d in decay)
        r.require(numbers, "key 'decay' must be a list of numbers, one a head")
        r.require(not numbers or heads is None or len(decay) == heads, f"'decay' must hold one number for each of the {heads} heads")
        r.require(not numbers or all(0.0 <= float(d) <= 1.0 for d in decay), "a decay lies between 0 and 1")
        r.finish()
        return LightningConfig(heads, dim, vdim, tuple(float(d) for d in decay))

    def to_dict(self) -> dict:
        return {"heads": self.heads, "dim": self.dim, "vdim": self.vdim, "decay": list(self.decay)}


@dataclass(frozen=True)
class PairConfig:
    left: KeptWindowConfig
    right: LightningConfig
    left_scale: float
    right_scale: float
    type: str = "parallel"

    @staticmethod
    def read(data: dict, where: str) -> "PairConfig":
        r = KeyReader(data, where)
        left, right = r.object("left"), r.object("right")
        scales = r.float("left_scale", 1.0), r.float("right_scale", 1.0)
        r.finish()
        return PairConfig(KeptWindowConfig.read(left, where + ".left"), LightningConfig.read(right, where + ".right"), *scales)

    def to_dict(self) -> dict:
        return {"left": self.left.to_dict(), "right": self.right.to_dict(), "left_scale": self.left_scale,
                "right_scale": self.right_scale}


MIXERS = {"attention": ChunkAttentionConfig, "parallel": PairConfig}


@dataclass(frozen=True)
class DenseConfig:
    ff: int

    def to_dict(self) -> dict:
        return {"kind": "dense", "ff": self.ff}


@dataclass(frozen=True)
class ClippedExpertsConfig:
    ff: int
    limit: float
    experts: int
    top: int
    shared: Optional[tuple]         # (ff, limit) of the expert that every token uses, or None

    def to_dict(self) -> dict:
        out = {"kind": "moe", "expert": {"ff": self.ff, "limit": self.limit}, "router": {"experts": self.experts, "top": self.top}}
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
        ff, limit = _expert(expert, where + ".expert")
        rr = KeyReader(router, where + ".router")
        experts, top = rr.int("experts"), rr.int("top")
        _positive(rr, experts=experts, top=top)
        rr.require(not experts or not top or top <= experts, f"a token cannot use {top} of {experts} experts")
        rr.finish()
        return ClippedExpertsConfig(ff, limit, experts, top, None if shared is None else _expert(shared, where + ".shared"))
    r.finish()
    raise ConfigError(f"{where}: unknown feed-forward kind {kind!r} (known: dense, moe)")


@dataclass(frozen=True)
class LayerConfig:
    mixer: object                   # one of MIXERS' classes
    mlp: object                     # DenseConfig, ClippedExpertsConfig or None


@dataclass(frozen=True)
class MedulornConfig:
    architecture: str
    vocab: int
    width: int
    norm_eps: float
    alpha: float
    embedding_scale: float
    logit_softcap: float            # 0: none
    layers: tuple                   # of LayerConfig
    max_positions: int
    eos_token_ids: tuple = ()
    bos_token_id: Optional[int] = None

    # the design names no longest context; the engine's tables are made for what a caller asks for, up to this
    DEFAULT_MAX_POSITIONS = 1 << 20

    @staticmethod
    def from_dict(data: dict, where: str = "config.json") -> "MedulornConfig":
        r = KeyReader(data, where)
        arch = r.str("architecture", "Medulorn")
        vocab, width = r.int("vocab"), r.int("width")
        norm, embedding = r.object("norm"), r.object("embedding", {})
        alpha, cap = r.float("postln_alpha", 1.0), r.float("logit_softcap", 0.0)
        layers = data.get("layers")
        r.require(isinstance(layers, list) and len(layers) > 0, "key 'layers' must be a non-empty list")
        _positive(r, vocab=vocab, width=width)
        r.require(cap is None or cap >= 0, "logit_softcap must not be negative")
        max_positions = r.int("max_positions", MedulornConfig.DEFAULT_MAX_POSITIONS)
        eos = r.int_or_list("eos_token_id", None)
        bos = r.int("bos_token_id", None)
        r.finish()
        rn = KeyReader(norm, where + ".norm")
        eps = rn.float("eps")
        rn.require(eps is None or eps >= 0, "eps must not be negative")
        rn.finish()
        rs = KeyReader(embedding, where + ".embedding")
        scale = rs.float("scale", 1.0)
        rs.finish()
        out = []
        for i, layer in enumerate(layers):
            at = f"{where}.layers[{i}]"
            rl = KeyReader(layer, at)
            kind = rl.str("type")
            mixer, mlp = rl.object("mixer"), rl.object("mlp", None)
            rl.require(kind is None or kind in MIXERS, f"unknown mixer type {kind!r} (known: {', '.join(sorted(MIXERS))})")
            rl.finish()
            out.append(LayerConfig(MIXERS[kind].read(mixer, at + ".mixer"), None if mlp is None else read_mlp(mlp, at + ".mlp")))
        return MedulornConfig(arch, vocab, width, eps, alpha, scale, cap, tuple(out), max_positions, tuple(eos), bos)

    def to_dict(self) -> dict:
        out = {"architecture": self.architecture, "vocab": self.vocab, "width": self.width, "norm": {"eps": self.norm_eps},
               "embedding": {"scale": self.embedding_scale}, "postln_alpha": self.alpha,
               "layers": [{"type": l.mixer.type, "mixer": l.mixer.to_dict(), "mlp": None if l.mlp is None else l.mlp.to_dict()}
                          for l in self.layers]}
        if self.logit_softcap:
            out["logit_softcap"] = self.logit_softcap
        if self.max_positions != self.DEFAULT_MAX_POSITIONS:
            out["max_positions"] = self.max_positions
        if self.eos_token_ids:
            out["eos_token_id"] = list(self.eos_token_ids)
        if self.bos_token_id is not None:
            out["bos_token_id"] = self.bos_token_id
        return out
