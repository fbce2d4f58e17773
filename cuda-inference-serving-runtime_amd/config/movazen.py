"""MovazenConfig: the keys of a Movazen config.json, typed and checked.

    {"architecture": "Movazen", "vocab": V, "width": H, "embedding": {"scale": s}, "norm": {"eps": e}, "token_side": {"dim": d},
     "layers": [{"type": "attention", "mixer": {...}, "mlp": {...} | null} | {"type": "parallel", ...}, ...]}

An "attention" mixer: heads, kv_heads, dim, vdim, scale, optionally mask {size, keep_first}.  A "parallel" mixer: left (heads,
kv_heads, dim, vdim, scale, optionally q_temp {coef, every}), right (heads, dim, vdim, decay: a number a head), left_scale,
right_scale.  A feed-forward: {"kind": "moe", "expert": {ff, limit}, "router": {experts, top, optionally groups {count,
keep}}, optionally "shared": {ff, limit}}.  Every size and every constant that differs between models of the design is read
from here; the order and kind of the layers is data.
"""
from dataclasses import dataclass
from typing import Optional, Tuple

from .base import ConfigError
from .novosun import _positive_ints, _take
from .zovozen import _count


def _attention_sizes(raw, where):
    heads, kv_heads, dim, vdim, scale = _take(raw, ("heads", "kv_heads", "dim", "vdim", "scale"), where)
    _positive_ints((heads, kv_heads, dim, vdim), where)
    if heads % kv_heads:
        raise ConfigError(f"{where}: {heads} heads are not a multiple of {kv_heads} kv_heads")
    if max(dim, vdim) > 256:
        raise ConfigError(f"{where}: head sizes of at most 256 are supported")
    if not float(scale) > 0:
        raise ConfigError(f"{where}: scale must be positive")
    return heads, kv_heads, dim, vdim, float(scale)


@dataclass(frozen=True)
class KeptWindowAttentionSpec:
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    scale: float
    window: Optional[int] = None
    keep_first: int = 0

    @classmethod
    def from_dict(cls, raw, where):
        sizes = _attention_sizes(raw, where)
        window, keep = None, 0
        if raw.get("mask") is not None:
            (window,) = _take(raw["mask"], ("size",), where + ".mask")
            _positive_ints((window,), where + ".mask")
            keep = _count(raw["mask"].get("keep_first", 0), where + ".mask.keep_first")
        return cls(*sizes, window, keep)

    def to_dict(self):
        out = {"heads": self.heads, "kv_heads": self.kv_heads, "dim": self.dim, "vdim": self.vdim, "scale": self.scale}
        if self.window is not None:
            out["mask"] = {"size": self.window, "keep_first": self.keep_first}
        return out


@dataclass(frozen=True)
class SinkAttentionSpec:
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    scale: float
    q_temp: Optional[Tuple[float, int]] = None      # (coef, every)

    @classmethod
    def from_dict(cls, raw, where):
        sizes = _attention_sizes(raw, where)
        temp = None
        if raw.get("q_temp") is not None:
            coef, every = _take(raw["q_temp"], ("coef", "every"), where + ".q_temp")
            if isinstance(every, float) and every == int(every):
                every = int(every)
            _positive_ints((every,), where + ".q_temp.every")
            temp = (float(coef), every)
        return cls(*sizes, temp)

    def to_dict(self):
        out = {"heads": self.heads, "kv_heads": self.kv_heads, "dim": self.dim, "vdim": self.vdim, "scale": self.scale}
        if self.q_temp is not None:
            out["q_temp"] = {"coef": self.q_temp[0], "every": self.q_temp[1]}
        return out


@dataclass(frozen=True)
class LightningSpec:
    heads: int
    dim: int
    vdim: int
    decay: Tuple[float, ...]

    @classmethod
    def from_dict(cls, raw, where):
        heads, dim, vdim, decay = _take(raw, ("heads", "dim", "vdim", "decay"), where)
        _positive_ints((heads, dim, vdim), where)
        if dim > 256:
            raise ConfigError(f"{where}: key sizes of at most 256 are supported")
        if not isinstance(decay, (list, tuple)) or len(decay) != heads:
            raise ConfigError(f"{where}.decay must be a list of {heads} numbers, one a head")
        return cls(heads, dim, vdim, tuple(float(d) for d in decay))

    def to_dict(self):
        return {"heads": self.heads, "dim": self.dim, "vdim": self.vdim, "decay": list(self.decay)}


@dataclass(frozen=True)
class PairSpec:
    left: SinkAttentionSpec
    right: LightningSpec
    left_scale: float
    right_scale: float

    @classmethod
    def from_dict(cls, raw, where):
        left, right, ls, rs = _take(raw, ("left", "right", "left_scale", "right_scale"), where)
        return cls(SinkAttentionSpec.from_dict(left, where + ".left"), LightningSpec.from_dict(right, where + ".right"), float(ls), float(rs))

    def to_dict(self):
        return {"left": self.left.to_dict(), "right": self.right.to_dict(), "left_scale": self.left_scale, "right_scale": self.right_scale}


@dataclass(frozen=True)
class MixtureSpec:
    ff: int
    limit: float
    experts: int
    top: int
    groups: Optional[Tuple[int, int]] = None          # (count, keep)
    shared: Optional[Tuple[int, float]] = None        # (ff, limit)

    @classmethod
    def from_dict(cls, raw, where):
        if raw.get("kind") != "moe":
            raise ConfigError(f"{where}: feed-forward kind {raw.get('kind')!r} is not moe")
        expert, router = _take(raw, ("expert", "router"), where)
        ff, limit = cls._expert(expert, where + ".expert")
        experts, top = _take(router, ("experts", "top"), where + ".router")
        _positive_ints((experts, top), where + ".router")
        if top > min(experts, 16) or experts > 4096:
            raise ConfigError(f"{where}.router: {top} of {experts} experts: at most all of them, at most 16, of at most 4096")
        groups = None
        if router.get("groups") is not None:
            count, keep = _take(router["groups"], ("count", "keep"), where + ".router.groups")
            _positive_ints((count, keep), where + ".router.groups")
            if experts % count or keep > count or count > 64:
                raise ConfigError(f"{where}.router.groups: {experts} experts in {count} equal groups (at most 64) of which {keep} are kept")
            if keep * (experts // count) < top:
                raise ConfigError(f"{where}.router: {top} experts cannot be chosen from {keep} groups of {experts // count}")
            groups = (count, keep)
        shared = None if raw.get("shared") is None else cls._expert(raw["shared"], where + ".shared")
        return cls(ff, limit, experts, top, groups, shared)

    @staticmethod
    def _expert(raw, where):
        ff, limit = _take(raw, ("ff", "limit"), where)
        _positive_ints((ff,), where)
        if not float(limit) > 0:
            raise ConfigError(f"{where}: limit must be positive")
        return ff, float(limit)

    def to_dict(self):
        router = {"experts": self.experts, "top": self.top}
        if self.groups is not None:
            router["groups"] = {"count": self.groups[0], "keep": self.groups[1]}
        out = {"kind": "moe", "expert": {"ff": self.ff, "limit": self.limit}, "router": router}
        if self.shared is not None:
            out["shared"] = {"ff": self.shared[0], "limit": self.shared[1]}
        return out


@dataclass(frozen=True)
class LayerSpec:
    type: str                                         # "attention" or "parallel"
    mixer: object                                     # KeptWindowAttentionSpec or PairSpec
    mlp: Optional[MixtureSpec] = None

    MIXERS = {"attention": KeptWindowAttentionSpec, "parallel": PairSpec}

    @classmethod
    def from_dict(cls, raw, where):
        kind, mixer = _take(raw, ("type", "mixer"), where)
        if kind not in cls.MIXERS:
            raise ConfigError(f"{where}: layer type {kind!r} is neither attention nor parallel")
        mlp = raw.get("mlp")
        return cls(kind, cls.MIXERS[kind].from_dict(mixer, where + ".mixer"), None if mlp is None else MixtureSpec.from_dict(mlp, where + ".mlp"))

    def to_dict(self):
        return {"type": self.type, "mixer": self.mixer.to_dict(), "mlp": None if self.mlp is None else self.mlp.to_dict()}


@dataclass(frozen=True)
class MovazenConfig:
    vocab: int
    width: int
    layers: Tuple[LayerSpec, ...]
    norm_eps: float
    embedding_scale: float
    side_dim: int
    # config.json names no longest context; this bounds the block tables.
    max_positions: int = 1 << 17

    architecture = "Movazen"

    @classmethod
    def from_dict(cls, raw):
        if raw.get("architecture", raw.get("model_type")) not in ("Movazen", "movazen") and "Movazen" not in (raw.get("architectures") or []):
            raise ConfigError(f"architecture {raw.get('architecture')!r} is not Movazen")
        vocab, width, layers, norm, embedding, side = _take(raw, ("vocab", "width", "layers", "norm", "embedding", "token_side"), "config.json")
        (scale,) = _take(embedding, ("scale",), "config.json embedding")
        (side_dim,) = _take(side, ("dim",), "config.json token_side")
        _positive_ints((vocab, width, side_dim), "config.json")
        if not isinstance(layers, list) or not layers:
            raise ConfigError("config.json: layers must be a list of at least one layer")
        if not isinstance(norm, dict) or "eps" not in norm or not float(norm["eps"]) >= 0:
            raise ConfigError("config.json: norm.eps must be a number >= 0")
        limit = raw.get("max_positions", cls.max_positions)
        _positive_ints((limit,), "config.json max_positions")
        return cls(vocab, width, tuple(LayerSpec.from_dict(layer, f"layers[{i}]") for i, layer in enumerate(layers)), float(norm["eps"]),
                   float(scale), side_dim, limit)

    def to_dict(self):
        out = {"architecture": self.architecture, "vocab": self.vocab, "width": self.width, "embedding": {"scale": self.embedding_scale},
               "norm": {"eps": self.norm_eps}, "token_side": {"dim": self.side_dim}, "layers": [layer.to_dict() for layer in self.layers]}
        if self.max_positions != type(self).max_positions:
            out["max_positions"] = self.max_positions
        return out
