"""GuduzenConfig: the keys of a Guduzen config.json, typed and checked.

    {"architecture": "Guduzen", "vocab": V, "width": H, "streams": s, "logit_softcap": c, "norm": {"eps": e},
     "layers": [{"type": "attention" | "latent_attention" | "channel_delta", "mixer": {...},
                 "mlp": {"kind": "dense", "ff": F} | null}, ...]}

An "attention" mixer gives heads, kv_heads, dim, vdim, scale, mask {size} (a sliding window; without it every earlier key)
and optionally kv_from: j, an earlier attention layer whose keys and values it reads; a "latent_attention" mixer heads,
dim, vdim, kv_rank, scale and q_rank (left out: the file decides); a "channel_delta" mixer heads, kv_heads, dim, vdim
and conv (taps).  Every size and every constant that differs between models of the design is read from here; the order
and kind of the layers is data.
"""
from dataclasses import dataclass
from typing import Optional, Tuple

from .base import ConfigError
from .novosun import _positive_ints, _take

LAYER_TYPES = ("attention", "latent_attention", "channel_delta")
MAX_STREAMS = 8            # streams of a residual that the row kernels hold in registers


@dataclass(frozen=True)
class WindowAttentionSpec:
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    scale: float
    window: Optional[int] = None
    kv_from: Optional[int] = None

    @classmethod
    def from_dict(cls, raw, where):
        heads, kv_heads, dim, vdim, scale = _take(raw, ("heads", "kv_heads", "dim", "vdim", "scale"), where)
        _positive_ints((heads, kv_heads, dim, vdim), where)
        if heads % kv_heads:
            raise ConfigError(f"{where}: {heads} heads are not a multiple of {kv_heads} kv_heads")
        if max(dim, vdim) > 256:
            raise ConfigError(f"{where}: head sizes of at most 256 are supported")
        if not float(scale) > 0:
            raise ConfigError(f"{where}: scale must be positive")
        window = None
        if raw.get("mask") is not None:
            (window,) = _take(raw["mask"], ("size",), where + ".mask")
            _positive_ints((window,), where + ".mask.size")
        source = raw.get("kv_from")
        if source is not None and (not isinstance(source, int) or isinstance(source, bool) or source < 0):
            raise ConfigError(f"{where}: kv_from must name a layer")
        return cls(heads, kv_heads, dim, vdim, float(scale), window, source)

    def to_dict(self):
        out = {"heads": self.heads, "kv_heads": self.kv_heads, "dim": self.dim, "vdim": self.vdim, "scale": self.scale}
        if self.window is not None:
            out["mask"] = {"size": self.window}
        if self.kv_from is not None:
            out["kv_from"] = self.kv_from
        return out


@dataclass(frozen=True)
class LatentAttentionSpec:
    heads: int
    dim: int
    vdim: int
    kv_rank: int
    scale: float
    q_rank: Optional[int] = None      # None: the file decides

    @classmethod
    def from_dict(cls, raw, where):
        heads, dim, vdim, kv_rank, scale = _take(raw, ("heads", "dim", "vdim", "kv_rank", "scale"), where)
        _positive_ints((heads, dim, vdim, kv_rank), where)
        if kv_rank > 640:
            raise ConfigError(f"{where}: kv_rank of at most 640 is supported")
        if not float(scale) > 0:
            raise ConfigError(f"{where}: scale must be positive")
        q_rank = raw.get("q_rank")
        if q_rank is not None:
            _positive_ints((q_rank,), where + ".q_rank")
        return cls(heads, dim, vdim, kv_rank, float(scale), q_rank)

    def to_dict(self):
        out = {"heads": self.heads, "dim": self.dim, "vdim": self.vdim, "kv_rank": self.kv_rank, "scale": self.scale}
        if self.q_rank is not None:
            out["q_rank"] = self.q_rank
        return out


@dataclass(frozen=True)
class ChannelDeltaSpec:
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    conv: int

    @classmethod
    def from_dict(cls, raw, where):
        values = _take(raw, ("heads", "kv_heads", "dim", "vdim", "conv"), where)
        _positive_ints(values, where)
        heads, kv_heads, dim, _, conv = values
        if heads % kv_heads:
            raise ConfigError(f"{where}: {heads} heads are not a multiple of {kv_heads} kv_heads")
        if conv > 16 or dim > 256:
            raise ConfigError(f"{where}: convolutions of at most 16 taps and heads of at most 256 are supported")
        return cls(*values)

    def to_dict(self):
        return {"heads": self.heads, "kv_heads": self.kv_heads, "dim": self.dim, "vdim": self.vdim, "conv": self.conv}


_MIXERS = {"attention": WindowAttentionSpec, "latent_attention": LatentAttentionSpec, "channel_delta": ChannelDeltaSpec}


@dataclass(frozen=True)
class GuduzenLayer:
    type: str
    mixer: object                     # the spec of its type
    ff: Optional[int] = None          # the feed-forward's inner size; None: a layer without one

    @classmethod
    def from_dict(cls, raw, where):
        kind, mixer = _take(raw, ("type", "mixer"), where)
        if kind not in _MIXERS:
            raise ConfigError(f"{where}: layer type {kind!r} is none of {LAYER_TYPES}")
        ff, mlp = None, raw.get("mlp")
        if mlp is not None:
            if mlp.get("kind", "dense") != "dense":
                raise ConfigError(f"{where}.mlp: feed-forward kind {mlp.get('kind')!r} is not dense")
            (ff,) = _take(mlp, ("ff",), where + ".mlp")
            _positive_ints((ff,), where + ".mlp")
        return cls(kind, _MIXERS[kind].from_dict(mixer, where + ".mixer"), ff)

    @property
    def attention(self):
        return self.mixer if self.type == "attention" else None

    def to_dict(self):
        return {"type": self.type, "mixer": self.mixer.to_dict(), "mlp": None if self.ff is None else {"kind": "dense", "ff": self.ff}}


@dataclass(frozen=True)
class GuduzenConfig:
    vocab: int
    width: int
    layers: Tuple[GuduzenLayer, ...]
    norm_eps: float
    streams: int
    logit_softcap: Optional[float] = None
    # config.json names no longest context; this bounds the block tables.
    max_positions: int = 1 << 17

    architecture = "Guduzen"

    @classmethod
    def from_dict(cls, raw):
        if raw.get("architecture", raw.get("model_type")) not in ("Guduzen", "guduzen") and "Guduzen" not in (raw.get("architectures") or []):
            raise ConfigError(f"architecture {raw.get('architecture')!r} is not Guduzen")
        vocab, width, streams, layers, norm = _take(raw, ("vocab", "width", "streams", "layers", "norm"), "config.json")
        _positive_ints((vocab, width, streams), "config.json")
        if streams > MAX_STREAMS:
            raise ConfigError(f"config.json: at most {MAX_STREAMS} streams are supported")
        if not isinstance(layers, list) or not layers:
            raise ConfigError("config.json: layers must be a list of at least one layer")
        if not isinstance(norm, dict) or "eps" not in norm or not float(norm["eps"]) >= 0:
            raise ConfigError("config.json: norm.eps must be a number >= 0")
        cap = raw.get("logit_softcap")
        if cap is not None and not float(cap) > 0:
            raise ConfigError("config.json: logit_softcap must be positive")
        limit = raw.get("max_positions", cls.max_positions)
        _positive_ints((limit,), "config.json max_positions")
        specs = tuple(GuduzenLayer.from_dict(layer, f"layers[{i}]") for i, layer in enumerate(layers))
        for i, spec in enumerate(specs):
            a = spec.attention
            if a is None or a.kv_from is None:
                continue
            source = specs[a.kv_from].attention if a.kv_from < i else None
            if source is None or source.kv_from is not None:
                raise ConfigError(f"layers[{i}].mixer.kv_from: layer {a.kv_from} is no earlier attention layer with keys of its own")
            if (source.kv_heads, source.dim, source.vdim) != (a.kv_heads, a.dim, a.vdim):
                raise ConfigError(f"layers[{i}].mixer: key heads and head sizes must equal layer {a.kv_from}'s")
        return cls(vocab, width, specs, float(norm["eps"]), streams, None if cap is None else float(cap), limit)

    def to_dict(self):
        out = {"architecture": self.architecture, "vocab": self.vocab, "width": self.width, "streams": self.streams,
               "norm": {"eps": self.norm_eps}, "layers": [layer.to_dict() for layer in self.layers]}
        if self.logit_softcap is not None:
            out["logit_softcap"] = self.logit_softcap
        if self.max_positions != type(self).max_positions:
            out["max_positions"] = self.max_positions
        return out
