"""Typed configuration of the Bobevik decoder, read from its config.json.

The file is nested: 'vocab', 'width', 'residual_mult', 'norm' {eps} and a list 'layers' whose entries give 'type' (the
mixer's kind: 'attention', 'retention' or 'parallel'), 'mixer' (its sizes and constants) and 'mlp' (the feed-forward, or
null for none). Every layer carries its own sizes, so layers of one model may differ in kind, in order and in every size.

  attention: heads, kv_heads, dim, vdim, scale, rot {base, dims}, v_mix
  retention: heads, dim, vdim, decay (one number a head), rot {base, dims}
  parallel:  left (heads, kv_heads, dim, vdim, scale, softcap, rot {base, dims, scaling {factor}}), right (heads, dim,
             vdim, decay)
  mlp:       kind 'dense', ff
"""
from __future__ import annotations

import dataclasses

from .base import ConfigError, ModelConfig, architecture_name, read_field, read_object


@dataclasses.dataclass
class BobevikRotation:
    base: float
    dims: int
    factor: float = 1.0     # every frequency is divided by it

    def to_dict(self) -> dict:
        d = {"base": self.base, "dims": self.dims}
        if self.factor != 1.0:
            d["scaling"] = {"factor": self.factor}
        return d


@dataclasses.dataclass
class BobevikAttention:
    heads: int
    kv_heads: int
    dim: int                # of a query and of a key
    vdim: int               # of a value
    scale: float            # on q . k
    rot: BobevikRotation | None = None
    softcap: float = 0.0    # 0: scores are not capped
    v_mix: bool = False     # values mixed with those of the first such layer

    def to_dict(self) -> dict:
        d = {"dim": self.dim, "heads": self.heads, "kv_heads": self.kv_heads, "scale": self.scale, "vdim": self.vdim}
        if self.rot is not None:
            d["rot"] = self.rot.to_dict()
        if self.softcap:
            d["softcap"] = self.softcap
        if self.v_mix:
            d["v_mix"] = True
        return d


@dataclasses.dataclass
class BobevikMemory:
    heads: int
    dim: int
    vdim: int
    decay: list
    rot: BobevikRotation | None = None

    def to_dict(self) -> dict:
        d = {"decay": list(self.decay), "dim": self.dim, "heads": self.heads, "vdim": self.vdim}
        if self.rot is not None:
            d["rot"] = self.rot.to_dict()
        return d


@dataclasses.dataclass
class BobevikParallel:
    left: BobevikAttention
    right: BobevikMemory

    def to_dict(self) -> dict:
        return {"left": self.left.to_dict(), "right": self.right.to_dict()}


@dataclasses.dataclass
class BobevikMLP:
    ff: int
    kind: str = "dense"

    def to_dict(self) -> dict:
        return {"ff": self.ff, "kind": self.kind}


@dataclasses.dataclass
class BobevikLayer:
    type: str
    mixer: BobevikAttention | BobevikMemory | BobevikParallel
    mlp: BobevikMLP | None

    def to_dict(self) -> dict:
        return {"mixer": self.mixer.to_dict(), "mlp": None if self.mlp is None else self.mlp.to_dict(), "type": self.type}


def _positive(where: str, **values) -> None:
    for key, v in values.items():
        if v <= 0:
            raise ConfigError(f"config key '{where}.{key}' must be positive, got {v}")


def _rotation(where: str, m: dict, dim: int) -> BobevikRotation | None:
    raw = read_object(m, "rot", None)
    if raw is None:
        return None
    scaling = read_object(raw, "scaling", None) or {}
    rot = BobevikRotation(base=read_field(raw, "base", float), dims=read_field(raw, "dims", int, dim),
                          factor=read_field(scaling, "factor", float, 1.0))
    _positive(f"{where}.rot", base=rot.base)
    _positive(f"{where}.rot.scaling", factor=rot.factor)
    if rot.dims < 0 or rot.dims % 2 or rot.dims > dim:
        raise ConfigError(f"config key '{where}.rot.dims' ({rot.dims}) must be even and at most dim ({dim})")
    return rot if rot.dims else None        # no dimension is rotated


def _attention(where: str, m: dict) -> BobevikAttention:
    heads, dim = read_field(m, "heads", int), read_field(m, "dim", int)
    a = BobevikAttention(heads=heads, kv_heads=read_field(m, "kv_heads", int, heads), dim=dim,
                         vdim=read_field(m, "vdim", int, dim), scale=read_field(m, "scale", float),
                         rot=_rotation(where, m, dim), softcap=read_field(m, "softcap", float, 0.0),
                         v_mix=read_field(m, "v_mix", bool, False))
    _positive(where, heads=a.heads, kv_heads=a.kv_heads, dim=a.dim, vdim=a.vdim, scale=a.scale)
    if a.softcap < 0:
        raise ConfigError(f"config key '{where}.softcap' must not be negative")
    if a.heads % a.kv_heads:
        raise ConfigError(f"config key '{where}.heads' ({a.heads}) must be a multiple of kv_heads ({a.kv_heads})")
    return a


def _memory(where: str, m: dict) -> BobevikMemory:
    dim = read_field(m, "dim", int)
    raw = m.get("decay")
    if not isinstance(raw, list) or not all(isinstance(d, (int, float)) and not isinstance(d, bool) for d in raw):
        raise ConfigError(f"config key '{where}.decay' must be a list of numbers")
    out = BobevikMemory(heads=read_field(m, "heads", int), dim=dim, vdim=read_field(m, "vdim", int, dim),
                        decay=[float(d) for d in raw], rot=_rotation(where, m, dim))
    _positive(where, heads=out.heads, dim=out.dim, vdim=out.vdim)
    if out.dim > 512:
        raise ConfigError(f"config key '{where}.dim' ({out.dim}) above 512")
    if len(out.decay) != out.heads or not all(0.0 <= d <= 1.0 for d in out.decay):
        raise ConfigError(f"config key '{where}.decay' must give a number in [0, 1] for each of the {out.heads} heads")
    return out


def _mixer(where: str, kind: str, m: dict):
    if kind == "attention":
        return _attention(where, m)
    if kind == "retention":
        return _memory(where, m)
    if kind == "parallel":
        return BobevikParallel(left=_attention(where + ".left", read_object(m, "left")),
                               right=_memory(where + ".right", read_object(m, "right")))
    raise ConfigError(f"config key '{where[:-6]}.type': unknown mixer '{kind}'")


def _mlp(where: str, m: dict | None) -> BobevikMLP | None:
    if m is None:
        return None
    out = BobevikMLP(ff=read_field(m, "ff", int), kind=read_field(m, "kind", str, "dense"))
    if out.kind != "dense":
        raise ConfigError(f"config key '{where}.kind': unknown feed-forward '{out.kind}'")
    _positive(where, ff=out.ff)
    return out


@dataclasses.dataclass
class BobevikConfig(ModelConfig):
    vocab: int = 0
    width: int = 0
    residual_mult: float = 1.0
    norm_eps: float = 1e-6
    layers: list = dataclasses.field(default_factory=list)
    torch_dtype: str = "bfloat16"

    @classmethod
    def from_dict(cls, data: dict) -> "BobevikConfig":
        raw = data.get("layers")
        if not isinstance(raw, list) or not raw:
            raise ConfigError("config key 'layers' must be a non-empty list")
        layers = []
        for i, entry in enumerate(raw):
            if not isinstance(entry, dict):
                raise ConfigError(f"config key 'layers[{i}]': expected an object")
            kind = read_field(entry, "type", str)
            layers.append(BobevikLayer(kind, _mixer(f"layers[{i}].mixer", kind, read_object(entry, "mixer")),
                                       _mlp(f"layers[{i}].mlp", read_object(entry, "mlp", None))))
        cfg = cls(architecture=architecture_name(data), vocab=read_field(data, "vocab", int),
                  width=read_field(data, "width", int), residual_mult=read_field(data, "residual_mult", float, 1.0),
                  norm_eps=read_field(read_object(data, "norm"), "eps", float), layers=layers,
                  torch_dtype=read_field(data, "torch_dtype", str, "bfloat16"))
        cfg.validate()
        return cfg

    def mixing_layers(self) -> list[int]:
        """The attention layers whose values are mixed; the first of them gives the values the others mix in."""
        return [i for i, l in enumerate(self.layers) if l.type == "attention" and l.mixer.v_mix]

    def validate(self) -> None:
        _positive("config", vocab=self.vocab, width=self.width, norm_eps=self.norm_eps)
        mixing = self.mixing_layers()
        for i in mixing[1:]:
            a, b = self.layers[i].mixer, self.layers[mixing[0]].mixer
            if (a.kv_heads, a.vdim) != (b.kv_heads, b.vdim):
                raise ConfigError(f"config key 'layers[{i}].mixer.v_mix': kv_heads and vdim ({a.kv_heads}, {a.vdim}) must equal "
                                  f"those of layer {mixing[0]} ({b.kv_heads}, {b.vdim})")

    def to_dict(self) -> dict:
        return {"architecture": self.architecture, "layers": [l.to_dict() for l in self.layers],
                "norm": {"eps": self.norm_eps}, "residual_mult": self.residual_mult, "torch_dtype": self.torch_dtype,
                "vocab": self.vocab, "width": self.width}
