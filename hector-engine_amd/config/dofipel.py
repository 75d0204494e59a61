"""Typed configuration of the Dofipel decoder, read from its config.json.

The file is nested: 'vocab', 'width', 'logit_scale', 'norm' {eps} and a list 'layers' whose entries give 'type' (the
mixer's kind: 'latent_attention' or 'attention'), 'mixer' (its sizes and constants) and 'mlp' (the feed-forward, or
null for none). Every layer carries its own sizes, so layers of one model may differ in kind, in order and in every size.

  latent_attention: heads, dim, rot_dim, vdim, kv_rank, scale, rot {base, dims}, kv_from (the layer whose latents this
                    one reads, or none)
  attention:        heads, kv_heads, dim, vdim, scale, softcap (or none), bias_max, mask {size} (or none: every
                    earlier position); a distance table has as many rows as are stored (in a random model 'bias_rows')
  mlp:              kind 'dense' {ff}, or kind 'moe' {expert {ff}, router {experts, top}, shared {ff} (or none)}
"""
from __future__ import annotations

import dataclasses

from .base import ConfigError, ModelConfig, architecture_name, read_field, read_object


@dataclasses.dataclass
class DofipelLatent:
    heads: int
    dim: int            # unrotated dims of a head's query and key
    rot_dim: int        # rotated dims
    vdim: int
    kv_rank: int
    scale: float
    rot_base: float = 10000.0
    kv_from: int | None = None

    def to_dict(self) -> dict:
        d = {"dim": self.dim, "heads": self.heads, "kv_rank": self.kv_rank,
             "rot": {"base": self.rot_base, "dims": self.rot_dim}, "rot_dim": self.rot_dim, "scale": self.scale,
             "vdim": self.vdim}
        if self.kv_from is not None:
            d["kv_from"] = self.kv_from
        return d


@dataclasses.dataclass
class DofipelAttention:
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    scale: float
    bias_max: int
    softcap: float = 0.0        # 0: scores are not capped
    window: int = 0             # 0: every earlier position

    def to_dict(self) -> dict:
        d = {"bias_max": self.bias_max, "dim": self.dim, "heads": self.heads, "kv_heads": self.kv_heads, "scale": self.scale,
             "vdim": self.vdim}
        if self.softcap:
            d["softcap"] = self.softcap
        if self.window:
            d["mask"] = {"size": self.window}
        return d


@dataclasses.dataclass
class DofipelMLP:
    kind: str                   # 'dense' or 'moe'
    ff: int = 0                 # dense: the intermediate width; moe: an expert's
    experts: int = 0
    top: int = 0
    shared_ff: int = 0          # 0: no shared expert

    def to_dict(self) -> dict:
        if self.kind == "dense":
            return {"ff": self.ff, "kind": "dense"}
        d = {"expert": {"ff": self.ff}, "kind": "moe", "router": {"experts": self.experts, "top": self.top}}
        if self.shared_ff:
            d["shared"] = {"ff": self.shared_ff}
        return d


@dataclasses.dataclass
class DofipelLayer:
    type: str
    mixer: DofipelLatent | DofipelAttention
    mlp: DofipelMLP | None

    def to_dict(self) -> dict:
        return {"mixer": self.mixer.to_dict(), "mlp": None if self.mlp is None else self.mlp.to_dict(), "type": self.type}


def _positive(where: str, **values) -> None:
    for key, v in values.items():
        if v <= 0:
            raise ConfigError(f"config key '{where}.{key}' must be positive, got {v}")


def _mixer(where: str, kind: str, m: dict):
    if kind == "latent_attention":
        rot = read_object(m, "rot", {})
        out = DofipelLatent(heads=read_field(m, "heads", int), dim=read_field(m, "dim", int),
                            rot_dim=read_field(m, "rot_dim", int, 0), vdim=read_field(m, "vdim", int),
                            kv_rank=read_field(m, "kv_rank", int), scale=read_field(m, "scale", float),
                            rot_base=read_field(rot, "base", float, 10000.0), kv_from=read_field(m, "kv_from", int, None))
        _positive(where, heads=out.heads, dim=out.dim, vdim=out.vdim, kv_rank=out.kv_rank, scale=out.scale)
        dims = read_field(rot, "dims", int, out.rot_dim)
        if out.rot_dim < 0 or out.rot_dim % 2 or dims != out.rot_dim:
            raise ConfigError(f"config key '{where}.rot_dim' must be even and equal to rot.dims, got {out.rot_dim} and {dims}")
        _positive(f"{where}.rot", base=out.rot_base)
        return out
    if kind != "attention":
        raise ConfigError(f"config key '{where[:-6]}.type': unknown mixer '{kind}'")
    mask = read_object(m, "mask", None)
    out = DofipelAttention(heads=read_field(m, "heads", int), kv_heads=read_field(m, "kv_heads", int),
                           dim=read_field(m, "dim", int), vdim=read_field(m, "vdim", int),
                           scale=read_field(m, "scale", float), bias_max=read_field(m, "bias_max", int),
                           softcap=read_field(m, "softcap", float, 0.0),
                           window=0 if mask is None else read_field(mask, "size", int))
    _positive(where, heads=out.heads, kv_heads=out.kv_heads, dim=out.dim, vdim=out.vdim, scale=out.scale, bias_max=out.bias_max)
    if mask is not None:
        _positive(f"{where}.mask", size=out.window)
    if out.softcap < 0:
        raise ConfigError(f"config key '{where}.softcap' must not be negative")
    if out.heads % out.kv_heads:
        raise ConfigError(f"config key '{where}.heads' ({out.heads}) must be a multiple of kv_heads ({out.kv_heads})")
    return out


def _mlp(where: str, m: dict | None):
    if m is None:
        return None
    kind = read_field(m, "kind", str)
    if kind == "dense":
        out = DofipelMLP("dense", ff=read_field(m, "ff", int))
        _positive(where, ff=out.ff)
        return out
    if kind != "moe":
        raise ConfigError(f"config key '{where}.kind': unknown feed-forward '{kind}'")
    router, shared = read_object(m, "router"), read_object(m, "shared", None)
    out = DofipelMLP("moe", ff=read_field(read_object(m, "expert"), "ff", int), experts=read_field(router, "experts", int),
                     top=read_field(router, "top", int), shared_ff=read_field(shared, "ff", int) if shared else 0)
    _positive(where, ff=out.ff, experts=out.experts, top=out.top)
    if out.top > out.experts:
        raise ConfigError(f"config key '{where}.router.top' ({out.top}) exceeds the {out.experts} experts")
    return out


@dataclasses.dataclass
class DofipelConfig(ModelConfig):
    vocab: int = 0
    width: int = 0
    logit_scale: float = 1.0
    norm_eps: float = 1e-6
    layers: list = dataclasses.field(default_factory=list)
    bias_rows: int = 32         # rows of the distance tables of a random model (a stored table has its own)
    torch_dtype: str = "bfloat16"

    @classmethod
    def from_dict(cls, data: dict) -> "DofipelConfig":
        raw = data.get("layers")
        if not isinstance(raw, list) or not raw:
            raise ConfigError("config key 'layers' must be a non-empty list")
        layers = []
        for i, entry in enumerate(raw):
            if not isinstance(entry, dict):
                raise ConfigError(f"config key 'layers[{i}]': expected an object")
            kind = read_field(entry, "type", str)
            layers.append(DofipelLayer(kind, _mixer(f"layers[{i}].mixer", kind, read_object(entry, "mixer")),
                                       _mlp(f"layers[{i}].mlp", read_object(entry, "mlp", None))))
        cfg = cls(architecture=architecture_name(data), vocab=read_field(data, "vocab", int),
                  width=read_field(data, "width", int), logit_scale=read_field(data, "logit_scale", float, 1.0),
                  norm_eps=read_field(read_object(data, "norm"), "eps", float), layers=layers,
                  bias_rows=read_field(data, "bias_rows", int, 32),
                  torch_dtype=read_field(data, "torch_dtype", str, "bfloat16"))
        cfg.validate()
        return cfg

    def validate(self) -> None:
        _positive("config", vocab=self.vocab, width=self.width, bias_rows=self.bias_rows)
        for i, layer in enumerate(self.layers):
            j = getattr(layer.mixer, "kv_from", None)
            if j is None:
                continue
            where = f"config key 'layers[{i}].mixer.kv_from' ({j})"
            if not 0 <= j < i or self.layers[j].type != "latent_attention" or self.layers[j].mixer.kv_from is not None:
                raise ConfigError(f"{where} must name an earlier latent_attention layer with latents of its own")
            a, b = layer.mixer, self.layers[j].mixer
            if (a.kv_rank, a.rot_dim, a.rot_base) != (b.kv_rank, b.rot_dim, b.rot_base):
                raise ConfigError(f"{where}: kv_rank, rot_dim and rot must equal those of that layer")

    def to_dict(self) -> dict:
        return {"architecture": self.architecture, "bias_rows": self.bias_rows, "layers": [l.to_dict() for l in self.layers],
                "logit_scale": self.logit_scale, "norm": {"eps": self.norm_eps}, "torch_dtype": self.torch_dtype,
                "vocab": self.vocab, "width": self.width}
