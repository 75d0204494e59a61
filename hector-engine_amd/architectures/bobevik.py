"""Bobevik as data: a decoder whose layers each name their kind and sizes.

Token embedding, normed on its way into the stream; per layer a block with norms on both sides of each branch,
x += m norm1b(mixer(norm1(x))) and, where the layer has one, x += m norm2b(ff(norm2(x))), all RMS norms whose stored
weight is the gain's difference from one, m a constant that is folded into the gains of the norms behind the branches. The
mixer is one of three: a grouped-query attention with a half-split rotation, q and k divided by their root mean square
behind it, a gate a head, and, where the layer says so, values mixed with those of the first layer that says so (options
of parts/attention.py); a retention, that is a memory that fades by a constant a head, on rotated queries and keys
(parts/decay_memory.py); or two mixers on the same input, each result RMS-normed with a gain of its own and the two
averaged (parts/parallel.py): an attention with biases, a rotation whose frequencies are divided by a factor, scores capped
by a tanh and a gate a head, and a fading memory on SiLU of its projections without a rotation, normed over all heads at
once. The feed-forward is dense and gated by relu. Final norm of the same kind, then an output matrix of its own.

Tensor names: 'embed', 'embed.norm', 'head', 'final.norm', and per layer i 'l<i>.norm1', 'l<i>.norm1b', 'l<i>.norm2',
'l<i>.norm2b', 'l<i>.mix.*' (attention: q, k, v, g, o, vmix; retention: q, k, v, g, o; parallel: left.{q,k,v} + '.b',
left.{g,o,out}, right.{q,k,v,g,o,norm,out}) and 'l<i>.mlp.{gate,up,down}'.
"""
from __future__ import annotations

from ..config.bobevik import BobevikAttention, BobevikConfig, BobevikMemory, BobevikRotation
from ..parts.base import LayerSpec, ModelSpec, PartSpec, ScheduleEntry
from ..registry import register_architecture

# positions are exact in the fp32 angles up to 2^24; the configuration names no bound of its own
_MAX_POSITIONS = 1 << 22
_MEMORY_NAMES = {"q": "q", "k": "k", "v": "v", "g": "g", "o": "o", "norm": "norm"}


def _position(rot: BobevikRotation | None, dim: int) -> PartSpec:
    if rot is None:
        return PartSpec("none")
    params = {"head_dim": dim, "rotary_dim": rot.dims, "theta": rot.base}
    if rot.factor != 1.0:
        params["scaling"] = {"kind": "linear", "factor": rot.factor}
    return PartSpec("rotary", params)


def _attention(cfg: BobevikConfig, a: BobevikAttention, role: str, side_by_side: bool) -> PartSpec:
    params = {"hidden_size": cfg.width, "num_heads": a.heads, "num_kv_heads": a.kv_heads, "head_dim": a.dim,
              "value_dim": a.vdim, "scale": a.scale, "score_cap": a.softcap, "head_gate": True, "qkv_bias": side_by_side,
              "position": _position(a.rot, a.dim),
              "names": {"q": "q", "k": "k", "v": "v", "o": "o", "gate": "g", "q_bias": "q.b", "k_bias": "k.b",
                        "v_bias": "v.b", "v_mix": "vmix"}}
    if not side_by_side:
        params.update({"qk_norm": "unit", "qk_norm_eps": cfg.norm_eps})
    if role:
        params["v_mix"] = {"role": role, "key": "first_values"}
    return PartSpec("attention", params)


def _memory(cfg: BobevikConfig, m: BobevikMemory, side_by_side: bool) -> PartSpec:
    params = {"hidden_size": cfg.width, "num_heads": m.heads, "head_dim": m.dim, "value_dim": m.vdim, "decay": m.decay,
              "eps": cfg.norm_eps, "position": _position(m.rot, m.dim), "names": _MEMORY_NAMES}
    if side_by_side:
        params.update({"activation": "silu", "out_norm": "row", "gate": "sigmoid"})
    else:
        params.update({"k_scale": m.dim ** -0.5, "out_norm": "heads", "gate": "silu"})
    return PartSpec("decay_memory", params)


def bobevik_spec(cfg: BobevikConfig) -> ModelSpec:
    def norm(scale: float = 1.0) -> PartSpec:
        return PartSpec("rmsnorm", {"size": cfg.width, "eps": cfg.norm_eps, "offset": 1.0, "scale": scale,
                                    "names": {"weight": ""}})

    branch_norm = PartSpec("rmsnorm", {"size": cfg.width, "eps": cfg.norm_eps, "names": {"weight": ""}})
    mixing = cfg.mixing_layers()
    layers = []
    for l, layer in enumerate(cfg.layers):
        m = layer.mixer
        if layer.type == "attention":
            role = "" if l not in mixing else "first" if l == mixing[0] else "mix"
            mixer = _attention(cfg, m, role, False)
        elif layer.type == "retention":
            mixer = _memory(cfg, m, False)
        else:
            mixer = PartSpec("parallel", {"branches": [
                {"name": "left", "scale": 0.5, "mixer": _attention(cfg, m.left, "", True), "norm": branch_norm,
                 "norm_name": "left.out"},
                {"name": "right", "scale": 0.5, "mixer": _memory(cfg, m.right, True), "norm": branch_norm,
                 "norm_name": "right.out"}]})
        params = {"mixer_norm": norm(), "mixer_post_norm": norm(cfg.residual_mult), "mixer": mixer,
                  "names": {"mixer_norm": "norm1", "mixer_post_norm": "norm1b", "mixer": "mix",
                            "feed_forward_norm": "norm2", "feed_forward_post_norm": "norm2b", "feed_forward": "mlp"}}
        if layer.mlp is not None:
            params["feed_forward_norm"], params["feed_forward_post_norm"] = norm(), norm(cfg.residual_mult)
            params["feed_forward"] = PartSpec("gated_mlp", {
                "hidden_size": cfg.width, "intermediate_size": layer.mlp.ff, "activation": "relu",
                "names": {"gate": "gate", "up": "up", "down": "down"}})
        layers.append(LayerSpec(f"l{l}.", PartSpec("sandwich_norm", params)))
    return ModelSpec(
        hidden_size=cfg.width,
        vocab_size=cfg.vocab,
        embedding=PartSpec("token_embedding", {"vocab_size": cfg.vocab, "hidden_size": cfg.width, "norm": norm(),
                                               "norm_prefix": "embed.norm.", "names": {"weight": ""}}),
        embedding_prefix="embed.",
        layers=layers,
        schedule=[ScheduleEntry(l) for l in range(len(cfg.layers))],
        final_norm=norm(),
        final_norm_prefix="final.norm.",
        head=PartSpec("linear_head", {"vocab_size": cfg.vocab, "hidden_size": cfg.width, "names": {"weight": ""}}),
        head_prefix="head.",
        max_positions=_MAX_POSITIONS,
    )


register_architecture("Bobevik", BobevikConfig, bobevik_spec)
