"""Dofipel as data: a decoder whose layers each name their kind and sizes.

Token embedding; per layer a parallel block, x += mixer(h) + ff(h) with h = norm1(x), the norm a Dynamic Tanh
(tanh(alpha x) * w + b); a layer may be without a feed-forward. The mixer is one of two: an attention through latents
(parts/latent_attention.py: one cached latent and one rotated key part a token for all heads, interleaved rotation, queries
straight from h, an element-wise output gate; a layer may read an earlier layer's latents, its own matrices on them), or a
grouped-query attention over a sliding window without rotation, whose scores are capped by a tanh and then shifted by a
stored table over the distance, with sinks (options of parts/attention.py). The feed-forward is dense (gated, gelu's tanh
form) or routed: the `top` experts by the router's logits with their biases, weighted by the softmax over the chosen logits
alone, plus a shared expert (gated SiLU both). Final Dynamic Tanh, then the embedding table as output matrix; the logits'
factor is folded into that last norm's weight and bias.

Tensor names: 'embed', 'final.norm' (+ '.b', '.alpha'), and per layer i 'l<i>.norm1' (+ '.b', '.alpha'), 'l<i>.mix.*' (latent:
q, dkv, dkv.norm, uk, uv, g, o; attention: q, k, v, rel, sink, o) and 'l<i>.mlp.*' (dense: gate, up, down; routed: router,
router.b, e<j>.{gate,up,down}, shared.{gate,up,down}).
"""
from __future__ import annotations

from ..config.dofipel import DofipelConfig
from ..parts.base import LayerSpec, ModelSpec, PartSpec, ScheduleEntry
from ..registry import register_architecture

# positions are exact in the fp32 angles up to 2^24; the configuration names no bound of its own
_MAX_POSITIONS = 1 << 22
_GATED = {"gate": "gate", "up": "up", "down": "down"}


def _mixer(cfg: DofipelConfig, kind: str, m) -> PartSpec:
    if kind == "latent_attention":
        position = PartSpec("none")
        if m.rot_dim:
            position = PartSpec("rotary", {"head_dim": m.rot_dim + m.kv_rank, "rotary_dim": m.rot_dim, "theta": m.rot_base,
                                           "interleaved": True})
        return PartSpec("latent_attention", {
            "hidden_size": cfg.width, "num_heads": m.heads, "head_dim": m.dim, "rotary_dim": m.rot_dim, "value_dim": m.vdim,
            "kv_rank": m.kv_rank, "scale": m.scale, "eps": cfg.norm_eps, "out_gate": True,
            "kv_projection": m.kv_from is None, "position": position,
            "names": {"q": "q", "dkv": "dkv", "dkv_norm": "dkv.norm", "uk": "uk", "uv": "uv", "gate": "g", "o": "o"}})
    return PartSpec("attention", {
        "hidden_size": cfg.width, "num_heads": m.heads, "num_kv_heads": m.kv_heads, "head_dim": m.dim, "value_dim": m.vdim,
        "scale": m.scale, "window": m.window, "sinks": True, "score_cap": m.softcap,
        "distance_table": {"rows": cfg.bias_rows, "far": m.bias_max},
        "names": {"q": "q", "k": "k", "v": "v", "o": "o", "sinks": "sink", "distance": "rel"}})


def _feed_forward(cfg: DofipelConfig, mlp) -> PartSpec:
    if mlp.kind == "dense":
        return PartSpec("gated_mlp", {"hidden_size": cfg.width, "intermediate_size": mlp.ff, "activation": "gelu_tanh",
                                      "names": _GATED})
    params = {"hidden_size": cfg.width, "intermediate_size": mlp.ff, "experts": mlp.experts, "top": mlp.top,
              "correction": False, "normalize": True, "router_bias": True,
              "names": {"router": "router", "router_bias": "router.b", "expert": "e{e}.", **_GATED}}
    if mlp.shared_ff:
        params["shared"] = {"name": "shared", "gate": None, "feed_forward": PartSpec("gated_mlp", {
            "hidden_size": cfg.width, "intermediate_size": mlp.shared_ff, "activation": "silu", "names": _GATED})}
    return PartSpec("routed_experts", params)


def dofipel_spec(cfg: DofipelConfig) -> ModelSpec:
    names = {"weight": "", "bias": "b", "alpha": "alpha"}
    norm = PartSpec("dynamic_tanh", {"size": cfg.width, "names": names})
    layers = []
    for l, layer in enumerate(cfg.layers):
        params = {"norm": norm, "mixer": _mixer(cfg, layer.type, layer.mixer),
                  "names": {"norm": "norm1", "mixer": "mix", "feed_forward": "mlp"}}
        if layer.mlp is not None:
            params["feed_forward"] = _feed_forward(cfg, layer.mlp)
        layers.append(LayerSpec(f"l{l}.", PartSpec("parallel_residual", params)))
    return ModelSpec(
        hidden_size=cfg.width,
        vocab_size=cfg.vocab,
        embedding=PartSpec("token_embedding", {"vocab_size": cfg.vocab, "hidden_size": cfg.width, "names": {"weight": ""}}),
        embedding_prefix="embed.",
        layers=layers,
        schedule=[ScheduleEntry(l, cache_from=getattr(layer.mixer, "kv_from", None)) for l, layer in enumerate(cfg.layers)],
        final_norm=PartSpec("dynamic_tanh", {"size": cfg.width, "scale": cfg.logit_scale, "names": names}),
        final_norm_prefix="final.norm.",
        head=PartSpec("linear_head", {"vocab_size": cfg.vocab, "hidden_size": cfg.width, "tied_to": "embed"}),
        head_prefix="",
        max_positions=_MAX_POSITIONS,
    )


register_architecture("Dofipel", DofipelConfig, dofipel_spec)
