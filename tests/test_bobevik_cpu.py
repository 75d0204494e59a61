"""Bobevik without a GPU: its configuration (every size from the file, defaults for what a layer leaves out, errors that
name the key), the tensors and the state its parts ask for, what the parts fold into their numbers (gains stored around
zero, a branch's factor, scaled frequencies, relu as a gate's constants), and the plain implementation against itself (a
prompt at once equals the same tokens one by one and in portions, through what it carries)."""
import copy
import math

import pytest
import torch

import hector_engine_amd  # noqa: F401
from hector_engine_amd.config.base import ConfigError
from hector_engine_amd.parts.base import BuildEnv, PartSpec, build_part
from hector_engine_amd.registry import build_model, config_from_dict, model_spec
from tests.plain import bobevik_plain as P

CPU = BuildEnv(torch.device("cpu"), torch.float32)


def rot(base, dims, factor=None):
    d = {"base": base, "dims": dims}
    if factor is not None:
        d["scaling"] = {"factor": factor}
    return d


def attn(heads, kv, dim, vdim, scale, rotation=None, softcap=None, v_mix=False):
    d = {"dim": dim, "heads": heads, "kv_heads": kv, "scale": scale, "vdim": vdim}
    if rotation is not None:
        d["rot"] = rotation
    if softcap is not None:
        d["softcap"] = softcap
    if v_mix:
        d["v_mix"] = True
    return d


def memory(decay, dim, vdim, rotation=None):
    d = {"decay": list(decay), "dim": dim, "heads": len(decay), "vdim": vdim}
    if rotation is not None:
        d["rot"] = rotation
    return d


def pair(left, right):
    return {"left": left, "right": right}


def layer(kind, mixer, ff=None):
    return {"mixer": mixer, "mlp": None if ff is None else {"ff": ff, "kind": "dense"}, "type": kind}


def model(layers, vocab, width, mult=1.0, eps=1e-6):
    return {"architecture": "Bobevik", "layers": layers, "norm": {"eps": eps}, "residual_mult": mult, "torch_dtype": "bfloat16",
            "vocab": vocab, "width": width}


SMALL = model([layer("parallel", pair(attn(4, 2, 8, 12, 0.3, rot(500.0, 4, 3.0), 9.0), memory((0.9, 0.5, 0.99), 6, 10)), 20),
               layer("attention", attn(3, 1, 10, 6, 0.25, rot(1000.0, 10), v_mix=True)),
               layer("retention", memory((0.97, 0.8), 12, 5, rot(10000.0, 8)), 14),
               layer("attention", attn(4, 4, 6, 8, 0.4), 12),
               layer("attention", attn(2, 1, 16, 6, 0.2, rot(100.0, 6), v_mix=True), 8)],
              vocab=53, width=24, mult=0.6, eps=1e-5)


def test_configuration_reads_back_and_every_size_comes_from_the_file():
    cfg = config_from_dict(copy.deepcopy(SMALL))
    assert cfg.to_dict() == SMALL
    assert [l.type for l in cfg.layers] == ["parallel", "attention", "retention", "attention", "attention"]
    p, a, r = cfg.layers[0].mixer, cfg.layers[1].mixer, cfg.layers[2].mixer
    assert (p.left.heads, p.left.kv_heads, p.left.dim, p.left.vdim, p.left.scale, p.left.softcap) == (4, 2, 8, 12, 0.3, 9.0)
    assert (p.left.rot.base, p.left.rot.dims, p.left.rot.factor) == (500.0, 4, 3.0)
    assert (p.right.heads, p.right.dim, p.right.vdim, p.right.decay, p.right.rot) == (3, 6, 10, [0.9, 0.5, 0.99], None)
    assert (a.heads, a.kv_heads, a.dim, a.vdim, a.rot.dims, a.rot.factor, a.softcap, a.v_mix) == (3, 1, 10, 6, 10, 1.0, 0.0, True)
    assert (r.heads, r.dim, r.vdim, r.decay, r.rot.dims, r.rot.base) == (2, 12, 5, [0.97, 0.8], 8, 10000.0)
    assert cfg.layers[0].mlp.ff == 20 and cfg.layers[1].mlp is None
    assert (cfg.vocab, cfg.width, cfg.residual_mult, cfg.norm_eps) == (53, 24, 0.6, 1e-5)
    assert cfg.mixing_layers() == [1, 4]


def test_defaults_for_what_a_layer_leaves_out():
    d = copy.deepcopy(SMALL)
    del d["layers"][3]["mixer"]["kv_heads"], d["layers"][3]["mixer"]["vdim"], d["residual_mult"]
    del d["layers"][0]["mixer"]["left"]["softcap"], d["layers"][0]["mixer"]["left"]["rot"]["scaling"]
    d["layers"][2]["mixer"]["rot"]["dims"] = 0                 # no dimension rotated: the same as no 'rot'
    d["layers"][1]["mixer"]["v_mix"] = False
    cfg = config_from_dict(d)
    a = cfg.layers[3].mixer
    assert (a.kv_heads, a.vdim, a.rot, cfg.residual_mult) == (4, 6, None, 1.0)
    assert cfg.layers[0].mixer.left.softcap == 0.0 and cfg.layers[0].mixer.left.rot.factor == 1.0
    assert cfg.layers[2].mixer.rot is None and cfg.mixing_layers() == [4]


@pytest.mark.parametrize("path,value,word", [
    (("layers", 0, "type"), "conv", r"layers\[0\].type"),
    (("layers", 3, "mixer", "kv_heads"), 3, "kv_heads"),
    (("layers", 1, "mixer", "rot", "dims"), 7, "rot.dims"),
    (("layers", 1, "mixer", "rot", "dims"), 12, "rot.dims"),
    (("layers", 1, "mixer", "scale"), 0.0, "scale"),
    (("layers", 0, "mixer", "left", "softcap"), -1.0, "left.softcap"),
    (("layers", 0, "mixer", "left", "rot", "scaling", "factor"), 0.0, "factor"),
    (("layers", 0, "mixer", "right", "decay"), [0.5, 0.5], "right.decay"),
    (("layers", 0, "mixer", "right", "decay"), 0.5, "right.decay"),
    (("layers", 2, "mixer", "decay"), [0.5, 1.5], "decay"),
    (("layers", 2, "mixer", "dim"), 600, "dim"),
    (("layers", 4, "mixer", "vdim"), 8, r"layers\[4\].mixer.v_mix"),
    (("layers", 0, "mlp", "kind"), "moe", "unknown feed-forward"),
    (("layers", 0, "mlp", "ff"), 0, "ff"),
    (("layers",), [], "layers"),
    (("width",), 0, "width"),
])
def test_errors_name_the_key(path, value, word):
    d = copy.deepcopy(SMALL)
    at = d
    for k in path[:-1]:
        at = at[k]
    at[path[-1]] = value
    with pytest.raises(ConfigError, match=word):
        config_from_dict(d)


def test_tensors_the_parts_ask_for_and_the_state_a_sequence_carries():
    m = build_model(config_from_dict(copy.deepcopy(SMALL)), CPU)
    specs = {k: tuple(v.shape) for k, v in m.tensor_specs().items()}
    assert specs.pop("embed") == specs.pop("head") == (53, 24) and specs.pop("embed.norm") == specs.pop("final.norm") == (24,)
    for l in range(5):
        assert specs.pop(f"l{l}.norm1") == specs.pop(f"l{l}.norm1b") == (24,)
    for l, ff in ((0, 20), (2, 14), (3, 12), (4, 8)):
        assert specs.pop(f"l{l}.norm2") == specs.pop(f"l{l}.norm2b") == (24,)
        assert specs.pop(f"l{l}.mlp.gate") == specs.pop(f"l{l}.mlp.up") == (ff, 24) and specs.pop(f"l{l}.mlp.down") == (24, ff)
    for l, (H, G, d, e, mixes) in {1: (3, 1, 10, 6, True), 3: (4, 4, 6, 8, False), 4: (2, 1, 16, 6, True)}.items():
        assert specs.pop(f"l{l}.mix.q") == (H * d, 24) and specs.pop(f"l{l}.mix.k") == (G * d, 24)
        assert specs.pop(f"l{l}.mix.v") == (G * e, 24) and specs.pop(f"l{l}.mix.g") == (H, 24)
        assert specs.pop(f"l{l}.mix.o") == (24, H * e)
        if mixes:
            assert specs.pop(f"l{l}.mix.vmix") == ()
    assert specs.pop("l2.mix.q") == specs.pop("l2.mix.k") == (24, 24)
    assert specs.pop("l2.mix.v") == specs.pop("l2.mix.g") == (10, 24) and specs.pop("l2.mix.o") == (24, 10)
    left, right = "l0.mix.left.", "l0.mix.right."
    assert specs.pop(left + "q") == (32, 24) and specs.pop(left + "q.b") == (32,)
    assert specs.pop(left + "k") == (16, 24) and specs.pop(left + "k.b") == (16,)
    assert specs.pop(left + "v") == (24, 24) and specs.pop(left + "v.b") == (24,)
    assert specs.pop(left + "g") == (4, 24) and specs.pop(left + "o") == (24, 48)
    assert specs.pop(right + "q") == specs.pop(right + "k") == (18, 24)
    assert specs.pop(right + "v") == specs.pop(right + "g") == (30, 24) and specs.pop(right + "o") == (24, 30)
    assert specs.pop(right + "norm") == (30,) and specs.pop(left + "out") == specs.pop(right + "out") == (24,)
    assert specs == {}                                       # and nothing else
    plans = m.run_plans()
    assert [p.kv is not None for p in plans] == [True, True, False, True, True]
    assert [p.state_bytes for p in plans][1::2] == [0, 0] and plans[4].state_bytes == 0
    assert plans[0].state_bytes >= 4 * 3 * 6 * 10 and plans[2].state_bytes >= 4 * 2 * 12 * 5


def test_roles_of_the_layers_that_mix_values():
    def roles(*flags):
        d = model([layer("attention", attn(2, 1, 4, 4, 0.5, v_mix=f)) if f is not None else
                   layer("retention", memory((0.5,), 4, 4)) for f in flags], 20, 8)
        found = []
        for spec in model_spec(config_from_dict(d)).layers:
            found.append((spec.block.params["mixer"].params.get("v_mix") or {}).get("role"))
        return found
    assert roles(False, True, None, False, True, True) == [None, "first", None, None, "mix", "mix"]
    assert roles(True) == ["first"] and roles(False, None) == [None, None]


def test_gains_stored_around_zero_and_a_branch_factor_are_folded():
    w = torch.tensor([0.25, -0.5, 0.0], dtype=torch.bfloat16)
    n = build_part("norm", PartSpec("rmsnorm", {"size": 3, "eps": 1e-6, "offset": 1.0, "scale": 0.3, "names": {"weight": ""}}),
                   "x.norm.", CPU)
    assert list(n.tensor_specs()) == ["x.norm"]
    n.bind({"x.norm": w})
    gain, eps = n.carried()
    assert eps == 1e-6 and gain.dtype == torch.float32
    assert torch.allclose(gain, torch.tensor([1.25, 0.5, 1.0]) * 0.3, rtol=1e-7, atol=0)
    n = build_part("norm", PartSpec("rmsnorm", {"size": 3, "eps": 1e-6}), "x.", CPU)
    n.bind({"x.weight": w})
    assert n.carried()[0] is w                                # no offset, no factor: the stored vector itself


def test_linear_scaling_divides_every_frequency():
    plain = build_part("position", PartSpec("rotary", {"head_dim": 12, "rotary_dim": 8, "theta": 500.0}), "", CPU)
    scaled = build_part("position", PartSpec("rotary", {"head_dim": 12, "rotary_dim": 8, "theta": 500.0,
                                                        "scaling": {"kind": "linear", "factor": 2.5}}), "", CPU)
    want = torch.tensor([500.0 ** (-2.0 * i / 8) / 2.5 for i in range(4)])
    assert torch.allclose(scaled.inv_freq, want, rtol=1e-6, atol=0) and torch.allclose(plain.inv_freq / 2.5, want, rtol=1e-6, atol=0)
    assert scaled.mscale == 1.0
    with pytest.raises(ValueError, match="factor"):
        build_part("position", PartSpec("rotary", {"head_dim": 8, "theta": 10.0, "scaling": {"kind": "linear", "factor": 0.0}}), "", CPU)


def test_relu_as_a_gates_constants():
    ff = build_part("feed_forward", PartSpec("gated_mlp", {"hidden_size": 8, "intermediate_size": 4, "activation": "relu"}), "", CPU)
    g = torch.tensor([-3e4, -5.0, -1e-3, -1e-20, 0.0, 1e-20, 1e-3, 5.0, 3e4])
    got = g / (1.0 + torch.exp(-(ff.act["alpha"] + ff.act.get("cubic", 0.0) * g * g) * g))
    assert torch.equal(got + 0.0, torch.clamp(g, min=0.0))


def test_parts_refuse_what_they_do_not_take():
    def memory_part(**kw):
        return build_part("mixer", PartSpec("decay_memory", {"hidden_size": 8, "num_heads": 2, "head_dim": 4, "decay": [0.5, 0.9],
                                                             "eps": 1e-6, **kw}), "m.", CPU)
    assert memory_part().state_bytes() >= 4 * 2 * 4 * 4
    for kw, word in (({"decay": [0.5]}, "decay"), ({"decay": [0.5, 1.1]}, "decay"), ({"head_dim": 513}, "head_dim"),
                     ({"gate": "tanh"}, "gate"), ({"out_norm": "none"}, "out_norm"), ({"activation": "relu"}, "activation"),
                     ({"position": PartSpec("rotary", {"head_dim": 4, "theta": 10.0, "interleaved": True})}, "half-split")):
        with pytest.raises(ValueError, match=word):
            memory_part(**kw)
    base = {"hidden_size": 8, "num_heads": 2, "num_kv_heads": 2, "head_dim": 4}
    for kw, word in (({"v_mix": {"role": "last", "key": "x"}}, "role"), ({"v_mix": {"role": "mix", "key": "x"}, "values": "keys"}, "v_mix"),
                     ({"qk_norm": "rows"}, "qk_norm")):
        with pytest.raises(ValueError, match=word):
            build_part("mixer", PartSpec("attention", {**base, **kw}), "m.", CPU)
    branch = {"mixer": PartSpec("attention", base), "name": "a"}
    normed = {**branch, "norm": PartSpec("rmsnorm", {"size": 8, "eps": 1e-6}), "norm_name": "n"}
    with pytest.raises(ValueError, match="every branch has a norm"):
        build_part("mixer", PartSpec("parallel", {"branches": [normed, {**branch, "mixer": PartSpec("decay_memory", {
            "hidden_size": 8, "num_heads": 1, "head_dim": 4, "decay": [0.5], "eps": 1e-6}), "name": "b"}]}), "m.", CPU)


# ------------------------------------------------------------------ the plain implementation against itself
def random_weights(cfg_dict, seed):
    m = build_model(config_from_dict(copy.deepcopy(cfg_dict)), CPU)
    g = torch.Generator().manual_seed(seed)
    return {name: torch.randn(tuple(spec.shape), generator=g, dtype=torch.float64) * (0.3 if len(spec.shape) == 2 else 0.4)
            for name, spec in m.tensor_specs().items()}


def test_plain_prompt_equals_plain_token_by_token_and_portions():
    w = random_weights(SMALL, 3)
    ids = torch.randint(0, 53, (23,), generator=torch.Generator().manual_seed(5)).tolist()
    whole, _ = P.forward(SMALL, w, ids)
    for cuts in ([1] * 23, [2, 1, 7, 2, 11]):
        carry, rows, at = None, [], 0
        for c in cuts:
            out, carry = P.forward(SMALL, w, ids[at:at + c], carry)
            rows.append(out)
            at += c
        assert torch.allclose(torch.cat(rows), whole, rtol=1e-9, atol=1e-9)


def test_plain_memory_equals_its_sum_form():
    """y_t = sum over s <= t of decay^(t - s) (q_t . k_s) v_s."""
    g = torch.Generator().manual_seed(1)
    T, H, d, e = 9, 3, 3, 4
    q, k = torch.randn(T, H, d, generator=g, dtype=torch.float64), torch.randn(T, H, d, generator=g, dtype=torch.float64)
    v = torch.randn(T, H, e, generator=g, dtype=torch.float64)
    decay = [0.9, 0.0, 1.0]
    y, S = P.decay_scan(q, k, v, decay)
    for a in range(H):
        for t in range(T):
            want = sum(decay[a] ** (t - s) * torch.dot(q[t, a], k[s, a]) * v[s, a] for s in range(t + 1))
            assert torch.allclose(y[t, a], want, rtol=1e-10, atol=1e-12)
    y2, _ = P.decay_scan(q[4:], k[4:], v[4:], decay, P.decay_scan(q[:4], k[:4], v[:4], decay)[1])
    assert torch.allclose(y2, y[4:], rtol=1e-12, atol=1e-12)


def test_plain_rotation_norm_cap_and_mixed_values():
    x = torch.arange(12, dtype=torch.float64).reshape(1, 1, 12) + 1
    y = P.rotate(x, 7, 8, 100.0, 2.0)
    ang = 7 * 100.0 ** (-2.0 / 8) / 2.0                   # pair (1, 5)
    assert abs(y[0, 0, 1].item() - (2 * math.cos(ang) - 6 * math.sin(ang))) < 1e-12
    assert abs(y[0, 0, 5].item() - (6 * math.cos(ang) + 2 * math.sin(ang))) < 1e-12
    assert torch.equal(y[..., 8:], x[..., 8:])            # what lies behind the rotated dims stays
    # a rotation does not change the root mean square: dividing by it before or behind is the same
    assert torch.allclose(P.rms(P.rotate(x, 7, 8, 100.0), 1e-5), P.rotate(P.rms(x, 1e-5), 7, 8, 100.0), rtol=1e-12, atol=1e-12)
    assert abs(P.capped(torch.tensor(1000.0, dtype=torch.float64), 5.0).item() - 5.0) < 1e-12
    assert abs(P.capped(torch.tensor(0.01, dtype=torch.float64), 5.0).item() - 0.01) < 1e-6
    # one token: softmax over a single key gives the (mixed) value itself, times the gate
    w = {"g": torch.zeros(1, 3, dtype=torch.float64), "o": torch.eye(3, dtype=torch.float64),
         **{n: torch.eye(3, dtype=torch.float64) for n in "qkv"}}
    m = {"heads": 1, "kv_heads": 1, "dim": 3, "vdim": 3, "scale": 1.0}
    h, first = torch.tensor([[1.0, 2.0, 3.0]], dtype=torch.float64), torch.tensor([[[5.0, 5.0, 5.0]]], dtype=torch.float64)
    out, (_, cached), own = P.attention_mixer(h, w, "", m, 1e-6, biases=False, unit=True, v_first=first, mix=0.25)
    assert torch.allclose(out[0], 0.5 * (0.75 * h[0] + 0.25 * 5.0)) and torch.equal(own[0, 0], h[0])
    assert torch.allclose(cached[0, 0], 0.75 * h[0] + 1.25)
