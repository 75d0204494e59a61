"""Dofipel without a GPU: its configuration (round trip, defaults, errors that name the key), the tensors and caches its
parts ask for, the rows of the distance table, and the plain implementation against direct sums."""
import json
import math

import pytest
import torch

from tests.plain import dofipel_plain as P

F64 = torch.float64


# ---- configurations as the tests write them ----------------------------------------
def latent(heads, dim, rot_dim, vdim, kv_rank, scale, base=10000.0, kv_from=None):
    m = {"dim": dim, "heads": heads, "kv_rank": kv_rank, "rot": {"base": base, "dims": rot_dim}, "rot_dim": rot_dim,
         "scale": scale, "vdim": vdim}
    if kv_from is not None:
        m["kv_from"] = kv_from
    return m


def windowed(heads, kv_heads, dim, vdim, scale, bias_max, softcap=0.0, window=0):
    m = {"bias_max": bias_max, "dim": dim, "heads": heads, "kv_heads": kv_heads, "scale": scale, "vdim": vdim}
    if softcap:
        m["softcap"] = softcap
    if window:
        m["mask"] = {"size": window}
    return m


def dense(ff):
    return {"ff": ff, "kind": "dense"}


def moe(ff, experts, top, shared=0):
    m = {"expert": {"ff": ff}, "kind": "moe", "router": {"experts": experts, "top": top}}
    if shared:
        m["shared"] = {"ff": shared}
    return m


def layer(kind, mixer, mlp):
    return {"mixer": mixer, "mlp": mlp, "type": kind}


def model(layers, vocab, width, logit_scale, bias_rows=32, eps=1e-6):
    return {"architecture": "Dofipel", "bias_rows": bias_rows, "layers": layers, "logit_scale": logit_scale, "norm": {"eps": eps},
            "torch_dtype": "bfloat16", "vocab": vocab, "width": width}


# A: every kind of layer and feed-forward, latents read by two later layers with other heads and widths than their
# owner's; B: what A makes equal or leaves in differs (no rotation, no cap, no window, one head, one expert a token, no shared
# expert, layers without a feed-forward, an odd number of table rows, a logit factor of 1); C: sizes that are no multiple of 8
MODELS = {
    "A": model([layer("latent_attention", latent(4, 16, 8, 24, 40, 0.25), dense(96)),
                layer("latent_attention", latent(6, 24, 8, 16, 40, 0.2, kv_from=0), moe(32, 9, 2, shared=48)),
                layer("attention", windowed(6, 2, 32, 16, 0.2, 50, softcap=6.0, window=37), moe(32, 9, 2, shared=32)),
                layer("latent_attention", latent(2, 16, 16, 8, 32, 0.25, base=500.0), dense(64)),
                layer("latent_attention", latent(4, 16, 8, 24, 40, 0.3, kv_from=0), None),
                layer("attention", windowed(2, 2, 24, 40, 0.3, 300, softcap=10.0, window=70), dense(40))],
               vocab=200, width=64, logit_scale=1.5, bias_rows=16),
    "B": model([layer("attention", windowed(3, 1, 16, 16, 0.3, 40), None),
                layer("latent_attention", latent(1, 8, 0, 8, 16, 0.4), moe(16, 5, 1)),
                layer("latent_attention", latent(3, 8, 4, 12, 24, 0.3, base=100.0), None),
                layer("latent_attention", latent(5, 16, 4, 8, 24, 0.25, base=100.0, kv_from=2), moe(24, 4, 4, shared=8)),
                layer("attention", windowed(4, 4, 48, 48, 0.15, 128, softcap=4.0, window=1), dense(32))],
               vocab=131, width=48, logit_scale=1.0, bias_rows=9, eps=1e-5),
    "C": model([layer("latent_attention", latent(5, 6, 2, 10, 12, 0.4), moe(10, 3, 2, shared=6)),
                layer("attention", windowed(3, 1, 20, 13, 0.25, 33, softcap=3.0, window=5), dense(22)),
                layer("latent_attention", latent(3, 7, 2, 5, 12, 0.35, kv_from=0), dense(14))],
               vocab=77, width=30, logit_scale=0.3, bias_rows=6),
}


def config_of(data):
    import hector_engine_amd  # noqa: F401
    from hector_engine_amd.registry import config_from_dict
    return config_from_dict(json.loads(json.dumps(data)))


@pytest.mark.parametrize("name", list(MODELS))
def test_configuration_round_trip(name):
    cfg = config_of(MODELS[name])
    assert cfg.to_dict() == MODELS[name]
    assert config_of(cfg.to_dict()).to_dict() == MODELS[name]


def test_defaults_of_what_a_layer_leaves_out():
    cfg = config_of(MODELS["B"])
    assert cfg.layers[0].mixer.softcap == 0.0 and cfg.layers[0].mixer.window == 0 and cfg.layers[0].mlp is None
    assert cfg.layers[1].mixer.kv_from is None and cfg.layers[1].mixer.rot_dim == 0 and cfg.layers[1].mlp.shared_ff == 0
    data = json.loads(json.dumps(MODELS["B"]))
    del data["logit_scale"], data["bias_rows"], data["torch_dtype"]
    cfg = config_of(data)
    assert cfg.logit_scale == 1.0 and cfg.bias_rows == 32


@pytest.mark.parametrize("change,key", [
    (lambda d: d["layers"][0].update(type="mamba"), "layers[0].type"),
    (lambda d: d["layers"][0]["mixer"].pop("bias_max"), "bias_max"),
    (lambda d: d["layers"][0]["mixer"].update(heads=4, kv_heads=3), "layers[0].mixer.heads"),
    (lambda d: d["layers"][0]["mixer"].update(mask={"size": 0}), "layers[0].mixer.mask.size"),
    (lambda d: d["layers"][0]["mixer"].update(softcap=-1.0), "layers[0].mixer.softcap"),
    (lambda d: d["layers"][2]["mixer"].update(rot_dim=3), "layers[2].mixer.rot_dim"),
    (lambda d: d["layers"][2]["mixer"].update(scale=0.0), "layers[2].mixer.scale"),
    (lambda d: d["layers"][3]["mixer"].update(kv_from=3), "layers[3].mixer.kv_from"),
    (lambda d: d["layers"][3]["mixer"].update(kv_from=0), "layers[3].mixer.kv_from"),
    (lambda d: d["layers"][3]["mixer"].update(kv_from=1), "layers[3].mixer.kv_from"),       # another rank
    (lambda d: d["layers"][3]["mlp"]["router"].update(top=5), "layers[3].mlp.router.top"),
    (lambda d: d["layers"][4]["mlp"].update(kind="glu"), "layers[4].mlp.kind"),
    (lambda d: d["layers"][4]["mlp"].update(ff=0), "layers[4].mlp.ff"),
    (lambda d: d["norm"].pop("eps"), "eps"),
    (lambda d: d.pop("vocab"), "vocab"),
    (lambda d: d.update(layers=[]), "layers"),
])
def test_errors_name_the_key(change, key):
    from hector_engine_amd.config.base import ConfigError
    data = json.loads(json.dumps(MODELS["B"]))
    change(data)
    with pytest.raises(ConfigError) as err:
        config_of(data)
    assert key in str(err.value)


def test_tensors_and_caches_the_parts_ask_for():
    import hector_engine_amd  # noqa: F401
    from hector_engine_amd.parts.base import BuildEnv
    from hector_engine_amd.registry import build_model
    m = build_model(config_of(MODELS["A"]), BuildEnv(torch.device("cpu"), torch.bfloat16))
    specs = m.tensor_specs()
    shape = {k: tuple(v.shape) for k, v in specs.items()}
    assert shape["embed"] == (200, 64) and "head" not in shape and shape["final.norm.alpha"] == () and shape["l4.norm1.b"] == (64,)
    assert "l0.norm2" not in shape and not any(k.startswith("l4.mlp") for k in shape)
    assert shape["l0.mix.q"] == (4 * 24, 64) and shape["l0.mix.dkv"] == (48, 64) and shape["l0.mix.dkv.norm"] == (40,)
    assert shape["l0.mix.uk"] == (64, 40) and shape["l0.mix.uv"] == (96, 40) and shape["l0.mix.g"] == (96, 64)
    assert "l1.mix.dkv" not in shape and "l1.mix.dkv.norm" not in shape and shape["l1.mix.uk"] == (6 * 24, 40)
    assert shape["l2.mix.rel"] == (None, 6) and specs["l2.mix.rel"].random_shape() == (16, 6) and shape["l2.mix.sink"] == (6,)
    assert specs["l2.mix.rel"].matches((7, 6)) and not specs["l2.mix.rel"].matches((7, 5)) and not specs["l2.mix.rel"].matches((6,))
    assert shape["l2.mix.v"] == (32, 64) and shape["l2.mix.o"] == (64, 96)
    assert shape["l1.mlp.router"] == (9, 64) and shape["l1.mlp.router.b"] == (9,) and shape["l1.mlp.shared.up"] == (48, 64)
    assert shape["l1.mlp.e8.down"] == (64, 32) and shape["l0.mlp.gate"] == (96, 64)
    plans = m.run_plans()
    assert [p.cache_from for p in plans] == [None, 0, None, None, 0, None] and all(p.state_bytes == 0 for p in plans)
    assert plans[1].kv is None and plans[0].kv.kv_heads == 1 and plans[0].kv.head_dim == 48 and plans[0].kv.window == 0
    assert (plans[2].kv.kv_heads, plans[2].kv.window, plans[2].kv.head_dim) == (2, 37, 32)


# ---- the distance table -------------------------------------------------------------
@pytest.mark.parametrize("rows,far", [(16, 200), (16, 128), (32, 128), (2, 5), (9, 40), (6, 33), (64, 100), (7, 1000), (8, 5)])
def test_rows_of_the_distance_table(rows, far):
    from hector_engine_amd.parts.attention import distance_bucket
    half = rows // 2
    got = [distance_bucket(n, rows, far) for n in range(3 * far)]
    assert got[:half] == list(range(half)) and max(got) == rows - 1 and got[far:] == [rows - 1] * (2 * far)
    assert all(a <= b for a, b in zip(got, got[1:]))
    for n in range(half, 3 * far):
        if far <= half:
            continue
        x = math.log(n / half) / math.log(far / half) * (rows - half)
        if abs(x - round(x)) > 1e-9:                    # (on an edge the logarithms round either way)
            assert got[n] == min(rows - 1, half + math.floor(x)), n
        assert got[n] == P.bucket_of(n, rows, far)
    if far == 128 and rows == 16:                        # 8 * 16^(k/8): 16, 32 and 64 are edges themselves
        assert [got[n] for n in (15, 16, 31, 32, 63, 64)] == [9, 10, 11, 12, 13, 14]


def test_a_table_of_any_number_of_stored_rows_is_spread_over_the_distances():
    import hector_engine_amd  # noqa: F401
    from hector_engine_amd.parts.base import BuildEnv, PartSpec, build_part
    for stored, window, entries in ((4, 0, 51), (30, 0, 51), (4, 20, 20), (200, 0, 101), (1, 3, 3)):
        part = build_part("mixer", PartSpec("attention", {
            "hidden_size": 16, "num_heads": 3, "num_kv_heads": 1, "head_dim": 8, "window": window, "score_cap": 2.0,
            "distance_table": {"rows": 9, "far": 50}}), "m.", BuildEnv(torch.device("cpu"), torch.float32))
        tensors = {k: torch.zeros(v.random_shape()) for k, v in part.tensor_specs().items()}
        assert tensors["m.distance_bias"].shape == (9, 3)
        tensors["m.distance_bias"] = torch.arange(stored * 3, dtype=torch.float32).view(stored, 3)
        part.bind(tensors)
        assert part.table.shape == (3, entries) and part.table.is_contiguous()
        for n in range(entries):
            row = P.bucket_of(n, stored, 50) if 0 < stored // 2 < 50 else n if n < stored // 2 else stored - 1
            assert part.table[:, n].tolist() == [3.0 * row, 3.0 * row + 1, 3.0 * row + 2]


def test_the_gated_gelu_is_a_sigmoid_of_a_cubic():
    import hector_engine_amd  # noqa: F401
    from hector_engine_amd.parts.base import BuildEnv, PartSpec, build_part
    ff = build_part("feed_forward", PartSpec("gated_mlp", {"hidden_size": 8, "intermediate_size": 8, "activation": "gelu_tanh"}),
                    "f.", BuildEnv(torch.device("cpu"), torch.float32))
    z = torch.linspace(-12, 12, 4001, dtype=F64)
    y = z * torch.sigmoid(ff.act["alpha"] * z + ff.act["cubic"] * z ** 3)
    assert torch.allclose(y, P.gelu_tanh(z), rtol=1e-12, atol=1e-12)


# ---- the plain implementation against direct sums -----------------------------------------
def rnd(*shape, seed=0, scale=1.0):
    g = torch.Generator().manual_seed(seed)
    return torch.randn(*shape, generator=g, dtype=F64) * scale


@pytest.mark.parametrize("window,cap", [(0, 0.0), (4, 2.0), (1, 3.0), (7, 0.0)])
def test_windowed_attention_key_by_key(window, cap):
    Tq, Tk, H, G, d, e, far = 9, 14, 4, 2, 5, 3, 11
    q, k, v, table, sinks = rnd(Tq, H, d, seed=1), rnd(Tk, G, d, seed=2), rnd(Tk, G, e, seed=3), rnd(6, H, seed=4), rnd(H, seed=5)
    got = P.window_attention(q, k, v, 0.7, cap, table, far, sinks, window, first_position=5)
    for t in range(Tq):
        i = 5 + t
        for h in range(H):
            num, den = torch.zeros(e, dtype=F64), math.exp(float(sinks[h]))
            for j in range(max(0, i - window + 1) if window else 0, i + 1):
                s = float(q[t, h] @ k[j, h // 2]) * 0.7
                if cap:
                    s = cap * math.tanh(s / cap)
                s += float(table[P.bucket_of(i - j, 6, far), h])
                num, den = num + math.exp(s) * v[j, h // 2], den + math.exp(s)
            assert torch.allclose(got[t, h], num / den, atol=1e-12)


def test_latent_attention_key_by_key_and_from_another_layer():
    T, D, m = 8, 10, {"heads": 3, "dim": 4, "rot_dim": 2, "vdim": 5, "kv_rank": 6, "scale": 0.4, "rot": {"base": 50.0}}
    w = {"q": rnd(18, D, seed=1), "dkv": rnd(8, D, seed=2), "dkv.norm": rnd(6, seed=3), "uk": rnd(12, 6, seed=4),
         "uv": rnd(15, 6, seed=5), "g": rnd(15, D, seed=6), "o": rnd(D, 15, seed=7)}
    h, other = rnd(T, D, seed=8), rnd(T, D, seed=9)
    pos = list(range(T))
    for source in (h, other):                  # its own latents, and those another layer made of other rows
        kept = P.latents(source, w, "", m, 1e-5, pos)
        got = P.latent_attention(h, w, "", m, 1e-5, pos, kept)
        down = source @ w["dkv"].T
        c = down[:, :6] / torch.sqrt((down[:, :6] ** 2).mean(-1, keepdim=True) + 1e-5) * w["dkv.norm"]
        want = torch.zeros(T, 15, dtype=F64)
        for t in range(T):
            for head in range(3):
                qt = (h[t] @ w["q"].T)[6 * head:6 * head + 6]
                ss, vs = [], []
                for j in range(t + 1):
                    # turning both by their positions is turning the query by the difference
                    a = float(t - j)
                    u, v = qt[4] * math.cos(a) - qt[5] * math.sin(a), qt[5] * math.cos(a) + qt[4] * math.sin(a)
                    key = w["uk"][4 * head:4 * head + 4] @ c[j]
                    ss.append((float(qt[:4] @ key) + float(u * down[j, 6] + v * down[j, 7])) * 0.4)
                    vs.append(w["uv"][5 * head:5 * head + 5] @ c[j])
                p = torch.softmax(torch.tensor(ss, dtype=F64), 0)
                want[t, 5 * head:5 * head + 5] = sum(a * b for a, b in zip(p, vs)) * torch.sigmoid(w["g"] @ h[t])[5 * head:5 * head + 5]
        assert torch.allclose(got, want @ w["o"].T, atol=1e-10)


def test_the_routed_weights():
    h = rnd(7, 10, seed=9)
    w = {"r.router": rnd(5, 10, seed=10), "r.router.b": rnd(5, seed=11, scale=3.0)}
    for e in ("e0", "e1", "e2", "e3", "e4", "shared"):
        for i, (k, s) in enumerate((("gate", (6, 10)), ("up", (6, 10)), ("down", (10, 6)))):
            w[f"r.{e}.{k}"] = rnd(*s, seed=20 + 7 * i + sum(map(ord, e)))
    z = h @ w["r.router"].T + w["r.router.b"]
    every = P.routed_ff(h, w, "r.", {"router": {"experts": 5, "top": 5}})
    want = sum(torch.softmax(z, -1)[:, e:e + 1] * P.gated_ff(h, w, f"r.e{e}.", P.silu) for e in range(5))
    assert torch.allclose(every, want, atol=1e-12)          # all experts chosen: the softmax over all logits
    one = P.routed_ff(h, w, "r.", {"router": {"experts": 5, "top": 1}, "shared": {"ff": 6}})
    want = P.gated_ff(h[2:3], w, f"r.e{int(z[2].argmax())}.", P.silu) + P.gated_ff(h[2:3], w, "r.shared.", P.silu)
    assert torch.allclose(one[2:3], want, atol=1e-12)       # one expert: weight 1


@pytest.mark.parametrize("name", list(MODELS))
def test_prefix_logits_do_not_depend_on_what_follows(name):
    import hector_engine_amd  # noqa: F401
    from hector_engine_amd.parts.base import BuildEnv
    from hector_engine_amd.registry import build_model
    from hector_engine_amd.weights.random_init import random_tensors
    specs = build_model(config_of(MODELS[name]), BuildEnv(torch.device("cpu"), torch.bfloat16)).tensor_specs()
    w = {k: v.to(F64) for k, v in random_tensors(specs, 5, torch.bfloat16, "cpu").items()}
    ids = [3, 70, 12, 12, 5, 44, 9, 1, 30, 2, 61]
    whole = P.forward(MODELS[name], w, ids)
    assert torch.allclose(P.forward(MODELS[name], w, ids[:6]), whole[:6], atol=1e-9)
    assert P.greedy(MODELS[name], w, ids[:4], 3) == P.greedy(MODELS[name], w, ids[:4], 5)[:3]
