"""Bobevik on the GPU against the plain implementation (tests/plain/bobevik_plain.py): each new mechanism alone at its
kernel, fed in portions and in batches through slots that are used again, with inputs planted so that a lost state or a
key that is not seen shows; then whole models of several shapes and layer orders through the engine's step function, cut
and batched in many ways, in 32-bit and in bfloat16; and greedy generation through the library's own entry point, its
command line and the trace replay."""
import json
import os
import subprocess
import sys

import pytest
import torch

from tests.helpers import argmax_agrees_where_clear, rand_ids
from tests.plain import bobevik_plain as P
from tests.test_bobevik_cpu import attn, layer, memory, model, pair, rot
from tests.test_kernels_gpu import PAGE, cached_k, cached_v, dev, paged_setup, rnd

pytestmark = pytest.mark.gpu
DTYPES = ["float32", "bfloat16"]
TORCH = {"float32": torch.float32, "bfloat16": torch.bfloat16}
F64 = torch.float64


@pytest.fixture(scope="module")
def ops():
    import hector_engine_amd  # noqa: F401
    from hector_engine_amd.kernels import ops as o
    return o


def i32(values):
    return torch.tensor(values, dtype=torch.int32, device="cuda")


# a schedule of steps over three sequences: (sequence, new tokens) per step; lengths 71, 9 and 140
SCHEDULE = [[(0, 3), (1, 1), (2, 64)], [(0, 1), (1, 1), (2, 1)], [(0, 2), (2, 2)], [(1, 7), (2, 70)],
            [(0, 64)], [(0, 1), (2, 1)], [(2, 2)]]
LENGTHS = [71, 9, 140]


def run_schedule(slots, per_step):
    """Feeds SCHEDULE; per_step(sequences, new tokens of each, first position of each, slots) runs one step."""
    done = [0, 0, 0]
    for step in SCHEDULE:
        seqs, q_lens = [s for s, _ in step], [n for _, n in step]
        per_step(seqs, q_lens, [done[s] for s in seqs], [slots[s] for s in seqs])
        for s, n in step:
            done[s] += n
    assert done == LENGTHS


def cu_of(q_lens):
    cu = [0]
    for n in q_lens:
        cu.append(cu[-1] + n)
    return cu


# ------------------------------------------------------------------ memories with a constant decay
def powers_of(ops, decay):
    e = torch.arange(ops.DECAY_POWERS, dtype=F64)
    return dev((torch.tensor(decay, dtype=F64)[:, None] ** e).float())


def inv_freq(r, base):
    return dev((base ** (-torch.arange(0, r, 2, dtype=F64) / r)).float()) if r else None


def plain_memory(x, H, dk, dv, decay, r, base, silu, k_scale, first=0, state=None):
    """(y [T, H dv], S) of rows [q | k | v] at positions first, first + 1, ..."""
    T = x.shape[0]
    f = P.silu if silu else (lambda z: z)
    x = x.double()
    q, k = f(x[:, :H * dk]).reshape(T, H, dk), f(x[:, H * dk:2 * H * dk]).reshape(T, H, dk)
    v = f(x[:, 2 * H * dk:2 * H * dk + H * dv]).reshape(T, H, dv)
    if r:
        q, k = P.rotate(q, first, r, base), P.rotate(k, first, r, base)
    y, S = P.decay_scan(q, k * k_scale, v, decay, state)
    return y.reshape(T, H * dv), S


def scan(ops, x, state, offset, positions, cu, slots, H, dk, dv, decay, r, base, silu, k_scale, most=None, rows=None):
    rows = x.shape[0] if rows is None else rows
    y = torch.full((rows, H * dv), float("nan"), device="cuda")
    q_lens = [b - a for a, b in zip(cu, cu[1:])]
    ops.decay_scan(y, x[:, :H * dk], x[:, H * dk:2 * H * dk], x[:, 2 * H * dk:2 * H * dk + H * dv], powers_of(ops, decay), state,
                   offset, i32(positions), i32(cu), i32(slots), rows, len(slots), most or max(q_lens), H, dk, dv, act=silu,
                   k_scale=k_scale, inv_freq=inv_freq(r, base))
    return y


SIZES = [(2, 64, 40, 64, False), (3, 12, 20, 8, False), (1, 5, 3, 2, False), (2, 130, 24, 0, True), (4, 16, 1, 0, True), (1, 1, 7, 0, True),
         (2, 48, 66, 48, False), (1, 300, 132, 300, False), (2, 128, 256, 128, False)]


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("H,dk,dv,r,silu", SIZES)
def test_a_memory_in_portions_and_batches_equals_the_whole(ops, dtype, H, dk, dv, r, silu):
    tdt = TORCH[dtype]
    wide = 2 * H * dk + H * dv + 8                                # q | k | v inside wider rows, as behind one product
    decay = [0.995, 0.6, 0.9, 0.99][:H]
    xs = [rnd(n, wide, seed=10 + i).to(tdt) for i, n in enumerate(LENGTHS)]
    k_scale = 1.0 if silu else dk ** -0.5
    want = [plain_memory(x, H, dk, dv, decay, r, 5000.0, silu, k_scale) for x in xs]
    offset, nbytes = 256, 4 * ops.decay_state_floats(H, dk, dv)
    assert nbytes >= 4 * H * dk * dv
    state = torch.zeros(6, offset + nbytes + 64, dtype=torch.uint8, device="cuda")
    state[:, :offset] = 55
    state[:, offset + nbytes:] = 77                               # what lies around the memory is not touched
    slots = [4, 0, 2]                                             # not in order, with gaps
    got = [torch.zeros(n, H * dv, dtype=F64) for n in LENGTHS]

    def per_step(seqs, q_lens, starts, sl):
        x = dev(torch.cat([xs[s][at:at + n] for s, n, at in zip(seqs, q_lens, starts)]))
        positions = [at + t for n, at in zip(q_lens, starts) for t in range(n)]
        y = scan(ops, x, state, offset, positions, cu_of(q_lens), sl, H, dk, dv, decay, r, 5000.0, silu, k_scale)
        at = 0
        for s, n, st in zip(seqs, q_lens, starts):
            got[s][st:st + n] = y[at:at + n].cpu().double()
            at += n

    run_schedule(slots, per_step)
    # (angles are 32-bit numbers: at position 139 off by 8e-6 rad, and so are the rotated rows)
    tol = 2e-5 if r else 3e-6
    for s, (g, (w, S)) in enumerate(zip(got, want)):
        assert torch.allclose(g, w, rtol=0, atol=tol * w.abs().max().item())
        kept = state[slots[s], offset:offset + nbytes].view(torch.float32).cpu().double().reshape(H, dk, -1)[:, :, :dv]
        assert torch.allclose(kept, S, rtol=0, atol=tol * S.abs().max().item())
    assert bool((state[:, :offset] == 55).all()) and bool((state[:, offset + nbytes:] == 77).all())
    assert bool((state[[1, 3, 5]][:, offset:offset + nbytes] == 0).all())     # rows of other slots stay as they were


@pytest.mark.parametrize("dtype", DTYPES)
def test_a_memory_that_was_lost_shows(ops, dtype):
    """One early token with a large value, and decays near one: hundreds of tokens later a query along its key still
    reads its value, faded by exactly decay^distance, whether the tokens came at once, one by one, in pairs, or so that the
    early one is the last or the first of a chunk. A decay of 1 keeps it whole, a decay of 0 forgets it at once."""
    H, dk, dv, T = 4, 8, 16, 330
    decay = [0.999, 1.0, 0.995, 0.0]
    for early in (5, 63, 64, 127):
        x = 0.02 * rnd(T, 2 * H * dk + H * dv, seed=1)
        for h in range(H):
            x[early, H * dk + h * dk + 3] = 2.0
            x[early, 2 * H * dk + h * dv:2 * H * dk + (h + 1) * dv] = 8.0 + h
            x[-1, h * dk + 3] = 2.0                              # the last query asks along the early key
        x = x.to(TORCH[dtype])
        want, _ = plain_memory(x, H, dk, dv, decay, 0, 1.0, False, 1.0)
        for h in range(H):
            faded = 4.0 * (8.0 + h) * decay[h] ** (T - 1 - early)
            assert (want[-1, h * dv:(h + 1) * dv] - faded).abs().max() < 0.3       # the early token answers
        for cuts in ([T], [1] * T, [2] * (T // 2), [early + 1, 1, T - early - 4, 2], [early, T - early], [64, 65, 9, 192]):
            state = torch.zeros(2, 4 * ops.decay_state_floats(H, dk, dv), dtype=torch.uint8, device="cuda")
            out, at = [], 0
            for c in cuts:
                out.append(scan(ops, dev(x[at:at + c].contiguous()), state, 0, list(range(at, at + c)), [0, c], [1], H, dk, dv, decay,
                                0, 1.0, False, 1.0).cpu())
                at += c
            assert torch.allclose(torch.cat(out).double(), want, rtol=1e-5, atol=1e-5)
            assert bool((state[0] == 0).all())


@pytest.mark.parametrize("most", [1, 5, 100])
def test_rows_of_no_sequence_get_zeros_and_empty_sequences_are_passed_over(ops, most):
    """A step that runs in the bucket of larger sizes: sequences without rows (slot -1) and rows behind the last one."""
    H, dk, dv = 2, 16, 24
    q_lens = [1, 0, min(most, 70), 0]
    rows = sum(q_lens) + 9
    x = dev(rnd(rows, 2 * H * dk + H * dv, seed=4))
    state = torch.zeros(3, 4 * ops.decay_state_floats(H, dk, dv), dtype=torch.uint8, device="cuda")
    positions = [0] + list(range(q_lens[2])) + [0] * 9
    y = scan(ops, x, state, 0, positions, cu_of(q_lens), [2, -1, 0, -1], H, dk, dv, [0.9, 0.8], 8, 100.0, False, 1.0, most, rows).cpu()
    assert bool((y[sum(q_lens):] == 0).all())
    at = 0
    for n in q_lens:
        if n:
            want, _ = plain_memory(x[at:at + n].cpu(), H, dk, dv, [0.9, 0.8], 8, 100.0, False, 1.0)
            assert torch.allclose(y[at:at + n].double(), want, rtol=0, atol=1e-5 * want.abs().max().item())
        at += n
    assert bool((state[1] == 0).all())


def test_more_sequences_than_a_wavefront_has_lanes(ops):
    """150 sequences of 1 to 140 rows: chunks are counted through all of them."""
    H, dk, dv = 1, 8, 8
    q_lens = [1 + (i * 37) % 9 for i in range(150)]
    for i in (3, 63, 64, 65, 128, 149):
        q_lens[i] = 60 + i % 81
    T = sum(q_lens)
    x = rnd(T, 3 * 8, seed=9)
    state = torch.zeros(150, 4 * ops.decay_state_floats(H, dk, dv), dtype=torch.uint8, device="cuda")
    slots = [(7 * i) % 150 for i in range(150)]
    positions = [t for n in q_lens for t in range(n)]
    y = scan(ops, dev(x), state, 0, positions, cu_of(q_lens), slots, H, dk, dv, [0.97], 4, 100.0, False, 0.5).cpu().double()
    at = 0
    for s, n in enumerate(q_lens):
        want, S = plain_memory(x[at:at + n], H, dk, dv, [0.97], 4, 100.0, False, 0.5)
        assert torch.allclose(y[at:at + n], want, rtol=0, atol=1e-5 * want.abs().max().item()), s
        kept = state[slots[s]].view(torch.float32).cpu().double().reshape(1, 8, 8)
        assert torch.allclose(kept, S, rtol=0, atol=1e-5 * S.abs().max().item()), s
        at += n


def test_memories_too_large_to_hold_for_all_chunks_at_once(ops):
    """40 heads of 512 x 512: the chunks of a step are walked in windows of a few. A head's rows have the bits they
    have when the head runs alone, in one window."""
    H, dk, dv, T = 40, 512, 512, 650
    x = torch.randn(T, 3 * H * dk, generator=torch.Generator(device="cuda").manual_seed(1), device="cuda").to(torch.bfloat16)
    decay = [0.9 + 0.0025 * h for h in range(H)]
    cu, slots = [0, 10, 300, T], [2, 0, 1]
    positions = [t for a, b in zip(cu, cu[1:]) for t in range(b - a)]
    state = torch.zeros(3, 4 * ops.decay_state_floats(H, dk, dv), dtype=torch.uint8, device="cuda")
    assert ops.decay_workspace_floats(T, 3, 350, H, dk, dv) < 10 * ops.decay_state_floats(H, dk, dv)     # not all 12 at once
    y = scan(ops, x, state, 0, positions, cu, slots, H, dk, dv, decay, 0, 1.0, False, 0.05)
    for h in (0, 17, 39):
        one = torch.cat([x[:, (p * H + h) * dk:(p * H + h + 1) * dk] for p in range(3)], 1).contiguous()
        alone = torch.zeros(3, 4 * ops.decay_state_floats(1, dk, dv), dtype=torch.uint8, device="cuda")
        y1 = scan(ops, one, alone, 0, positions, cu, slots, 1, dk, dv, [decay[h]], 0, 1.0, False, 0.05)
        assert torch.equal(y[:, h * dv:(h + 1) * dv], y1)
        assert torch.equal(state.view(torch.float32).reshape(3, H, -1)[:, h], alone.view(torch.float32))


def test_a_scan_refuses_sizes_that_do_not_fit(ops):
    x = torch.zeros(4, 3 * 8, device="cuda")
    y = torch.zeros(4, 8, device="cuda")
    state = torch.zeros(1, 4 * ops.decay_state_floats(1, 8, 8), dtype=torch.uint8, device="cuda")
    pw, meta = powers_of(ops, [0.5]), (i32([0, 1, 2, 3]), i32([0, 4]), i32([0]), 4, 1, 4, 1, 8, 8)
    with pytest.raises(ValueError, match="room"):
        ops.decay_scan(y, x[:, :8], x[:, 8:16], x[:, 16:], pw, state[:, :64], 0, *meta)
    with pytest.raises(ValueError, match="powers"):
        ops.decay_scan(y, x[:, :8], x[:, 8:16], x[:, 16:], pw[:, :64].contiguous(), state, 0, *meta)
    with pytest.raises(RuntimeError, match="rotated"):
        ops.decay_scan(y, x[:, :8], x[:, 8:16], x[:, 16:], pw, state, 0, *meta, inv_freq=inv_freq(16, 10.0))


# ------------------------------------------------------------------ rows, norms, gates
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("D", [24, 37, 320, 2048, 4096, 16384])
def test_an_embedding_normed_on_its_way_into_the_stream(ops, dtype, D):
    table = rnd(50, D, seed=1, scale=3.0).to(TORCH[dtype])
    gain = 1 + 0.3 * rnd(D, seed=2)
    ids = torch.tensor([3, 49, 0, -1, 50, 17], dtype=torch.int32)
    out = torch.empty(6, D, device="cuda")
    ops.embedding(out, dev(table), dev(ids), 6, 1.5, dev(gain), 1e-5)
    want = P.rms(1.5 * table.double()[[3, 49, 0, 0, 0, 17]], 1e-5) * gain.double()
    want[3:5] = 0                                                  # ids outside the table
    assert torch.allclose(out.cpu().double(), want, rtol=2e-6, atol=2e-6)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("rows,D", [(1, 24), (7, 37), (70, 320), (5, 2048), (3, 4096), (2, 10000)])
@pytest.mark.parametrize("reader", ["norm", "rows", "none", "pair alone"])
def test_two_normed_branches_into_the_stream_and_the_next_reader(ops, dtype, rows, D, reader):
    tdt = TORCH[dtype]
    resid = rnd(rows, D, seed=1, scale=4.0)
    a, b = rnd(rows, D, seed=2, scale=30.0).to(tdt), rnd(rows, D, seed=5, scale=0.2).to(tdt)
    wa, wb = (1 + 0.3 * rnd(D, seed=6)).to(tdt), 1 + 0.3 * rnd(D, seed=7).to(tdt)
    post, nxt = 0.5 * (1 + 0.3 * rnd(D, seed=3)), 1 + 0.3 * rnd(D, seed=4)
    delta = 0.7 * (P.rms(a.double(), 1e-4) * wa.double() + P.rms(b.double(), 1e-4) * wb.double())
    tol = 3e-6 if dtype == "float32" else 2 ** -7
    if reader == "pair alone":
        out = torch.empty(rows, D, dtype=tdt, device="cuda")
        ops.add_normed_pair(None, dev(a), dev(b), dev(wa), dev(wb), 1e-4, 0.7, None, 0.0, None, 0.0, out, rows)
        assert torch.allclose(out.cpu().double(), delta, rtol=tol, atol=tol)
        return
    r = dev(resid.clone())
    out = None if reader == "none" else torch.empty(rows, D, dtype=tdt, device="cuda")
    ops.add_normed_pair(r, dev(a), dev(b), dev(wa), dev(wb), 1e-4, 0.7, dev(post), 1e-5, dev(nxt) if reader == "norm" else None,
                        2e-6, out, rows)
    want = resid.double() + P.rms(delta, 1e-5) * post.double()
    assert torch.allclose(r.cpu().double(), want, rtol=2e-6, atol=2e-6)          # the stream itself stays in 32 bits
    if reader != "none":
        read = P.rms(want, 2e-6) * nxt.double() if reader == "norm" else want
        assert torch.allclose(out.cpu().double(), read, rtol=tol, atol=tol * read.abs().max().item())


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("rows,parts,width,shift", [(5, 2, 32, 4), (3, 1, 60, 4), (2, 3, 20, 1), (70, 8, 256, 8), (300, 4, 128, 0),
                                                    (4, 1, 2048, 16), (3, 1, 5000, 4), (2, 1, 700, 0), (2, 2, 7, 3)])
@pytest.mark.parametrize("gate", ["silu", True, False])
def test_heads_or_rows_normed_and_gated(ops, dtype, rows, parts, width, shift, gate):
    """Every part by its own root mean square (heads), or all of them by one (a row), then the gate; and the form
    whose gate comes before the norm."""
    tdt = TORCH[dtype]
    W = parts * width
    y, z = rnd(rows, W, seed=1, scale=3.0), rnd(rows, W + 24, seed=2, scale=2.0).to(tdt)
    weight = torch.ones(W) if gate == "silu" else (1 + 0.3 * rnd(W, seed=3)).to(tdt)
    out = torch.empty(rows, W, dtype=tdt, device="cuda")
    ops.gated_group_norm(out, dev(y), dev(z)[:, shift:shift + W], dev(weight), rows, parts, 1e-5, gate_after=gate)
    g = z[:, shift:shift + W].double()
    if gate:
        want = P.rms(y.double().reshape(rows, parts, width), 1e-5).reshape(rows, W) * weight.double()
        want = want * (P.silu(g) if gate == "silu" else torch.sigmoid(g))
    else:
        want = P.rms((y.double() * P.silu(g)).reshape(rows, parts, width), 1e-5).reshape(rows, W) * weight.double()
    tol = 4e-6 if dtype == "float32" else 2 ** -7
    assert torch.allclose(out.cpu().double(), want, rtol=tol, atol=tol)


RELU = {"alpha": 1e30}


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("rows,I", [(3, 20), (130, 136), (9, 33)])
def test_the_relu_gate(ops, dtype, rows, I):
    x = rnd(rows, 2 * I, seed=2, scale=2.0).to(TORCH[dtype])
    x[0, :6] = torch.tensor([0.0, 3.0, -1e-6, 5.0, 1e-6, 7.0])
    out = torch.empty(rows, I, dtype=TORCH[dtype], device="cuda")
    ops.silu_mul(out, dev(x), rows, True, **RELU)
    g, u = x.double()[:, 0::2], x.double()[:, 1::2]
    want = (torch.clamp(g, min=0.0) * u).to(TORCH[dtype])
    assert torch.allclose(out.cpu().double(), want.double(), rtol=1e-6 if dtype == "float32" else 2 ** -8, atol=1e-30)


@pytest.mark.parametrize("M", [1, 8, 16, 17, 40, 64, 200])
def test_the_relu_gate_through_the_feed_forward_part(M):
    """The gated feed-forward at every kernel's row counts: the epilogue of the products of up to 16 and of up to 64
    rows, and the activation's own kernel behind the library's product."""
    import hector_engine_amd  # noqa: F401
    from hector_engine_amd.engine.scratch import ScratchPool
    from hector_engine_amd.parts.base import BuildEnv, PartSpec, StepContext, build_part
    D, I = 96, 72
    env = BuildEnv(torch.device("cuda"), torch.bfloat16)
    part = build_part("feed_forward", PartSpec("gated_mlp", {"hidden_size": D, "intermediate_size": I, "activation": "relu",
                                                            "names": {"gate": "gate", "up": "up", "down": "down"}}), "mlp.", env)
    w = {n: rnd(*s, seed=i, scale=0.2).to(torch.bfloat16) for i, (n, s) in
         enumerate((("mlp.gate", (I, D)), ("mlp.up", (I, D)), ("mlp.down", (D, I))))}
    part.bind({n: dev(t) for n, t in w.items()})
    x = rnd(M, D, seed=9).to(torch.bfloat16)
    pool = ScratchPool(env.device)
    pool.reset()
    ctx = StepContext(rows=M, num_seqs=1, positions=None, row_seq=None, seq_slot=None, cu_seqlens=None, seq_start=None,
                      max_q_len=M, max_keys=M, all_single=False, env=env, scratch=pool)
    got = part.forward(dev(x), ctx).cpu().double()
    want = P.gated_ff(x.double(), {n: t.double() for n, t in w.items()}, "mlp.")
    assert torch.allclose(got[:M], want, rtol=2 ** -6, atol=2 ** -7 * want.abs().max().item())


# ------------------------------------------------------------------ q and k at unit size, mixed values, on the way into the cache
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("H,KVH,kd,vd,pd,r", [(4, 2, 48, 32, 48, 48), (6, 1, 32, 64, 64, 16), (3, 3, 16, 16, 16, 0),
                                              (4, 2, 40, 24, 48, 8), (2, 1, 10, 14, 16, 6), (8, 8, 128, 128, 128, 64),
                                              (40, 4, 64, 64, 64, 64)])
@pytest.mark.parametrize("biased,mixed", [(False, True), (True, False), (False, False), (True, True)])
def test_unit_queries_and_keys_and_mixed_values(ops, dtype, H, KVH, kd, vd, pd, r, biased, mixed):
    tdt = TORCH[dtype]
    starts, new, theta, eps, lam = [70, 5, 130], [3, 64, 1], 50000.0, 1e-3, 0.3
    slots, table, kpool, vpool = paged_setup([a + b for a, b in zip(starts, new)], KVH, pd, tdt, 20)
    rows = sum(new)
    width = (H + KVH) * kd + KVH * vd
    qkv = rnd(rows + 1, width, seed=21, scale=0.2).to(tdt)        # eps matters: mean squares of 0.04
    qkv[-1] = 0                                                    # a padding row at the end must be left alone
    bias = (0.2 * rnd(width, seed=22)).to(tdt) if biased else None
    others = rnd(rows + 1, KVH * vd + 11, seed=23).to(tdt)        # another layer's rows, its values inside them
    positions = torch.cat([torch.arange(a, a + b) for a, b in zip(starts, new)] + [torch.zeros(1, dtype=torch.int64)]).int()
    row_seq = torch.cat([torch.full((b,), i) for i, b in enumerate(new)] + [torch.full((1,), -1)]).int()
    q_out = torch.zeros(rows + 1, H * pd, dtype=tdt, device="cuda")
    kp, vp = dev(kpool), dev(vpool)
    ops.qkv_rope_cache(q_out, kp, vp, dev(qkv), H * kd, KVH * kd, dev(bias) if biased else None, dev(positions), dev(row_seq),
                       i32(slots), dev(table), inv_freq(r, theta), r, rows + 1, H, KVH, pd, True, key_dim=kd, value_dim=vd,
                       unit_eps=eps, v_mix=(lam, dev(others)[:, 5:5 + KVH * vd]) if mixed else None)
    x = qkv[:rows].double() + (bias.double() if biased else 0.0)
    q, k = x[:, :H * kd].reshape(rows, H, kd), x[:, H * kd:(H + KVH) * kd].reshape(rows, KVH, kd)
    v = x[:, (H + KVH) * kd:].reshape(rows, KVH, vd)
    at = 0
    for s, n in zip(starts, new):
        q[at:at + n], k[at:at + n] = P.rotate(q[at:at + n], s, r, theta), P.rotate(k[at:at + n], s, r, theta)
        at += n
    q, k = P.rms(q, eps), P.rms(k, eps)
    if mixed:
        v = (1 - lam) * v + lam * others[:rows, 5:5 + KVH * vd].double().reshape(rows, KVH, vd)
    tol = 2e-5 if dtype == "float32" else 2 ** -7
    got = q_out.cpu()[:rows].double().reshape(rows, H, pd)
    assert torch.allclose(got[:, :, :kd], q, rtol=tol, atol=tol * 2) and bool((got[:, :, kd:] == 0).all())
    assert bool((q_out[rows] == 0).all())
    kp, vp = kp.cpu(), vp.cpu()
    for i in range(rows):
        page = table[slots[row_seq[i]], positions[i] // PAGE].item()
        assert torch.allclose(cached_k(kp, page, positions[i] % PAGE, pd)[:, :kd].double(), k[i], rtol=tol, atol=tol * 2)
        assert torch.allclose(cached_v(vp, page, positions[i] % PAGE, pd)[:, :vd].double(), v[i], rtol=tol, atol=tol * 2)
    # nothing else in the pools was touched
    assert (kp != 0).sum().item() <= rows * KVH * kd and (vp != 0).sum().item() <= rows * KVH * vd


# ------------------------------------------------------------------ whole models
# C1: every kind of layer; the layer whose values the others mix in is not the first attention; one memory head and
#     several, key and value widths that differ everywhere, partial rotations, a layer without feed-forward
# C2: sizes that are no multiples of 8; no rotation in the retention; no cap, no scaling; one head everywhere
# C3: whole-head rotations and equal widths; residual factor 1; memories wider than a block of 64 dims
MODELS = {
    "C1": model([layer("parallel", pair(attn(4, 2, 32, 16, 0.3, rot(500.0, 16, 3.0), 8.0), memory((0.9, 0.5, 0.995), 12, 20)), 72),
                 layer("attention", attn(3, 3, 16, 24, 0.5, rot(1000.0, 8)), 40),
                 layer("attention", attn(6, 2, 16, 8, 0.4, rot(10000.0, 16), v_mix=True)),
                 layer("retention", memory((0.97, 0.9985), 24, 8, rot(10000.0, 16)), 48),
                 layer("attention", attn(4, 2, 48, 8, 0.3, rot(10000.0, 48), v_mix=True), 56)],
                vocab=97, width=48, mult=0.6),
    "C2": model([layer("retention", memory((0.9,), 10, 6)), layer("attention", attn(1, 1, 10, 7, 0.6, v_mix=True), 30),
                 layer("parallel", pair(attn(3, 1, 12, 6, 0.5), memory((0.98,), 9, 13)), 22),
                 layer("attention", attn(5, 1, 14, 7, 0.5, rot(100.0, 6), v_mix=True), 18)],
                vocab=131, width=36, mult=1.3, eps=1e-4),
    "C3": model([layer("attention", attn(4, 4, 32, 32, 0.3, rot(10000.0, 32), v_mix=True), 64),
                 layer("retention", memory((0.95, 0.995, 0.6), 72, 136, rot(10000.0, 72)), 64),
                 layer("parallel", pair(attn(2, 1, 64, 64, 0.2, rot(10000.0, 64, 2.0), 4.0), memory((0.7, 0.99), 68, 80)), 64)],
                vocab=64, width=64, mult=1.0),
}


def sharpened(path, calm):
    """Makes the stored matrices larger than the random default, so that attention weights are far from uniform and a
    key that is wrongly seen or missed, a gate or a memory matters."""
    from hector_engine_amd.weights.safetensors_io import write_safetensors
    from safetensors.torch import load_file
    tensors = load_file(path)
    for k in tensors:
        f = 1.0
        if k.endswith((".left.q", ".left.k")):
            f = 5.0 if calm else 12.0
        elif tensors[k].dim() == 2 and k not in ("embed", "head"):
            f = 4.0 if calm else 8.0
        elif k.endswith(".b"):
            f = 10.0
        if f != 1.0:
            tensors[k] = (tensors[k].float() * f).to(torch.bfloat16)
    write_safetensors(path, tensors, {"format": "pt"})


@pytest.fixture(scope="module")
def folders(tmp_path_factory):
    """name -> model folder."""
    import hector_engine_amd  # noqa: F401
    from hector_engine_amd.registry import config_from_dict
    from hector_engine_amd.weights import write_random_model
    out = {}
    for i, (name, cfg) in enumerate(MODELS.items()):
        for calm in (False, True):
            folder = str(tmp_path_factory.mktemp(f"bobevik_{name}"))
            write_random_model(config_from_dict(json.loads(json.dumps(cfg))), 60 + i, folder, "bfloat16")
            sharpened(folder + "/model.safetensors", calm)
            out[name + "_calm" if calm else name] = folder
    return out


def variant(name, dtype):
    """The folder a precision is tested on: under bfloat16 the matrices are raised less (the rounding of q and k moves
    attention weights by the size of the scores times 2^-9)."""
    return name if dtype == "float32" else name + "_calm"


@pytest.fixture(scope="module")
def plain(folders):
    return {name: P.read_model(f) for name, f in folders.items()}


@pytest.fixture(scope="module")
def engines(folders):
    import hector_engine_amd as he
    cache = {}

    def get(name, dtype, **kw):
        key = (name, dtype, tuple(sorted(kw.items())))
        if key not in cache:
            opts = dict(max_tokens=4096, max_slots=8, max_seq_len=1024)
            opts.update(kw)
            cache[key] = he.Engine(folders[variant(name, dtype)], dtype=dtype, **opts)
        return cache[key]

    return get


class Want:
    """The plain logits of a request at some of its places, and how far they move when every matrix entry is off by a
    rounding to 8 bits (the largest of some draws; formed when asked for)."""

    def __init__(self, cfg, w, ids, rows=None):
        self.cfg, self.w, self.ids = cfg, w, list(ids)
        self.rows = list(range(len(self.ids))) if rows is None else [r % len(self.ids) for r in rows]
        self.logits = P.forward(cfg, w, self.ids)[0][self.rows]

    def at(self, rows):
        out = Want.__new__(Want)
        out.cfg, out.w, out.ids = self.cfg, self.w, self.ids
        out.rows = [self.rows[r] for r in rows]
        out.logits = self.logits[list(rows)]
        return out

    def moved(self, draws):
        worst = torch.zeros(len(self.rows), dtype=F64)
        for seed in range(draws):
            g = torch.Generator().manual_seed(seed)
            w = {k: t * (1 + 2.0 ** -9 * torch.randn(t.shape, generator=g, dtype=F64)) if t.dim() == 2 else t
                 for k, t in self.w.items()}
            worst = torch.maximum(worst, relative(P.forward(self.cfg, w, self.ids)[0][self.rows], self.logits))
        return worst


def relative(got, want):
    """Per position, the root mean square of the difference (mean taken off) against that of the logits."""
    d = got - want
    d = d - d.mean(-1, keepdim=True)
    w = want - want.mean(-1, keepdim=True)
    return d.pow(2).mean(-1).sqrt() / w.pow(2).mean(-1).sqrt()


def same(got, want: Want, dtype, tol32=3e-5, against=None):
    """float32: every logit within tol32 of the logits' size (or of 1); the angles of the rotation are 32-bit numbers, off
    by up to 6e-8 of themselves, so long requests are given more. bfloat16, per position (relative): a median of 2.5 % at
    most, and at most 5 % or three times what the plain logits of that place move by themselves. (A retention's head is
    divided by its own size: where an answer is almost nothing, as over the first tokens of a sequence, a rounding of q or
    k can turn it round.) against: compare with these logits in place of the plain ones, by the same bounds."""
    ref = want.logits if against is None else against.detach().cpu().double()
    got = got.detach().cpu().double()
    assert got.shape == ref.shape, (got.shape, ref.shape)
    if dtype == "float32":
        scale = ref.abs().max().item()
        err = (got - ref).abs().max().item()
        assert err <= tol32 * max(scale, 1.0), f"max error {err:.3g} above {tol32 * max(scale, 1.0):.3g} (logit scale {scale:.3g})"
        return
    r = relative(got, ref)
    assert bool(torch.isfinite(r).all())
    limit = torch.full_like(r, 0.05)
    for draws in (3, 24):
        if bool((r > limit).any()):
            limit = torch.clamp(3 * want.moved(draws), min=0.05)
    assert bool((r <= limit).all()), (r[r > limit], limit[r > limit])
    if len(r) >= 8:
        assert r.median().item() <= 0.025, r


def entry(slot, tokens, want):
    from hector_engine_amd.engine.engine import StepEntry
    return StepEntry(slot, list(tokens), list(want))


def test_the_folder_written_from_a_configuration_reads_back(folders):
    from hector_engine_amd.registry import load_config
    for name, folder in folders.items():
        assert load_config(folder).to_dict() == json.load(open(folder + "/config.json")) == MODELS[name.split("_")[0]]


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", list(MODELS))
def test_each_request_alone_and_whole(engines, plain, name, dtype):
    eng = engines(name, dtype)
    cfg, w = plain[variant(name, dtype)]
    for seed, n in enumerate([1, 2, 8, 9, 23, 64, 65, 150]):
        ids = rand_ids(cfg["vocab"], n, seed)
        s = eng.acquire()
        got = eng.step([entry(s, ids, range(n))])
        want = Want(cfg, w, ids)
        same(got, want, dtype)
        if dtype == "float32":
            argmax_agrees_where_clear(got, want.logits, 0.05 * want.logits.abs().max().item())
        eng.release(s)


def test_every_mechanism_matters_to_the_logits(plain, monkeypatch):
    """The models are such that leaving a mechanism out moves the logits by far more than the tests' bounds."""
    cfg, w = plain["C1"]
    ids = rand_ids(cfg["vocab"], 60, 3)
    want = P.forward(cfg, w, ids)[0]
    scale = want.abs().max().item()

    def moved(c=None, changed_w=None, **patches):
        with monkeypatch.context() as mp:
            for k, v in patches.items():
                mp.setattr(P, k, v)
            return (P.forward(c or cfg, changed_w or w, ids)[0] - want).abs().max().item() / scale

    def with_mixer(i, side=None, **changes):
        c = json.loads(json.dumps(cfg))
        m = c["layers"][i]["mixer"]
        (m[side] if side else m).update(changes)
        return c

    rotate, rms, capped = P.rotate, P.rms, P.capped
    assert moved(capped=lambda s, c: s) > 1e-3 and moved(with_mixer(0, "left", softcap=9.0)) > 1e-3
    assert moved(with_mixer(0, "left", rot=rot(500.0, 16))) > 1e-3                      # the frequencies' factor
    assert moved(rotate=lambda x, *a: x) > 1e-2
    assert moved(with_mixer(0, "right", decay=[0.9, 0.5, 0.99])) > 1e-3
    assert moved(with_mixer(3, decay=[0.97, 0.99])) > 1e-3
    assert moved(with_mixer(3, rot=None)) > 1e-3
    assert moved(with_mixer(4, v_mix=False)) > 1e-3
    assert moved(changed_w={**w, "l4.mix.vmix": 1.2 * w["l4.mix.vmix"]}) > 1e-3
    assert moved(changed_w={**w, "l2.mix.vmix": 1.2 * w["l2.mix.vmix"]}) == 0.0         # the first one's is unused
    for name in ("l0.mix.left.g", "l1.mix.g", "l3.mix.g", "l0.mix.right.g"):
        assert moved(changed_w={**w, name: 0 * w[name]}) > 1e-3
    for name in ("l0.mix.left.q.b", "l0.mix.left.v.b", "embed.norm", "l0.norm1b", "l3.norm2b"):
        assert moved(changed_w={**w, name: 0 * w[name]}) > 1e-3
    for name in ("l0.mix.left.out", "l0.mix.right.out", "l0.mix.right.norm"):
        assert moved(changed_w={**w, name: 0 * w[name] + 1.0}) > 1e-3
    assert moved({**cfg, "residual_mult": 0.7}) > 1e-2
    assert moved(gated_ff=lambda h, ww, pre: (P.silu(h @ ww[pre + "gate"].T) * (h @ ww[pre + "up"].T)) @ ww[pre + "down"].T) > 1e-3


@pytest.mark.parametrize("name", list(MODELS))
def test_the_stream_after_every_layer(engines, plain, name):
    eng = engines(name, "float32", use_graphs=False)
    cfg, w = plain[name]
    ids = rand_ids(cfg["vocab"], 70, 9)
    want, seen = [], []
    P.forward(cfg, w, ids, None, want)
    originals = [b.forward for b in eng.model.blocks]
    try:
        for b, orig in zip(eng.model.blocks, originals):
            def fwd(stream, ctx, cache, orig=orig):
                orig(stream, ctx, cache)
                seen.append(stream.materialize(ctx)[:ctx.rows].clone())
            b.forward = fwd
        s = eng.acquire()
        eng.step([entry(s, ids, [69])])
        eng.release(s)
    finally:
        for b, orig in zip(eng.model.blocks, originals):
            b.forward = orig
    assert len(seen) == len(want) == len(cfg["layers"])
    for got, ref in zip(seen, want):
        assert torch.allclose(got.cpu().double(), ref, rtol=0, atol=2e-5 * ref.abs().max().item())


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", list(MODELS))
def test_prompt_then_token_by_token_over_page_edges(engines, plain, name, dtype):
    eng = engines(name, dtype)
    cfg, w = plain[variant(name, dtype)]
    n, tail = 210, 150                  # the decoded positions 60..209 cross two page edges
    ids = rand_ids(cfg["vocab"], n, 11)
    want = Want(cfg, w, ids)
    s = eng.acquire()
    whole = eng.step([entry(s, ids, range(n))]).clone()
    eng.release(s)
    same(whole, want, dtype)
    s = eng.acquire()
    assert eng.step([entry(s, ids[:n - tail], [])]) is None
    dec = torch.cat([eng.step([entry(s, [t], [0])]).clone() for t in ids[n - tail:]])
    eng.release(s)
    same(dec, want.at(range(n - tail, n)), dtype)
    same(dec, want.at(range(n - tail, n)), dtype, against=whole[n - tail:])


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", list(MODELS))
@pytest.mark.parametrize("cuts", [[2] * 40, [3, 2, 61, 17, 64, 2, 70], [1, 1, 2, 1, 25, 47, 48, 2], [128, 2, 2, 65], [8, 9, 7, 63, 10]])
def test_prompts_fed_in_portions(engines, plain, name, dtype, cuts):
    eng = engines(name, dtype)
    cfg, w = plain[variant(name, dtype)]
    n = sum(cuts)
    ids = rand_ids(cfg["vocab"], n, 12)
    want = Want(cfg, w, ids)
    s = eng.acquire()
    whole = eng.step([entry(s, ids, range(n))]).clone()
    eng.release(s)
    s = eng.acquire()
    parts, at = [], 0
    for c in cuts:
        parts.append(eng.step([entry(s, ids[at:at + c], range(c))]).clone())
        at += c
    eng.release(s)
    got = torch.cat(parts)
    same(got, want, dtype)
    same(got, want, dtype, against=whole)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", list(MODELS))
def test_unequal_batches_equal_each_request_alone_and_slots_are_used_again(engines, plain, name, dtype):
    eng = engines(name, dtype, max_slots=4)
    cfg, w = plain[variant(name, dtype)]
    free = eng.cache.free_pages
    for round_no, lengths in enumerate([[1, 67, 140, 25], [90, 3, 49], [200, 2, 2, 64]]):
        prompts = [rand_ids(cfg["vocab"], n, 20 * round_no + i) for i, n in enumerate(lengths)]
        decode = 12
        full = [p + rand_ids(cfg["vocab"], decode - i, 500 + i) for i, p in enumerate(prompts)]   # shorter ones end earlier
        want = [Want(cfg, w, f, range(len(p) - 1, len(f))) for p, f in zip(prompts, full)]
        slots = [eng.acquire() for _ in prompts]
        got = [[] for _ in prompts]
        logits = eng.step([entry(s, p, [len(p) - 1]) for s, p in zip(slots, prompts)])
        for i in range(len(prompts)):
            got[i].append(logits[i:i + 1].clone())
        for t in range(decode):
            live = [i for i in range(len(prompts)) if len(prompts[i]) + t < len(full[i])]
            if not live:
                break
            logits = eng.step([entry(slots[i], [full[i][len(prompts[i]) + t]], [0]) for i in live])
            for j, i in enumerate(live):
                got[i].append(logits[j:j + 1].clone())
        for i, s in enumerate(slots):
            eng.release(s)          # the next round's requests take these slots, pages and memories again
            same(torch.cat(got[i]), want[i], dtype)
    assert eng.cache.free_pages == free


@pytest.mark.parametrize("dtype", DTYPES)
def test_batches_of_every_kernel_size(engines, plain, dtype):
    """Decoding batches of 1, 3, 17 and 70 requests: products of up to 16, of up to 64 and of more rows."""
    eng = engines("C1", dtype, max_slots=72, max_tokens=8192)
    cfg, w = plain[variant("C1", dtype)]
    for batch in (1, 3, 17, 70):
        prompts = [rand_ids(cfg["vocab"], 3 + i % 5, 900 + i) for i in range(batch)]
        tails = [rand_ids(cfg["vocab"], 4, 950 + i) for i in range(batch)]
        slots = [eng.acquire() for _ in prompts]
        got = [eng.step([entry(s, p, [len(p) - 1]) for s, p in zip(slots, prompts)]).clone()]
        for t in range(4):
            got.append(eng.step([entry(s, [tail[t]], [0]) for s, tail in zip(slots, tails)]).clone())
        for s in slots:
            eng.release(s)
        for i in range(0, batch, 4):
            n = len(prompts[i])
            same(torch.stack([g[i] for g in got]), Want(cfg, w, prompts[i] + tails[i], range(n - 1, n + 4)), dtype)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", list(MODELS))
def test_a_mixed_step_of_a_prompt_and_decoding_requests(engines, plain, name, dtype):
    eng = engines(name, dtype)
    cfg, w = plain[variant(name, dtype)]
    a, b, c = rand_ids(cfg["vocab"], 80, 30), rand_ids(cfg["vocab"], 137, 31), rand_ids(cfg["vocab"], 20, 32)
    sa, sb, sc = (eng.acquire() for _ in range(3))
    eng.step([entry(sa, a[:79], []), entry(sc, c[:18], [])])
    got = eng.step([entry(sa, a[79:], [0]), entry(sb, b, range(137)), entry(sc, c[18:], [0, 1])])
    same(got[:1], Want(cfg, w, a, [79]), dtype)
    same(got[1:138], Want(cfg, w, b), dtype)
    same(got[138:], Want(cfg, w, c, [18, 19]), dtype)
    for s in (sa, sb, sc):
        eng.release(s)


@pytest.mark.parametrize("dtype", DTYPES)
def test_a_long_request_and_long_decoding(engines, plain, dtype):
    eng = engines("C1", dtype)
    cfg, w = plain[variant("C1", dtype)]
    n = 700
    ids = rand_ids(cfg["vocab"], n, 41)
    want = Want(cfg, w, ids, [0, 63, 64, 399, *range(400, n)])
    s = eng.acquire()
    got = [eng.step([entry(s, ids[:400], [0, 63, 64, 399])]).clone()]
    got += [eng.step([entry(s, [t], [0])]).clone() for t in ids[400:]]
    eng.release(s)
    same(torch.cat(got), want, dtype, 1e-4)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("far", [0, 1, 63, 64, 127, 128, 255])
def test_a_token_far_back_answers(tmp_path, dtype, far):
    """Queries and keys are made the same rows of the input (k's matrix is q's), without rotation: an earlier occurrence
    of the asking token stands out by 16 in the unit attention and by the cap in the capped one. The rare token stands once far
    back (the first positions, both sides of page borders) and asks 150 to 300 tokens later, in the prompt and decoded."""
    import hector_engine_amd as he
    from hector_engine_amd.registry import config_from_dict
    from hector_engine_amd.weights import write_random_model
    from hector_engine_amd.weights.safetensors_io import write_safetensors
    from safetensors.torch import load_file
    cfg = model([layer("attention", attn(2, 2, 16, 16, 1.0, v_mix=True)),
                 layer("parallel", pair(attn(1, 1, 16, 24, 1.0, None, 15.0), memory((0.998, 0.9), 8, 8))),
                 layer("attention", attn(2, 2, 16, 16, 1.0, v_mix=True), 32)], 80, 32, 0.8)
    folder = str(tmp_path)
    write_random_model(config_from_dict(json.loads(json.dumps(cfg))), 5, folder, "bfloat16")
    path = folder + "/model.safetensors"
    t = load_file(path)
    for k in t:
        if t[k].dim() == 2 and k not in ("embed", "head"):
            t[k] = (t[k].float() * 6).to(torch.bfloat16)
    for l in ("l0.mix.", "l2.mix."):
        t[l + "k"] = t[l + "q"].clone()
    t["l1.mix.left.q"] = (t["l1.mix.left.q"].float() * 2).to(torch.bfloat16)
    t["l1.mix.left.k"], t["l1.mix.left.k.b"] = t["l1.mix.left.q"].clone(), t["l1.mix.left.q.b"].clone()
    write_safetensors(path, t, {"format": "pt"})
    c, w = P.read_model(folder)
    n, asks = 420, (300, 330, 401, 419)
    ids = [i % 70 for i in rand_ids(70, n, 5)]
    for at in (far, *asks):
        ids[at] = 77
    want = Want(c, w, ids)
    # the planted token is what the first asking one reads: with another one in its place the logits move
    other = list(ids)
    other[far] = 78
    d = (P.forward(c, w, other)[0] - want.logits)[300].abs().max().item() / want.logits.abs().max().item()
    assert d > 0.05, d
    eng = he.Engine(folder, dtype=dtype, max_tokens=2048, max_slots=2, max_seq_len=512)
    s = eng.acquire()
    whole = eng.step([entry(s, ids, range(n))]).clone()
    eng.release(s)
    same(whole, want, dtype)
    same(whole[list(asks)], want.at(asks), dtype)
    s = eng.acquire()
    eng.step([entry(s, ids[:290], [])])
    dec = torch.cat([eng.step([entry(s, [x], [0])]).clone() for x in ids[290:]])
    eng.release(s)
    same(dec, want.at(range(290, n)), dtype)
    same(dec[[a - 290 for a in asks]], want.at(asks), dtype)


@pytest.mark.parametrize("name", list(MODELS))
def test_greedy_generation_through_the_library(folders, plain, name):
    import hector_engine_amd as he
    cfg, w = plain[name]
    prompts = [rand_ids(cfg["vocab"], n, 70 + i) for i, n in enumerate([5, 30, 61])]
    steps = 40
    want = [P.greedy(cfg, w, p, steps) for p in prompts]
    eng = he.Engine(folders[name], dtype="float32", max_tokens=2048, max_seq_len=512)
    got = he.generate(eng, prompts, max_new_tokens=steps, stop_ids=())
    assert [r.tokens for r in got] == want
    small = he.Engine(folders[name], dtype="float32", max_tokens=2048, max_slots=2, max_seq_len=512)
    assert [r.tokens for r in he.generate(small, prompts, max_new_tokens=steps, stop_ids=())] == want
    assert small.cache.free_pages == small.cache.num_pages
    cfg, w = plain[name + "_calm"]
    want = [P.greedy(cfg, w, p, steps) for p in prompts]
    eng16 = he.Engine(folders[name + "_calm"], dtype="bfloat16", max_tokens=2048, max_seq_len=512)
    for p, r, t in zip(prompts, he.generate(eng16, prompts, max_new_tokens=steps, stop_ids=()), want):
        seq = list(p)
        for x, y in zip(r.tokens, t):
            if x != y:
                logits = P.forward(cfg, w, seq)[0][-1]
                top = logits.topk(2).values
                assert (top[0] - top[1]).item() < 0.1 * logits.std().item() + 1e-3      # a near tie
                break
            seq.append(x)


def test_the_command_line_and_the_trace_replay_serve_it(folders, plain, tmp_path):
    import numpy as np
    from tests.conftest import ROOT
    cfg, w = plain["C1"]
    exe = os.path.join(ROOT, "bin", "hector_generate")
    out = subprocess.run([sys.executable, exe, folders["C1"], "5,17,3;9,2,77,13", "6", "--dtype", "float32",
                          "--stop-ids", ""], capture_output=True, text=True, timeout=180)
    assert out.returncode == 0, out.stderr
    for i, p in enumerate(([5, 17, 3], [9, 2, 77, 13])):
        assert f"[{i}] prompt" in out.stdout and ",".join(map(str, P.greedy(cfg, w, p, 6))) in out.stdout
    assert "Bobevik" in out.stdout
    reqs = {"a": rand_ids(cfg["vocab"], 4, 1), "b": rand_ids(cfg["vocab"], 68, 2), "c": rand_ids(cfg["vocab"], 133, 3)}
    steps = [{"step": 0, "entries": [{"id": k, "tokens": v[:-3], "want": [len(v) - 4]} for k, v in reqs.items()], "end": []}]
    for t in range(3):
        steps.append({"step": t + 1, "entries": [{"id": k, "tokens": [v[len(v) - 3 + t]], "want": [0]} for k, v in reqs.items()],
                      "end": list(reqs) if t == 2 else []})
    for dtype in DTYPES:
        out_dir = str(tmp_path / dtype)
        cfg, w = plain[variant("C1", dtype)]
        proc = subprocess.run([sys.executable, os.path.join(ROOT, "bin", "trace_run"), "--model", folders[variant("C1", dtype)],
                               "--dtype", dtype, "--out", out_dir, "--max-tokens", "205"],
                              input="".join(json.dumps(s) + "\n" for s in steps), capture_output=True, text=True, timeout=180)
        assert proc.returncode == 0, proc.stderr
        assert [l for l in proc.stdout.splitlines() if l.startswith("done")] == [f"done {i}" for i in range(4)]
        for s in range(4):
            got = torch.from_numpy(np.fromfile(os.path.join(out_dir, f"{s}.f32"), dtype="<f4").reshape(3, -1).copy())
            for i, v in enumerate(reqs.values()):
                same(got[i:i + 1], Want(cfg, w, v, [len(v) - 4 + s]), dtype)


# ------------------------------------------------------------------ random configurations
def random_configuration(rng):
    """Layers of any kind in any order, with sizes drawn from small sets that hold odd ones, ones, and pairs that are
    equal as well as pairs that differ."""
    def rotation(dim, may_scale):
        r = rng.choice([None] + [r for r in (2, 4, 8, 12, 16, 24, 32, 64) if r <= dim])
        return None if r is None else rot(rng.choice([100.0, 10000.0, 1000000.0]), r,
                                          rng.choice([2.0, 3.5]) if may_scale and rng.random() < 0.7 else None)

    shared = (rng.choice([1, 2, 3]), rng.choice([4, 7, 8, 20, 32]))      # kv heads and value width of the mixing layers
    layers = []
    for _ in range(rng.randint(1, 5)):
        kind = rng.choice(["attention", "retention", "parallel"])
        dim = rng.choice([4, 8, 12, 16, 24, 32, 72])
        if kind == "attention":
            mixes = rng.random() < 0.6
            kv, e = shared if mixes else (rng.choice([1, 2, 3]), rng.choice([4, 8, 20, 32, 40]))
            mixer = attn(kv * rng.choice([1, 2, 3]), kv, dim, e, rng.choice([0.2, 0.4]), rotation(dim, False), v_mix=mixes)
        else:
            H = rng.choice([1, 2, 3, 5])
            mixer = memory([rng.choice([0.5, 0.9, 0.99, 0.998, 1.0 - 2.0 ** -10]) for _ in range(H)],
                           rng.choice([4, 5, 12, 16, 40, 66, 72]), rng.choice([1, 4, 6, 16, 36, 68]))
            if kind == "retention":
                r = rotation(mixer["dim"], False)
                if r is not None and r["dims"] <= mixer["dim"]:
                    mixer["rot"] = r
            else:
                kv = rng.choice([1, 2])
                left = attn(kv * rng.choice([1, 2, 4]), kv, dim, rng.choice([4, 8, 20, 40]), rng.choice([0.2, 0.4]),
                            rotation(dim, True), rng.choice([None, 3.0, 20.0]))
                mixer = pair(left, mixer)
        layers.append(layer(kind, mixer, rng.choice([None, 6, 16, 40, 72])))
    return model(layers, rng.choice([50, 97, 130]), rng.choice([24, 36, 40, 64, 72, 96]), rng.choice([0.5, 1.0, 0.7]),
                 rng.choice([1e-6, 1e-5]))


@pytest.mark.parametrize("dtype,seed", [("float32", s) for s in range(14)] + [("bfloat16", s) for s in range(14, 26)])
def test_random_configurations(tmp_path, dtype, seed):
    """A prompt batch in portions, then one-token steps of the batch, twice through the same slots, against the plain
    implementation; in 32-bit, and with other configurations under bfloat16 (whose kernels have needs of their own: whole
    pieces of 8, padded heads)."""
    import random
    import hector_engine_amd as he
    from hector_engine_amd.registry import config_from_dict
    from hector_engine_amd.weights import write_random_model
    rng = random.Random(seed)
    cfg = random_configuration(rng)
    folder = str(tmp_path)
    write_random_model(config_from_dict(json.loads(json.dumps(cfg))), seed, folder, "bfloat16")
    sharpened(folder + "/model.safetensors", dtype == "bfloat16")
    c, w = P.read_model(folder)
    lens = [rng.choice([1, 2, 5, 63, 64, 65, 130]) for _ in range(3)]
    fulls = [rand_ids(c["vocab"], n + 6, seed * 10 + i) for i, n in enumerate(lens)]
    wants = [Want(c, w, f) for f in fulls]
    eng = he.Engine(folder, dtype=dtype, max_tokens=2048, max_slots=4, max_seq_len=512)
    for _ in range(2):
        slots = [eng.acquire() for _ in fulls]
        got = [[] for _ in fulls]
        cut = [max(1, n // 2) for n in lens]
        logits = eng.step([entry(s, f[:k], range(k)) for s, f, k in zip(slots, fulls, cut)])
        at = 0
        for i, k in enumerate(cut):
            got[i].append(logits[at:at + k].clone())
            at += k
        for i, (s, f, k, n) in enumerate(zip(slots, fulls, cut, lens)):
            if n > k:
                got[i].append(eng.step([entry(s, f[k:n], range(n - k))]).clone())
        for t in range(6):
            logits = eng.step([entry(s, [f[n + t]], [0]) for s, f, n in zip(slots, fulls, lens)])
            for i in range(len(fulls)):
                got[i].append(logits[i:i + 1].clone())
        for s in slots:
            eng.release(s)
        for g, want in zip(got, wants):
            same(torch.cat(g), want, dtype, 6e-5)
