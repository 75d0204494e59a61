"""A plain, slow Bobevik in float64 torch on the CPU, one function per mechanism, written from
the design's equations and sharing nothing with the library. It reads config.json with `json`
and model.safetensors with the safetensors package.

Notation: x the residual stream [T, D]; p the position of a token in its sequence (from 0).
Attention: H query heads, G key/value heads, key width d, value width e, r rotated dims.
Decaying memory: H heads with a constant decay each and a memory S [d, e] per head.
"""
from __future__ import annotations

import json
import math
import os

import torch

F64 = torch.float64


def read_model(folder: str):
    """(config dict, {name: float64 tensor})."""
    from safetensors.torch import load_file
    with open(os.path.join(folder, "config.json")) as f:
        cfg = json.load(f)
    w = {k: (v.to(F64) if v.is_floating_point() else v) for k, v in
         load_file(os.path.join(folder, "model.safetensors")).items()}
    return cfg, w


# ---- small functions -------------------------------------------------------------

def rms(x, eps):
    """x / sqrt(mean(x^2) + eps) over the last axis."""
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def shifted_norm(x, w, eps):
    """The model's norm: its weight is stored as the difference from one."""
    return rms(x, eps) * (1.0 + w)


def silu(z):
    return z * torch.sigmoid(z)


def capped(s, c: float):
    return c * torch.tanh(s / c)


# ---- rotation ---------------------------------------------------------------------

def rotate(x, first: int, r: int, base: float, factor: float = 1.0):
    """x [T, heads, d] at positions first, first + 1, ...; of the first r dims of every head the pair (i, i + r/2)
    turns by p * base^(-2i/r) / factor; the other dims stay."""
    out = x.clone()
    p = torch.arange(first, first + x.shape[0], dtype=F64)
    for i in range(r // 2):
        a = p * (base ** (-2.0 * i / r) / factor)
        c, s = torch.cos(a)[:, None], torch.sin(a)[:, None]
        u, v = x[:, :, i], x[:, :, i + r // 2]
        out[:, :, i] = u * c - v * s
        out[:, :, i + r // 2] = v * c + u * s
    return out


def rotate_by(x, first: int, rot):
    if not rot:
        return x
    return rotate(x, first, rot["dims"], rot["base"], (rot.get("scaling") or {}).get("factor", 1.0))


# ---- attention ---------------------------------------------------------------------

def softmax_attention(q, k, v, scale, first_pos: int, softcap: float = 0.0):
    """q [T, d] at positions first_pos.., k [S, d], v [S, e] at positions 0..: causal."""
    s = (q @ k.T) * scale
    if softcap:
        s = capped(s, softcap)
    seen = torch.arange(k.shape[0])[None, :] <= first_pos + torch.arange(q.shape[0])[:, None]
    s = torch.where(seen, s, torch.full_like(s, -math.inf))
    e = torch.exp(s - s.amax(-1, keepdim=True))
    return (e / e.sum(-1, keepdim=True)) @ v


def attention_mixer(h, w, pre, m, eps, *, biases: bool, unit: bool, v_first=None, mix=None, carry=None):
    """h [T, D] -> ([T, D], (k, v) of the whole sequence, this layer's own values of the new tokens).
    biases: q, k and v have them. unit: q and k are divided by their root mean square behind the rotation.
    With mix (a number) the values are (1 - mix) v + mix v_first. carry = (k [S, G, d], v [S, G, e])."""
    T = h.shape[0]
    H, G, d, e = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q, k, v = h @ w[pre + "q"].T, h @ w[pre + "k"].T, h @ w[pre + "v"].T
    if biases:
        q, k, v = q + w[pre + "q.b"], k + w[pre + "k.b"], v + w[pre + "v.b"]
    q, k, v = q.reshape(T, H, d), k.reshape(T, G, d), v.reshape(T, G, e)
    first = 0 if carry is None else carry[0].shape[0]
    q, k = rotate_by(q, first, m.get("rot")), rotate_by(k, first, m.get("rot"))
    if unit:
        q, k = rms(q, eps), rms(k, eps)
    own = v
    if mix is not None:
        v = (1.0 - mix) * v + mix * v_first
    if carry is not None:
        k, v = torch.cat([carry[0], k]), torch.cat([carry[1], v])
    heads = [softmax_attention(q[:, a], k[:, a // (H // G)], v[:, a // (H // G)], m["scale"], first, m.get("softcap") or 0.0)
             for a in range(H)]
    y = torch.stack(heads, 1) * torch.sigmoid(h @ w[pre + "g"].T)[:, :, None]
    return y.reshape(T, H * e) @ w[pre + "o"].T, (k, v), own


# ---- memories with a constant decay -------------------------------------------------

def decay_scan(q, k, v, decay, state=None):
    """q, k [T, H, d], v [T, H, e], decay [H]; state S [H, d, e] or None for zeros:
    S <- decay S + k v^T, y = S^T q. Returns (y [T, H, e], S)."""
    T, H, d = q.shape
    S = torch.zeros((H, d, v.shape[2]), dtype=F64) if state is None else state.clone()
    g = torch.tensor(decay, dtype=F64)[:, None, None]
    y = torch.zeros((T, H, v.shape[2]), dtype=F64)
    for t in range(T):
        S = g * S + k[t, :, :, None] * v[t, :, None, :]
        y[t] = (q[t, :, :, None] * S).sum(1)
    return y, S


def retention_mixer(h, w, pre, m, eps, carry=None):
    """h [T, D] -> [T, D]; carry = (tokens before, S)."""
    T = h.shape[0]
    H, d, e = m["heads"], m["dim"], m["vdim"]
    first, S = (0, None) if carry is None else carry
    q = rotate_by((h @ w[pre + "q"].T).reshape(T, H, d), first, m.get("rot"))
    k = rotate_by((h @ w[pre + "k"].T).reshape(T, H, d), first, m.get("rot")) * d ** -0.5
    v = (h @ w[pre + "v"].T).reshape(T, H, e)
    y, S = decay_scan(q, k, v, m["decay"], S)
    y = rms(y, eps).reshape(T, H * e) * silu(h @ w[pre + "g"].T)
    return y @ w[pre + "o"].T, (first + T, S)


def lightning_mixer(h, w, pre, m, eps, carry=None):
    """h [T, D] -> [T, D]; carry = S."""
    T = h.shape[0]
    H, d, e = m["heads"], m["dim"], m["vdim"]
    q = silu(h @ w[pre + "q"].T).reshape(T, H, d)
    k = silu(h @ w[pre + "k"].T).reshape(T, H, d)
    v = silu(h @ w[pre + "v"].T).reshape(T, H, e)
    y, S = decay_scan(q, k, v, m["decay"], carry)
    y = rms(y.reshape(T, H * e), eps) * w[pre + "norm"] * torch.sigmoid(h @ w[pre + "g"].T)
    return y @ w[pre + "o"].T, S


def side_by_side(h, w, pre, m, eps, carry=None):
    left, c_left, _ = attention_mixer(h, w, pre + "left.", m["left"], eps, biases=True, unit=False,
                                      carry=None if carry is None else carry[0])
    right, c_right = lightning_mixer(h, w, pre + "right.", m["right"], eps, None if carry is None else carry[1])
    return 0.5 * (rms(left, eps) * w[pre + "left.out"] + rms(right, eps) * w[pre + "right.out"]), (c_left, c_right)


# ---- feed-forward ------------------------------------------------------------------

def gated_ff(h, w, pre):
    return (torch.clamp(h @ w[pre + "gate"].T, min=0.0) * (h @ w[pre + "up"].T)) @ w[pre + "down"].T


# ---- the model -----------------------------------------------------------------------

def forward(cfg, w, tokens, carry=None, layers_out=None):
    """Logits [T, vocab] of `tokens` that continue the sequence `carry` describes (None: its
    start), and the new carry: one entry for every layer."""
    eps, mult = cfg["norm"]["eps"], cfg.get("residual_mult", 1.0)
    x = shifted_norm(w["embed"][torch.tensor(tokens)], w["embed.norm"], eps)
    v_first = None
    new_carry = []
    for l, layer in enumerate(cfg["layers"]):
        pre, m = f"l{l}.", layer["mixer"]
        h = shifted_norm(x, w[pre + "norm1"], eps)
        c = None if carry is None else carry[l]
        if layer["type"] == "attention":
            mixes = bool(m.get("v_mix"))
            mix = w[pre + "mix.vmix"] if mixes and v_first is not None else None
            y, c, own = attention_mixer(h, w, pre + "mix.", m, eps, biases=False, unit=True, v_first=v_first, mix=mix, carry=c)
            if mixes and v_first is None:
                v_first = own
        elif layer["type"] == "retention":
            y, c = retention_mixer(h, w, pre + "mix.", m, eps, c)
        else:
            y, c = side_by_side(h, w, pre + "mix.", m, eps, c)
        new_carry.append(c)
        x = x + mult * shifted_norm(y, w[pre + "norm1b"], eps)
        if layer.get("mlp") is not None:
            y = gated_ff(shifted_norm(x, w[pre + "norm2"], eps), w, pre + "mlp.")
            x = x + mult * shifted_norm(y, w[pre + "norm2b"], eps)
        if layers_out is not None:
            layers_out.append(x.clone())
    return shifted_norm(x, w["final.norm"], eps) @ w["head"].T, new_carry


def greedy(cfg, w, prompt, steps: int) -> list[int]:
    """`steps` tokens after `prompt`, each the argmax of the last logits (lowest id on ties)."""
    logits, carry = forward(cfg, w, list(prompt))
    out = []
    for _ in range(steps):
        out.append(int(torch.argmax(logits[-1]).item()))
        logits, carry = forward(cfg, w, [out[-1]], carry)
    return out
