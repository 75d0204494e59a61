"""A plain, slow Dofipel in float64 torch on the CPU, one function per mechanism, written from the
design's equations and sharing nothing with the library. It reads config.json with `json` and
model.safetensors with the safetensors package.

Notation: x the residual stream [T, D]; p the position of a token in its sequence (from 0); h = norm1(x), the
input of a layer's mixer and of its feed-forward alike.
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

def dynamic_tanh(x, w, name):
    """tanh(alpha x) * weight + bias, element by element: alpha a stored number, weight and bias stored vectors."""
    return torch.tanh(w[name + ".alpha"] * x) * w[name] + w[name + ".b"]


def rms(x, eps):
    """x / sqrt(mean(x^2) + eps) over the last axis."""
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def gelu_tanh(z):
    return 0.5 * z * (1.0 + torch.tanh(math.sqrt(2.0 / math.pi) * (z + 0.044715 * z ** 3)))


def silu(z):
    return z / (1.0 + torch.exp(-z))


# ---- attention with a distance table ------------------------------------------------

def bucket_of(n: int, buckets: int, far: int) -> int:
    """The row of the table for distance n >= 0: the first half of the rows are the distances 0, 1, 2, ...; the
    others divide [half, far) into steps of equal ratio, and the last row takes all that is farther.
    floor(m ln(n / half) / ln(far / half)) >= k exactly when (n / half)^m >= (far / half)^k: in integers."""
    half = buckets // 2
    if n < half:
        return n
    m = buckets - half
    k = 0
    while k + 1 < m and n ** m * half ** (k + 1) >= far ** (k + 1) * half ** m:
        k += 1
    return min(buckets - 1, half + k)


def distance_bias(table, far: int, reach: int):
    """[reach, H]: row n is the bias of a key n positions back."""
    B = table.shape[0]
    return torch.stack([table[bucket_of(n, B, far)] for n in range(reach)])


def capped_scores(q, k, scale: float, cap: float):
    """cap * tanh(q . k * scale / cap) for all pairs of rows (cap 0: no cap)."""
    s = (q @ k.T) * scale
    return cap * torch.tanh(s / cap) if cap else s


def window_attention(q, k, v, scale, cap, table, far, sinks, window, first_position=0):
    """q [Tq, H, d] at the positions first_position.., k [Tk, G, d] and v [Tk, G, e] at the positions 0..: query i
    sees the keys j with 0 <= i - j < window (window 0: every j <= i); the score is capped, then the table's entry for
    the distance is added; exp(sink_h) joins the denominator of head h (sinks None: it does not)."""
    Tq, H, _ = q.shape
    Tk, G, e = v.shape
    back = first_position + torch.arange(Tq)[:, None] - torch.arange(Tk)[None, :]
    seen = back >= 0
    if window:
        seen &= back < window
    bias = distance_bias(table, far, int(back.max()) + 1) if table is not None else None
    out = torch.zeros((Tq, H, e), dtype=F64)
    for h in range(H):
        g = h // (H // G)
        s = capped_scores(q[:, h], k[:, g], scale, cap)
        if bias is not None:
            s = s + bias[back.clamp(min=0), h]
        s = s.masked_fill(~seen, -math.inf)
        top = s.max(-1).values
        if sinks is not None:
            top = torch.maximum(top, sinks[h])
        p = torch.exp(s - top[:, None])
        total = p.sum(-1)
        if sinks is not None:
            total = total + torch.exp(sinks[h] - top)
        out[:, h] = (p @ v[:, g]) / total[:, None]
    return out


def attention(h, w, pre, m):
    T = h.shape[0]
    H, G, d, e = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q = (h @ w[pre + "q"].T).reshape(T, H, d)
    k = (h @ w[pre + "k"].T).reshape(T, G, d)
    v = (h @ w[pre + "v"].T).reshape(T, G, e)
    out = window_attention(q, k, v, m["scale"], m.get("softcap", 0.0), w[pre + "rel"], m["bias_max"], w[pre + "sink"],
                           (m.get("mask") or {}).get("size", 0))
    return out.reshape(T, H * e) @ w[pre + "o"].T


# ---- latent attention ---------------------------------------------------------------

def rotate_pairs(x, positions, r: int, base: float):
    """x [T, heads, d]: of every head's first r dims, dims 2i and 2i + 1 turn together by p * base^(-2i/r)."""
    out = x.clone()
    p = torch.tensor(positions, dtype=F64)[:, None]
    for i in range(r // 2):
        c, s = torch.cos(p * base ** (-2.0 * i / r)), torch.sin(p * base ** (-2.0 * i / r))
        u, v = x[:, :, 2 * i], x[:, :, 2 * i + 1]
        out[:, :, 2 * i] = u * c - v * s
        out[:, :, 2 * i + 1] = v * c + u * s
    return out


def latents(h, w, pre, m, eps, positions):
    """(c [T, rank], the rotated key part [T, r]): what a sequence keeps per token."""
    rank, r = m["kv_rank"], m["rot_dim"]
    down = h @ w[pre + "dkv"].T
    c = rms(down[:, :rank], eps) * w[pre + "dkv.norm"]
    k_rot = rotate_pairs(down[:, rank:].reshape(len(h), 1, r), positions, r, m["rot"]["base"])[:, 0] if r else down[:, rank:]
    return c, k_rot


def latent_attention(h, w, pre, m, eps, positions, kept):
    """kept: (c, rotated key part) of the layer whose latents this one reads (its own or another's)."""
    T = h.shape[0]
    H, d, r, e = m["heads"], m["dim"], m["rot_dim"], m["vdim"]
    c, k_rot = kept
    q = (h @ w[pre + "q"].T).reshape(T, H, d + r)
    q_rot = rotate_pairs(q[:, :, d:], positions, r, m["rot"]["base"]) if r else q[:, :, d:]
    k_plain = (c @ w[pre + "uk"].T).reshape(-1, H, d)
    v = (c @ w[pre + "uv"].T).reshape(-1, H, e)
    ahead = torch.arange(len(c))[None, :] > torch.tensor(positions)[:, None]
    out = torch.zeros((T, H, e), dtype=F64)
    for head in range(H):
        s = (q[:, head, :d] @ k_plain[:, head].T + q_rot[:, head] @ k_rot.T) * m["scale"]
        out[:, head] = torch.softmax(s.masked_fill(ahead, -math.inf), -1) @ v[:, head]
    gated = out.reshape(T, H * e) * torch.sigmoid(h @ w[pre + "g"].T)
    return gated @ w[pre + "o"].T


# ---- feed-forwards ----------------------------------------------------------------

def gated_ff(h, w, pre, act):
    return (act(h @ w[pre + "gate"].T) * (h @ w[pre + "up"].T)) @ w[pre + "down"].T


def routed_ff(h, w, pre, mlp):
    """The `top` experts of the largest router logits (bias included), weighted by the softmax over those logits."""
    z = h @ w[pre + "router"].T + w[pre + "router.b"]
    out = torch.zeros_like(h)
    for t in range(h.shape[0]):
        chosen = torch.topk(z[t], mlp["router"]["top"]).indices
        share = torch.softmax(z[t][chosen], 0)
        for s, e in zip(share, chosen.tolist()):
            out[t] = out[t] + s * gated_ff(h[t:t + 1], w, f"{pre}e{e}.", silu)[0]
    if mlp.get("shared"):
        out = out + gated_ff(h, w, pre + "shared.", silu)
    return out


# ---- the model --------------------------------------------------------------------

def forward(cfg, w, tokens, streams=None):
    """Logits [T, vocab] of one sequence from its first token on. streams: a list that receives the residual
    stream after every layer."""
    eps = cfg["norm"]["eps"]
    positions = list(range(len(tokens)))
    x = w["embed"][torch.tensor(tokens, dtype=torch.long)]
    kept = {}
    for i, layer in enumerate(cfg["layers"]):
        pre, m = f"l{i}.mix.", layer["mixer"]
        h = dynamic_tanh(x, w, f"l{i}.norm1")
        if layer["type"] == "latent_attention":
            if m.get("kv_from") is None:
                kept[i] = latents(h, w, pre, m, eps, positions)
            y = latent_attention(h, w, pre, m, eps, positions, kept[i if m.get("kv_from") is None else m["kv_from"]])
        elif layer["type"] == "attention":
            y = attention(h, w, pre, m)
        else:
            raise ValueError(layer["type"])
        mlp = layer.get("mlp")
        if mlp:
            pre = f"l{i}.mlp."
            y = y + (gated_ff(h, w, pre, gelu_tanh) if mlp["kind"] == "dense" else routed_ff(h, w, pre, mlp))
        x = x + y
        if streams is not None:
            streams.append(x)
    return dynamic_tanh(x, w, "final.norm") @ w["embed"].T * cfg["logit_scale"]


def greedy(cfg, w, prompt, new_tokens: int):
    tokens = list(prompt)
    for _ in range(new_tokens):
        tokens.append(int(forward(cfg, w, tokens)[-1].argmax()))
    return tokens[len(prompt):]
