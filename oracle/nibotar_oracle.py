"""CPU oracle for Nibotar models: plain, slow torch, one function per mechanism.

TEST INFRASTRUCTURE ONLY, like the other oracles of this package: only tests and scripts that check the product import
it, and it shares no code with it.  A model is (config dict, weights dict); the weights are torch tensors under the
checkpoint's names, and everything is computed in `dtype` (float32 or float64).  There is no cache: `forward` evaluates a
whole sequence, and a decoded token is checked against the last row of the sequence that ends with it.

Parity pinning: parity unpinned by a third implementation (no library has the design).  The functions are the equations
written out, loops over heads and positions where that is plainest; tests/test_nibotar_oracle.py holds closed forms.
"""
from __future__ import annotations

import math
from typing import Dict, List, Optional, Sequence

import torch


def rms(x, eps):
    """x / sqrt(mean(x^2) + eps) over the last dimension."""
    return x / torch.sqrt((x * x).mean(dim=-1, keepdim=True) + eps)


def norm_one_plus(x, w, eps):
    """RMS norm whose stored weight is an offset from one."""
    return rms(x, eps) * (1.0 + w)


def rotate_pairs(x, positions, dims, base):
    """Rotary positions, dimension 2i paired with 2i+1, over the first `dims` of the last dimension; x [T, heads, D]."""
    out = x.clone()
    for i in range(dims // 2):
        a = positions.to(torch.float64) * base ** (-2.0 * i / dims)
        c, s = torch.cos(a).to(x.dtype)[:, None], torch.sin(a).to(x.dtype)[:, None]
        u, v = x[..., 2 * i], x[..., 2 * i + 1]
        out[..., 2 * i] = u * c - v * s
        out[..., 2 * i + 1] = v * c + u * s
    return out


def may_see(i, j, chunk: Optional[int]):
    """Causal, and inside one chunk of `chunk` positions counted from position 0 (None: causal only)."""
    ok = j <= i
    return ok if not chunk else ok & (torch.div(i, chunk, rounding_mode="floor") == torch.div(j, chunk, rounding_mode="floor"))


def sink_attention(q, k, v, scale, sink, chunk):
    """q [T, H, D], k [T, G, D], v [T, G, Dv], sink [H] -> [T, H, Dv].  The softmax of head h has one more term in its
    denominator, exp(sink_h)."""
    T, H, G = q.shape[0], q.shape[1], k.shape[1]
    pos = torch.arange(T)
    see = may_see(pos[:, None], pos[None, :], chunk)
    out = torch.zeros(T, H, v.shape[2], dtype=q.dtype)
    for h in range(H):
        g = h // (H // G)
        s = (q[:, h] @ k[:, g].T) * scale
        s = s.masked_fill(~see, -math.inf)
        top = torch.maximum(s.max(dim=1).values, sink[h])
        e = torch.exp(s - top[:, None])
        den = e.sum(dim=1) + torch.exp(sink[h] - top)
        out[:, h] = (e @ v[:, g]) / den[:, None]
    return out


def attention(w, pre, mx, eps, h, v_first):
    """The mixer on h [T, width].  Returns (output, the values it would cache)."""
    T = h.shape[0]
    H, G, D, Dv = mx["heads"], mx["kv_heads"], mx["dim"], mx["vdim"]
    q = h @ w[pre + "q"].T + w[pre + "q.b"]
    k = h @ w[pre + "k"].T + w[pre + "k.b"]
    v = h @ w[pre + "v"].T + w[pre + "v.b"]
    q = (rms(q, eps) * w[pre + "q.norm"]).reshape(T, H, D)
    k = (rms(k, eps) * w[pre + "k.norm"]).reshape(T, G, D)
    pos = torch.arange(T)
    rot = mx.get("rot")
    if rot:
        q = rotate_pairs(q, pos, rot["dims"], rot["base"])
        k = rotate_pairs(k, pos, rot["dims"], rot["base"])
    if mx.get("v_mix") and v_first is not None:
        lam = w[pre + "vmix"]
        v = (1.0 - lam) * v + lam * v_first
    chunk = (mx.get("mask") or {}).get("size")
    o = sink_attention(q, k, v.reshape(T, G, Dv), mx["scale"], w[pre + "sink"], chunk)
    return o.reshape(T, H * Dv) @ w[pre + "o"].T, v


def relu_squared_mlp(w, pre, h):
    u = torch.relu(h @ w[pre + "up"].T)
    return (u * u) @ w[pre + "down"].T


def gated_mlp(w, pre, h):
    z = h @ w[pre + "gate"].T
    return (z * torch.sigmoid(z) * (h @ w[pre + "up"].T)) @ w[pre + "down"].T


def table_experts(w, pre, mlp, tokens, h):
    """Each token's experts come from a table indexed by the token id; equal weights; a shared expert is added."""
    top = mlp["router"]["top"]
    table = w[pre + "table"].long()
    out = torch.zeros_like(h)
    for t, tok in enumerate(tokens):
        for j in range(top):
            out[t] += gated_mlp(w, f"{pre}e{int(table[tok, j])}.", h[t:t + 1])[0] / top
    if mlp.get("shared"):
        out = out + gated_mlp(w, pre + "shared.", h)
    return out


def softcap(z, cap):
    return cap * torch.tanh(z / cap) if cap else z


def forward(config: dict, weights: Dict[str, torch.Tensor], tokens: Sequence[int], dtype=torch.float64,
            residuals: Optional[List[torch.Tensor]] = None) -> torch.Tensor:
    """Logits [T, vocab] of one whole sequence.  `residuals` (a list) receives the residual stream after every layer."""
    w = {n: (t.to(dtype) if t.is_floating_point() else t) for n, t in weights.items()}
    eps, alpha = config["norm"]["eps"], config["postln_alpha"]
    x = w["embed"][torch.tensor(list(tokens), dtype=torch.long)]
    v_first = None
    for i, layer in enumerate(config["layers"]):
        pre = f"l{i}."
        y, v = attention(w, pre + "mix.", layer["mixer"], eps, x, v_first)
        if layer["mixer"].get("v_mix") and v_first is None:
            v_first = v
        x = norm_one_plus(alpha * x + y, w[pre + "norm1"], eps)
        mlp = layer["mlp"]
        if mlp is not None:
            if mlp["kind"] == "dense":
                y = relu_squared_mlp(w, pre + "mlp.", x)
            else:
                y = table_experts(w, pre + "mlp.", mlp, tokens, x)
            x = norm_one_plus(alpha * x + y, w[pre + "norm2"], eps)
        if residuals is not None:
            residuals.append(x.clone())
    x = norm_one_plus(x, w["final.norm"], eps)
    return softcap(x @ w["head"].T, config.get("logit_softcap"))
