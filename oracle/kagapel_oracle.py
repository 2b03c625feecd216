"""CPU oracle for Kagapel models: plain, slow torch, one function per mechanism.

TEST INFRASTRUCTURE ONLY, like the other oracles of this package: only tests and scripts that check the product import
it, and it shares no code with it.  A model is (config dict, weights dict); the weights are torch tensors under the
checkpoint's names, and everything is computed in `dtype` (float32 or float64).  There is no cache: `forward` evaluates a
whole sequence, and a decoded token is checked against the last row of the sequence that ends with it.

Parity pinning: parity unpinned by a third implementation (no library has the design).  The functions are the equations
written out, loops over heads and streams where that is plainest; tests/test_kagapel_oracle.py holds closed forms.
"""
from __future__ import annotations

import math
from typing import Dict, List, Optional, Sequence

import torch


def rms_norm(x, w, eps):
    """w x / sqrt(mean(x^2) + eps) over the last dimension."""
    return x / torch.sqrt((x * x).mean(dim=-1, keepdim=True) + eps) * w


def yarn_frequencies(dims, base, scaling: Optional[dict]):
    """Angle per position of every pair, and the factor on cos and sin.  Without scaling: base^(-2i/dims) and 1."""
    freq = [base ** (-2.0 * i / dims) for i in range(dims // 2)]
    if not scaling:
        return freq, 1.0
    s, L = scaling["factor"], scaling["original"]

    def index_of(turns):
        """The (real-valued) pair index, in dimensions, that makes `turns` turns over L positions."""
        return dims * math.log(L / (2.0 * math.pi * turns)) / (2.0 * math.log(base))
    lo = max(math.floor(index_of(scaling["fast"])), 0)
    hi = min(math.ceil(index_of(scaling["slow"])), dims - 1)
    out = []
    for i, f in enumerate(freq):
        r = (i - lo) / max(hi - lo, 0.001)
        r = min(max(r, 0.0), 1.0)
        out.append(f / s * r + f * (1.0 - r))
    return out, 0.1 * math.log(s) + 1.0


def rotate_halves(x, rot):
    """x [T, heads, R], token t at position t: dimension i is paired with dimension i + dims/2."""
    T, n = x.shape[0], rot["dims"] // 2
    freq, m = yarn_frequencies(rot["dims"], rot["base"], rot.get("scaling"))
    out = x.clone()
    pos = torch.arange(T, dtype=torch.float64)
    for i in range(n):
        c, s = (m * torch.cos(pos * freq[i])).to(x.dtype)[:, None], (m * torch.sin(pos * freq[i])).to(x.dtype)[:, None]
        u, v = x[..., i], x[..., i + n]
        out[..., i] = u * c - v * s
        out[..., i + n] = v * c + u * s
    return out


def latents(w, pre, mx, eps, h):
    """What a layer caches: the normed latent [T, rank] and the rotated key part that all heads share [T, rot_dim]."""
    r = mx["kv_rank"]
    z = h @ w[pre + "dkv"].T
    c = rms_norm(z[:, :r], w[pre + "dkv.norm"], eps)
    return c, rotate_halves(z[:, None, r:], mx["rot"])[:, 0]


def causal_softmax(s, sink=None):
    """Weights [T, T] of one head from its scores; `sink` (a number): one more term exp(sink) in the denominator."""
    T = s.shape[0]
    s = s.masked_fill(~torch.ones(T, T).tril().bool(), -math.inf)
    top = s.max(dim=1).values
    if sink is not None:
        top = torch.maximum(top, sink)
    e = torch.exp(s - top[:, None])
    den = e.sum(dim=1)
    if sink is not None:
        den = den + torch.exp(sink - top)
    return e / den[:, None]


def latent_attention(w, pre, mx, h, c, kr, sink, gated):
    """h [T, width] and the cached parts -> the mixer's output [T, width]."""
    T, H, D, R, Dv = h.shape[0], mx["heads"], mx["dim"], mx["rot_dim"], mx["vdim"]
    q = (h @ w[pre + "q"].T).reshape(T, H, D + R)
    qu, qr = q[..., :D], rotate_halves(q[..., D:], mx["rot"])
    ku, v = (c @ w[pre + "uk"].T).reshape(T, H, D), (c @ w[pre + "uv"].T).reshape(T, H, Dv)
    o = torch.zeros(T, H, Dv, dtype=h.dtype)
    for i in range(H):
        s = (qu[:, i] @ ku[:, i].T + qr[:, i] @ kr.T) * mx["scale"]
        o[:, i] = causal_softmax(s, sink[i] if sink is not None else None) @ v[:, i]
    o = o.reshape(T, H * Dv)
    if gated:
        o = o * torch.sigmoid(h @ w[pre + "g"].T)
    return o @ w[pre + "o"].T


def gated_mlp(w, pre, h):
    z = h @ w[pre + "gate"].T + w[pre + "gate.b"]
    return (z * torch.sigmoid(z) * (h @ w[pre + "up"].T + w[pre + "up.b"])) @ w[pre + "down"].T + w[pre + "down.b"]


def streams_in(w, pre, xs):
    """The sublayer's input: a weighted sum of the streams."""
    return sum(w[pre + "in"][s] * x for s, x in enumerate(xs))


def streams_out(w, pre, xs, y):
    """The streams after the sublayer: each a mixture of the old ones plus its share of the output."""
    n = len(xs)
    return [sum(w[pre + "mix"][s, t] * xs[s] for s in range(n)) + w[pre + "out"][t] * y for t in range(n)]


def forward(config: dict, weights: Dict[str, torch.Tensor], tokens: Sequence[int], dtype=torch.float64,
            residuals: Optional[List[torch.Tensor]] = None) -> torch.Tensor:
    """Logits [T, vocab] of one whole sequence.  `residuals` (a list) receives the sum of the streams after every layer."""
    w = {n: t.to(dtype) for n, t in weights.items()}
    eps, T = config["norm"]["eps"], len(tokens)
    x = w["embed"][torch.tensor(list(tokens), dtype=torch.long)] + w["pos"][:T]
    xs = [x.clone() for _ in range(config["streams"])]
    cached = {}
    for i, layer in enumerate(config["layers"]):
        p, mx = f"l{i}.", layer["mixer"]
        second = layer["type"] == "latent_attention_2"
        h = rms_norm(streams_in(w, p + "hc1.", xs), w[p + "norm1"], eps)
        if "kv_from" in mx:
            c, kr = cached[mx["kv_from"]]
        else:
            c, kr = cached[i] = latents(w, p + "mix.", mx, eps, h)
        y = latent_attention(w, p + "mix.", mx, h, c, kr, w[p + "mix.sink"] if second else None, not second)
        xs = streams_out(w, p + "hc1.", xs, y)
        if layer["mlp"] is not None:
            h = rms_norm(streams_in(w, p + "hc2.", xs), w[p + "norm2"], eps)
            xs = streams_out(w, p + "hc2.", xs, gated_mlp(w, p + "mlp.", h))
        if residuals is not None:
            residuals.append(sum(xs))
    return rms_norm(sum(xs), w["final.norm"], eps) @ w["head"].T * config["logit_scale"]
