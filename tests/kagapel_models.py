"""Small Kagapel models with random weights for the tests."""
import torch

from oracle import kagapel_oracle as O
from tests.nibotar_models import error, prompt  # noqa: F401  (shared by the tests of both designs)


def yarn(factor, original, fast=32.0, slow=1.0):
    return {"factor": factor, "original": original, "fast": fast, "slow": slow}


def mixer(heads, dim, rot, vdim, rank, scale=None, base=10000.0, scaling=None, kv_from=None):
    m = {"heads": heads, "dim": dim, "rot_dim": rot, "vdim": vdim, "kv_rank": rank, "scale": scale if scale is not None else (dim + rot) ** -0.5,
         "rot": {"base": base, "dims": rot}}
    if scaling:
        m["rot"]["scaling"] = scaling
    if kv_from is not None:
        m["kv_from"] = kv_from
    return m


def gated(*a, ff=None, **kw):
    """A layer with an output gate."""
    return {"type": "latent_attention", "mixer": mixer(*a, **kw), "mlp": {"kind": "dense", "ff": ff} if ff else None}


def sunk(*a, ff=None, **kw):
    """A layer with sinks."""
    return {"type": "latent_attention_2", "mixer": mixer(*a, **kw), "mlp": {"kind": "dense", "ff": ff} if ff else None}


def model(width, vocab, layers, streams=2, eps=1e-5, logit_scale=1.5, positions=512):
    return {"architecture": "Kagapel", "width": width, "vocab": vocab, "streams": streams, "norm": {"eps": eps}, "logit_scale": logit_scale,
            "max_positions": positions, "layers": layers}


def weights(cfg, seed=0, peak=1.5, sink=1.0):
    """bf16 weights by name.  `peak` scales the queries: attention that picks single keys instead of averaging many, so that a
    wrong key shows; `sink` scales the sinks."""
    g = torch.Generator().manual_seed(seed)

    def rn(*shape, std=1.0, mean=0.0):
        return (torch.randn(shape, generator=g) * std + mean).bfloat16()

    W, V, S = cfg["width"], cfg["vocab"], cfg["streams"]
    w = {"embed": rn(V, W), "pos": rn(cfg["max_positions"], W, std=0.5), "head": rn(V, W, std=3 * W ** -0.5), "final.norm": rn(W, std=0.2, mean=1.0)}
    for i, layer in enumerate(cfg["layers"]):
        m, p = layer["mixer"], f"l{i}."
        H, D, R, Dv, r = m["heads"], m["dim"], m["rot_dim"], m["vdim"], m["kv_rank"]
        w[p + "mix.q"] = rn(H * (D + R), W, std=peak * W ** -0.5)
        if "kv_from" not in m:
            w[p + "mix.dkv"] = rn(r + R, W, std=W ** -0.5)
            w[p + "mix.dkv.norm"] = rn(r, std=0.2, mean=1.0)
        w[p + "mix.uk"] = rn(H * D, r, std=r ** -0.5)
        w[p + "mix.uv"] = rn(H * Dv, r, std=r ** -0.5)
        w[p + "mix.o"] = rn(W, H * Dv, std=2 * (H * Dv) ** -0.5)
        if layer["type"] == "latent_attention":
            w[p + "mix.g"] = rn(H * Dv, W, std=2 * W ** -0.5)
        else:
            w[p + "mix.sink"] = rn(H, std=sink)
        subs = [1]
        f = layer["mlp"]
        if f is not None:
            subs.append(2)
            for n in ("gate", "up"):
                w[p + f"mlp.{n}"] = rn(f["ff"], W, std=W ** -0.5)
                w[p + f"mlp.{n}.b"] = rn(f["ff"], std=0.5)
            w[p + "mlp.down"] = rn(W, f["ff"], std=2 * f["ff"] ** -0.5)
            w[p + "mlp.down.b"] = rn(W, std=0.3)
        for q in subs:
            w[p + f"norm{q}"] = rn(W, std=0.2, mean=1.0)
            w[p + f"hc{q}.in"] = rn(S, std=0.3, mean=1.0 / S)
            w[p + f"hc{q}.out"] = rn(S, std=0.3, mean=1.0)
            w[p + f"hc{q}.mix"] = (torch.eye(S) * 0.8 + torch.randn((S, S), generator=g) * 0.15).bfloat16()
    return w


# one model per mechanism, and some with everything
CASES = {
    "one_stream": model(96, 67, [gated(4, 32, 16, 32, 48)], streams=1),
    "streams": model(80, 67, [gated(2, 16, 8, 16, 24), gated(3, 16, 8, 16, 24, ff=40), gated(2, 16, 8, 16, 24)], streams=4),
    "many_streams": model(64, 51, [gated(2, 16, 8, 16, 24, ff=48), sunk(2, 16, 8, 16, 24, ff=48)], streams=7),
    "sinks": model(64, 51, [sunk(5, 24, 8, 16, 40), sunk(3, 16, 16, 24, 16, ff=64)]),
    "rotated_part_only_matters": model(64, 51, [gated(4, 8, 40, 16, 32, scale=0.4, base=300.0)]),
    "yarn": model(64, 51, [gated(4, 16, 32, 16, 32, scaling=yarn(4.0, 64), scale=0.4), gated(2, 16, 20, 16, 32, scaling=yarn(1.5, 40, 8.0, 2.0), base=500.0)]),
    "yarn_edges": model(64, 51, [sunk(2, 8, 24, 16, 32, scaling=yarn(8.0, 20, 1.0, 1.0), scale=0.4, base=50.0),     # the blend is a step
                                 gated(2, 8, 12, 16, 32, scaling=yarn(2.0, 100000, 2.0, 1e-4), scale=0.4)]),         # clamped at both ends
    "shared_latents": model(72, 51, [sunk(4, 16, 12, 24, 36, base=777.0), sunk(6, 24, 12, 8, 36, base=777.0, kv_from=0),
                                     gated(2, 40, 12, 16, 36, base=777.0, kv_from=0, ff=56), sunk(3, 16, 12, 16, 36, base=777.0),
                                     sunk(2, 8, 12, 40, 36, base=777.0, kv_from=3), sunk(5, 16, 12, 16, 36, base=777.0, kv_from=0)]),
    "twenty_heads": model(64, 51, [gated(20, 8, 8, 8, 24, ff=32), sunk(33, 8, 4, 16, 16)]),
    "seventy_heads": model(64, 51, [sunk(70, 8, 8, 8, 40)]),
    "large_rank": model(96, 51, [gated(3, 24, 64, 24, 512), sunk(18, 16, 128, 16, 300), gated(40, 8, 2, 8, 130)], streams=3),
    "large_heads": model(128, 60, [gated(2, 192, 64, 160, 96, ff=96), sunk(2, 100, 60, 250, 64), gated(4, 128, 64, 128, 96)]),
    "one_of_each": model(48, 51, [sunk(1, 1, 2, 1, 1, scale=1.3), gated(1, 2, 2, 3, 5, ff=1)], streams=3, eps=0.3),
    "width_not_of_fours": model(70, 41, [gated(3, 18, 6, 22, 37, ff=51), sunk(5, 30, 10, 11, 19, ff=25), sunk(2, 7, 10, 5, 19, kv_from=1)], streams=3),
    "everything": model(160, 301, [sunk(6, 40, 24, 56, 72, ff=100, base=5000.0, scale=0.2),
                                   gated(5, 64, 16, 28, 48, ff=200, scaling=yarn(3.0, 100), scale=0.15),
                                   sunk(8, 24, 24, 32, 72, ff=60, base=5000.0, kv_from=0),
                                   gated(4, 16, 32, 80, 150),
                                   sunk(3, 48, 24, 40, 72, ff=44, base=5000.0, kv_from=0)], streams=3, logit_scale=0.7, eps=1e-3),
}


def oracle(cfg, w, tokens, residuals=None, dtype=torch.float64):
    return O.forward(cfg, w, tokens, dtype, residuals)


def far_key_model(heads, rank, length, at, rotated=False, seed=5):
    """One key that outweighs every other: position `at` holds token 0, which alone has feature 0; its plain key (or its
    rotated part, at angles that hardly move) points along a direction that every query has (feature 1, the same in all
    tokens), so whoever sees it, takes it."""
    D, R, Dv = 16, 8, 24
    cfg = model(64, 40, [sunk(heads, D, R, Dv, rank, scale=0.5, base=1e6, scaling=yarn(1e6, 1, 1e6, 1e5) if rotated else None)], positions=length, eps=1e-5)
    w = weights(cfg, seed, peak=0.3, sink=0.3)
    g = torch.Generator().manual_seed(seed)

    def unit(n):
        u = torch.randn(n, generator=g)
        return u / u.norm()
    for n in ("embed", "pos"):
        w[n][:, :2] = 0
    w["embed"][:, 1] = 3.0
    w["embed"][0, 0] = 12.0
    m = "l0.mix."
    w["l0.norm1"][:2] = 1.0
    for n in ("q", "dkv"):
        w[m + n][:, :2] = 0
    if rotated:
        u = unit(R)
        q = w[m + "q"].view(heads, D + R, -1)
        q[:, D:, 1] = u * 2
        w[m + "dkv"][rank:, 0] = u * 4
    else:
        u = unit(D)
        q = w[m + "q"].view(heads, D + R, -1)
        q[:, :D, 1] = u * 3
        w[m + "dkv"][0, :] = 0
        w[m + "dkv"][0, 0] = 2.0                                    # latent 0 is this feature alone
        w[m + "uk"].view(heads, D, rank)[:, :, 0] = u * 3
    toks = [t if t else 1 for t in prompt(cfg, length, seed)]
    toks[at] = 0
    return cfg, w, toks
