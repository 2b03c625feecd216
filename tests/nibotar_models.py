"""Small Nibotar models with random weights for the tests."""
import torch

from oracle import nibotar_oracle as O


def attn(heads, kv_heads, dim, vdim, scale=None, chunk=None, rot=None, base=10000.0, v_mix=False):
    m = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale if scale is not None else dim ** -0.5, "v_mix": v_mix}
    if chunk:
        m["mask"] = {"size": chunk}
    if rot is None or rot > 0:
        m["rot"] = {"base": base, "dims": rot if rot is not None else dim}
    return m


def dense(ff):
    return {"kind": "dense", "ff": ff}


def moe(ff, experts, top, shared=None):
    m = {"kind": "moe", "expert": {"ff": ff}, "router": {"experts": experts, "top": top}}
    if shared:
        m["shared"] = {"ff": shared}
    return m


def model(width, vocab, layers, alpha=2.0, eps=1e-5, softcap=20.0):
    return {"architecture": "Nibotar", "width": width, "vocab": vocab, "norm": {"eps": eps}, "postln_alpha": alpha, "logit_softcap": softcap,
            "layers": [{"type": "attention", "mixer": m, "mlp": f} for m, f in layers]}


def weights(cfg, seed=0, peak=1.5, sink=1.0, head=1.0):
    """bf16 weights by name.  `peak` scales the query norms: attention that picks single keys instead of averaging many, so
    that a key too many or too few shows; `sink` scales the sinks."""
    g = torch.Generator().manual_seed(seed)

    def rn(*shape, std=1.0, mean=0.0):
        return (torch.randn(shape, generator=g) * std + mean).bfloat16()

    W, V = cfg["width"], cfg["vocab"]
    w = {"embed": rn(V, W), "head": rn(V, W, std=head * 3 * W ** -0.5), "final.norm": rn(W, std=0.2)}
    for i, layer in enumerate(cfg["layers"]):
        m, p = layer["mixer"], f"l{i}."
        for n, rows in (("q", m["heads"] * m["dim"]), ("k", m["kv_heads"] * m["dim"]), ("v", m["kv_heads"] * m["vdim"])):
            w[p + f"mix.{n}"] = rn(rows, W, std=W ** -0.5)
            w[p + f"mix.{n}.b"] = rn(rows, std=0.3)
            if n != "v":
                w[p + f"mix.{n}.norm"] = rn(rows, std=0.2, mean=peak)
        w[p + "mix.vmix"] = (torch.rand((), generator=g) * 0.6 + 0.2).bfloat16()
        w[p + "mix.sink"] = rn(m["heads"], std=sink)
        w[p + "mix.o"] = rn(W, m["heads"] * m["vdim"], std=(m["heads"] * m["vdim"]) ** -0.5)
        w[p + "norm1"] = rn(W, std=0.2)
        f = layer["mlp"]
        if f is None:
            continue
        w[p + "norm2"] = rn(W, std=0.2)
        if f["kind"] == "dense":
            w[p + "mlp.up"] = rn(f["ff"], W, std=W ** -0.5)
            w[p + "mlp.down"] = rn(W, f["ff"], std=f["ff"] ** -0.5)
        else:
            E, top = f["router"]["experts"], f["router"]["top"]
            parts = [(f"e{e}", f["expert"]["ff"]) for e in range(E)] + ([("shared", f["shared"]["ff"])] if f.get("shared") else [])
            for name, ff in parts:
                w[p + f"mlp.{name}.gate"] = rn(ff, W, std=2 * W ** -0.5)
                w[p + f"mlp.{name}.up"] = rn(ff, W, std=W ** -0.5)
                w[p + f"mlp.{name}.down"] = rn(W, ff, std=2 * ff ** -0.5)
            w[p + "mlp.table"] = torch.stack([torch.randperm(E, generator=g)[:top] for _ in range(V)]).int()
    return w


def prompt(cfg, n, seed=1):
    return torch.randint(0, cfg["vocab"], (n,), generator=torch.Generator().manual_seed(seed)).tolist()


def error(got, want):
    """Root mean square of the difference per row, in units of the rows' own spread."""
    got, want = got.double().cpu(), want.double()
    return ((got - want).pow(2).mean(-1).sqrt() / want.std()).max().item()


# one model per mechanism, and some with everything
CASES = {
    "plain": model(96, 67, [(attn(4, 4, 32, 32, rot=0), None)]),
    "projection_norms": model(80, 67, [(attn(6, 3, 24, 16, rot=0, scale=0.4), None)], eps=0.3),
    "rotation_partial": model(64, 51, [(attn(4, 2, 40, 24, rot=14, base=333.0), None)]),
    "rotation_whole": model(64, 51, [(attn(2, 1, 48, 64, base=1e6), None)]),
    "chunks": model(64, 51, [(attn(4, 2, 32, 40, chunk=13), None), (attn(3, 3, 16, 16, chunk=5), None)]),
    "many_heads_per_group": model(72, 51, [(attn(20, 1, 16, 8, chunk=50), None), (attn(34, 2, 8, 24), None)]),
    "tiny_chunks": model(64, 51, [(attn(2, 1, 16, 16, chunk=1), None), (attn(4, 2, 24, 8, chunk=2), dense(40)), (attn(2, 2, 16, 16, chunk=3), None)]),
    "more_experts_than_tokens": model(64, 51, [(attn(2, 2, 16, 16), moe(16, 300, 5, shared=24)), (attn(2, 2, 16, 16), moe(24, 2, 2))]),
    "value_mixing": model(64, 51, [(attn(2, 1, 16, 32), None), (attn(4, 2, 24, 20, v_mix=True), None), (attn(2, 2, 16, 20, chunk=9), None),
                                   (attn(8, 4, 16, 10, v_mix=True), None)]),
    "relu_squared": model(100, 51, [(attn(2, 2, 16, 16), dense(77)), (attn(2, 2, 16, 16), dense(260))]),
    "experts": model(64, 73, [(attn(2, 2, 16, 16), moe(24, 5, 3)), (attn(2, 2, 16, 16), moe(36, 9, 1))]),
    "experts_and_shared": model(64, 73, [(attn(2, 2, 16, 16), moe(20, 6, 2, shared=44)), (attn(2, 2, 16, 16), moe(70, 4, 4, shared=9))]),
    "soft_cap_low": model(64, 51, [(attn(2, 1, 16, 16), dense(64))], softcap=2.0, alpha=1.0),
    "no_soft_cap": model(64, 51, [(attn(2, 1, 16, 16), dense(64))], softcap=None, alpha=0.7),
    "width_not_of_fours": model(70, 41, [(attn(3, 1, 18, 22, rot=6, chunk=11, v_mix=True), moe(25, 3, 2, shared=13)),
                                         (attn(6, 2, 30, 11, rot=4, chunk=17, v_mix=True), dense(51))]),
    "large_heads": model(128, 60, [(attn(2, 1, 192, 160, chunk=70), dense(96)), (attn(4, 2, 96, 128, rot=32), dense(96))]),
    "everything": model(160, 301, [(attn(6, 2, 40, 56, rot=20, base=5000.0, chunk=37, v_mix=True, scale=0.2), moe(60, 7, 3, shared=100)),
                                   (attn(8, 4, 64, 28, chunk=61, v_mix=True), dense(200)),
                                   (attn(5, 1, 72, 80, rot=72), None),
                                   (attn(4, 2, 16, 56, chunk=24, v_mix=True, rot=8), moe(44, 10, 2))], alpha=1.7, softcap=9.0),
}


def oracle(cfg, w, tokens, residuals=None, dtype=torch.float64):
    return O.forward(cfg, w, tokens, dtype, residuals)


def edge_model(chunk, length, at, seed=5):
    """One key that outweighs every other: position `at` holds token 0, whose key is made long along the direction of all
    queries (their bias), so whoever can see it, takes it."""
    cfg = model(64, 40, [(attn(4, 2, 32, 24, chunk=chunk, rot=0, scale=0.5), None)])
    w = weights(cfg, seed, peak=1.0, sink=0.3)
    g = torch.Generator().manual_seed(seed)
    u = torch.randn(32, generator=g)
    u = u / u.norm()
    # queries: a common part along u; keys: token 0 carries feature 0, which no other token has
    w["l0.mix.q"] = (w["l0.mix.q"].float() * 0.2).bfloat16()
    w["l0.mix.q.b"] = (u.repeat(4) * 4).bfloat16()
    w["embed"][:, 0] = 0
    w["embed"][0, 0] = 12.0
    w["l0.mix.k"][:, 0] = (u.repeat(2) * 3).bfloat16()
    toks = [t if t else 1 for t in prompt(cfg, length, seed)]
    toks[at] = 0
    return cfg, w, toks
