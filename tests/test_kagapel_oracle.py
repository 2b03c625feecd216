"""Closed forms for the Kagapel oracle, and that the test models show the faults they are made to show (CPU only)."""
import copy
import math

import pytest
import torch

from oracle import kagapel_oracle as O
from tests import kagapel_models as M


def test_rms_norm():
    x = torch.tensor([[3.0, -4.0]]).double()
    assert torch.allclose(O.rms_norm(x, torch.tensor([1.0, 2.0]).double(), 0.0), torch.tensor([[3.0, -8.0]]).double() / math.sqrt(12.5))
    assert torch.allclose(O.rms_norm(x, torch.ones(2).double(), 12.5), x / 5.0)          # eps is inside the root


def test_rotation_pairs_halves():
    x = torch.zeros(3, 1, 4).double()
    x[:, 0, 0], x[:, 0, 3] = 1.0, 2.0
    y = O.rotate_halves(x, {"dims": 4, "base": 100.0})
    for p in range(3):
        a, b = p * 1.0, p * 0.1
        assert torch.allclose(y[p, 0], torch.tensor([math.cos(a), -2 * math.sin(b), math.sin(a), 2 * math.cos(b)]).double())


def test_yarn_frequencies():
    plain, one = O.yarn_frequencies(8, 10000.0, None)
    assert plain == pytest.approx([1.0, 0.1, 0.01, 0.001]) and one == 1.0
    f, m = O.yarn_frequencies(8, 10000.0, M.yarn(4.0, 1000, 20.0, 0.2))
    assert m == pytest.approx(0.1 * math.log(4.0) + 1.0)
    # turns over 1000 positions: 159, 15.9, 1.59, 0.159.  index(20) = 0.9 -> 0; index(0.2) = 2.9 -> 3
    assert f == pytest.approx([1.0, 0.1 * (2 / 3 + 1 / 12), 0.01 * (1 / 3 + 2 / 12), 0.001 / 4])
    f, _ = O.yarn_frequencies(8, 10000.0, M.yarn(4.0, 1000, 1e-9, 1e-9))                 # every pair makes more turns
    assert f == pytest.approx(plain)
    f, _ = O.yarn_frequencies(8, 10000.0, M.yarn(4.0, 1000, 1e9, 1e6))                   # the blend starts and ends at pair 0
    assert f[1:] == pytest.approx([v / 4 for v in plain[1:]])


def test_sink_takes_its_share():
    s = torch.zeros(4, 4).double()
    for sink, extra in ((None, 0.0), (torch.tensor(0.0).double(), 1.0), (torch.tensor(math.log(3.0)).double(), 3.0)):
        p = O.causal_softmax(s, sink)
        for t in range(4):
            assert p[t, :t + 1].tolist() == pytest.approx([1.0 / (t + 1 + extra)] * (t + 1)) and not p[t, t + 1:].any()


def test_latent_attention_equals_attention_over_expanded_heads():
    """The same mixer written over the latents: queries taken through W_uk, one shared key and value row per position."""
    cfg = M.CASES["sinks"]
    w = {n: t.double() for n, t in M.weights(cfg).items()}
    mx, T = cfg["layers"][0]["mixer"], 9
    h = torch.randn(T, cfg["width"], generator=torch.Generator().manual_seed(1)).double()
    c, kr = O.latents(w, "l0.mix.", mx, 1e-5, h)
    want = O.latent_attention(w, "l0.mix.", mx, h, c, kr, w["l0.mix.sink"], False)
    H, D, R, Dv = mx["heads"], mx["dim"], mx["rot_dim"], mx["vdim"]
    q = (h @ w["l0.mix.q"].T).reshape(T, H, D + R)
    outs = []
    for i in range(H):
        ql = q[:, i, :D] @ w["l0.mix.uk"][i * D:(i + 1) * D]
        qr = O.rotate_halves(q[:, i:i + 1, D:], mx["rot"])[:, 0]
        p = O.causal_softmax((ql @ c.T + qr @ kr.T) * mx["scale"], w["l0.mix.sink"][i])
        outs.append((p @ c) @ w["l0.mix.uv"][i * Dv:(i + 1) * Dv].T)
    assert torch.allclose(torch.cat(outs, dim=1) @ w["l0.mix.o"].T, want)


def test_streams():
    w = {"in": torch.tensor([1.0, 10.0]), "out": torch.tensor([2.0, 3.0]), "mix": torch.tensor([[1.0, 5.0], [0.0, 7.0]])}
    xs = [torch.tensor([1.0]), torch.tensor([2.0])]
    assert O.streams_in(w, "", xs).item() == 21.0
    assert [x.item() for x in O.streams_out(w, "", xs, torch.tensor([100.0]))] == [201.0, 319.0]     # from stream 0: 1 and 5


def test_feed_forward():
    w = {"gate": torch.tensor([[1.0]]), "gate.b": torch.tensor([0.5]), "up": torch.tensor([[2.0]]), "up.b": torch.tensor([-1.0]),
         "down": torch.tensor([[1.0]]), "down.b": torch.tensor([10.0])}
    assert O.gated_mlp(w, "", torch.tensor([[3.0]])).item() == pytest.approx(3.5 / (1 + math.exp(-3.5)) * 5.0 + 10.0)


def test_prefixes_agree():
    """Position i does not depend on later tokens."""
    cfg = M.CASES["everything"]
    w, toks = M.weights(cfg), M.prompt(cfg, 50)
    assert torch.allclose(M.oracle(cfg, w, toks)[:31], M.oracle(cfg, w, toks[:31]), atol=1e-9)


@pytest.mark.parametrize("rotated", [False, True])
def test_the_far_key_model_shows_its_key(rotated):
    cfg, w, toks = M.far_key_model(3, 20, 70, 30, rotated)
    right = M.oracle(cfg, w, toks)
    other = list(toks)
    other[30] = 1
    assert M.error(M.oracle(cfg, w, other)[31:], right[31:]) > 0.4
    off = dict(w)
    off["l0.mix.sink"] = torch.full((3,), 25.0).bfloat16()
    assert M.error(M.oracle(cfg, off, toks), right) > 0.1


@pytest.mark.parametrize("plant", ["no_sink", "no_gate", "no_yarn", "yarn_factor_off", "neighbour_pairs", "rotated_part_normed", "latent_not_normed",
                                   "mix_transposed", "one_stream_read", "own_latents", "no_position", "position_shift", "no_bias", "unscaled"])
def test_planted_faults_show_in_the_logits(plant, monkeypatch):
    cfg = copy.deepcopy(M.CASES["everything"])
    w, toks = M.weights(cfg, 3), M.prompt(cfg, 60, 4)
    right = M.oracle(cfg, w, toks)
    if plant == "no_sink":
        w = {n: (torch.full_like(t, -50.0) if n.endswith("sink") else t) for n, t in w.items()}
    elif plant == "no_gate":
        old = O.latent_attention
        monkeypatch.setattr(O, "latent_attention", lambda *a: old(*a[:-1], False))
    elif plant == "no_yarn":
        del cfg["layers"][1]["mixer"]["rot"]["scaling"]
    elif plant == "yarn_factor_off":
        old = O.yarn_frequencies
        monkeypatch.setattr(O, "yarn_frequencies", lambda *a: (old(*a)[0], 1.0))
    elif plant == "neighbour_pairs":
        old = O.rotate_halves

        def neighbours(x, rot):
            p = torch.cat([torch.arange(0, rot["dims"], 2), torch.arange(1, rot["dims"], 2)])
            return old(x[..., p], rot)[..., torch.argsort(p)]
        monkeypatch.setattr(O, "rotate_halves", neighbours)
    elif plant == "rotated_part_normed":
        old = O.latents

        def normed(*a):
            c, k = old(*a)
            return c, O.rms_norm(k, torch.ones(k.shape[-1], dtype=k.dtype), 1e-5)
        monkeypatch.setattr(O, "latents", normed)
    elif plant == "latent_not_normed":
        old = O.rms_norm
        monkeypatch.setattr(O, "rms_norm", lambda x, n, e: x * n if x.shape[-1] in (48, 72, 150) else old(x, n, e))
    elif plant == "mix_transposed":
        w = {n: (t.T if n.endswith(".mix") else t) for n, t in w.items()}
    elif plant == "one_stream_read":
        monkeypatch.setattr(O, "streams_in", lambda w, p, xs: xs[0])
    elif plant == "own_latents":
        del cfg["layers"][4]["mixer"]["kv_from"]
        w = {**w, "l4.mix.dkv": w["l0.mix.dkv"], "l4.mix.dkv.norm": w["l0.mix.dkv.norm"]}
    elif plant == "no_position":
        w = {**w, "pos": torch.zeros_like(w["pos"])}
    elif plant == "position_shift":
        w = {**w, "pos": w["pos"].roll(1, 0)}
    elif plant == "no_bias":
        w = {n: (torch.zeros_like(t) if n.endswith("gate.b") else t) for n, t in w.items()}
    else:
        cfg["logit_scale"] = 1.0
    assert M.error(M.oracle(cfg, w, toks), right) > 0.1
