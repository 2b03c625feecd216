"""Closed forms for the Nibotar oracle, and that the test models show the faults they are made to show (CPU only)."""
import copy
import math

import pytest
import torch

from oracle import nibotar_oracle as O
from tests import nibotar_models as M


def test_rms_norm():
    x = torch.tensor([[3.0, -4.0]]).double()
    assert torch.allclose(O.rms(x, 0.0), x / math.sqrt(12.5))
    assert torch.allclose(O.rms(x, 12.5), x / 5.0)                   # eps is inside the root
    assert torch.allclose(O.norm_one_plus(x, torch.tensor([1.0, 0.0]).double(), 0.0), torch.tensor([[6.0, -4.0]]).double() / math.sqrt(12.5))


def test_rotation_pairs_neighbours():
    x = torch.zeros(3, 1, 6).double()
    x[:, 0, 0], x[:, 0, 2], x[:, 0, 5] = 1.0, 1.0, 7.0
    y = O.rotate_pairs(x, torch.arange(3), 4, 100.0)
    for p in range(3):
        a, b = p * 1.0, p * 100.0 ** -0.5
        assert torch.allclose(y[p, 0], torch.tensor([math.cos(a), math.sin(a), math.cos(b), math.sin(b), 0.0, 7.0]).double())
    # scores depend on the distance of the positions only
    g = torch.Generator().manual_seed(0)
    q, k = torch.randn(1, 1, 8, generator=g).double(), torch.randn(1, 1, 8, generator=g).double()

    def score(i, j):
        return float((O.rotate_pairs(q, torch.tensor([i]), 8, 50.0) * O.rotate_pairs(k, torch.tensor([j]), 8, 50.0)).sum())
    assert abs(score(9, 4) - score(105, 100)) < 1e-9 and abs(score(9, 4) - score(9, 5)) > 1e-3


def test_chunked_visibility():
    see = O.may_see(torch.arange(7)[:, None], torch.arange(7)[None, :], 3)
    assert see.int().tolist() == [[1, 0, 0, 0, 0, 0, 0], [1, 1, 0, 0, 0, 0, 0], [1, 1, 1, 0, 0, 0, 0], [0, 0, 0, 1, 0, 0, 0],
                                  [0, 0, 0, 1, 1, 0, 0], [0, 0, 0, 1, 1, 1, 0], [0, 0, 0, 0, 0, 0, 1]]
    assert torch.equal(O.may_see(torch.arange(4)[:, None], torch.arange(4)[None, :], None), torch.ones(4, 4).tril().bool())


def test_sink_takes_its_share():
    T = 4
    q, k = torch.zeros(T, 2, 3).double(), torch.zeros(T, 1, 3).double()
    v = torch.arange(1, T + 1).double().reshape(T, 1, 1)
    out = O.sink_attention(q, k, v, 1.0, torch.tensor([0.0, math.log(3.0)]).double(), None)
    for t in range(T):
        s = sum(range(1, t + 2))
        assert out[t, 0, 0] == pytest.approx(s / (t + 2)) and out[t, 1, 0] == pytest.approx(s / (t + 4))
    # the sink is not scaled
    assert torch.allclose(O.sink_attention(q, k, v, 0.1, torch.tensor([0.0, math.log(3.0)]).double(), None), out)


def test_value_mixing_starts_at_the_second_such_layer():
    cfg = M.CASES["value_mixing"]
    w, toks = M.weights(cfg), M.prompt(cfg, 20)
    base = M.oracle(cfg, w, toks)
    first = dict(w)
    first["l1.mix.vmix"] = torch.tensor(5.0).bfloat16()              # the first mixing layer's own factor is not used
    first["l0.mix.vmix"] = first["l2.mix.vmix"] = torch.tensor(5.0).bfloat16()
    assert torch.equal(M.oracle(cfg, first, toks), base)
    later = dict(w)
    later["l3.mix.vmix"] = torch.tensor(0.0).bfloat16()
    assert M.error(M.oracle(cfg, later, toks), base) > 0.05


def test_feed_forwards():
    w = {"m.up": torch.tensor([[1.0, 0.0], [0.0, 1.0]]), "m.down": torch.tensor([[1.0, 10.0]])}
    assert O.relu_squared_mlp(w, "m.", torch.tensor([[3.0, -2.0]])).tolist() == [[9.0]]
    g = {"m.gate": torch.tensor([[1.0]]), "m.up": torch.tensor([[2.0]]), "m.down": torch.tensor([[1.0]])}
    assert O.gated_mlp(g, "m.", torch.tensor([[3.0]])).item() == pytest.approx(18.0 / (1 + math.exp(-3.0)))
    # equal experts: the choice does not matter; each weighs 1 / top
    mlp = {"router": {"experts": 3, "top": 2}}
    e = {f"m.e{i}.{n}": t for i in range(3) for n, t in (("gate", g["m.gate"]), ("up", g["m.up"]), ("down", g["m.down"] * (i + 1)))}
    e["m.table"] = torch.tensor([[0, 1], [2, 0]]).int()
    one = O.gated_mlp(g, "m.", torch.tensor([[3.0]])).item()
    assert O.table_experts(e, "m.", mlp, [0, 1], torch.tensor([[3.0], [3.0]])).flatten().tolist() == pytest.approx([1.5 * one, 2.0 * one])


def test_soft_cap():
    z = torch.tensor([0.0, 1e-3, 100.0])
    assert O.softcap(z, 5.0).tolist() == pytest.approx([0.0, 1e-3, 5.0], rel=1e-6)
    assert O.softcap(z, None) is z


def test_prefixes_agree():
    """Position i does not depend on later tokens."""
    cfg = M.CASES["everything"]
    w, toks = M.weights(cfg), M.prompt(cfg, 50)
    assert torch.allclose(M.oracle(cfg, w, toks)[:31], M.oracle(cfg, w, toks[:31]), atol=1e-9)


def test_the_edge_model_shows_its_key():
    """A chunk that is one position off, or sinks left out, are far outside every limit the tests use."""
    cfg, w, toks = M.edge_model(20, 70, 39)
    right = M.oracle(cfg, w, toks)
    for wrong in (19, 21, None):
        bad = copy.deepcopy(cfg)
        bad["layers"][0]["mixer"]["mask"] = {"size": wrong} if wrong else None
        assert M.error(M.oracle(bad, w, toks), right) > 0.4
    off = dict(w)
    off["l0.mix.sink"] = torch.full((4,), -30.0).bfloat16()
    assert M.error(M.oracle(cfg, off, toks), right) > 0.1


@pytest.mark.parametrize("plant", ["shift", "norm_per_head", "half_split_rotation", "wrong_group", "no_bias"])
def test_planted_faults_show_in_the_logits(plant, monkeypatch):
    cfg = M.CASES["everything"]
    w, toks = M.weights(cfg, 3), M.prompt(cfg, 60, 4)
    right = M.oracle(cfg, w, toks)
    if plant == "shift":                                             # positions off by one: chunk edges move
        old = O.may_see
        monkeypatch.setattr(O, "may_see", lambda i, j, c: old(i + 1, j + 1, c))
    elif plant == "norm_per_head":
        old = O.rms
        monkeypatch.setattr(O, "rms", lambda x, eps: old(x.reshape(x.shape[0], 2, -1), eps).reshape(x.shape) if x.shape[1] != cfg["width"] else old(x, eps))
    elif plant == "half_split_rotation":
        old = O.rotate_pairs
        def halves(x, pos, dims, base):
            p = torch.cat([torch.arange(0, dims, 2), torch.arange(1, dims, 2), torch.arange(dims, x.shape[-1])])
            return old(x[..., torch.argsort(p)], pos, dims, base)[..., p]
        monkeypatch.setattr(O, "rotate_pairs", halves)
    elif plant == "wrong_group":
        old = O.sink_attention
        monkeypatch.setattr(O, "sink_attention", lambda q, k, v, *a: old(q, k.flip(1), v.flip(1), *a))
    else:
        w = {n: (torch.zeros_like(t) if n.endswith("k.b") else t) for n, t in w.items()}
    assert M.error(M.oracle(cfg, w, toks), right) > 0.1
