"""Host side of the sequence models: configuration, checkpoint files, registry, engine, C ABI layout (no GPU)."""
import ctypes
import json
import os
import re
import subprocess

import pytest
import torch

from clusterfusionplus_amd import engine as E
from clusterfusionplus_amd import kagapel, nibotar, registry, seq_model, trace, weights
from tests import kagapel_models as KM
from tests import nibotar_models as M

ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))


# ---- configuration and weights -------------------------------------------------------------------------------------

def test_config_is_read_in_full():
    c = nibotar.parse_config(M.CASES["everything"])
    assert (c.width, c.vocab, c.alpha, c.softcap, c.eps) == (160, 301, 1.7, 9.0, 1e-5)
    a = c.layers[0].attention
    assert (a.heads, a.kv_heads, a.dim, a.vdim, a.scale, a.chunk, a.rot_dims, a.rot_base, a.v_mix) == (6, 2, 40, 56, 0.2, 37, 20, 5000.0, True)
    assert c.layers[0].mlp == nibotar.FeedForwardConfig("moe", 60, 7, 3, 100)
    assert c.layers[1].mlp == nibotar.FeedForwardConfig("dense", 200)
    assert c.layers[2].mlp is None and c.layers[2].attention.chunk == 0 and not c.layers[2].attention.v_mix
    assert c.layers[3].mlp.shared_ff == 0
    assert nibotar.parse_config(M.CASES["no_soft_cap"]).softcap == 0.0


@pytest.mark.parametrize("change", [lambda c: c["layers"][0].update(type="recurrent"), lambda c: c["layers"][0]["mixer"].update(kv_heads=4),
                                    lambda c: c["layers"][0]["mlp"].update(kind="sparse")])
def test_what_the_design_does_not_have_is_refused(change):
    cfg = json.loads(json.dumps(M.CASES["everything"]))
    change(cfg)
    with pytest.raises(ValueError):
        nibotar.parse_config(cfg)


def test_packed_weights():
    cfg = M.CASES["width_not_of_fours"]
    w = M.weights(cfg)
    p = nibotar.pack_weights(nibotar.parse_config(cfg), w, torch.bfloat16, "cpu")
    l0, l1 = p.layers
    assert l0.w_qkv.shape == (3 * 18 + 18 + 22, 128) and not l0.w_qkv[:, 70:].any()
    assert torch.equal(l0.w_qkv[54:72, :70], w["l0.mix.k"]) and torch.equal(l0.w_qkv[72:, :70], w["l0.mix.v"])
    assert torch.equal(l0.b_qkv, torch.cat([w["l0.mix.q.b"], w["l0.mix.k.b"], w["l0.mix.v.b"]]).float())
    assert l0.w_up.shape == (3, 50, 128) and torch.equal(l0.w_up[2, 0::2, :70], w["l0.mlp.e2.gate"]) and torch.equal(l0.w_up[2, 1::2, :70], w["l0.mlp.e2.up"])
    assert torch.equal(l0.w_shared_down[:, :13], w["l0.mlp.shared.down"]) and l0.table.dtype == torch.int32
    assert l0.v_lambda == 0.0 and l1.v_lambda == float(w["l1.mix.vmix"])
    f = nibotar.pack_weights(nibotar.parse_config(cfg), w, torch.float32, "cpu")
    assert f.layers[1].w_down.shape == (70, 64) and f.embed.shape == (41, 96)


def test_missing_and_misshapen_tensors_are_named():
    cfg = M.CASES["everything"]
    for name, t in (("l1.mix.k.norm", None), ("l0.mlp.e3.down", torch.zeros(2, 2)), ("l3.mlp.table", M.weights(cfg)["l3.mlp.table"] + 9)):
        w = M.weights(cfg)
        if t is None:
            del w[name]
        else:
            w[name] = t
        with pytest.raises(ValueError, match=re.escape(name)):
            nibotar.pack_weights(nibotar.parse_config(cfg), w, torch.bfloat16, "cpu")


def test_value_mixing_needs_equal_values():
    """The library refuses it (a GPU is not needed to see the rule in the packed sizes)."""
    cfg = M.CASES["value_mixing"]
    sizes = {l.kv_heads * l.vdim for l in nibotar.pack_weights(nibotar.parse_config(cfg), M.weights(cfg), torch.bfloat16, "cpu").layers if l.v_mix}
    assert len(sizes) == 1


def test_kagapel_config_is_read_in_full():
    c = kagapel.parse_config(KM.CASES["everything"])
    assert (c.width, c.vocab, c.eps, c.streams, c.max_positions, c.logit_scale) == (160, 301, 1e-3, 3, 512, 0.7)
    a, b = c.layers[0].mixer, c.layers[1].mixer
    assert (a.heads, a.dim, a.rot_dim, a.vdim, a.kv_rank, a.scale, a.rot_base, a.yarn, a.gated, a.sink, a.kv_from) == \
        (6, 40, 24, 56, 72, 0.2, 5000.0, None, False, True, -1)
    assert (b.yarn, b.gated, b.sink) == (kagapel.Yarn(3.0, 100.0, 32.0, 1.0), True, False)
    assert [l.mixer.kv_from for l in c.layers] == [-1, -1, 0, -1, 0] and [l.ff for l in c.layers] == [100, 200, 60, 0, 44]


@pytest.mark.parametrize("change", [lambda c: c["layers"][0].update(type="attention"), lambda c: c["layers"][0]["mlp"].update(kind="moe"),
                                    lambda c: c["layers"][0]["mixer"].update(kv_from=2), lambda c: c["layers"][4]["mixer"].update(kv_from=2),
                                    lambda c: c["layers"][2]["mixer"].update(kv_rank=71), lambda c: c["layers"][2]["mixer"]["rot"].update(base=1.5),
                                    lambda c: c["layers"][4]["mixer"].update(kv_from=1), lambda c: c["layers"][1]["mixer"].update(rot_dim=18)])
def test_kagapel_configs_that_do_not_fit_are_refused(change):
    cfg = json.loads(json.dumps(KM.CASES["everything"]))
    change(cfg)
    with pytest.raises(ValueError):
        kagapel.parse_config(cfg)


def test_kagapel_packed_weights():
    cfg = KM.CASES["width_not_of_fours"]
    w = KM.weights(cfg)
    p = kagapel.pack_weights(kagapel.parse_config(cfg), w, torch.bfloat16, "cpu")
    l0, l1, l2 = p.layers
    assert l0.w_qkv.shape == (3 * 24 + 43 + 66, 128) and l1.w_qkv.shape == (5 * 40 + 29, 128) and l2.w_qkv.shape == (2 * 17, 128)
    assert torch.equal(l0.w_qkv[72:115, :70], w["l0.mix.dkv"]) and torch.equal(l0.w_qkv[115:, :70], w["l0.mix.g"])
    assert l0.w_ukv.shape == (3 * 40, 64) and torch.equal(l0.w_ukv[54:, :37], w["l0.mix.uv"]) and not l0.w_ukv[:, 37:].any()
    assert torch.equal(l1.w_up[0::2, :70], w["l1.mlp.gate"]) and torch.equal(l1.b_up[1::2], w["l1.mlp.up.b"].float())
    assert l0.sink is None and l1.kv_norm.shape == (19,) and l2.kv_norm is None and l2.kv_from == 1 and l2.ff_kind == seq_model.FF_NONE
    assert torch.equal(l1.hc2.mix, w["l1.hc2.mix"].float()) and l2.hc2 is None and p.norm_offset == 0.0 and p.pos.shape == (512, 128)
    for name in ("l0.mix.dkv.norm", "l1.hc1.mix", "l1.mlp.down.b", "pos"):
        bad = {n: (t[:-1] if n == name else t) for n, t in w.items()}
        with pytest.raises(ValueError, match=re.escape(name)):
            kagapel.pack_weights(kagapel.parse_config(cfg), bad, torch.bfloat16, "cpu")


def test_safetensors_files(tmp_path):
    from safetensors.torch import load_file, save_file
    t = {"a": torch.randn(3, 5), "b": torch.arange(7).int(), "c": torch.randn(2, 3).bfloat16(), "s": torch.tensor(0.5).bfloat16(), "e": torch.zeros(0, 4)}
    save_file(t, str(tmp_path / "x.safetensors"), metadata={"format": "pt"})
    got = weights.read_weights(str(tmp_path))
    assert set(got) == set(t) and all(torch.equal(got[n], t[n]) and got[n].dtype == t[n].dtype for n in t)
    weights.write_safetensors(str(tmp_path / "y.safetensors"), t)
    back = load_file(str(tmp_path / "y.safetensors"))
    assert all(torch.equal(back[n], t[n]) for n in t)
    (tmp_path / "bad").mkdir()
    with pytest.raises(FileNotFoundError):
        weights.read_weights(str(tmp_path / "bad"))
    (tmp_path / "bad" / "z.safetensors").write_bytes(b"\xff" * 20)
    with pytest.raises(ValueError):
        weights.read_weights(str(tmp_path / "bad"))


def test_registry(tmp_path):
    assert registry.architectures() == ["GPTNeoXForCausalLM", "Kagapel", "Nibotar"]
    assert registry.dtypes_of({"architecture": "Nibotar"}) == registry.dtypes_of({"architecture": "Kagapel"}) == ("bfloat16", "float32")
    assert registry.architecture_of({"architectures": ["GPTNeoXForCausalLM"]}) == "GPTNeoXForCausalLM"
    with pytest.raises(ValueError):
        registry.architecture_of({"architectures": ["Other"]})
    (tmp_path / "config.json").write_text(json.dumps({"architectures": ["GPTNeoXForCausalLM"]}))
    with pytest.raises(ValueError):
        registry.load_model(str(tmp_path), "float32")
    assert trace.main(["--model", str(tmp_path), "--dtype", "float32", "--out", str(tmp_path)]) == 3


def test_there_is_no_cpu_path():
    cfg = M.CASES["plain"]
    with pytest.raises(RuntimeError):
        nibotar.from_tensors(cfg, M.weights(cfg), device="cpu")


# ---- engine --------------------------------------------------------------------------------------------------------

class Counting:
    """A stand-in model: the next token is the number of tokens the sequence has seen, modulo the vocabulary."""
    vocab, architecture = 50, "counting"

    def __init__(self, slots, capacity):
        self.slots, self.capacity, self.seen, self.calls = slots, capacity, [0] * slots, []

    def forward(self, slot, tokens, pos, want=()):
        if pos == 0:
            self.seen[slot] = 0
        assert self.seen[slot] == pos and len(tokens) > 0 and pos + len(tokens) <= self.capacity
        self.seen[slot] += len(tokens)
        self.calls.append(("forward", slot, pos, len(tokens)))
        out = torch.zeros(len(want), self.vocab)
        for r, w in enumerate(want):
            out[r, (pos + w + 1) % self.vocab] = 1
        return out

    def decode(self, slot, token, pos, n):
        assert self.seen[slot] == pos and token == pos % self.vocab and pos + n <= self.capacity
        self.seen[slot] += n
        self.calls.append(("decode", slot, pos, n))
        return [(pos + i + 1) % self.vocab for i in range(n)]


@pytest.mark.parametrize("slots,portion,burst", [(1, 100, 100), (1, 3, 2), (2, 4, 1), (5, 1, 7)])
def test_engine_runs_every_request(slots, portion, burst):
    m = Counting(slots, 60)
    prompts = [[1] * n for n in (5, 1, 17, 9)]
    e = E.Engine(m, portion, burst)
    assert e.generate(prompts, 20) == [[(len(p) + i) % 50 for i in range(20)] for p in prompts]
    assert e.states.free == slots and max(n for k, _, _, n in m.calls if k == "forward") <= portion
    assert max([n for k, _, _, n in m.calls if k == "decode"]) <= burst
    assert e.generate(prompts[:1], 0) == [[]] and e.generate([[1]], 1) == [[1]]
    assert e.generate([[1] * 5], 20, stop=[8]) == [[5, 6, 7, 8]]


def test_engine_takes_turns_and_keeps_order():
    m = Counting(2, 60)
    e = E.Engine(m, portion=4, burst=2)
    a, b, c = (e.add(E.Request(n, [1] * 8, 4)) for n in "abc")
    assert [e.step().id for _ in range(4)] == ["a", "b", "a", "b"]
    e.run()
    assert a.done and b.done and c.done and [r.tokens for r in (a, b, c)] == [[8, 9, 10, 11]] * 3
    assert e.step() is None


def test_engine_refuses():
    e = E.Engine(Counting(1, 10))
    for bad in (E.Request("x", [], 3), E.Request("x", [1], -1), E.Request("x", [1] * 8, 4)):
        with pytest.raises(ValueError):
            e.add(bad)
    e.feed("k", [1, 2])
    with pytest.raises(RuntimeError):
        e.feed("other", [1])
    with pytest.raises(RuntimeError):
        e.feed("k", [1] * 9)
    assert e.states.position("k") == 2
    e.finish("k")
    assert e.states.free == 1
    with pytest.raises(ValueError):
        E.Engine(Counting(1, 10), portion=0)


# ---- C ABI ---------------------------------------------------------------------------------------------------------

def test_every_declared_function_is_exported():
    text = open(os.path.join(ROOT, "include", "cfpp_seq.h")).read()
    names = set(re.findall(r"\b(cfpp_seq_\w+)\s*\(", re.sub(r"/\*.*?\*/", "", text, flags=re.S)))
    lib = ctypes.CDLL(os.path.join(ROOT, "clusterfusionplus_amd", "libcfpp_seq.so"))
    assert len(names) >= 11 and not [n for n in names if not hasattr(lib, n)]


def test_structures_match_the_header(tmp_path):
    """Size and field offsets of the ctypes structures against a C compiler's."""
    checks = []
    for cls, name in ((seq_model._Layer, "cfpp_seq_layer"), (seq_model._Desc, "cfpp_seq_desc")):
        checks.append((f"sizeof({name})", ctypes.sizeof(cls)))
        checks += [(f"offsetof({name}, {f})", getattr(cls, f).offset) for f, _ in cls._fields_]
    src = '#include "cfpp_seq.h"\n#include <stdio.h>\nint main(void) {' + "".join(f'printf("%zu\\n", {c});' for c, _ in checks) + "return 0;}"
    (tmp_path / "t.c").write_text(src)
    subprocess.run(["gcc", "-I" + os.path.join(ROOT, "include"), str(tmp_path / "t.c"), "-o", str(tmp_path / "t")], check=True)
    out = subprocess.run([str(tmp_path / "t")], capture_output=True, text=True, check=True).stdout.split()
    assert [int(x) for x in out] == [v for _, v in checks]


def test_row_pitch():
    lib = seq_model._load()
    for k in (1, 63, 64, 65, 100, 4096):
        for code, dt in ((0, torch.bfloat16), (1, torch.float32)):
            assert lib.cfpp_seq_row_pitch(k, code) == seq_model.pad_rows(torch.zeros(1, k), dt, "cpu").shape[1] * (2 if code == 0 else 4)
