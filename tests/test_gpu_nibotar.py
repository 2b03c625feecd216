"""Nibotar on the GPU against the plain oracle: every mechanism, portions, decoding, slots, generation, entry points."""
import functools
import io
import json
import os
import subprocess
import sys

import numpy as np
import pytest
import torch

from tests import nibotar_models as M

pytestmark = pytest.mark.gpu
LIMIT = {torch.float32: 3e-5, torch.bfloat16: 4e-2}
DTYPES = [torch.float32, torch.bfloat16]
IDS = ["f32", "bf16"]


def build(cfg, w, dtype, capacity=400, slots=1, max_portion=2048):
    from clusterfusionplus_amd import nibotar
    return nibotar.from_tensors(cfg, w, dtype, capacity=capacity, slots=slots, max_portion=max_portion)


@functools.lru_cache(maxsize=None)
def reference(name, n=90, seed=3):
    cfg = M.CASES[name]
    w, toks, res = M.weights(cfg, seed), M.prompt(cfg, n, seed + 1), []
    return cfg, w, toks, M.oracle(cfg, w, toks, res), torch.stack(res)


def run_portions(m, toks, sizes, slot=0):
    """All logits of a sequence fed in portions of the given sizes (cycled)."""
    out, pos, i = [], 0, 0
    while pos < len(toks):
        n = min(sizes[i % len(sizes)], len(toks) - pos)
        out.append(m.forward(slot, toks[pos:pos + n], pos, range(n)))
        pos, i = pos + n, i + 1
    return torch.cat(out)


@pytest.mark.parametrize("dtype", DTYPES, ids=IDS)
@pytest.mark.parametrize("name", list(M.CASES))
def test_prompt_and_decoding_match_the_oracle(name, dtype):
    cfg, w, toks, want, res = reference(name)
    m = build(cfg, w, dtype)
    logits, layers = m.forward(0, toks, 0, range(len(toks)), residuals=True)
    for i in range(len(cfg["layers"])):
        assert M.error(layers[i], res[i]) < LIMIT[dtype], f"residual stream after layer {i}"
    assert M.error(logits, want) < LIMIT[dtype]
    # token by token, in the same slot: the decode kernels, from the first position on
    rows = [m.forward(0, [t], i, [0], residuals=True) for i, t in enumerate(toks)]
    for i in range(len(cfg["layers"])):
        assert M.error(torch.stack([r[1][i, 0] for r in rows]), res[i]) < LIMIT[dtype], f"decoded: residual stream after layer {i}"
    assert M.error(torch.cat([r[0] for r in rows]), want) < LIMIT[dtype]


@pytest.mark.parametrize("dtype", DTYPES, ids=IDS)
@pytest.mark.parametrize("sizes", [(2,), (3, 1, 2), (37,), (24, 13, 61), (1, 50, 1, 1)], ids=str)
def test_portions(sizes, dtype):
    cfg, w, toks, want, _ = reference("everything", 150)
    assert M.error(run_portions(build(cfg, w, dtype), toks, sizes), want) < LIMIT[dtype]


@pytest.mark.parametrize("portion", [2, 7, 37, 64])
def test_passes_inside_one_call(portion):
    """A call longer than the model's pass size is cut into passes."""
    cfg, w, toks, want, res = reference("everything", 150)
    m = build(cfg, w, torch.float32, max_portion=portion)
    logits, layers = m.forward(0, toks, 0, range(len(toks)), residuals=True)
    assert M.error(logits, want) < LIMIT[torch.float32]
    assert M.error(layers[-1], res[-1]) < LIMIT[torch.float32]


def test_wanted_places_in_any_number_and_order():
    cfg, w, toks, want, _ = reference("everything")
    m = build(cfg, w, torch.float32)
    assert m.forward(0, toks, 0, []).shape == (0, cfg["vocab"])
    for places in ([0], [len(toks) - 1], [5, 3, 3, 80]):
        assert M.error(m.forward(0, toks, 0, places), want[places]) < LIMIT[torch.float32]


def test_results_do_not_depend_on_the_cut_beyond_rounding():
    cfg, w, toks, _, _ = reference("everything", 150)
    m = build(cfg, w, torch.float32)
    whole = m.forward(0, toks, 0, range(len(toks)))
    for sizes in ((2,), (1,), (36, 2), (61, 3)):
        assert M.error(run_portions(m, toks, sizes), whole.cpu()) < LIMIT[torch.float32]


# ---- chunk edges, far keys, sinks ----------------------------------------------------------------------------------

@pytest.mark.parametrize("dtype", DTYPES, ids=IDS)
@pytest.mark.parametrize("at", [0, 1, 19, 20, 39, 40, 41, 59])
def test_key_at_a_chunk_edge(at, dtype):
    cfg, w, toks = M.edge_model(20, 70, at)
    want = M.oracle(cfg, w, toks)
    m = build(cfg, w, dtype)
    assert M.error(m.forward(0, toks, 0, range(len(toks))), want) < LIMIT[dtype]
    assert M.error(run_portions(m, toks, (1,)), want) < LIMIT[dtype]
    for sizes in ((19, 1, 20), (at + 1, 2), (max(at, 1), 3), (21, 38)):
        assert M.error(run_portions(m, toks, sizes), want) < LIMIT[dtype]


@pytest.mark.parametrize("dtype", DTYPES, ids=IDS)
@pytest.mark.parametrize("chunk,length,at", [(None, 1500, 3), (None, 1500, 1400), (1024, 1300, 700), (700, 1401, 700), (700, 1401, 699)])
def test_far_key_with_many_splits(chunk, length, at, dtype):
    """Long caches: decode steps that share a head's keys among many workgroups, prompts of many key tiles."""
    cfg, w, toks = M.edge_model(chunk, length, at)
    want = M.oracle(cfg, w, toks)
    m = build(cfg, w, dtype, capacity=1600)
    assert M.error(m.forward(0, toks, 0, range(length)), want) < LIMIT[dtype]
    cut = length - 45
    m.forward(0, toks[:cut], 0)
    assert M.error(torch.cat([m.forward(0, [t], cut + i, [0]) for i, t in enumerate(toks[cut:])]), want[cut:]) < LIMIT[dtype]
    assert M.error(run_portions(m, toks, (611, 2, 300)), want) < LIMIT[dtype]


@pytest.mark.parametrize("dtype", DTYPES, ids=IDS)
@pytest.mark.parametrize("level", [-20.0, 0.0, 12.0])
def test_sinks_of_any_size(level, dtype):
    cfg, w, toks, _, _ = reference("chunks")
    w = {n: (torch.full_like(t, level) if n.endswith("sink") else t) for n, t in w.items()}
    want = M.oracle(cfg, w, toks)
    m = build(cfg, w, dtype)
    assert M.error(m.forward(0, toks, 0, range(len(toks))), want) < LIMIT[dtype]
    assert M.error(run_portions(m, toks, (1,)), want) < LIMIT[dtype]


def test_long_decoding_over_many_chunks():
    cfg, w, toks, want, _ = reference("everything", 330, seed=11)
    m = build(cfg, w, torch.float32)
    m.forward(0, toks[:3], 0)
    got = torch.cat([m.forward(0, [t], 3 + i, [0]) for i, t in enumerate(toks[3:])])
    assert M.error(got, want[3:]) < LIMIT[torch.float32]


# ---- slots ---------------------------------------------------------------------------------------------------------

@pytest.mark.parametrize("dtype", DTYPES, ids=IDS)
def test_sequences_in_turns_and_slots_used_again(dtype):
    cfg, w, _, _, _ = reference("everything")
    seqs = [M.prompt(cfg, n, 20 + n) for n in (90, 7, 64, 33)]
    m = build(cfg, w, dtype, slots=3)
    alone = [build(cfg, w, dtype).forward(0, s, 0, range(len(s))).cpu() for s in seqs]
    for s, want in zip(seqs, alone):
        assert M.error(want, M.oracle(cfg, w, s)) < LIMIT[dtype]
    # three live sequences take turns; the fourth takes over the slot of the first that ends
    feeds = {0: (0, 5), 1: (1, 3), 2: (2, 11)}
    pos, out = {i: 0 for i in range(4)}, {i: [] for i in range(4)}
    while feeds:
        for i, (slot, size) in list(feeds.items()):
            n = min(size, len(seqs[i]) - pos[i])
            out[i].append(m.forward(slot, seqs[i][pos[i]:pos[i] + n], pos[i], range(n)).cpu())
            pos[i] += n
            if pos[i] == len(seqs[i]):
                del feeds[i]
                if i == 1:
                    feeds[3] = (slot, 1)
    tight = 3e-5 if dtype == torch.float32 else 2e-2
    for i in range(4):
        assert M.error(torch.cat(out[i]), alone[i]) < tight, f"sequence {i}"


# ---- generation ----------------------------------------------------------------------------------------------------

def oracle_greedy(cfg, w, toks, n):
    out = []
    for _ in range(n):
        out.append(int(M.oracle(cfg, w, toks + out)[-1].argmax()))
    return out


@pytest.mark.parametrize("portion,burst,slots", [(2048, 32, 1), (5, 3, 2), (16, 1, 3)])
def test_generation_through_the_engine(portion, burst, slots):
    from clusterfusionplus_amd import Engine
    cfg, w, _, _, _ = reference("everything")
    prompts = [M.prompt(cfg, n, 40 + n) for n in (1, 12, 41)]
    want = [oracle_greedy(cfg, w, p, 30) for p in prompts]
    m = build(cfg, w, torch.float32, capacity=80, slots=slots)
    engine = Engine(m, portion=portion, burst=burst)
    assert engine.generate(prompts, 30) == want
    assert engine.states.free == slots
    # again, with a stop token, in slots that have been used
    stop = want[1][10]
    k = want[1].index(stop)
    assert engine.generate(prompts[1:2], 30, stop=[stop]) == [want[1][:k + 1]]


@pytest.mark.parametrize("dtype", DTYPES, ids=IDS)
def test_graph_replays_equal_eager_steps(dtype):
    cfg, w, toks, _, _ = reference("everything")
    m = build(cfg, w, dtype, slots=2)
    for slot in (0, 1):
        m.forward(slot, toks[:60], 0)
    m.set_state(toks[60], 60, slot=0)
    m.step(25)
    eager, logits = m.generated(), m.logits.clone()
    for _ in range(2):
        # (a chunk's cache rows are taken over by the next chunk: a sequence cannot be wound back, it is run again)
        m.forward(1, toks[:60], 0)
        m.set_state(toks[60], 60, slot=1)
        m.graph_steps(25)
        assert m.generated() == eager and torch.equal(m.logits, logits)
    m.forward(1, toks[:60], 0)
    # replays one at a time, with other work on the same scratch memory and reads between them
    for i in range(25):
        m.set_state(toks[60] if i == 0 else eager[i - 1], 60 + i, slot=1)
        m.graph_steps(1)
        torch.cuda.synchronize()
        assert m.generated() == [eager[i]]
        assert m.state.tolist() == [eager[i], 61 + i, 1, 1]
        last = m.logits.clone()
        m.forward(0, toks[:2 + i], 0)
    assert torch.equal(last, logits)


def test_capacity_and_arguments_are_checked():
    from clusterfusionplus_amd import Engine, Request
    cfg, w, toks, _, _ = reference("plain")
    m = build(cfg, w, torch.float32, capacity=20)
    m.forward(0, toks[:20], 0)
    for bad in (lambda: m.forward(0, toks[:1], 20), lambda: m.forward(0, toks[:21], 0), lambda: m.forward(1, toks[:1], 0),
                lambda: m.forward(0, [cfg["vocab"]], 0), lambda: m.forward(0, [-1], 0), lambda: m.forward(0, toks[:4], 0, [4]),
                lambda: m.forward(0, [], 0), lambda: m.set_state(0, 20), lambda: m.set_state(cfg["vocab"], 0)):
        with pytest.raises(RuntimeError):
            bad()
    m.set_state(1, 17)
    m.graph_steps(3)
    with pytest.raises(RuntimeError):
        m.graph_steps(1)
    with pytest.raises(ValueError):
        Engine(m).add(Request("a", toks[:15], 7))
    engine = Engine(m)
    with pytest.raises(RuntimeError):
        engine.feed("b", toks[:21], [])
    assert engine.states.free == 1


# ---- checkpoints and entry points ----------------------------------------------------------------------------------

@pytest.fixture(scope="module")
def checkpoint(tmp_path_factory):
    from clusterfusionplus_amd.weights import write_safetensors
    d = tmp_path_factory.mktemp("nibotar")
    cfg, w, _, _, _ = reference("everything")
    (d / "config.json").write_text(json.dumps(cfg))
    write_safetensors(str(d / "model.safetensors"), w)
    return str(d)


def test_command_line_generates(checkpoint, capsys):
    from clusterfusionplus_amd.__main__ import main
    cfg, w, _, _, _ = reference("everything")
    p = M.prompt(cfg, 9, 77)
    assert main(["generate", "--model", checkpoint, "--tokens", ",".join(map(str, p)), "--max-new", "6", "--dtype", "float32"]) == 0
    assert json.loads(capsys.readouterr().out.strip().splitlines()[-1]) == oracle_greedy(cfg, w, p, 6)


def trace_lines(toks):
    return [{"step": 0, "entries": [{"id": "a", "tokens": toks[:40], "want": [0, 39]}], "end": []},
            {"step": 1, "entries": [{"id": "a", "tokens": toks[40:42], "want": []}], "end": []},
            {"step": 2, "entries": [{"id": "a", "tokens": toks[42:43], "want": [0]}], "end": ["a"]},
            {"step": 3, "entries": [{"id": "b", "tokens": toks[:7], "want": [6]}], "end": ["b"]}]


def check_trace(out, text, want, vocab, limit):
    assert [ln for ln in text.splitlines() if ln.startswith("done")] == [f"done {i}" for i in range(4)]
    assert not os.path.exists(os.path.join(out, "1.f32"))
    for step, places in ((0, [0, 39]), (2, [42]), (3, [6])):
        got = torch.from_numpy(np.fromfile(os.path.join(out, f"{step}.f32"), dtype="<f4").reshape(-1, vocab))
        assert M.error(got, want[places]) < limit


def test_trace_replay(checkpoint, tmp_path, monkeypatch, capsys):
    from clusterfusionplus_amd import trace
    cfg, _, toks, want, _ = reference("everything")
    monkeypatch.setattr(sys, "stdin", io.StringIO("".join(json.dumps(s) + "\n" for s in trace_lines(toks))))
    assert trace.main(["--model", checkpoint, "--dtype", "float32", "--out", str(tmp_path), "--max-tokens", "43"]) == 0
    check_trace(str(tmp_path), capsys.readouterr().out, want, cfg["vocab"], LIMIT[torch.float32])


def test_trace_program(checkpoint, tmp_path):
    cfg, _, toks, want, _ = reference("everything")
    root = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
    r = subprocess.run([os.path.join(root, "bin", "trace_run"), "--model", checkpoint, "--dtype", "bfloat16", "--out", str(tmp_path),
                        "--max-tokens", "64"], input="".join(json.dumps(s) + "\n" for s in trace_lines(toks)), text=True,
                       capture_output=True, timeout=100, cwd=str(tmp_path))
    assert r.returncode == 0, r.stderr[-2000:]
    check_trace(str(tmp_path), r.stdout, want, cfg["vocab"], LIMIT[torch.bfloat16])


def test_neox_through_the_same_engine(tmp_path):
    """The registry's other family: a small GPT-NeoX checkpoint, generated from by the same engine."""
    from clusterfusionplus_amd import Engine, load_model
    from clusterfusionplus_amd.weights import write_safetensors
    from oracle import neox_oracle as N
    dims, L, V = N.NeoxDims(hidden=512, heads=8, head_dim=64, rotary_dim=16, ffn=2048), 2, 256
    layers = [N.make_layer_weights(dims, layer=i) for i in range(L)]
    g = torch.Generator().manual_seed(3)
    embed, head = torch.randn((V, 512), generator=g).half(), (torch.randn((V, 512), generator=g) * 0.1).half()
    fw, fb = torch.ones(512).half(), torch.zeros(512).half()
    from clusterfusionplus_amd.model import _hf_names
    t = {"gpt_neox.embed_in.weight": embed, "embed_out.weight": head, "gpt_neox.final_layer_norm.weight": fw, "gpt_neox.final_layer_norm.bias": fb}
    for i, lw in enumerate(layers):
        t.update({f"gpt_neox.layers.{i}.{n}": lw[k] for k, n in _hf_names.items()})
    write_safetensors(str(tmp_path / "model.safetensors"), t)
    (tmp_path / "config.json").write_text(json.dumps({
        "architectures": ["GPTNeoXForCausalLM"], "hidden_size": 512, "num_attention_heads": 8, "intermediate_size": 2048, "num_hidden_layers": L,
        "vocab_size": V, "layer_norm_eps": 1e-5, "rotary_pct": 0.25, "rotary_emb_base": 10000, "use_parallel_residual": True}))
    prompt = [5, 17, 200, 3]
    kc, vc = [torch.zeros(32, 512).half() for _ in range(L)], [torch.zeros(32, 512).half() for _ in range(L)]
    toks, out = list(prompt), []
    for i in range(len(prompt) + 5):
        r = N.neox_stack_decode(toks[i], embed, layers, fw, fb, head, kc, vc, i, dims)
        if i >= len(prompt) - 1:
            out.append(int(torch.argmax(r["logits"])))
            toks.append(out[-1])
    assert Engine(load_model(str(tmp_path), capacity=32)).generate([prompt], 6) == [out]
