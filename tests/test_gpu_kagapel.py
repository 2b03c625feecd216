"""Kagapel on the GPU against the plain oracle: every mechanism, portions, decoding, slots, generation, entry points; and the
sequence library's mechanisms in other combinations than the two designs have."""
import functools
import io
import json
import os
import subprocess
import sys

import numpy as np
import pytest
import torch

from oracle import kagapel_oracle as KO
from oracle import nibotar_oracle as NO
from tests import kagapel_models as M
from tests import nibotar_models as NM

pytestmark = pytest.mark.gpu
LIMIT = {torch.float32: 3e-5, torch.bfloat16: 4e-2}
DTYPES = [torch.float32, torch.bfloat16]
IDS = ["f32", "bf16"]


def build(cfg, w, dtype, capacity=400, slots=1, max_portion=2048):
    from clusterfusionplus_amd import kagapel
    return kagapel.from_tensors(cfg, w, dtype, capacity=capacity, slots=slots, max_portion=max_portion)


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


# (norms over one or two values: bf16 inputs alone move the logits by a tenth of their spread)
@pytest.mark.parametrize("name,dtype", [(n, d) for n in M.CASES for d in DTYPES if n != "one_of_each" or d == torch.float32],
                         ids=lambda v: v if isinstance(v, str) else IDS[DTYPES.index(v)])
def test_prompt_and_decoding_match_the_oracle(name, dtype):
    cfg, w, toks, want, res = reference(name)
    m = build(cfg, w, dtype)
    logits, layers = m.forward(0, toks, 0, range(len(toks)), residuals=True)
    for i in range(len(cfg["layers"])):
        assert M.error(layers[i], res[i]) < LIMIT[dtype], f"residual streams after layer {i}"
    assert M.error(logits, want) < LIMIT[dtype]
    # token by token, in the same slot: the decode kernels, from the first position on
    rows = [m.forward(0, [t], i, [0], residuals=True) for i, t in enumerate(toks)]
    for i in range(len(cfg["layers"])):
        assert M.error(torch.stack([r[1][i, 0] for r in rows]), res[i]) < LIMIT[dtype], f"decoded: residual streams after layer {i}"
    assert M.error(torch.cat([r[0] for r in rows]), want) < LIMIT[dtype]


@pytest.mark.parametrize("dtype", DTYPES, ids=IDS)
@pytest.mark.parametrize("sizes", [(2,), (3, 1, 2), (37,), (24, 13, 61), (1, 50, 1, 1), (32, 64)], ids=str)
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


# ---- far keys, sinks ------------------------------------------------------------------------------------------------

@pytest.mark.parametrize("dtype", DTYPES, ids=IDS)
@pytest.mark.parametrize("rotated", [False, True], ids=["plain", "rotated"])
@pytest.mark.parametrize("at", [0, 1, 15, 16, 31, 32, 63, 64, 69])
def test_key_at_a_tile_edge(at, rotated, dtype):
    cfg, w, toks = M.far_key_model(5, 24, 75, at, rotated)
    want = M.oracle(cfg, w, toks)
    m = build(cfg, w, dtype)
    assert M.error(m.forward(0, toks, 0, range(len(toks))), want) < LIMIT[dtype]
    assert M.error(run_portions(m, toks, (1,)), want) < LIMIT[dtype]
    for sizes in ((at + 1, 2), (max(at, 1), 3), (33, 31)):
        assert M.error(run_portions(m, toks, sizes), want) < LIMIT[dtype]


@pytest.mark.parametrize("dtype", DTYPES, ids=IDS)
@pytest.mark.parametrize("heads,rank,length,at", [(3, 24, 1500, 3), (20, 136, 1500, 1400), (40, 24, 1300, 700), (3, 300, 2300, 1023)])
def test_far_key_with_many_splits(heads, rank, length, at, dtype):
    """Long caches: decode steps that share the keys among many workgroups, some with several tiles; prompts of many tiles."""
    cfg, w, toks = M.far_key_model(heads, rank, length, at)
    want = M.oracle(cfg, w, toks)
    m = build(cfg, w, dtype, capacity=2400)
    assert M.error(m.forward(0, toks, 0, range(length)), want) < LIMIT[dtype]
    cut = length - 45
    m.forward(0, toks[:cut], 0)
    assert M.error(torch.cat([m.forward(0, [t], cut + i, [0]) for i, t in enumerate(toks[cut:])]), want[cut:]) < LIMIT[dtype]
    assert M.error(run_portions(m, toks, (611, 2, 300)), want) < LIMIT[dtype]


@pytest.mark.parametrize("dtype", DTYPES, ids=IDS)
@pytest.mark.parametrize("heads,rank", [(3, 500), (40, 60)])
def test_very_long_caches_decoded_like_a_prompt(heads, rank, dtype):
    """More splits than a workgroup that merges them takes at a time, against the same positions of a whole prompt."""
    length, n = 9000, 4
    for at in (8990, 77):
        cfg, w, toks = M.far_key_model(heads, rank, length, at)
        m = build(cfg, w, dtype, capacity=length, max_portion=length)
        want = m.forward(0, toks, 0, range(length - n, length)).cpu()
        other = m.forward(0, [1 if t == 0 else t for t in toks], 0, [length - 1]).cpu()
        assert M.error(other, want[-1:]) > 0.2       # the key is seen
        m.forward(0, toks[:length - n], 0)
        got = torch.cat([m.forward(0, [t], length - n + i, [0]) for i, t in enumerate(toks[length - n:])])
        assert M.error(got, want) < LIMIT[dtype]


@pytest.mark.parametrize("dtype", DTYPES, ids=IDS)
@pytest.mark.parametrize("level", [-20.0, 0.0, 12.0])
def test_sinks_of_any_size(level, dtype):
    cfg, w, toks, _, _ = reference("sinks")
    w = {n: (torch.full_like(t, level) if n.endswith("sink") else t) for n, t in w.items()}
    want = M.oracle(cfg, w, toks)
    m = build(cfg, w, dtype)
    assert M.error(m.forward(0, toks, 0, range(len(toks))), want) < LIMIT[dtype]
    assert M.error(run_portions(m, toks, (1,)), want) < LIMIT[dtype]


def test_long_decoding():
    cfg, w, toks, want, _ = reference("everything", 330, seed=11)
    m = build(cfg, w, torch.float32)
    m.forward(0, toks[:3], 0)
    got = torch.cat([m.forward(0, [t], 3 + i, [0]) for i, t in enumerate(toks[3:])])
    assert M.error(got, want[3:]) < LIMIT[torch.float32]


def test_shared_latents_cost_no_cache():
    """A layer that reads another one's latents has no cache rows of its own."""
    cfg, w, _, _, _ = reference("shared_latents")
    own = {**cfg, "layers": [{**l, "mixer": {k: v for k, v in l["mixer"].items() if k != "kv_from"}} for l in cfg["layers"]]}
    row = 128 + 64                                       # 36 bf16 latents padded to 128 bytes, 12 rotated values to 64
    sizes = [build(c, M.weights(c), torch.bfloat16, capacity=512, slots=s).bytes_allocated for c in (cfg, own) for s in (1, 9)]
    assert sizes[1] - sizes[0] == 8 * 512 * row * 2 and sizes[3] - sizes[2] == 8 * 512 * row * 6


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
    tight = 3e-5 if dtype == torch.float32 else 3e-2
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
@pytest.mark.parametrize("name", ["everything", "twenty_heads"])
def test_graph_replays_equal_eager_steps(name, dtype):
    cfg, w, toks, _, _ = reference(name)
    m = build(cfg, w, dtype, slots=2)
    for slot in (0, 1):
        m.forward(slot, toks[:60], 0)
    m.set_state(toks[60], 60, slot=0)
    m.step(25)
    eager, logits = m.generated(), m.logits.clone()
    for _ in range(2):
        # nothing is taken over: the sequence is wound back and goes on from the same position
        m.set_state(toks[60], 60, slot=1)
        m.graph_steps(25)
        assert m.generated() == eager and torch.equal(m.logits, logits)
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
    cfg, w, toks, _, _ = reference("one_stream")
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
    # a sequence ends where the position vectors end
    short = {**cfg, "max_positions": 30}
    m = build(short, {**w, "pos": w["pos"][:30]}, torch.float32, capacity=400)
    assert m.capacity == 30
    with pytest.raises(RuntimeError):
        m.forward(0, toks[:31], 0)
    assert M.error(m.forward(0, toks[:30], 0, range(30)), M.oracle(cfg, w, toks[:30])) < LIMIT[torch.float32]


def test_descriptions_the_library_refuses():
    from clusterfusionplus_amd import kagapel
    from clusterfusionplus_amd.seq_model import SeqModel
    cfg, w, _, _, _ = reference("shared_latents")

    def packed():
        return kagapel.pack_weights(kagapel.parse_config(cfg), w, torch.bfloat16, "cuda")
    for change in (dict(kv_from=1), dict(kv_from=4), dict(kv_rank=35), dict(kv_rank=513), dict(rot_dims=130), dict(dim=257), dict(rot_dims=7),
                   dict(w_ukv=None), dict(hc1=None), dict(mixer=2), dict(chunk=5), dict(rot_factor=-1.0)):
        p = packed()
        for n, v in change.items():
            setattr(p.layers[1], n, v)
        with pytest.raises(RuntimeError):
            SeqModel(p, capacity=64)
    for n, v in (("streams", 9), ("streams", 0), ("pos", packed().pos[:40])):
        p = packed()
        setattr(p, n, v)
        with pytest.raises(RuntimeError):
            SeqModel(p, capacity=64)


# ---- checkpoints and entry points ----------------------------------------------------------------------------------

@pytest.fixture(scope="module")
def checkpoint(tmp_path_factory):
    from clusterfusionplus_amd.weights import write_safetensors
    d = tmp_path_factory.mktemp("kagapel")
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


# ---- other combinations of the library's mechanisms ----------------------------------------------------------------

def grouped_layer_in_streams():
    """A Nibotar layer (chunked grouped attention; experts chosen by a table, and a shared one) inside three streams."""
    from clusterfusionplus_amd import nibotar
    from clusterfusionplus_amd.seq_model import Connections
    cfg = NM.model(64, 51, [(NM.attn(4, 2, 24, 16, chunk=13), NM.moe(20, 6, 2, shared=44)), (NM.attn(2, 1, 16, 16), NM.dense(40))], softcap=None)
    w, S = NM.weights(cfg, 7), 3
    like = M.weights(M.model(64, 51, [M.gated(1, 8, 8, 8, 8, ff=8)] * 2, streams=S), 8)

    def pack(dtype):
        p = nibotar.pack_weights(nibotar.parse_config(cfg), w, dtype, "cuda")
        p.streams, p.logit_scale, p.norm_offset = S, 0.5, 1.0
        for i, l in enumerate(p.layers):
            l.hc1, l.hc2 = (Connections(*(like[f"l{i}.hc{q}.{n}"].float().cuda().contiguous() for n in ("in", "mix", "out"))) for q in (1, 2))
        return p

    def forward(toks):
        d = {n: (t.double() if t.is_floating_point() else t) for n, t in {**like, **w}.items()}
        x, eps = d["embed"][torch.tensor(toks)], cfg["norm"]["eps"]
        xs = [x] * S
        for i, layer in enumerate(cfg["layers"]):
            pre = f"l{i}."
            h = NO.norm_one_plus(KO.streams_in(d, pre + "hc1.", xs), d[pre + "norm1"], eps)
            xs = KO.streams_out(d, pre + "hc1.", xs, NO.attention(d, pre + "mix.", layer["mixer"], eps, h, None)[0])
            h = NO.norm_one_plus(KO.streams_in(d, pre + "hc2.", xs), d[pre + "norm2"], eps)
            y = NO.relu_squared_mlp(d, pre + "mlp.", h) if layer["mlp"]["kind"] == "dense" else NO.table_experts(d, pre + "mlp.", layer["mlp"], toks, h)
            xs = KO.streams_out(d, pre + "hc2.", xs, y)
        return 0.5 * NO.norm_one_plus(sum(xs), d["final.norm"], eps) @ d["head"].T
    return pack, forward, 51


def latent_layer_with_norms_after():
    """A Kagapel layer inside Nibotar's residual sum, x <- norm(alpha x + f(x))."""
    from clusterfusionplus_amd import kagapel
    cfg = M.model(64, 51, [M.gated(3, 16, 8, 24, 40, ff=72), M.sunk(5, 8, 8, 8, 24)], streams=1, logit_scale=2.0)
    w = M.weights(cfg, 9)

    def pack(dtype):
        p = kagapel.pack_weights(kagapel.parse_config(cfg), w, dtype, "cuda")
        p.streams, p.pos, p.alpha, p.softcap = 0, None, 1.3, 6.0
        return p

    def forward(toks):
        d = {n: t.double() for n, t in w.items()}
        x, eps = d["embed"][torch.tensor(toks)], cfg["norm"]["eps"]
        for i, layer in enumerate(cfg["layers"]):
            pre = f"l{i}."
            c, kr = KO.latents(d, pre + "mix.", layer["mixer"], eps, x)
            second = layer["type"] == "latent_attention_2"
            y = KO.latent_attention(d, pre + "mix.", layer["mixer"], x, c, kr, d[pre + "mix.sink"] if second else None, not second)
            x = KO.rms_norm(1.3 * x + y, d[pre + "norm1"], eps)
            if layer["mlp"]:
                x = KO.rms_norm(1.3 * x + KO.gated_mlp(d, pre + "mlp.", x), d[pre + "norm2"], eps)
        return NO.softcap(2.0 * KO.rms_norm(x, d["final.norm"], eps) @ d["head"].T, 6.0)
    return pack, forward, 51


@pytest.mark.parametrize("dtype", DTYPES, ids=IDS)
@pytest.mark.parametrize("make", [grouped_layer_in_streams, latent_layer_with_norms_after])
def test_mechanisms_combine(make, dtype):
    from clusterfusionplus_amd.seq_model import SeqModel
    pack, forward, vocab = make()
    toks = torch.randint(0, vocab, (60,), generator=torch.Generator().manual_seed(4)).tolist()
    want = forward(toks)
    m = SeqModel(pack(dtype), capacity=64)
    for sizes in ((60,), (1,), (7, 2, 1)):
        assert M.error(run_portions(m, toks, sizes), want) < LIMIT[dtype]
