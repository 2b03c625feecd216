"""Nibotar: a decoder-only language model with norms after the residual sums, chunked attention with sinks, values mixed
across layers, and feed-forwards that are squared-relu layers or experts chosen by a table of token ids.

This file reads its configuration and its checkpoint; the computation is the sequence-model library's
(`seq_model.SeqModel`, include/cfpp_seq.h), which any design made of the same pieces can use."""
from __future__ import annotations

from dataclasses import dataclass
from typing import Dict, List, Optional

import torch

from .seq_model import FF_NONE, FF_RELU2, FF_TABLE_EXPERTS, SeqLayer, SeqModel, SeqWeights, interleave, pad_rows, vector
from .weights import read_config, read_weights, take

ARCHITECTURE = "Nibotar"


@dataclass(frozen=True)
class AttentionConfig:
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    scale: float
    chunk: int            # 0: causal only
    rot_dims: int         # 0: no rotation
    rot_base: float
    v_mix: bool


@dataclass(frozen=True)
class FeedForwardConfig:
    kind: str             # "dense" or "moe"
    ff: int               # of one expert with "moe"
    experts: int = 0
    top: int = 0
    shared_ff: int = 0    # 0: no shared expert


@dataclass(frozen=True)
class LayerConfig:
    attention: AttentionConfig
    mlp: Optional[FeedForwardConfig]


@dataclass(frozen=True)
class NibotarConfig:
    width: int
    vocab: int
    eps: float
    alpha: float
    softcap: float        # 0: none
    layers: List[LayerConfig]


def parse_config(cfg: dict) -> NibotarConfig:
    layers = []
    for i, entry in enumerate(cfg["layers"]):
        if entry["type"] != "attention":
            raise ValueError(f"layer {i}: unknown mixer {entry['type']!r}")
        m, rot = entry["mixer"], entry["mixer"].get("rot") or {}
        if m["heads"] % m["kv_heads"]:
            raise ValueError(f"layer {i}: {m['heads']} query heads do not share {m['kv_heads']} key/value heads evenly")
        att = AttentionConfig(heads=int(m["heads"]), kv_heads=int(m["kv_heads"]), dim=int(m["dim"]), vdim=int(m["vdim"]),
                              scale=float(m["scale"]), chunk=int((m.get("mask") or {}).get("size") or 0),
                              rot_dims=int(rot.get("dims") or 0), rot_base=float(rot.get("base") or 10000.0), v_mix=bool(m.get("v_mix", False)))
        f = entry.get("mlp")
        if f is None:
            mlp = None
        elif f["kind"] == "dense":
            mlp = FeedForwardConfig("dense", int(f["ff"]))
        elif f["kind"] == "moe":
            mlp = FeedForwardConfig("moe", int(f["expert"]["ff"]), int(f["router"]["experts"]), int(f["router"]["top"]),
                                    int((f.get("shared") or {}).get("ff") or 0))
        else:
            raise ValueError(f"layer {i}: unknown feed-forward {f['kind']!r}")
        layers.append(LayerConfig(att, mlp))
    return NibotarConfig(width=int(cfg["width"]), vocab=int(cfg["vocab"]), eps=float(cfg["norm"]["eps"]), alpha=float(cfg["postln_alpha"]),
                         softcap=float(cfg.get("logit_softcap") or 0.0), layers=layers)


def pack_weights(cfg: NibotarConfig, weights: Dict[str, torch.Tensor], dtype: torch.dtype, device) -> SeqWeights:
    """Checkpoint tensors -> the library's layout: q, k and v rows in one matrix, gate and up rows interleaved, experts one
    after the other, rows padded."""
    W = cfg.width

    def mat(t):
        return pad_rows(t, dtype, device)

    layers = []
    for i, l in enumerate(cfg.layers):
        p, a = f"l{i}.", l.attention
        nq, nk, nv = a.heads * a.dim, a.kv_heads * a.dim, a.kv_heads * a.vdim
        m = p + "mix."
        rows = ((m + "q", nq), (m + "k", nk), (m + "v", nv))
        kw = dict(heads=a.heads, kv_heads=a.kv_heads, dim=a.dim, vdim=a.vdim, scale=a.scale, chunk=a.chunk, rot_dims=a.rot_dims,
                  rot_base=a.rot_base, v_mix=a.v_mix,
                  w_qkv=mat(torch.cat([take(weights, n, (r, W)) for n, r in rows])),
                  b_qkv=vector(torch.cat([take(weights, n + ".b", (r,)) for n, r in rows]), device),
                  q_norm=vector(take(weights, m + "q.norm", (nq,)), device), k_norm=vector(take(weights, m + "k.norm", (nk,)), device),
                  sink=vector(take(weights, m + "sink", (a.heads,)), device), w_o=mat(take(weights, m + "o", (W, a.heads * a.vdim))),
                  norm1=vector(take(weights, p + "norm1", (W,)), device))
        if a.v_mix and any(e.attention.v_mix for e in cfg.layers[:i]):
            kw["v_lambda"] = float(take(weights, m + "vmix", ()).float())
        f, m = l.mlp, p + "mlp."
        if f is None:
            kw["ff_kind"] = FF_NONE
        elif f.kind == "dense":
            kw.update(ff_kind=FF_RELU2, ff=f.ff, w_up=mat(take(weights, m + "up", (f.ff, W))), w_down=mat(take(weights, m + "down", (W, f.ff))))
        else:
            table = take(weights, m + "table", (cfg.vocab, f.top))
            if int(table.min()) < 0 or int(table.max()) >= f.experts:
                raise ValueError(f"checkpoint: {m}table names experts outside 0 .. {f.experts - 1}")
            # (expert by expert: the interleaved copy of one is all that exists beside the packed matrices)
            up = torch.stack([mat(interleave(take(weights, f"{m}e{e}.gate", (f.ff, W)), take(weights, f"{m}e{e}.up", (f.ff, W))))
                              for e in range(f.experts)])
            down = torch.stack([mat(take(weights, f"{m}e{e}.down", (W, f.ff))) for e in range(f.experts)])
            kw.update(ff_kind=FF_TABLE_EXPERTS, ff=f.ff, experts=f.experts, top=f.top, shared_ff=f.shared_ff, w_up=up, w_down=down,
                      table=table.to(device=device, dtype=torch.int32).contiguous())
            if f.shared_ff:
                kw.update(w_shared_up=mat(interleave(take(weights, m + "shared.gate", (f.shared_ff, W)), take(weights, m + "shared.up", (f.shared_ff, W)))),
                          w_shared_down=mat(take(weights, m + "shared.down", (W, f.shared_ff))))
        if f is not None:
            kw["norm2"] = vector(take(weights, p + "norm2", (W,)), device)
        layers.append(SeqLayer(**kw))
    return SeqWeights(dtype=dtype, width=W, vocab=cfg.vocab, eps=cfg.eps, alpha=cfg.alpha, softcap=cfg.softcap, layers=layers,
                      embed=mat(take(weights, "embed", (cfg.vocab, W))), final_norm=vector(take(weights, "final.norm", (W,)), device),
                      head=mat(take(weights, "head", (cfg.vocab, W))), architecture=ARCHITECTURE)


def from_tensors(config: dict, weights: Dict[str, torch.Tensor], dtype=torch.bfloat16, capacity: int = 4096, slots: int = 1,
                 max_portion: int = 2048, device="cuda") -> SeqModel:
    """A model on the device from a config.json dictionary and the checkpoint's tensors."""
    return SeqModel(pack_weights(parse_config(config), weights, dtype, device), capacity=capacity, slots=slots, max_portion=max_portion)


def load(path: str, dtype=torch.bfloat16, capacity: int = 4096, slots: int = 1, max_portion: int = 2048, device="cuda") -> SeqModel:
    from .build import ensure_seq
    ensure_seq()
    return from_tensors(read_config(path), read_weights(path), dtype, capacity, slots, max_portion, device)
