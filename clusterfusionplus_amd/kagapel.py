"""Kagapel: a decoder-only language model with latent attention, several residual streams with learned connections, and
learned positions beside the rotary ones.

Two kinds of mixer: `latent_attention` (output gate, rotary angles that may be scaled with YaRN) and `latent_attention_2` (a
sink per head; may read another layer's cached latents).  This file reads the configuration and the checkpoint; the
computation is the sequence-model library's (`seq_model.SeqModel`, include/cfpp_seq.h), which any design made of the same
pieces can use."""
from __future__ import annotations

from dataclasses import dataclass
from typing import Dict, List, Optional

import torch

from .seq_model import FF_GATED, FF_NONE, MIX_LATENT, Connections, SeqLayer, SeqModel, SeqWeights, interleave, pad_rows, vector
from .weights import read_config, read_weights, take

ARCHITECTURE = "Kagapel"


@dataclass(frozen=True)
class Yarn:
    factor: float
    original: float
    fast: float
    slow: float


@dataclass(frozen=True)
class MixerConfig:
    heads: int
    dim: int              # plain query / key dimensions of a head
    rot_dim: int          # rotated ones
    vdim: int
    kv_rank: int
    scale: float
    rot_base: float
    yarn: Optional[Yarn]
    gated: bool
    sink: bool
    kv_from: int          # -1: the layer has latents of its own


@dataclass(frozen=True)
class LayerConfig:
    mixer: MixerConfig
    ff: int               # 0: no feed-forward


@dataclass(frozen=True)
class KagapelConfig:
    width: int
    vocab: int
    eps: float
    streams: int
    max_positions: int
    logit_scale: float
    layers: List[LayerConfig]


def parse_config(cfg: dict) -> KagapelConfig:
    layers: List[LayerConfig] = []
    for i, entry in enumerate(cfg["layers"]):
        if entry["type"] not in ("latent_attention", "latent_attention_2"):
            raise ValueError(f"layer {i}: unknown mixer {entry['type']!r}")
        second = entry["type"] == "latent_attention_2"
        m, rot = entry["mixer"], entry["mixer"]["rot"]
        if rot["dims"] != m["rot_dim"]:
            raise ValueError(f"layer {i}: rotation of {rot['dims']} dimensions on a rotated part of {m['rot_dim']}")
        sc = rot.get("scaling")
        yarn = Yarn(*(float(sc[k]) for k in ("factor", "original", "fast", "slow"))) if sc else None
        source = m.get("kv_from")
        mixer = MixerConfig(heads=int(m["heads"]), dim=int(m["dim"]), rot_dim=int(m["rot_dim"]), vdim=int(m["vdim"]), kv_rank=int(m["kv_rank"]),
                            scale=float(m["scale"]), rot_base=float(rot["base"]), yarn=yarn, gated=not second, sink=second,
                            kv_from=-1 if source is None else int(source))
        if mixer.kv_from >= 0:
            if mixer.kv_from >= i:
                raise ValueError(f"layer {i}: its latents are to come from layer {mixer.kv_from}, which is not before it")
            o = layers[mixer.kv_from].mixer
            if o.kv_from >= 0 or (o.kv_rank, o.rot_dim, o.rot_base, o.yarn) != (mixer.kv_rank, mixer.rot_dim, mixer.rot_base, mixer.yarn):
                raise ValueError(f"layer {i}: layer {mixer.kv_from} has no latents that fit it")
        f = entry.get("mlp")
        if f is not None and f["kind"] != "dense":
            raise ValueError(f"layer {i}: unknown feed-forward {f['kind']!r}")
        layers.append(LayerConfig(mixer, int(f["ff"]) if f is not None else 0))
    return KagapelConfig(width=int(cfg["width"]), vocab=int(cfg["vocab"]), eps=float(cfg["norm"]["eps"]), streams=int(cfg["streams"]),
                         max_positions=int(cfg["max_positions"]), logit_scale=float(cfg["logit_scale"]), layers=layers)


def pack_weights(cfg: KagapelConfig, weights: Dict[str, torch.Tensor], dtype: torch.dtype, device) -> SeqWeights:
    """Checkpoint tensors -> the library's layout: all rows that read the mixer's input in one matrix, W_uk and W_uv in one,
    gate and up rows interleaved, rows padded."""
    W, S = cfg.width, cfg.streams

    def mat(t):
        return pad_rows(t, dtype, device)

    def vec(name, *shape):
        return vector(take(weights, name, shape), device)

    layers = []
    for i, l in enumerate(cfg.layers):
        p, a = f"l{i}.", l.mixer
        m = p + "mix."

        def connections(q):
            return Connections(read=vec(f"{p}hc{q}.in", S), mix=vec(f"{p}hc{q}.mix", S, S), write=vec(f"{p}hc{q}.out", S))

        rows = [take(weights, m + "q", (a.heads * (a.dim + a.rot_dim), W))]
        if a.kv_from < 0:
            rows.append(take(weights, m + "dkv", (a.kv_rank + a.rot_dim, W)))
        if a.gated:
            rows.append(take(weights, m + "g", (a.heads * a.vdim, W)))
        up = torch.cat([take(weights, m + "uk", (a.heads * a.dim, a.kv_rank)), take(weights, m + "uv", (a.heads * a.vdim, a.kv_rank))])
        kw = dict(mixer=MIX_LATENT, heads=a.heads, dim=a.dim, vdim=a.vdim, scale=a.scale, rot_dims=a.rot_dim, rot_half=True, rot_base=a.rot_base,
                  kv_rank=a.kv_rank, kv_from=a.kv_from, gated=a.gated, w_qkv=mat(torch.cat(rows)), w_ukv=mat(up),
                  w_o=mat(take(weights, m + "o", (W, a.heads * a.vdim))), norm1=vec(p + "norm1", W), hc1=connections(1))
        if a.yarn:
            kw.update(rot_factor=a.yarn.factor, rot_original=a.yarn.original, rot_fast=a.yarn.fast, rot_slow=a.yarn.slow)
        if a.kv_from < 0:
            kw["kv_norm"] = vec(m + "dkv.norm", a.kv_rank)
        if a.sink:
            kw["sink"] = vec(m + "sink", a.heads)
        f, m = l.ff, p + "mlp."
        if f:
            kw.update(ff_kind=FF_GATED, ff=f, w_up=mat(interleave(take(weights, m + "gate", (f, W)), take(weights, m + "up", (f, W)))),
                      b_up=vector(torch.stack([take(weights, m + "gate.b", (f,)), take(weights, m + "up.b", (f,))], dim=1).flatten(), device),
                      w_down=mat(take(weights, m + "down", (W, f))), b_down=vec(m + "down.b", W), norm2=vec(p + "norm2", W), hc2=connections(2))
        else:
            kw["ff_kind"] = FF_NONE
        layers.append(SeqLayer(**kw))
    return SeqWeights(dtype=dtype, width=W, vocab=cfg.vocab, eps=cfg.eps, streams=S, norm_offset=0.0, logit_scale=cfg.logit_scale, layers=layers,
                      embed=mat(take(weights, "embed", (cfg.vocab, W))), pos=mat(take(weights, "pos", (cfg.max_positions, W))),
                      final_norm=vec("final.norm", W), head=mat(take(weights, "head", (cfg.vocab, W))), architecture=ARCHITECTURE)


def from_tensors(config: dict, weights: Dict[str, torch.Tensor], dtype=torch.bfloat16, capacity: int = 4096, slots: int = 1,
                 max_portion: int = 2048, device="cuda") -> SeqModel:
    """A model on the device from a config.json dictionary and the checkpoint's tensors.  A sequence has at most as many
    positions as the model has position vectors."""
    cfg = parse_config(config)
    return SeqModel(pack_weights(cfg, weights, dtype, device), capacity=min(capacity, cfg.max_positions), slots=slots, max_portion=max_portion)


def load(path: str, dtype=torch.bfloat16, capacity: int = 4096, slots: int = 1, max_portion: int = 2048, device="cuda") -> SeqModel:
    from .build import ensure_seq
    ensure_seq()
    return from_tensors(read_config(path), read_weights(path), dtype, capacity, slots, max_portion, device)
