"""Binding of libcfpp_seq.so (include/cfpp_seq.h): decoder stacks described as a list of layers, with portions of prompts,
single tokens and greedy decode from one captured hipGraph, all in HIP.  There is no other path: without the library, or
without a GPU, construction fails."""
from __future__ import annotations

import ctypes as C
import os
from dataclasses import dataclass, field
from typing import List, Optional, Sequence

import torch

_HERE = os.path.dirname(os.path.abspath(__file__))
_DTYPE_CODE = {torch.bfloat16: 0, torch.float32: 1}
ROW_BYTES = 128
FF_NONE, FF_RELU2, FF_TABLE_EXPERTS, FF_GATED = 0, 1, 2, 3
MIX_GROUPED, MIX_LATENT = 0, 1


class _Streams(C.Structure):
    _fields_ = [(n, C.c_void_p) for n in ("in", "mix", "out")]


class _Layer(C.Structure):
    _fields_ = [(n, C.c_int32) for n in ("mixer", "heads", "kv_heads", "dim", "vdim", "chunk", "rot_dims", "rot_half", "v_mix", "kv_rank", "kv_from", "gated")] + \
        [(n, C.c_float) for n in ("scale", "v_lambda")] + \
        [(n, C.c_double) for n in ("rot_base", "rot_factor", "rot_original", "rot_fast", "rot_slow")] + \
        [(n, C.c_void_p) for n in ("w_qkv", "b_qkv", "q_norm", "k_norm", "kv_norm", "w_ukv", "sink", "w_o", "norm1")] + \
        [("hc1", _Streams)] + \
        [(n, C.c_int32) for n in ("ff_kind", "ff", "experts", "top", "shared_ff")] + \
        [(n, C.c_void_p) for n in ("w_up", "w_down", "b_up", "b_down", "w_shared_up", "w_shared_down", "table", "norm2")] + \
        [("hc2", _Streams)]


class _Desc(C.Structure):
    _fields_ = [(n, C.c_int32) for n in ("dtype", "n_layers", "width", "vocab", "streams", "positions")] + \
        [(n, C.c_float) for n in ("eps", "alpha", "norm_offset", "logit_scale", "softcap")] + \
        [("layers", C.POINTER(_Layer)), ("embed", C.c_void_p), ("pos", C.c_void_p), ("final_norm", C.c_void_p), ("head", C.c_void_p)] + \
        [(n, C.c_int32) for n in ("slots", "capacity", "max_portion")]


_lib = None


def _load():
    global _lib
    if _lib is None:
        path = os.path.join(_HERE, "libcfpp_seq.so")
        if not os.path.exists(path):
            raise ImportError(f"clusterfusionplus_amd: native library libcfpp_seq.so is missing from {_HERE}; "
                              "run `python -m clusterfusionplus_amd.build`. There is no fallback path.")
        lib = C.CDLL(path)
        p, i = C.c_void_p, C.c_int32
        for name, res, args in (
                ("cfpp_seq_create", C.c_int, [C.POINTER(_Desc), C.POINTER(p)]), ("cfpp_seq_destroy", C.c_int, [p]),
                ("cfpp_seq_bytes", C.c_size_t, [p]), ("cfpp_seq_row_pitch", C.c_size_t, [i, i]), ("cfpp_seq_version", C.c_char_p, []),
                ("cfpp_seq_forward", C.c_int, [p, i, C.POINTER(i), i, i, C.POINTER(i), i, p, p, p]),
                ("cfpp_seq_set_state", C.c_int, [p, i, i, i, p]), ("cfpp_seq_steps", C.c_int, [p, i, p]),
                ("cfpp_seq_graph_steps", C.c_int, [p, i, p]), ("cfpp_seq_launches_per_step", C.c_int, [p]),
                ("cfpp_seq_buffers", C.c_int, [p, C.POINTER(p), C.POINTER(p), C.POINTER(p), C.POINTER(i)])):
            f = getattr(lib, name)
            f.restype, f.argtypes = res, args
        _lib = lib
    return _lib


_STATUS = {-1: "a required pointer is NULL", -2: "unsupported dimensions, token ids or places", -3: "position beyond the capacity",
           -5: "unknown slot", -6: "unknown mode or element type"}


def _check(rc: int, what: str):
    if rc != 0:
        raise RuntimeError(f"{what}: " + (_STATUS.get(rc, f"status {rc}") if rc < 0 else f"HIP error {rc}"))


def pad_rows(rows: torch.Tensor, dtype: torch.dtype, device) -> torch.Tensor:
    """[..., K] -> [..., K'] of `dtype` on the device, rows padded with zeros to a multiple of ROW_BYTES bytes."""
    unit = ROW_BYTES // torch.empty(0, dtype=dtype).element_size()
    K = rows.shape[-1]
    out = torch.zeros((*rows.shape[:-1], (K + unit - 1) // unit * unit), dtype=dtype, device=device)
    out[..., :K] = rows.to(device=device)
    return out


def interleave(gate: torch.Tensor, up: torch.Tensor) -> torch.Tensor:
    """Gate and up matrices [..., F, K] as one matrix [..., 2 F, K]: row 2j = gate row j, row 2j + 1 = up row j."""
    return torch.stack((gate, up), dim=-2).flatten(-3, -2)


def _ptr(t: Optional[torch.Tensor]) -> Optional[int]:
    return t.data_ptr() if t is not None else None


def vector(v: torch.Tensor, device) -> torch.Tensor:
    return v.detach().to(device=device, dtype=torch.float32).contiguous()


@dataclass
class Connections:
    """How a sublayer reads and updates the residual streams (fp32 on the device)."""
    read: torch.Tensor        # [streams]
    mix: torch.Tensor         # [streams, streams], indexed [from, to]
    write: torch.Tensor       # [streams]


@dataclass
class SeqLayer:
    """One layer: sizes and constants as numbers, tensors on the device (matrices through pad_rows, vectors fp32).  What a
    mixer or a feed-forward does not use stays at its default; include/cfpp_seq.h says what each one is."""
    heads: int
    dim: int
    vdim: int
    scale: float
    w_qkv: torch.Tensor
    w_o: torch.Tensor
    norm1: torch.Tensor
    mixer: int = MIX_GROUPED
    sink: Optional[torch.Tensor] = None
    rot_dims: int = 0
    rot_half: bool = False
    rot_base: float = 10000.0
    rot_factor: float = 0.0
    rot_original: float = 0.0
    rot_fast: float = 0.0
    rot_slow: float = 0.0
    hc1: Optional[Connections] = None
    # grouped heads
    kv_heads: int = 0
    chunk: int = 0
    v_mix: bool = False
    v_lambda: float = 0.0
    b_qkv: Optional[torch.Tensor] = None
    q_norm: Optional[torch.Tensor] = None
    k_norm: Optional[torch.Tensor] = None
    # latent
    kv_rank: int = 0
    kv_from: int = -1
    gated: bool = False
    kv_norm: Optional[torch.Tensor] = None
    w_ukv: Optional[torch.Tensor] = None
    # feed-forward
    ff_kind: int = FF_NONE
    ff: int = 0
    experts: int = 0
    top: int = 0
    shared_ff: int = 0
    w_up: Optional[torch.Tensor] = None
    w_down: Optional[torch.Tensor] = None
    b_up: Optional[torch.Tensor] = None
    b_down: Optional[torch.Tensor] = None
    w_shared_up: Optional[torch.Tensor] = None
    w_shared_down: Optional[torch.Tensor] = None
    table: Optional[torch.Tensor] = None
    norm2: Optional[torch.Tensor] = None
    hc2: Optional[Connections] = None


@dataclass
class SeqWeights:
    dtype: torch.dtype
    width: int
    vocab: int
    eps: float
    layers: List[SeqLayer]
    embed: torch.Tensor
    final_norm: torch.Tensor
    head: torch.Tensor
    alpha: float = 1.0
    streams: int = 0                      # residual streams with norms in front; 0: norms after the sums
    pos: Optional[torch.Tensor] = None    # learned positions
    norm_offset: float = 1.0              # norm weight = norm_offset + stored weight
    logit_scale: float = 1.0
    softcap: float = 0.0
    architecture: str = ""
    extra: dict = field(default_factory=dict)


class SeqModel:
    """A sequence model on the device: weights, caches for `slots` sequences of up to `capacity` positions, and the step
    functions.  Implements the interface the engine drives (`forward`, `decode`)."""

    def __init__(self, weights: SeqWeights, capacity: int, slots: int = 1, max_portion: int = 2048):
        if weights.embed.device.type != "cuda":
            raise RuntimeError("sequence models run on a GPU; there is no CPU path")
        lib = _load()
        self.weights = weights                                    # keeps the storage alive
        self.architecture = weights.architecture
        self.vocab, self.width, self.n_layers = weights.vocab, weights.width, len(weights.layers)
        self.capacity, self.slots, self.dtype = int(capacity), int(slots), weights.dtype
        self.device = weights.embed.device
        arr = (_Layer * self.n_layers)()
        for s, l in zip(arr, weights.layers):
            for name, kind in _Layer._fields_:
                v = getattr(l, name)
                if kind is C.c_void_p:
                    v = _ptr(v)
                elif kind is C.c_int32:
                    v = int(v)
                elif kind is _Streams:
                    v = _Streams(_ptr(v.read), _ptr(v.mix), _ptr(v.write)) if v is not None else _Streams()
                setattr(s, name, v)
        desc = _Desc(_DTYPE_CODE[weights.dtype], self.n_layers, self.width, self.vocab, weights.streams,
                     weights.pos.shape[0] if weights.pos is not None else 0, weights.eps, weights.alpha, weights.norm_offset, weights.logit_scale,
                     weights.softcap, arr, _ptr(weights.embed), _ptr(weights.pos), _ptr(weights.final_norm), _ptr(weights.head),
                     self.slots, self.capacity, int(max_portion))
        handle = C.c_void_p()
        with torch.cuda.device(self.device):
            torch.cuda.synchronize()
            _check(lib.cfpp_seq_create(C.byref(desc), C.byref(handle)), "cfpp_seq_create")
        self._lib, self._h = lib, handle
        ptrs = [C.c_void_p() for _ in range(3)]
        cap = C.c_int32()
        _check(lib.cfpp_seq_buffers(handle, *[C.byref(p) for p in ptrs], C.byref(cap)), "cfpp_seq_buffers")
        self._logits, self._state, self._history = (
            _device_view(p.value, n, d, self.device) for p, n, d in zip(ptrs, (self.vocab, 4, cap.value), ("<f4", "<i4", "<i4")))

    def __del__(self):
        h, self._h = getattr(self, "_h", None), None
        if h:
            self._lib.cfpp_seq_destroy(h)

    def _stream(self):
        return C.c_void_p(torch.cuda.current_stream(self.device).cuda_stream)

    # ---- the engine's interface
    def forward(self, slot: int, tokens: Sequence[int], pos: int, want: Sequence[int] = (), residuals: bool = False):
        """Runs `tokens` at positions pos, pos + 1, ... of the sequence in `slot` and returns the logits (fp32,
        [len(want), vocab]) at the places `want`.  With `residuals`: (logits, residual stream after every layer)."""
        n, order = len(tokens), sorted(set(int(w) for w in want))
        logits = torch.empty((len(order), self.vocab), dtype=torch.float32, device=self.device)
        res = torch.empty((self.n_layers, n, self.width), dtype=torch.float32, device=self.device) if residuals else None
        _check(self._lib.cfpp_seq_forward(self._h, slot, (C.c_int32 * n)(*tokens), n, pos, (C.c_int32 * len(order))(*order), len(order),
                                          C.c_void_p(logits.data_ptr()) if order else None,
                                          C.c_void_p(res.data_ptr()) if residuals else None, self._stream()), "cfpp_seq_forward")
        if list(want) != order:
            place = {w: i for i, w in enumerate(order)}
            logits = logits[[place[int(w)] for w in want]]
        return (logits, res) if residuals else logits

    def decode(self, slot: int, token: int, pos: int, n: int) -> List[int]:
        """`n` greedy steps from `token` at position `pos`; the tokens picked."""
        self.set_state(token, pos, slot)
        self.graph_steps(n)
        return self.generated()

    # ---- the pieces of it, named as in NeoxDecoder
    def set_state(self, token: int, pos: int, slot: int = 0):
        _check(self._lib.cfpp_seq_set_state(self._h, slot, int(token), int(pos), self._stream()), "cfpp_seq_set_state")

    def step(self, n: int = 1):
        """Eager greedy steps (one launch per kernel)."""
        _check(self._lib.cfpp_seq_steps(self._h, int(n), self._stream()), "cfpp_seq_steps")

    def graph_steps(self, n: int):
        """Greedy steps, each one replay of the captured hipGraph.  Raises instead of going past the capacity."""
        _check(self._lib.cfpp_seq_graph_steps(self._h, int(n), self._stream()), "cfpp_seq_graph_steps")

    @property
    def launches_per_step(self) -> int:
        return int(self._lib.cfpp_seq_launches_per_step(self._h))

    @property
    def bytes_allocated(self) -> int:
        return int(self._lib.cfpp_seq_bytes(self._h))

    @property
    def logits(self) -> torch.Tensor:
        return self._logits

    @property
    def state(self) -> torch.Tensor:
        """int32 [token, position, steps since set_state, slot] on the device; to read."""
        return self._state

    def generated(self) -> List[int]:
        """The tokens picked since `set_state`."""
        n = int(self._state[2].item())
        return self._history[:n].tolist()


class _DeviceArray:
    """Library memory offered to torch.as_tensor through the array interface it reads."""

    def __init__(self, ptr, count, typestr):
        self.__cuda_array_interface__ = {"data": (ptr, False), "shape": (count,), "typestr": typestr, "version": 2}


def _device_view(ptr, count, typestr, device):
    return torch.as_tensor(_DeviceArray(ptr, count, typestr), device=device)
