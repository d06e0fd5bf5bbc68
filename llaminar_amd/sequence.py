"""ctypes door onto sequence models (include/llaminar_amd/sequence_model.h): layer descriptions,
the weight layouts the kernels take, and the runner the engine steps.

A model is described layer by layer (``LatentAttention``, ``GroupedAttention``, ``MatrixMemory`` or
``DeltaRule``, then ``GatedFfn``, ``Experts`` or nothing); which tensors hold the weights is the model family's business
(llaminar_amd/models).  Needs no PyTorch: device memory belongs to the library.
"""
from __future__ import annotations

import ctypes
import sys
from ctypes import POINTER, c_bool, c_char_p, c_float, c_int, c_int32, c_long, c_size_t, c_void_p
from dataclasses import dataclass, field
from pathlib import Path

import numpy as np

LIB_PATH = Path(__file__).resolve().parent / "lib" / "libllaminar_seq.so"

BF16, F32 = 0, 1
DTYPES = {"bfloat16": BF16, "float32": F32}
OUT_F32, OUT_ADD, OUT_ELEM, OUT_GATED, OUT_RELU2, OUT_GATED_CLAMP = range(6)
MIXER_LATENT_ATTENTION, MIXER_MATRIX_MEMORY, MIXER_ATTENTION, MIXER_DELTA = 1, 2, 3, 4
FFN_NONE, FFN_GATED, FFN_EXPERTS, FFN_GATED_CLAMP = 0, 1, 2, 3


class SequenceError(RuntimeError):
    """A call into the library failed; the message is llam_seqm_last_error()."""


class Config(ctypes.Structure):
    _fields_ = [(n, c_int) for n in ("width", "vocab", "n_layers", "slots", "cap", "max_rows", "dtype")] + \
               [("eps", c_float), ("device_id", c_int)]


class Layer(ctypes.Structure):
    _fields_ = [("mixer", c_int), ("heads", c_int), ("dim", c_int), ("vdim", c_int), ("norm1", c_void_p),
                ("w_in", c_void_p), ("w_out", c_void_p), ("q_rank", c_int), ("kv_rank", c_int), ("kv_from", c_int),
                ("scale", c_float), ("q_norm", c_void_p), ("kv_norm", c_void_p), ("w_uq", c_void_p),
                ("w_uk_t", c_void_p), ("w_uv", c_void_p), ("gate_cap", c_float), ("gate_bias", c_void_p),
                ("head_norm", c_void_p), ("kv_heads", c_int), ("rot_dims", c_int), ("chunk", c_int), ("turns", c_void_p),
                ("taps", c_int), ("conv", c_void_p), ("a_log", c_void_p), ("dt_bias", c_void_p), ("parallel", c_int),
                ("ffn", c_int), ("norm2", c_void_p), ("limit", c_float), ("ff", c_int), ("w_up", c_void_p),
                ("w_down", c_void_p), ("experts", c_int), ("top", c_int), ("shared_ff", c_int), ("w_router", c_void_p),
                ("router_bias", c_void_p), ("w_shared_up", c_void_p), ("w_shared_down", c_void_p)]


class Globals(ctypes.Structure):
    _fields_ = [("embed", c_void_p), ("final_norm", c_void_p), ("head", c_void_p), ("embed_scale", c_float),
                ("pairs", c_void_p), ("buckets", c_int), ("mul_prev", c_long), ("mul_cur", c_long)]


class LinearArgs(ctypes.Structure):
    _fields_ = [(n, c_void_p) for n in ("d_a", "d_w", "d_y", "d_bias", "d_norm", "d_h_out")] + \
               [("eps", c_float)] + [(n, c_int) for n in ("k_real", "M", "N", "K", "lda", "ldy", "out", "batch")] + \
               [(n, c_long) for n in ("a_stride", "w_stride", "y_stride")] + [("limit", c_float)]


class EmbedArgs(ctypes.Structure):
    _fields_ = [("d_table", c_void_p), ("vocab", c_int), ("width", c_int), ("scale", c_float), ("d_pairs", c_void_p),
                ("buckets", c_int), ("mul_prev", c_long), ("mul_cur", c_long)] + \
               [(n, c_void_p) for n in ("d_row_slot", "d_row_pos", "d_history")] + [("cap", c_int)]


class Entries(ctypes.Structure):
    _fields_ = [(n, c_void_p) for n in ("d_row0", "d_ntok", "d_slot", "d_pos")]


class MemoryArgs(ctypes.Structure):
    _fields_ = [("d_proj", c_void_p), ("ldp", c_int)] + \
               [(n, c_void_p) for n in ("d_gate_bias", "d_norm", "d_state", "d_m", "d_y")] + \
               [(n, c_int) for n in ("ldy", "heads", "dim", "vdim", "vdim_real")] + \
               [(n, c_float) for n in ("q_scale", "gate_cap", "eps")]


class AttentionArgs(ctypes.Structure):
    _fields_ = [(n, c_int) for n in ("heads", "kv_heads", "dim", "vdim", "ring", "chunk")] + \
               [("scale", c_float), ("d_k", c_void_p), ("d_v", c_void_p)]


class DeltaArgs(ctypes.Structure):
    _fields_ = [("d_proj", c_void_p), ("ldp", c_int)] + \
               [(n, c_void_p) for n in ("d_conv", "d_a_log", "d_dt_bias", "d_norm", "d_state", "d_recent", "d_y")] + \
               [(n, c_int) for n in ("ldy", "heads", "kv_heads", "dim", "vdim", "dim_real", "vdim_real", "taps")] + \
               [("eps", c_float)]


class ExpertsArgs(ctypes.Structure):
    _fields_ = [("d_logits", c_void_p), ("ldz", c_int)] + \
               [(n, c_void_p) for n in ("d_up", "d_down", "d_shared_up", "d_shared_down")] + \
               [("up_stride", c_long), ("down_stride", c_long)] + \
               [(n, c_int) for n in ("experts", "top", "ff", "shared_ff", "K", "N")] + \
               [("d_h", c_void_p), ("d_x", c_void_p), ("ldx", c_int)]


_I32P = POINTER(c_int32)
# name -> (restype, argtypes); mirrors seq_api.h and sequence_model.h declaration by declaration
SIGNATURES = {
    "llam_seq_linear": (c_bool, [POINTER(LinearArgs), c_int, c_int, c_void_p]),
    "llam_seq_linear_pair": (c_bool, [POINTER(LinearArgs), POINTER(LinearArgs), c_int, c_int, c_void_p]),
    "llam_seq_embed": (c_bool, [POINTER(EmbedArgs), c_void_p, c_void_p, c_int, c_int, c_int, c_void_p]),
    "llam_seq_rmsnorm": (c_bool, [c_void_p, c_int, c_void_p, c_void_p, c_float, c_int, c_void_p, c_int, c_int, c_int,
                                  c_int, c_void_p]),
    "llam_seq_rmsnorm_pair": (c_bool, [c_void_p, c_int, c_void_p, c_void_p, c_float, c_int, c_void_p, c_void_p, c_int, c_int,
                                       c_int, c_int, c_void_p]),
    "llam_seq_rotary": (c_bool, [POINTER(AttentionArgs), c_void_p, c_int, c_bool, c_void_p, c_int, c_void_p, c_void_p, c_void_p,
                                 c_int, c_int, c_int, c_void_p]),
    "llam_seq_attention_scratch_floats": (c_size_t, [c_int]),
    "llam_seq_attention": (c_bool, [POINTER(AttentionArgs), c_void_p, POINTER(Entries), c_int, c_int, c_int, c_int, c_void_p,
                                    c_int, c_void_p, c_size_t, c_int, c_int, c_void_p]),
    "llam_seq_delta_scratch_bytes": (c_size_t, [c_int, c_int, c_int, c_int, c_int]),
    "llam_seq_delta_decode": (c_bool, [POINTER(DeltaArgs), POINTER(Entries), c_int, c_int, c_int, c_int, c_void_p]),
    "llam_seq_delta_prefill": (c_bool, [POINTER(DeltaArgs), POINTER(Entries), c_int, c_int, c_void_p, c_size_t, c_int, c_int,
                                        c_void_p]),
    "llam_seq_latent_append": (c_bool, [c_void_p, c_int, c_void_p, c_float, c_int, c_void_p, c_void_p, c_void_p, c_int,
                                        c_int, c_int, c_int, c_int, c_void_p]),
    "llam_seq_latent_scratch_floats": (c_size_t, [c_int, c_int, c_int, c_int, c_int]),
    "llam_seq_latent_attention": (c_bool, [c_void_p, c_void_p, POINTER(Entries), c_int, c_int, c_int, c_int, c_int,
                                           c_int, c_int, c_float, c_void_p, c_void_p, c_size_t, c_int, c_int, c_void_p]),
    "llam_seq_memory_scratch_bytes": (c_size_t, [c_int, c_int, c_int, c_int]),
    "llam_seq_memory_decode": (c_bool, [POINTER(MemoryArgs), POINTER(Entries), c_int, c_int, c_void_p, c_size_t, c_int,
                                        c_int, c_void_p]),
    "llam_seq_memory_prefill": (c_bool, [POINTER(MemoryArgs), POINTER(Entries), c_int, c_int, c_void_p, c_size_t, c_int,
                                         c_int, c_void_p]),
    "llam_seq_experts_scratch_bytes": (c_size_t, [c_int, c_int, c_int, c_int, c_int, c_int]),
    "llam_seq_experts": (c_bool, [POINTER(ExpertsArgs), c_int, c_void_p, c_size_t, c_int, c_int, c_void_p]),
    "llam_seq_record": (c_bool, [c_void_p, c_int, c_void_p, c_void_p, c_int, c_int, c_void_p]),
    "llam_seqm_create": (c_void_p, [POINTER(Config)]),
    "llam_seqm_destroy": (None, [c_void_p]),
    "llam_seqm_upload": (c_void_p, [c_void_p, c_void_p, c_size_t]),
    "llam_seqm_set_layer": (c_bool, [c_void_p, c_int, POINTER(Layer)]),
    "llam_seqm_set_globals": (c_bool, [c_void_p, POINTER(Globals)]),
    "llam_seqm_forward": (c_bool, [c_void_p, c_int, _I32P, _I32P, _I32P, _I32P, c_int, _I32P, c_void_p, _I32P]),
    "llam_seqm_decode": (c_bool, [c_void_p, c_int, _I32P, _I32P, _I32P, c_int, _I32P, POINTER(c_float)]),
    "llam_seqm_trace": (c_bool, [c_void_p, c_void_p]),
    "llam_seqm_slot_bytes": (c_size_t, [c_void_p]),
    "llam_seqm_device_bytes": (c_size_t, [c_void_p]),
    "llam_seqm_last_error": (c_char_p, []),
    "llam_ql_last_error": (c_char_p, []),
}

_lib = None


def load() -> ctypes.CDLL:
    """Load the library (once).  Raises if it has not been built: there is no fallback."""
    global _lib
    if _lib is None:
        if not LIB_PATH.exists():
            raise ImportError(f"{LIB_PATH} is missing: build it with `python -m llaminar_amd.build --seq-only`")
        # a process uses one HIP runtime: where PyTorch is around, the one it has brought along already
        torch = sys.modules.get("torch")
        if torch is not None:
            torch.cuda.is_available()
        lib = ctypes.CDLL(str(LIB_PATH))
        for name, (res, args) in SIGNATURES.items():
            fn = getattr(lib, name)
            fn.restype, fn.argtypes = res, args
        _lib = lib
    return _lib


# ---- weight layouts -------------------------------------------------------------------------------

def pad_to(n: int, to: int) -> int:
    return -(-n // to) * to


def P(n: int) -> int:
    """Inner dimensions are padded with zeros to multiples of 64."""
    return pad_to(n, 64)


def A(n: int) -> int:
    """Heads of the grouped-query attention are padded to 64, 128 or 256 (and may not be larger)."""
    return 64 if n <= 64 else 128 if n <= 128 else 256


def bf16_bits(x) -> np.ndarray:
    """float array -> bfloat16 bit patterns, to nearest even."""
    u = np.ascontiguousarray(x, dtype=np.float32).view(np.uint32)
    return ((u + 0x7FFF + ((u >> 16) & 1)) >> 16).astype(np.uint16)


def bf16_to_f32(bits) -> np.ndarray:
    return (np.asarray(bits).astype(np.uint32) << 16).view(np.float32)


def padded(w: np.ndarray, *shape: int) -> np.ndarray:
    """w in the corner of a zero array of the given shape."""
    if w.shape == shape:
        return w
    out = np.zeros(shape, w.dtype)
    out[tuple(slice(0, n) for n in w.shape)] = w
    return out


def head_rows(w: np.ndarray, heads: int, dim: int, pad=P) -> np.ndarray:
    """[heads * dim, K] -> [heads * pad(dim), K]: zero rows after each head's."""
    return padded(w.reshape(heads, dim, -1), heads, pad(dim), w.shape[1]).reshape(heads * pad(dim), -1)


def head_columns(w: np.ndarray, heads: int, dim: int, pad=P) -> np.ndarray:
    """[N, heads * dim] -> [N, heads * pad(dim)]."""
    return padded(w.reshape(-1, heads, dim), w.shape[0], heads, pad(dim)).reshape(w.shape[0], -1)


def tiled(w: np.ndarray) -> np.ndarray:
    """[N, K] -> the tiles of seq_api.h, N padded to a multiple of 16, K of 64."""
    w = padded(w, pad_to(w.shape[0], 16), P(w.shape[1]))
    n, k = w.shape
    return np.ascontiguousarray(w.reshape(n // 16, 16, k // 32, 4, 8).transpose(0, 2, 3, 1, 4))


def gate_up_tiles(gate: np.ndarray, up: np.ndarray) -> np.ndarray:
    """Two [ff, K] matrices as one whose 16-row tiles alternate between them."""
    ff, k = P(gate.shape[0]), gate.shape[1]
    g, u = padded(gate, ff, k).reshape(ff // 16, 16, k), padded(up, ff, k).reshape(ff // 16, 16, k)
    return tiled(np.stack([g, u], axis=1).reshape(2 * ff, k))


# ---- layer descriptions ----------------------------------------------------------------------------
# Every tensor field is a bfloat16 bit pattern array in the orientation [out, in] (vectors [n], norms also as float32).

@dataclass
class LatentAttention:
    heads: int
    dim: int
    vdim: int
    q_rank: int
    kv_rank: int
    scale: float
    kv_from: int | None
    dq: np.ndarray
    q_norm: np.ndarray
    uq: np.ndarray
    dkv: np.ndarray | None
    kv_norm: np.ndarray | None
    uk: np.ndarray
    uv: np.ndarray
    out: np.ndarray


@dataclass
class MatrixMemory:
    heads: int
    dim: int
    vdim: int
    gate_cap: float
    q: np.ndarray
    k: np.ndarray
    v: np.ndarray
    gate: np.ndarray
    i: np.ndarray
    i_bias: np.ndarray
    f: np.ndarray
    f_bias: np.ndarray
    head_norm: np.ndarray
    out: np.ndarray


@dataclass
class GroupedAttention:
    """Rotary attention, heads / kv_heads query heads on every key/value head."""
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    scale: float
    turns: np.ndarray          # float64: revolutions per position of the rotated pairs
    chunk: int | None          # positions see their own chunk only
    kv_from: int | None
    q: np.ndarray
    k: np.ndarray | None
    v: np.ndarray | None
    out: np.ndarray


@dataclass
class DeltaRule:
    """Gated delta rule, heads / kv_heads heads on every q/k head."""
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    q: np.ndarray
    q_conv: np.ndarray         # [channels, taps]
    k: np.ndarray
    k_conv: np.ndarray
    v: np.ndarray
    v_conv: np.ndarray
    gate: np.ndarray
    b: np.ndarray
    a: np.ndarray
    a_log: np.ndarray
    dt_bias: np.ndarray
    head_norm: np.ndarray      # [vdim], of all heads
    out: np.ndarray


@dataclass
class GatedFfn:
    gate: np.ndarray
    up: np.ndarray
    down: np.ndarray
    limit: float | None = None   # gelu(gate) * up, or with a limit the clamped activation of seq_api.h


@dataclass
class Experts:
    top: int
    router: np.ndarray
    router_bias: np.ndarray
    up: list            # per expert [ff, width]
    down: list          # per expert [width, ff]
    shared_up: np.ndarray | None = None
    shared_down: np.ndarray | None = None
    shared_gate: np.ndarray | None = None


@dataclass
class LayerWeights:
    norm1: np.ndarray
    mixer: object
    norm2: np.ndarray | None = None
    ffn: object = None
    parallel: bool = False   # mixer and feed-forward take the same x


@dataclass
class Pairs:
    """Embedding of pairs of neighbouring tokens: row (previous * mul_prev + current * mul_cur) mod buckets of the
    table, whose last row is for a sequence's first token."""
    buckets: int
    mul_prev: int
    mul_cur: int
    table: np.ndarray


@dataclass
class ModelWeights:
    width: int
    vocab: int
    eps: float
    embed: np.ndarray
    final_norm: np.ndarray
    head: np.ndarray
    layers: list = field(default_factory=list)   # of callables -> LayerWeights: a layer's host copies are
                                                 # made, uploaded and dropped one after the other
    embed_scale: float = 1.0
    pairs: Pairs | None = None


def _i32(values) -> np.ndarray:
    return np.ascontiguousarray(values, dtype=np.int32)


def _p32(a: np.ndarray):
    return a.ctypes.data_as(_I32P)


class SequenceModel:
    """A model on the device and the state of its sequences: the runner behind llaminar_amd.engine."""

    def __init__(self, weights: ModelWeights, slots: int, cap: int, max_rows: int = 2048, dtype: str = "bfloat16",
                 device_id: int = 0):
        self.L = load()
        self.width, self.vocab, self.slots, self.cap, self.max_rows = weights.width, weights.vocab, slots, cap, max_rows
        self.n_layers = len(weights.layers)
        self.h = self.L.llam_seqm_create(ctypes.byref(Config(weights.width, weights.vocab, self.n_layers, slots, cap, max_rows,
                                                             DTYPES[dtype], weights.eps, device_id)))
        if not self.h:
            raise SequenceError(self._error())
        for n, make in enumerate(weights.layers):
            layer = self._layer(make())
            self._check(self.L.llam_seqm_set_layer(self.h, n, ctypes.byref(layer)))
        g = Globals(self._raw(np.ascontiguousarray(weights.embed)), self._vector(weights.final_norm), self._matrix(weights.head),
                    weights.embed_scale)
        if weights.pairs is not None:
            p = weights.pairs
            g.pairs, g.buckets, g.mul_prev, g.mul_cur = self._raw(np.ascontiguousarray(p.table)), p.buckets, p.mul_prev, p.mul_cur
        self._check(self.L.llam_seqm_set_globals(self.h, ctypes.byref(g)))

    # -- weights
    def _raw(self, a: np.ndarray) -> int:
        p = self.L.llam_seqm_upload(self.h, a.ctypes.data, a.nbytes)
        if not p:
            raise SequenceError(self._error())
        return p

    def _matrix(self, w: np.ndarray) -> int:
        return self._raw(tiled(w))

    def _vector(self, bits: np.ndarray, *shape: int) -> int:
        v = bits if bits.dtype == np.float32 else bf16_to_f32(bits)
        return self._raw(np.ascontiguousarray(padded(v, *(shape or (P(v.shape[0]),)))))

    def _layer(self, w: LayerWeights) -> Layer:
        out = Layer(norm1=self._vector(w.norm1))
        m = w.mixer
        out.heads, out.dim, out.vdim, out.kv_from = m.heads, m.dim, m.vdim, -1
        pad = A if isinstance(m, GroupedAttention) else P
        w_out = padded(head_columns(m.out, m.heads, m.vdim, pad), P(self.width), m.heads * pad(m.vdim))
        out.parallel = w.parallel and w.ffn is not None
        if out.parallel:
            down = w.ffn.down
            w_out = np.concatenate([w_out, padded(down, P(self.width), P(down.shape[1]))], axis=1)
        out.w_out = self._matrix(w_out)
        if isinstance(m, LatentAttention):
            out.mixer = MIXER_LATENT_ATTENTION
            out.q_rank, out.kv_rank, out.scale = m.q_rank, m.kv_rank, m.scale
            out.kv_from = -1 if m.kv_from is None else m.kv_from
            rows = [padded(m.dq, P(m.q_rank), self.width)]
            if m.kv_from is None:
                rows.append(padded(m.dkv, P(m.kv_rank), self.width))
                out.kv_norm = self._vector(m.kv_norm)
            out.w_in = self._matrix(np.concatenate(rows))
            out.q_norm = self._vector(m.q_norm)
            out.w_uq = self._matrix(head_rows(m.uq, m.heads, m.dim))
            uk = padded(m.uk.reshape(m.heads, m.dim, m.kv_rank), m.heads, P(m.dim), P(m.kv_rank))
            out.w_uk_t = self._raw(np.stack([tiled(np.ascontiguousarray(uk[a].T)) for a in range(m.heads)]))
            uv = padded(m.uv.reshape(m.heads, m.vdim, m.kv_rank), m.heads, P(m.vdim), P(m.kv_rank))
            out.w_uv = self._raw(np.stack([tiled(uv[a]) for a in range(m.heads)]))
        elif isinstance(m, MatrixMemory):
            out.mixer = MIXER_MATRIX_MEMORY
            out.gate_cap, out.scale = m.gate_cap, m.dim ** -0.5
            out.w_in = self._matrix(np.concatenate([head_rows(m.q, m.heads, m.dim), head_rows(m.k, m.heads, m.dim),
                                                    head_rows(m.v, m.heads, m.vdim), head_rows(m.gate, m.heads, m.vdim),
                                                    m.i, m.f]))
            out.gate_bias = self._vector(np.concatenate([m.i_bias, m.f_bias]), 2 * m.heads)
            out.head_norm = self._vector(m.head_norm.reshape(m.heads, m.vdim), m.heads, P(m.vdim))
        elif isinstance(m, GroupedAttention):
            out.mixer, out.kv_heads, out.scale, out.chunk = MIXER_ATTENTION, m.kv_heads, m.scale, m.chunk or 0
            out.kv_from = -1 if m.kv_from is None else m.kv_from
            rows = [head_rows(m.q, m.heads, m.dim, A)]
            if m.kv_from is None:
                rows += [head_rows(m.k, m.kv_heads, m.dim, A), head_rows(m.v, m.kv_heads, m.vdim, A)]
            out.w_in = self._matrix(np.concatenate(rows))
            out.rot_dims = 2 * len(m.turns)
            if out.rot_dims:
                out.turns = self._raw(np.ascontiguousarray(m.turns, dtype=np.float64))
        elif isinstance(m, DeltaRule):
            out.mixer, out.kv_heads, out.taps = MIXER_DELTA, m.kv_heads, m.q_conv.shape[1]
            out.w_in = self._matrix(np.concatenate([head_rows(m.q, m.kv_heads, m.dim), head_rows(m.k, m.kv_heads, m.dim),
                                                    head_rows(m.v, m.heads, m.vdim), head_rows(m.gate, m.heads, m.vdim), m.b, m.a]))
            taps = np.concatenate([head_rows(m.q_conv, m.kv_heads, m.dim), head_rows(m.k_conv, m.kv_heads, m.dim),
                                   head_rows(m.v_conv, m.heads, m.vdim)])
            out.conv = self._vector(np.ascontiguousarray(taps.T), *taps.T.shape)
            out.a_log, out.dt_bias = self._vector(m.a_log, m.heads), self._vector(m.dt_bias, m.heads)
            out.head_norm = self._vector(m.head_norm)
        else:
            raise TypeError(f"mixer {type(m).__name__}")
        f = w.ffn
        if f is None:
            return out
        out.norm2 = self._vector(w.norm2)
        if isinstance(f, GatedFfn):
            out.ffn, out.ff = FFN_GATED if f.limit is None else FFN_GATED_CLAMP, f.gate.shape[0]
            out.limit = f.limit or 0.0
            out.w_up = self._raw(gate_up_tiles(f.gate, f.up))
            if not out.parallel:
                out.w_down = self._matrix(padded(f.down, P(self.width), P(out.ff)))
        elif isinstance(f, Experts):
            out.ffn, out.ff, out.experts, out.top = FFN_EXPERTS, f.up[0].shape[0], len(f.up), f.top
            ff, wp = P(out.ff), P(self.width)
            out.w_up = self._raw(np.stack([tiled(padded(u, ff, self.width)) for u in f.up]))
            out.w_down = self._raw(np.stack([tiled(padded(d, wp, ff)) for d in f.down]))
            rows, bias = f.router, f.router_bias
            if f.shared_up is not None:
                out.shared_ff = f.shared_up.shape[0]
                out.w_shared_up = self._matrix(padded(f.shared_up, P(out.shared_ff), self.width))
                out.w_shared_down = self._matrix(padded(f.shared_down, wp, P(out.shared_ff)))
                rows = np.concatenate([rows, f.shared_gate])
            out.w_router = self._matrix(rows)
            out.router_bias = self._vector(bias, pad_to(rows.shape[0], 16))
        else:
            raise TypeError(f"feed-forward {type(f).__name__}")
        return out

    # -- errors and life
    def _error(self) -> str:
        return self.L.llam_seqm_last_error().decode()

    def _check(self, ok: bool):
        if not ok:
            raise SequenceError(self._error())

    def close(self):
        if getattr(self, "h", None):
            self.L.llam_seqm_destroy(self.h)
            self.h = None

    def __del__(self):
        try:
            self.close()
        except Exception:
            pass

    # -- steps
    def forward(self, entries, want=(), best: bool = False):
        """One step.  entries: (slot, position of the first token, token ids); want: places among all tokens of the
        step.  Returns the logits there, [len(want), vocab], or with ``best`` the index of each row's largest."""
        slot, pos, ntok = _i32([e[0] for e in entries]), _i32([e[1] for e in entries]), _i32([len(e[2]) for e in entries])
        ids, want = _i32([t for e in entries for t in e[2]]), _i32(list(want))
        logits = None if best else np.empty((len(want), self.vocab), np.float32)
        chosen = np.empty(len(want), np.int32) if best else None
        self._check(self.L.llam_seqm_forward(self.h, len(entries), _p32(slot), _p32(pos), _p32(ntok), _p32(ids), len(want),
                                             _p32(want), None if best else logits.ctypes.data,
                                             _p32(chosen) if best else None))
        return chosen if best else logits

    def decode(self, slots, pos, ids, steps: int) -> np.ndarray:
        """`steps` greedy tokens of several sequences, [steps, n]; ids are their newest tokens, not yet in the state."""
        slots, pos, ids = _i32(slots), _i32(pos), _i32(ids)
        out = np.empty((steps, len(slots)), np.int32)
        ms = c_float()
        self._check(self.L.llam_seqm_decode(self.h, len(slots), _p32(slots), _p32(pos), _p32(ids), steps, _p32(out),
                                            ctypes.byref(ms)))
        self.last_decode_ms = ms.value
        return out

    def max_decode_steps(self, n: int) -> int:
        """Most steps of one decode call for n sequences (the tokens stay on the device meanwhile)."""
        return 4096 // n

    def trace_layers(self, entries) -> np.ndarray:
        """The residual stream after every layer of one step, [layers, tokens, width]."""
        rows = sum(len(e[2]) for e in entries)
        out = np.zeros((self.n_layers, rows, self.width), np.float32)
        self._check(self.L.llam_seqm_trace(self.h, out.ctypes.data))
        try:
            self.forward(entries)
        finally:
            self.L.llam_seqm_trace(self.h, None)
        return out

    def slot_bytes(self) -> int:
        return int(self.L.llam_seqm_slot_bytes(self.h))

    def device_bytes(self) -> int:
        return int(self.L.llam_seqm_device_bytes(self.h))
