"""Seeded synthetic GGUF weight blocks and activations.

Block fields are uniform over their whole range: every packed byte uniform
0..255 (which makes Q4_K's 6-bit scales/mins uniform 0..63, its nibbles uniform
0..15, Q6_K's int8 sub-scales uniform -128..127 and IQ3_S's 9-bit codebook
indices uniform 0..511 with random signs and 4-bit sub-scales), and the fp16
super-block scales d (and dmin) uniform in [0.001, 0.02).  Activations and
router logits are N(0,1).
"""
from __future__ import annotations

import numpy as np

from .capi import BLOCK_BYTES, FMT_IQ3_S, FMT_Q4_K, FMT_Q6_K

# byte offsets of the fp16 scale fields inside one super-block
_FP16_FIELDS = {FMT_Q4_K: (0, 2), FMT_Q6_K: (208,), FMT_IQ3_S: (0,)}


def weights_numpy(fmt: int, N: int, K: int, seed: int, d_lo: float = 0.001, d_hi: float = 0.02) -> np.ndarray:
    """uint8 array [N, K/256, block_bytes] of raw GGUF super-blocks."""
    assert K % 256 == 0
    rng = np.random.default_rng(seed)
    bb = BLOCK_BYTES[fmt]
    sb = K // 256
    w = rng.integers(0, 256, size=(N, sb, bb), dtype=np.uint8)
    for off in _FP16_FIELDS[fmt]:
        d = rng.uniform(d_lo, d_hi, size=(N, sb)).astype(np.float16)
        w[:, :, off:off + 2] = d.view(np.uint8).reshape(N, sb, 2)
    return w


def weights_torch(fmt: int, N: int, K: int, seed: int, device, d_lo: float = 0.001, d_hi: float = 0.02):
    """Same distribution generated directly on `device` (for matrices too big to
    build on the host every run).  uint8 tensor of N*(K/256)*block_bytes bytes."""
    import torch

    g = torch.Generator(device=device)
    g.manual_seed(seed)
    bb = BLOCK_BYTES[fmt]
    sb = K // 256
    w = torch.randint(0, 256, (N * sb, bb), dtype=torch.uint8, device=device, generator=g)
    for off in _FP16_FIELDS[fmt]:
        d = (torch.rand(N * sb, device=device, generator=g) * (d_hi - d_lo) + d_lo).to(torch.float16)
        w[:, off:off + 2] = d.view(torch.uint8).reshape(N * sb, 2)
    return w.reshape(-1)


def activations_numpy(M: int, K: int, seed: int) -> np.ndarray:
    rng = np.random.default_rng(seed)
    return rng.standard_normal((M, K)).astype(np.float32)


def gemv_bytes(fmt: int, N: int, K: int, M: int = 1) -> int:
    """Algorithmic bytes of one GEMV: weights + Q8_1 activations + fp32 outputs."""
    return N * (K // 256) * BLOCK_BYTES[fmt] + M * (K // 32) * 36 + M * N * 4


def sequence_model_torch(layers, width: int, vocab: int, device, slots: int, cap: int, max_rows: int = 2048,
                         dtype: str = "bfloat16", eps: float = 1e-5, seed: int = 0, pairs: int = 0):
    """A sequence.SequenceModel of random bf16 weights made on the device (matrices too big to build on the host
    every run).  ``layers``: sequence.Layer descriptions with sizes only; every tensor is filled in here, N(0, 1/in)
    (random weights need no particular order of tiles).  ``pairs``: buckets of an embedding of token pairs.  The tensors
    live as long as the model."""
    import ctypes

    import torch

    from . import sequence as sq

    g = torch.Generator(device=device)
    g.manual_seed(seed)
    P = sq.P
    model = sq.SequenceModel.__new__(sq.SequenceModel)
    model.L, model.keep = sq.load(), []
    model.width, model.vocab, model.slots, model.cap, model.max_rows, model.n_layers = width, vocab, slots, cap, max_rows, len(layers)
    model.weight_bytes = []   # per layer: bf16 bytes a decode step reads at batch 1
    model.h = model.L.llam_seqm_create(ctypes.byref(sq.Config(width, vocab, len(layers), slots, cap, max_rows, sq.DTYPES[dtype],
                                                              eps, device.index or 0)))
    if not model.h:
        raise sq.SequenceError(model._error())

    def matrix(rows, columns, count=1):
        t = torch.empty(count * sq.pad_to(rows, 16) * P(columns), dtype=torch.bfloat16, device=device)
        t.normal_(0.0, columns ** -0.5, generator=g)
        model.keep.append(t)
        return t.data_ptr(), t.numel() * 2

    def vector(n, value=1.0):
        t = torch.full((n,), value, device=device) if isinstance(value, float) else value.to(device)
        model.keep.append(t)
        return t.data_ptr()

    for n, w in enumerate(layers):
        H, d, v, wp, read = w.heads, P(w.dim), P(w.vdim), P(width), 0
        if w.mixer == sq.MIXER_ATTENTION:
            d, v = sq.A(w.dim), sq.A(w.vdim)
        w.norm1 = vector(wp)
        w.w_out, b = matrix(wp, H * v + (P(w.ff) if w.parallel and w.ffn else 0))
        read += b
        if w.mixer == sq.MIXER_LATENT_ATTENTION:
            own = w.kv_from < 0
            w.w_in, b1 = matrix(P(w.q_rank) + (P(w.kv_rank) if own else 0), wp)
            w.w_uq, b2 = matrix(H * d, w.q_rank)
            w.w_uk_t, b3 = matrix(H * P(w.kv_rank), d)
            w.w_uv, b4 = matrix(H * v, w.kv_rank)
            read += b1 + b2 + b3 + b4
            w.q_norm, w.kv_norm = vector(P(w.q_rank)), vector(P(w.kv_rank))
            w.scale = w.scale or w.dim ** -0.5
        elif w.mixer == sq.MIXER_ATTENTION:
            w.w_in, b = matrix(H * d + (w.kv_heads * (d + v) if w.kv_from < 0 else 0), wp)
            read += b
            w.scale, w.rot_dims = w.scale or w.dim ** -0.5, w.rot_dims or w.dim
            w.turns = vector(w.rot_dims // 2, 10000.0 ** (-torch.arange(0, w.rot_dims, 2, dtype=torch.float64) / w.rot_dims) / 6.283185307179586)
        elif w.mixer == sq.MIXER_DELTA:
            w.w_in, b = matrix(2 * w.kv_heads * d + 2 * H * v + 2 * H, wp)
            read += b
            w.conv = vector(w.taps * (2 * w.kv_heads * d + H * v), 0.5)
            w.a_log, w.dt_bias, w.head_norm = vector(H, -2.0), vector(H, -1.0), vector(v)
        else:
            w.w_in, b = matrix(2 * H * (d + v) + 2 * H, wp)
            read += b
            w.gate_bias, w.head_norm = vector(2 * H, 2.0), vector(H * v)
            w.gate_cap, w.scale = w.gate_cap or 15.0, w.dim ** -0.5
        if w.ffn:
            w.norm2 = vector(wp)
        if w.ffn in (sq.FFN_GATED, sq.FFN_GATED_CLAMP):
            w.w_up, b1 = matrix(2 * P(w.ff), wp)
            read += b1
            if not w.parallel:
                w.w_down, b2 = matrix(wp, P(w.ff))
                read += b2
        elif w.ffn == sq.FFN_EXPERTS:
            w.w_up, b1 = matrix(P(w.ff), wp, w.experts)
            w.w_down, b2 = matrix(wp, P(w.ff), w.experts)
            rows = w.experts + (1 if w.shared_ff else 0)
            w.w_router, b3 = matrix(rows, wp)
            w.router_bias = vector(sq.pad_to(rows, 16), 0.0)
            read += (b1 + b2) * w.top // w.experts + b3
            if w.shared_ff:
                w.w_shared_up, b4 = matrix(P(w.shared_ff), wp)
                w.w_shared_down, b5 = matrix(wp, P(w.shared_ff))
                read += b4 + b5
        model.weight_bytes.append(read)
        model._check(model.L.llam_seqm_set_layer(model.h, n, ctypes.byref(w)))
    embed = torch.randn(vocab, width, device=device, generator=g).to(torch.bfloat16)
    model.keep.append(embed)
    head, b = matrix(vocab, P(width))
    model.weight_bytes.append(b)
    torch.cuda.synchronize()
    g_ = sq.Globals(embed.data_ptr(), vector(P(width)), head, 1.0)
    if pairs:
        table = torch.randn(pairs + 1, width, device=device, generator=g).to(torch.bfloat16)
        model.keep.append(table)
        g_.pairs, g_.buckets, g_.mul_prev, g_.mul_cur = table.data_ptr(), pairs, 40503, 19
    torch.cuda.synchronize()
    model._check(model.L.llam_seqm_set_globals(model.h, ctypes.byref(g_)))
    return model
