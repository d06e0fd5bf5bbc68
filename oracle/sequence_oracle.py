"""Plain, slow restatement of the sequence-model mechanisms (numpy, double precision).

One function per mechanism, written from the equations and sharing no code with the
product.  Every function takes a whole sequence; recurrences run token by token.

Notation: a linear weight W is [out, in] and is applied to rows, y = x W^T.
``w`` below is a dict of tensors of one layer, keyed by the name behind the layer's
prefix ("mix.q", "mlp.e0.up", ...).
"""
from __future__ import annotations

import math

import numpy as np


def rms(x, eps):
    """x over its root mean square along the last axis, eps inside the root."""
    return x / np.sqrt(np.mean(x * x, axis=-1, keepdims=True) + eps)


def rms_norm(x, weight, eps):
    return rms(x, eps) * weight


def gelu_tanh(z):
    return 0.5 * z * (1.0 + np.tanh(math.sqrt(2.0 / math.pi) * (z + 0.044715 * z ** 3)))


def relu_squared(z):
    return np.maximum(z, 0.0) ** 2


def sigmoid(z):
    return 1.0 / (1.0 + np.exp(-z))


def log_sigmoid(z):
    return -np.logaddexp(0.0, -z)


def latent_rows(h, w, eps):
    """The cached latent of every position."""
    return rms_norm(h @ w["mix.dkv"].T, w["mix.dkv.norm"], eps)


def latent_attention(h, latent, w, heads, dim, vdim, scale, eps):
    """Causal softmax attention whose keys and values are up-projections of the latent rows."""
    T = h.shape[0]
    cq = rms_norm(h @ w["mix.dq"].T, w["mix.dq.norm"], eps)
    q = (cq @ w["mix.uq"].T).reshape(T, heads, dim)
    k = (latent @ w["mix.uk"].T).reshape(T, heads, dim)
    v = (latent @ w["mix.uv"].T).reshape(T, heads, vdim)
    out = np.zeros((T, heads, vdim))
    for i in range(T):
        for a in range(heads):
            s = (k[:i + 1, a] @ q[i, a]) * scale
            e = np.exp(s - s.max())
            out[i, a] = (e / e.sum()) @ v[:i + 1, a]
    return out.reshape(T, heads * vdim) @ w["mix.o"].T


def mlstm_gates(h, w, cap):
    """(log input gate, log forget gate), [T, heads] each: soft-capped, the forget gate through log sigmoid."""
    i = cap * np.tanh((h @ w["mix.i"].T + w["mix.i.b"]) / cap)
    f = log_sigmoid(cap * np.tanh((h @ w["mix.f"].T + w["mix.f.b"]) / cap))
    return i, f


def mlstm_recurrence(q, k, v, i, f):
    """One head's matrix memory over a sequence: q, k [T, dim], v [T, vdim], i, f [T] -> (o [T, vdim], S, n, m)."""
    S = np.zeros((q.shape[1], v.shape[1]))
    n = np.zeros(q.shape[1])
    m = 0.0
    out = np.zeros((q.shape[0], v.shape[1]))
    for t in range(q.shape[0]):
        m_new = max(f[t] + m, i[t])
        keep, take = math.exp(f[t] + m - m_new), math.exp(i[t] - m_new)
        S = keep * S + take * np.outer(k[t], v[t])
        n = keep * n + take * k[t]
        m = m_new
        out[t] = (q[t] @ S) / (max(abs(n @ q[t]), math.exp(-m)) + 1e-6)
    return out, S, n, m


def mlstm(h, w, heads, dim, vdim, cap, eps):
    T = h.shape[0]
    q = (h @ w["mix.q"].T).reshape(T, heads, dim) * dim ** -0.5
    k = (h @ w["mix.k"].T).reshape(T, heads, dim)
    v = (h @ w["mix.v"].T).reshape(T, heads, vdim)
    i, f = mlstm_gates(h, w, cap)
    o = np.stack([mlstm_recurrence(q[:, a], k[:, a], v[:, a], i[:, a], f[:, a])[0] for a in range(heads)], axis=1)
    o = rms(o, eps).reshape(T, heads * vdim) * w["mix.norm"] * sigmoid(h @ w["mix.g"].T)
    return o @ w["mix.o"].T


def gated_ffn(h, w):
    return (gelu_tanh(h @ w["mlp.gate"].T) * (h @ w["mlp.up"].T)) @ w["mlp.down"].T


def expert_ffn(h, up, down):
    return relu_squared(h @ up.T) @ down.T


def route(z, top):
    """Indices of the largest logits of one token and the softmax over them alone (a tie goes to the lower index)."""
    order = sorted(range(len(z)), key=lambda e: (-z[e], e))[:top]
    e = np.exp(z[order] - max(z[order]))
    return order, e / e.sum()


def routed_ffn(h, w, experts, top, shared):
    z = h @ w["mlp.router"].T + w["mlp.router.b"]
    assert z.shape[1] == experts
    y = np.zeros_like(h)
    for t in range(h.shape[0]):
        for e, p in zip(*route(z[t], top)):
            y[t] += p * expert_ffn(h[t], w[f"mlp.e{e}.up"], w[f"mlp.e{e}.down"])
        if shared:
            gate = sigmoid(h[t] @ w["mlp.shared.sg"].T)
            y[t] += gate * expert_ffn(h[t], w["mlp.shared.up"], w["mlp.shared.down"])
    return y


def kogilix(config, tensors, tokens, layers_out=None):
    """Logits [T, vocab] of one sequence.  ``layers_out`` (a list) receives the residual stream after every layer."""
    eps = config["norm"]["eps"]
    tensors = {n: np.asarray(t, dtype=np.float64) for n, t in tensors.items()}
    x = tensors["embed"][np.asarray(tokens)]
    latents = {}
    for n, layer in enumerate(config["layers"]):
        w = {name[len(f"l{n}."):]: t for name, t in tensors.items() if name.startswith(f"l{n}.")}
        mx = layer["mixer"]
        h = rms_norm(x, w["norm1"], eps)
        if layer["type"] == "latent_attention":
            source = mx.get("kv_from")
            if source is None:
                latents[n] = latent_rows(h, w, eps)
            y = latent_attention(h, latents[n if source is None else source], w, mx["heads"], mx["dim"], mx["vdim"],
                                 mx["scale"], eps)
        else:
            assert layer["type"] == "mlstm"
            y = mlstm(h, w, mx["heads"], mx["dim"], mx["vdim"], mx["gate_cap"], eps)
        x = x + y
        ff = layer.get("mlp")
        if ff is not None:
            h = rms_norm(x, w["norm2"], eps)
            if ff["kind"] == "dense":
                x = x + gated_ffn(h, w)
            else:
                x = x + routed_ffn(h, w, ff["router"]["experts"], ff["router"]["top"], ff.get("shared") is not None)
        if layers_out is not None:
            layers_out.append(x.copy())
    return rms_norm(x, tensors["final.norm"], eps) @ tensors["head"].T


# ---- rotary grouped-query attention, gated delta rule, parallel layers -------------------------------

def centred_norm(x, weight, eps):
    """RMS norm whose weight is stored as its distance from one."""
    return rms(x, eps) * (1.0 + weight)


def rotary_frequencies(dims, base, scaling=None):
    """Angle per position of every pair; ``scaling`` {factor, low, high, original} stretches the long wavelengths."""
    out = []
    for i in range(dims // 2):
        f = float(base) ** (-2.0 * i / dims)
        if scaling is not None:
            wave = 2.0 * math.pi / f
            if wave > scaling["original"] / scaling["low"]:
                f = f / scaling["factor"]
            elif wave >= scaling["original"] / scaling["high"]:
                s = (scaling["original"] / wave - scaling["low"]) / (scaling["high"] - scaling["low"])
                f = (1.0 - s) * f / scaling["factor"] + s * f
        out.append(f)
    return np.array(out)


def rotate(x, positions, freq):
    """x [T, heads, dim]: dimension i turns with dimension i + len(freq), the rest stays."""
    n = len(freq)
    y = x.copy()
    for t, p in enumerate(positions):
        c, s = np.cos(p * freq), np.sin(p * freq)
        u, v = x[t, :, :n], x[t, :, n:2 * n]
        y[t, :, :n] = u * c - v * s
        y[t, :, n:2 * n] = v * c + u * s
    return y


def sees(i, j, chunk):
    return j <= i and (chunk is None or i // chunk == j // chunk)


def grouped_attention(q, k, v, scale, chunk):
    """q [T, H, dim], k [T, G, dim], v [T, G, vdim] -> [T, H, vdim]; positions see their own chunk up to themselves."""
    T, H = q.shape[:2]
    out = np.zeros((T, H, v.shape[2]))
    for i in range(T):
        seen = [j for j in range(T) if sees(i, j, chunk)]
        for h in range(H):
            g = h // (H // k.shape[1])
            s = (k[seen, g] @ q[i, h]) * scale
            e = np.exp(s - s.max())
            out[i, h] = (e / e.sum()) @ v[seen, g]
    return out


def short_convolution(x, taps):
    """Causal, per channel: taps [channels, n], the last of them for the current token; silu behind."""
    T, n = x.shape[0], taps.shape[1]
    y = np.zeros_like(x)
    for t in range(T):
        for j in range(n):
            if t - (n - 1) + j >= 0:
                y[t] += taps[:, j] * x[t - (n - 1) + j]
    return y * sigmoid(y)


def unit(x):
    return x / np.sqrt(np.sum(x * x, axis=-1, keepdims=True) + 1e-6)


def delta_recurrence(q, k, v, decay, beta):
    """One head: q, k [T, dim], v [T, vdim], decay, beta [T] -> (o [T, vdim], S [dim, vdim])."""
    S = np.zeros((q.shape[1], v.shape[1]))
    out = np.zeros((q.shape[0], v.shape[1]))
    for t in range(q.shape[0]):
        S = decay[t] * S
        u = beta[t] * (v[t] - S.T @ k[t])
        S = S + np.outer(k[t], u)
        out[t] = S.T @ q[t]
    return out, S


def gated_delta(h, w, heads, groups, dim, vdim, eps):
    T = h.shape[0]
    q = unit(short_convolution(h @ w["mix.q"].T, w["mix.q.conv"]).reshape(T, groups, dim)) * dim ** -0.5
    k = unit(short_convolution(h @ w["mix.k"].T, w["mix.k.conv"]).reshape(T, groups, dim))
    v = short_convolution(h @ w["mix.v"].T, w["mix.v.conv"]).reshape(T, heads, vdim)
    beta = sigmoid(h @ w["mix.b"].T)
    decay = np.exp(-np.exp(w["mix.A_log"]) * np.logaddexp(0.0, h @ w["mix.a"].T + w["mix.dt_bias"]))
    per = heads // groups
    o = np.stack([delta_recurrence(q[:, a // per], k[:, a // per], v[:, a], decay[:, a], beta[:, a])[0] for a in range(heads)], axis=1)
    z = (h @ w["mix.g"].T).reshape(T, heads, vdim)
    return (rms(o, eps) * w["mix.norm"] * z * sigmoid(z)).reshape(T, heads * vdim) @ w["mix.o"].T


def clamped_ffn(h, w, limit):
    g = np.minimum(h @ w["mlp.gate"].T, limit)
    u = np.clip(h @ w["mlp.up"].T, -limit, limit)
    return (g * sigmoid(1.702 * g) * (u + 1.0)) @ w["mlp.down"].T


def bigram_rows(tokens, mul_prev, mul_cur, buckets):
    """Row of the pair table for every token; the first token of a sequence has the last row."""
    return [buckets if t == 0 else (int(tokens[t - 1]) * mul_prev + int(tokens[t]) * mul_cur) % buckets for t in range(len(tokens))]


def bosirax(config, tensors, tokens, layers_out=None):
    """Logits [T, vocab] of one sequence.  ``layers_out`` (a list) receives the residual stream after every layer."""
    eps = config["norm"]["eps"]
    tensors = {n: np.asarray(t, dtype=np.float64) for n, t in tensors.items()}
    x = tensors["embed"][np.asarray(tokens)] * config["embedding"]["scale"]
    pairs = config["embedding"].get("bigram")
    if pairs is not None:
        x = x + tensors["bigram"][bigram_rows(tokens, pairs["mul_prev"], pairs["mul_cur"], pairs["buckets"])]
    T, cached = len(tokens), {}
    for n, layer in enumerate(config["layers"]):
        w = {name[len(f"l{n}."):]: t for name, t in tensors.items() if name.startswith(f"l{n}.")}
        mx = layer["mixer"]
        H, G, dim, vdim = mx["heads"], mx["kv_heads"], mx["dim"], mx["vdim"]
        h = centred_norm(x, w["norm1"], eps)
        if layer["type"] == "attention":
            freq = rotary_frequencies(mx["rot"]["dims"], mx["rot"]["base"], mx["rot"].get("scaling"))
            source = mx.get("kv_from")
            if source is None:
                cached[n] = (rotate((h @ w["mix.k"].T).reshape(T, G, dim), range(T), freq), (h @ w["mix.v"].T).reshape(T, G, vdim))
            k, v = cached[n if source is None else source]
            q = rotate((h @ w["mix.q"].T).reshape(T, H, dim), range(T), freq)
            mask = mx.get("mask")
            y = grouped_attention(q, k, v, mx["scale"], None if mask is None else mask["size"])
            y = y.reshape(T, H * vdim) @ w["mix.o"].T
        else:
            assert layer["type"] == "delta"
            y = gated_delta(h, w, H, G, dim, vdim, eps)
        if layer.get("mlp") is not None:
            assert layer["mlp"]["kind"] == "dense"
            y = y + clamped_ffn(centred_norm(x, w["norm2"], eps), w, layer["mlp"]["limit"])
        x = x + y
        if layers_out is not None:
            layers_out.append(x.copy())
    return centred_norm(x, tensors["final.norm"], eps) @ tensors["head"].T
