"""The Bosirax family: rotary grouped-query attention and gated delta-rule layers in any order, every layer parallel (mixer
and feed-forward take the same x), norms around one, embeddings of tokens and of pairs of them.

config.json: "vocab", "width", "norm" {"eps"}, "embedding" {"scale" [, "bigram" {buckets, mul_prev, mul_cur}]} and
"layers", a list of {"type", "mixer", "mlp"}:
  type "attention": mixer {heads, kv_heads, dim, vdim, scale, rot {dims, base [, scaling {factor, low, high,
                    original}]} [, mask {size}] [, kv_from]}
  type "delta":     mixer {heads, kv_heads, dim, vdim, conv}
  mlp null or {kind "dense", ff, limit}
Weights: model.safetensors, bfloat16, layer i under "l<i>.".
"""
from __future__ import annotations

import math
from pathlib import Path

import numpy as np

from ..safetensors_io import SafeTensors
from ..sequence import DeltaRule, GatedFfn, GroupedAttention, LayerWeights, ModelWeights, Pairs, SequenceModel, bf16_to_f32
from . import ConfigError, integer, number, register


def rotary_turns(rot: dict) -> np.ndarray:
    """Revolutions per position of every rotated pair, long wavelengths stretched as "scaling" says."""
    dims, base = integer(rot, "dims", 0), number(rot, "base")
    if dims % 2 or not base > 0:
        raise ConfigError(f"config: rotation of {dims} dimensions with base {base}")
    turns = base ** (-2.0 * np.arange(dims // 2, dtype=np.float64) / max(dims, 1)) / (2.0 * math.pi)
    scaling = rot.get("scaling")
    if scaling is None:
        return turns
    factor, low, high, original = (number(scaling, k) for k in ("factor", "low", "high", "original"))
    if not (factor > 0 and high > low > 0 and original > 0):
        raise ConfigError(f"config: rotary scaling {scaling!r}")
    # (a wavelength is 1 / turns): all of a frequency is kept up to original / high, 1 / factor of it from original / low on
    kept = np.clip((original * turns - low) / (high - low), 0.0, 1.0)
    return turns * (kept + (1.0 - kept) / factor)


def _grouped(mx: dict) -> tuple[int, int, int, int]:
    heads, kv_heads, dim, vdim = (integer(mx, k) for k in ("heads", "kv_heads", "dim", "vdim"))
    if heads % kv_heads:
        raise ConfigError(f"config: {heads} heads over {kv_heads} key/value heads")
    return heads, kv_heads, dim, vdim


def _attention(t, at: str, mx: dict, width: int, index: int, layers: list) -> GroupedAttention:
    heads, kv_heads, dim, vdim = _grouped(mx)
    turns = rotary_turns(mx.get("rot"))
    if 2 * len(turns) > dim:
        raise ConfigError(f"config: layer {index} rotates {2 * len(turns)} of {dim} dimensions")
    mask, source = mx.get("mask"), mx.get("kv_from")
    if source is not None:
        source = integer(mx, "kv_from", 0)
        from_mx = (layers[source].get("mixer") or {}) if source < index else None
        if from_mx is None or layers[source].get("type") != "attention" or from_mx.get("kv_from") is not None or \
                any(from_mx.get(k) != mx[k] for k in ("kv_heads", "dim", "vdim")):
            raise ConfigError(f"config: layer {index} takes keys and values from layer {source}, which has none of its sizes before it")
    own = source is None
    return GroupedAttention(
        heads, kv_heads, dim, vdim, number(mx, "scale"), turns, None if mask is None else integer(mask, "size"), source,
        q=t.bf16(at + "q", (heads * dim, width)),
        k=t.bf16(at + "k", (kv_heads * dim, width)) if own else None,
        v=t.bf16(at + "v", (kv_heads * vdim, width)) if own else None,
        out=t.bf16(at + "o", (width, heads * vdim)))


def _delta(t, at: str, mx: dict, width: int) -> DeltaRule:
    heads, kv_heads, dim, vdim = _grouped(mx)
    taps = integer(mx, "conv")
    return DeltaRule(
        heads, kv_heads, dim, vdim,
        q=t.bf16(at + "q", (kv_heads * dim, width)), q_conv=t.bf16(at + "q.conv", (kv_heads * dim, taps)),
        k=t.bf16(at + "k", (kv_heads * dim, width)), k_conv=t.bf16(at + "k.conv", (kv_heads * dim, taps)),
        v=t.bf16(at + "v", (heads * vdim, width)), v_conv=t.bf16(at + "v.conv", (heads * vdim, taps)),
        gate=t.bf16(at + "g", (heads * vdim, width)), b=t.bf16(at + "b", (heads, width)), a=t.bf16(at + "a", (heads, width)),
        a_log=t.bf16(at + "A_log", (heads,)), dt_bias=t.bf16(at + "dt_bias", (heads,)),
        head_norm=t.bf16(at + "norm", (vdim,)), out=t.bf16(at + "o", (width, heads * vdim)))


def _feed_forward(t, at: str, mlp: dict, width: int) -> GatedFfn:
    if mlp.get("kind") != "dense":
        raise ConfigError(f"config: feed-forward kind {mlp.get('kind')!r}")
    ff = integer(mlp, "ff")
    return GatedFfn(t.bf16(at + "gate", (ff, width)), t.bf16(at + "up", (ff, width)), t.bf16(at + "down", (width, ff)),
                    limit=number(mlp, "limit"))


def weights(config: dict, tensors) -> ModelWeights:
    """The model's weights; ``tensors`` offers bf16(name, shape)."""
    width, vocab, layers = integer(config, "width"), integer(config, "vocab"), config.get("layers")
    if not isinstance(layers, list) or not layers or not all(isinstance(x, dict) and isinstance(x.get("mixer"), dict) for x in layers):
        raise ConfigError("config: 'layers' must be a list of layers with mixers")

    def norm(name: str) -> np.ndarray:
        return 1.0 + bf16_to_f32(tensors.bf16(name, (width,)))

    def layer(n: int):
        d, at = layers[n], f"l{n}."

        def make() -> LayerWeights:
            if d.get("type") == "attention":
                mixer = _attention(tensors, at + "mix.", d["mixer"], width, n, layers)
            elif d.get("type") == "delta":
                mixer = _delta(tensors, at + "mix.", d["mixer"], width)
            else:
                raise ConfigError(f"config: layer {n} is of type {d.get('type')!r}")
            out = LayerWeights(norm(at + "norm1"), mixer, parallel=True)
            if d.get("mlp") is not None:
                out.norm2 = norm(at + "norm2")
                out.ffn = _feed_forward(tensors, at + "mlp.", d["mlp"], width)
            return out
        return make

    embedding = config.get("embedding")
    scale, bigram, pairs = number(embedding, "scale"), embedding.get("bigram"), None
    if bigram is not None:
        buckets = integer(bigram, "buckets")
        pairs = Pairs(buckets, integer(bigram, "mul_prev", 0), integer(bigram, "mul_cur", 0), tensors.bf16("bigram", (buckets + 1, width)))
    return ModelWeights(width, vocab, number(config.get("norm"), "eps"), embed=tensors.bf16("embed", (vocab, width)),
                        final_norm=norm("final.norm"), head=tensors.bf16("head", (vocab, width)),
                        layers=[layer(n) for n in range(len(layers))], embed_scale=scale, pairs=pairs)


@register("Bosirax", sequence=True)
def load(config: dict, model_dir: Path, slots: int = 8, cap: int = 4096, max_rows: int = 2048, dtype: str = "bfloat16",
         device_id: int = 0) -> SequenceModel:
    return SequenceModel(weights(config, SafeTensors(model_dir / "model.safetensors")), slots, cap, max_rows, dtype, device_id)
