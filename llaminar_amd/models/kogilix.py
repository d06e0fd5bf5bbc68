"""The Kogilix family: latent-attention and mLSTM layers in any order, dense or routed feed-forwards.

config.json: "vocab", "width", "norm" {"eps"} and "layers", a list of {"type", "mixer", "mlp"}:
  type "latent_attention": mixer {heads, dim, vdim, q_rank, kv_rank, scale [, kv_from]}
  type "mlstm":            mixer {heads, dim, vdim, gate_cap}
  mlp null, {kind "dense", ff}, or
      {kind "moe", expert {ff}, router {experts, top} [, shared {ff}]}
Weights: model.safetensors, bfloat16, layer i under "l<i>.".
"""
from __future__ import annotations

from pathlib import Path

from ..safetensors_io import SafeTensors
from ..sequence import Experts, GatedFfn, LatentAttention, LayerWeights, MatrixMemory, ModelWeights, SequenceModel
from . import ConfigError, integer, number, register


def _latent_attention(t, at: str, mx: dict, width: int, index: int, layers: list) -> LatentAttention:
    heads, dim, vdim = integer(mx, "heads"), integer(mx, "dim"), integer(mx, "vdim")
    q_rank, kv_rank = integer(mx, "q_rank"), integer(mx, "kv_rank")
    source = mx.get("kv_from")
    if source is not None:
        source = integer(mx, "kv_from", 0)
        if source >= index:
            raise ConfigError(f"config: layer {index} takes its latent from layer {source}, which does not precede it")
        from_mx = layers[source].get("mixer") or {}
        if layers[source].get("type") != "latent_attention" or from_mx.get("kv_from") is not None or \
                from_mx.get("kv_rank") != kv_rank:
            raise ConfigError(f"config: layer {index} takes its latent from layer {source}, which has none of rank {kv_rank}")
    return LatentAttention(
        heads, dim, vdim, q_rank, kv_rank, number(mx, "scale"), source,
        dq=t.bf16(at + "dq", (q_rank, width)), q_norm=t.bf16(at + "dq.norm", (q_rank,)),
        uq=t.bf16(at + "uq", (heads * dim, q_rank)),
        dkv=None if source is not None else t.bf16(at + "dkv", (kv_rank, width)),
        kv_norm=None if source is not None else t.bf16(at + "dkv.norm", (kv_rank,)),
        uk=t.bf16(at + "uk", (heads * dim, kv_rank)), uv=t.bf16(at + "uv", (heads * vdim, kv_rank)),
        out=t.bf16(at + "o", (width, heads * vdim)))


def _mlstm(t, at: str, mx: dict, width: int) -> MatrixMemory:
    heads, dim, vdim = integer(mx, "heads"), integer(mx, "dim"), integer(mx, "vdim")
    return MatrixMemory(
        heads, dim, vdim, number(mx, "gate_cap"),
        q=t.bf16(at + "q", (heads * dim, width)), k=t.bf16(at + "k", (heads * dim, width)),
        v=t.bf16(at + "v", (heads * vdim, width)), gate=t.bf16(at + "g", (heads * vdim, width)),
        i=t.bf16(at + "i", (heads, width)), i_bias=t.bf16(at + "i.b", (heads,)),
        f=t.bf16(at + "f", (heads, width)), f_bias=t.bf16(at + "f.b", (heads,)),
        head_norm=t.bf16(at + "norm", (heads * vdim,)), out=t.bf16(at + "o", (width, heads * vdim)))


def _feed_forward(t, at: str, mlp: dict, width: int):
    kind = mlp.get("kind")
    if kind == "dense":
        ff = integer(mlp, "ff")
        return GatedFfn(t.bf16(at + "gate", (ff, width)), t.bf16(at + "up", (ff, width)), t.bf16(at + "down", (width, ff)))
    if kind != "moe":
        raise ConfigError(f"config: feed-forward kind {kind!r}")
    ff, experts, top = integer(mlp.get("expert"), "ff"), integer(mlp.get("router"), "experts"), integer(mlp.get("router"), "top")
    if top > experts:
        raise ConfigError(f"config: top {top} of {experts} experts")
    out = Experts(top, t.bf16(at + "router", (experts, width)), t.bf16(at + "router.b", (experts,)),
                  up=[t.bf16(f"{at}e{e}.up", (ff, width)) for e in range(experts)],
                  down=[t.bf16(f"{at}e{e}.down", (width, ff)) for e in range(experts)])
    if mlp.get("shared") is not None:
        shared_ff = integer(mlp["shared"], "ff")
        out.shared_up = t.bf16(at + "shared.up", (shared_ff, width))
        out.shared_down = t.bf16(at + "shared.down", (width, shared_ff))
        out.shared_gate = t.bf16(at + "shared.sg", (1, width))
    return out


def weights(config: dict, tensors) -> ModelWeights:
    """The model's weights; ``tensors`` offers bf16(name, shape)."""
    width, vocab, layers = integer(config, "width"), integer(config, "vocab"), config.get("layers")
    if not isinstance(layers, list) or not layers or not all(isinstance(x, dict) for x in layers):
        raise ConfigError("config: 'layers' must be a list of layers")

    def layer(n: int):
        d, at = layers[n], f"l{n}."

        def make() -> LayerWeights:
            if d.get("type") == "latent_attention":
                mixer = _latent_attention(tensors, at + "mix.", d.get("mixer"), width, n, layers)
            elif d.get("type") == "mlstm":
                mixer = _mlstm(tensors, at + "mix.", d.get("mixer"), width)
            else:
                raise ConfigError(f"config: layer {n} is of type {d.get('type')!r}")
            out = LayerWeights(tensors.bf16(at + "norm1", (width,)), mixer)
            if d.get("mlp") is not None:
                out.norm2 = tensors.bf16(at + "norm2", (width,))
                out.ffn = _feed_forward(tensors, at + "mlp.", d["mlp"], width)
            return out
        return make

    return ModelWeights(width, vocab, number(config.get("norm"), "eps"), embed=tensors.bf16("embed", (vocab, width)),
                        final_norm=tensors.bf16("final.norm", (width,)), head=tensors.bf16("head", (vocab, width)),
                        layers=[layer(n) for n in range(len(layers))])


@register("Kogilix", sequence=True)
def load(config: dict, model_dir: Path, slots: int = 8, cap: int = 4096, max_rows: int = 2048, dtype: str = "bfloat16",
         device_id: int = 0) -> SequenceModel:
    return SequenceModel(weights(config, SafeTensors(model_dir / "model.safetensors")), slots, cap, max_rows, dtype, device_id)
