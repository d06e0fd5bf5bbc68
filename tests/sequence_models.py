"""Small random sequence models for the tests: configurations, weights and the plain implementation's view of them."""
import numpy as np

from llaminar_amd.sequence import bf16_bits, bf16_to_f32


class Tensors:
    """Weights in memory, as a model family reads them and as the plain implementation takes them."""

    def __init__(self):
        self.bits = {}

    def put(self, name, values):
        self.bits[name] = bf16_bits(values).reshape(np.shape(values))

    def bf16(self, name, shape):
        t = self.bits[name]
        assert t.shape == tuple(shape), (name, t.shape, shape)
        return t

    def plain(self):
        return {n: bf16_to_f32(b).astype(np.float64) for n, b in self.bits.items()}


def latent(heads=3, dim=24, vdim=40, q_rank=56, kv_rank=88, scale=0.3, kv_from=None, mlp=None):
    mixer = dict(heads=heads, dim=dim, vdim=vdim, q_rank=q_rank, kv_rank=kv_rank, scale=scale)
    if kv_from is not None:
        mixer["kv_from"] = kv_from
    return {"type": "latent_attention", "mixer": mixer, "mlp": mlp}


def mlstm(heads=3, dim=40, vdim=24, gate_cap=9.0, mlp=None):
    return {"type": "mlstm", "mixer": dict(heads=heads, dim=dim, vdim=vdim, gate_cap=gate_cap), "mlp": mlp}


def dense(ff=104):
    return {"kind": "dense", "ff": ff}


def moe(ff=72, experts=7, top=2, shared=None):
    return {"kind": "moe", "expert": {"ff": ff}, "router": {"experts": experts, "top": top},
            "shared": None if shared is None else {"ff": shared}}


def config(*layers, width=136, vocab=203, eps=3e-5):
    return {"architecture": "Kogilix", "width": width, "vocab": vocab, "norm": {"eps": eps}, "layers": list(layers)}


def random_weights(cfg, seed=0, forget_bias=2.0, input_bias=0.0):
    rng = np.random.default_rng(seed)
    t = Tensors()
    width, vocab = cfg["width"], cfg["vocab"]

    def linear(name, out, inp, gain=1.0):
        t.put(name, rng.standard_normal((out, inp)) * gain / np.sqrt(inp))

    def norm(name, n):
        t.put(name, rng.uniform(0.5, 1.5, n))

    t.put("embed", rng.standard_normal((vocab, width)))
    for n, layer in enumerate(cfg["layers"]):
        at, m = f"l{n}.", layer["mixer"]
        norm(at + "norm1", width)
        H, d, v = m["heads"], m["dim"], m["vdim"]
        if layer["type"] == "latent_attention":
            linear(at + "mix.dq", m["q_rank"], width)
            norm(at + "mix.dq.norm", m["q_rank"])
            linear(at + "mix.uq", H * d, m["q_rank"])
            if m.get("kv_from") is None:
                linear(at + "mix.dkv", m["kv_rank"], width)
                norm(at + "mix.dkv.norm", m["kv_rank"])
            linear(at + "mix.uk", H * d, m["kv_rank"])
            linear(at + "mix.uv", H * v, m["kv_rank"])
        else:
            linear(at + "mix.q", H * d, width)
            linear(at + "mix.k", H * d, width)
            linear(at + "mix.v", H * v, width)
            linear(at + "mix.g", H * v, width)
            linear(at + "mix.i", H, width, 3.0)
            linear(at + "mix.f", H, width, 3.0)
            t.put(at + "mix.i.b", rng.standard_normal(H) + input_bias)
            t.put(at + "mix.f.b", rng.standard_normal(H) + forget_bias)
            norm(at + "mix.norm", H * v)
        linear(at + "mix.o", width, H * v)
        mlp = layer["mlp"]
        if mlp is None:
            continue
        norm(at + "norm2", width)
        if mlp["kind"] == "dense":
            linear(at + "mlp.gate", mlp["ff"], width)
            linear(at + "mlp.up", mlp["ff"], width)
            linear(at + "mlp.down", width, mlp["ff"])
            continue
        E, ff = mlp["router"]["experts"], mlp["expert"]["ff"]
        linear(at + "mlp.router", E, width, 2.0)
        t.put(at + "mlp.router.b", rng.standard_normal(E))
        for e in range(E):
            linear(f"{at}mlp.e{e}.up", ff, width)
            linear(f"{at}mlp.e{e}.down", width, ff)
        if mlp["shared"] is not None:
            linear(at + "mlp.shared.up", mlp["shared"]["ff"], width)
            linear(at + "mlp.shared.down", width, mlp["shared"]["ff"])
            linear(at + "mlp.shared.sg", 1, width)
    norm("final.norm", width)
    linear("head", vocab, width)
    return t


def row_errors(got, want):
    """Per row: rms of the difference over the rms of all of ``want``."""
    want = np.asarray(want, np.float64)
    return np.sqrt(np.mean((np.asarray(got, np.float64) - want) ** 2, axis=1)) / np.sqrt(np.mean(want ** 2))
