"""Small random sequence models for the tests: configurations, weights, the plain implementation's view of them, and how
results are compared."""
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


def scaling(factor=3.0, low=1.0, high=5.0, original=90):
    """Short enough for all three bands to occur among a few pairs."""
    return dict(factor=factor, low=low, high=high, original=original)


def attention(heads=4, kv_heads=2, dim=24, vdim=40, scale=0.3, rot=12, base=500.0, stretch=None, chunk=None, kv_from=None, mlp=None):
    mixer = dict(heads=heads, kv_heads=kv_heads, dim=dim, vdim=vdim, scale=scale, rot=dict(dims=rot, base=base))
    if stretch is not None:
        mixer["rot"]["scaling"] = stretch
    if chunk is not None:
        mixer["mask"] = {"size": chunk}
    if kv_from is not None:
        mixer["kv_from"] = kv_from
    return {"type": "attention", "mixer": mixer, "mlp": mlp}


def delta(heads=4, kv_heads=2, dim=40, vdim=24, conv=4, mlp=None):
    return {"type": "delta", "mixer": dict(heads=heads, kv_heads=kv_heads, dim=dim, vdim=vdim, conv=conv), "mlp": mlp}


def clamped(ff=104, limit=0.8):
    return {"kind": "dense", "ff": ff, "limit": limit}


def bosirax(*layers, width=136, vocab=203, eps=3e-5, scale=1.7, pairs=(97, 13, 5)):
    embedding = {"scale": scale}
    if pairs is not None:
        embedding["bigram"] = dict(zip(("buckets", "mul_prev", "mul_cur"), pairs))
    return {"architecture": "Bosirax", "width": width, "vocab": vocab, "norm": {"eps": eps}, "embedding": embedding,
            "layers": list(layers)}


def random_bosirax(cfg, seed=0, a_log=-1.0, dt_bias=0.0, gates=2.0):
    rng = np.random.default_rng(seed)
    t = Tensors()
    width, vocab = cfg["width"], cfg["vocab"]

    def linear(name, out, inp, gain=1.0):
        t.put(name, rng.standard_normal((out, inp)) * gain / np.sqrt(inp))

    def norm(name, n, about=0.0):
        t.put(name, about + rng.uniform(-0.5, 0.5, n))

    t.put("embed", rng.standard_normal((vocab, width)))
    if "bigram" in cfg["embedding"]:
        t.put("bigram", rng.standard_normal((cfg["embedding"]["bigram"]["buckets"] + 1, width)))
    for n, layer in enumerate(cfg["layers"]):
        at, m = f"l{n}.", layer["mixer"]
        H, G, d, v = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
        norm(at + "norm1", width)
        if layer["type"] == "attention":
            linear(at + "mix.q", H * d, width)
            if "kv_from" not in m:
                linear(at + "mix.k", G * d, width)
                linear(at + "mix.v", G * v, width)
        else:
            for name, rows in (("q", G * d), ("k", G * d), ("v", H * v)):
                linear(at + "mix." + name, rows, width)
                linear(f"{at}mix.{name}.conv", rows, m["conv"], 1.5)
            linear(at + "mix.g", H * v, width)
            linear(at + "mix.b", H, width, gates)
            linear(at + "mix.a", H, width, gates)
            t.put(at + "mix.A_log", rng.standard_normal(H) + a_log)
            t.put(at + "mix.dt_bias", rng.standard_normal(H) + dt_bias)
            norm(at + "mix.norm", v, 1.0)
        linear(at + "mix.o", width, H * v)
        if layer["mlp"] is not None:
            norm(at + "norm2", width)
            linear(at + "mlp.gate", layer["mlp"]["ff"], width)
            linear(at + "mlp.up", layer["mlp"]["ff"], width)
            linear(at + "mlp.down", width, layer["mlp"]["ff"])
    norm("final.norm", width)
    linear("head", vocab, width)
    return t


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


def run(model, slot, tokens, cuts, at=0):
    """Logits of every token, fed in the given portions."""
    rows = []
    for n in cuts:
        rows.append(model.forward([(slot, at, tokens[at:at + n])], range(n)))
        at += n
    return np.concatenate(rows)


def tokens_of(cfg, n, seed=0):
    return np.random.default_rng(seed + 1000).integers(0, cfg["vocab"], n).tolist()


def check(got, want, dtype, f32=2e-5, bf16=0.02, note=""):
    e = row_errors(got, want)
    print(f"[sequence] {note} {dtype}: worst {e.max():.2e} median {np.median(e):.2e}", flush=True)
    if dtype == "float32":
        # where a memory's output nearly cancels, the norm behind it magnifies the last bits (weights changed by half
        # a 32-bit rounding move such rows by 1e-5): a few rows may be further off, a wrong one is off by 1e-2
        ok = np.median(e) < f32 / 5 and np.mean(e > f32) <= 0.05 and e.max() < 30 * f32
        assert ok, (note, int(e.argmax()), float(e.max()), float(np.median(e)))
    else:
        # a router may choose otherwise where two logits are within a bfloat16 rounding: a few rows
        assert np.median(e) < bf16 and np.mean(e > 4 * bf16) <= 0.05, (note, int(e.argmax()), float(e.max()), float(np.median(e)))
