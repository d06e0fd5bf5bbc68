"""Sequence models on the CPU: weight layouts, configuration and weight files, the scheduler and its slots, the
exported C ABI, and the plain implementation against closed forms."""
import ctypes
import json
import re
from pathlib import Path

import numpy as np
import pytest

from llaminar_amd import engine, models, safetensors_io, sequence, trace
from llaminar_amd.models import bosirax, kogilix
from oracle import sequence_oracle as so
from tests import sequence_models as sm

ROOT = Path(__file__).resolve().parent.parent


# ---- C ABI -----------------------------------------------------------------------------------------

def test_library_exports_every_declared_symbol():
    assert sequence.LIB_PATH.exists(), "build the library first: python -m llaminar_amd.build"
    lib = ctypes.CDLL(str(sequence.LIB_PATH))
    text = "".join((ROOT / "include" / "llaminar_amd" / h).read_text() for h in ("seq_api.h", "sequence_model.h"))
    names = set(re.findall(r"\b(llam_seqm?_[a-z0-9_]+)\s*\(", re.sub(r"/\*.*?\*/", "", text, flags=re.S)))
    assert len(names) >= 18
    for n in names:
        assert hasattr(lib, n), n
    assert names | {"llam_ql_last_error"} == set(sequence.SIGNATURES)


def test_bad_arguments_are_refused_before_any_launch():
    lib = sequence.load()
    buf = np.zeros(4096, np.uint8)
    p = buf.ctypes.data + (-buf.ctypes.data % 16)
    err = lambda: lib.llam_ql_last_error().decode()
    a = sequence.LinearArgs(d_a=p, d_w=p, d_y=p, M=1, N=20, K=64, lda=64, ldy=32, batch=1)
    assert not lib.llam_seq_linear(ctypes.byref(a), 0, 0, None) and "multiple of" in err()
    a = sequence.LinearArgs(d_a=p, d_w=p, d_y=p, d_norm=p, M=17, N=16, K=64, lda=64, ldy=16, batch=1, k_real=64)
    assert not lib.llam_seq_linear(ctypes.byref(a), 0, 0, None) and "fused norm" in err()
    a = sequence.LinearArgs(d_a=p, d_w=p, d_y=p, M=2, N=16, K=64, lda=32, ldy=16, batch=1)
    assert not lib.llam_seq_linear(ctypes.byref(a), 0, 0, None) and "strides" in err()
    m = sequence.MemoryArgs(d_proj=p, ldp=4096, d_gate_bias=p, d_norm=p, d_state=p, d_m=p, d_y=p, heads=1, dim=576, vdim=64,
                            vdim_real=64, q_scale=1.0, gate_cap=1.0, eps=1e-5)
    e = sequence.Entries(p, p, p, p)
    assert not lib.llam_seq_memory_decode(ctypes.byref(m), ctypes.byref(e), 0, 1, p, 1 << 30, 0, 0, None) and "512" in err()
    x = sequence.ExpertsArgs(d_logits=p, ldz=16, d_up=p, d_down=p, experts=4, top=5, ff=64, K=64, N=64, d_h=p, d_x=p, ldx=64)
    assert not lib.llam_seq_experts(ctypes.byref(x), 1, p, 1 << 30, 0, 0, None) and "top=5" in err()
    assert not lib.llam_seq_latent_attention(p, p, ctypes.byref(e), 0, 1, 1, 65, 1, 64, 64, 1.0, p, p, 1 << 30, 0, 0, None)
    assert "max_len=65" in err()
    g = sequence.AttentionArgs(5, 2, 64, 64, 128, 0, 1.0, p, p)
    assert not lib.llam_seq_attention(ctypes.byref(g), p, ctypes.byref(e), 0, 1, 1, 65, p, 320, p, 1 << 30, 0, 0, None) and "kv_heads" in err()
    g = sequence.AttentionArgs(4, 2, 96, 64, 128, 0, 1.0, p, p)
    assert not lib.llam_seq_attention(ctypes.byref(g), p, ctypes.byref(e), 0, 1, 1, 65, p, 256, p, 1 << 30, 0, 0, None) and "padded" in err()
    g = sequence.AttentionArgs(4, 2, 64, 64, 128, 0, 1.0, p, p)
    assert not lib.llam_seq_attention(ctypes.byref(g), p, ctypes.byref(e), 0, 1, 1, 129, p, 256, p, 1 << 30, 0, 0, None) and "129 positions" in err()
    assert not lib.llam_seq_rotary(ctypes.byref(g), p, 256, True, p, 4, p, p, p, 1, 0, 0, None) and "ldp=256" in err()
    d = sequence.DeltaArgs(d_proj=p, ldp=4096, d_conv=p, d_a_log=p, d_dt_bias=p, d_norm=p, d_state=p, d_recent=p, d_y=p, ldy=64, heads=1,
                           kv_heads=1, dim=320, vdim=64, dim_real=300, vdim_real=64, taps=4, eps=1e-5)
    assert not lib.llam_seq_delta_decode(ctypes.byref(d), ctypes.byref(e), 0, 1, 0, 0, None) and "256" in err()
    d.dim, d.dim_real, d.taps = 64, 64, 0
    assert not lib.llam_seq_delta_prefill(ctypes.byref(d), ctypes.byref(e), 0, 5, p, 1 << 30, 0, 0, None) and "taps=0" in err()
    m = sequence.EmbedArgs(d_table=p, vocab=9, width=64, scale=1.0, d_pairs=p, buckets=0)
    assert not lib.llam_seq_embed(ctypes.byref(m), p, p, 1, 64, 0, None) and "buckets=0" in err()
    a = sequence.LinearArgs(d_a=p, d_w=p, d_y=p, M=1, N=16, K=64, lda=64, ldy=16, batch=1)
    b = sequence.LinearArgs(d_a=p, d_w=p, d_y=p, M=1, N=16, K=128, lda=128, ldy=16, batch=1)
    assert not lib.llam_seq_linear_pair(ctypes.byref(a), ctypes.byref(b), 0, 0, None) and "same rows" in err()
    assert not lib.llam_seqm_create(ctypes.byref(sequence.Config(0, 1, 1, 1, 1, 1, 0, 1e-5, 0)))


# ---- layouts ---------------------------------------------------------------------------------------

def test_weight_tiles_follow_the_documented_order():
    rng = np.random.default_rng(0)
    w = rng.integers(0, 1 << 16, (37, 100)).astype(np.uint16)
    t = sequence.tiled(w)
    assert t.shape == (3, 4, 4, 16, 8) and t.flags.c_contiguous
    for row, col in rng.integers(0, (48, 128), (500, 2)):
        want = w[row, col] if row < 37 and col < 100 else 0
        assert t[row // 16, col // 32, (col % 32) // 8, row % 16, col % 8] == want


def test_gate_and_up_alternate_by_tiles():
    g, u = np.full((24, 64), 1, np.uint16), np.full((24, 64), 2, np.uint16)
    t = sequence.gate_up_tiles(g, u)
    assert t.shape[0] == 8 and [int(t[i].max()) for i in range(8)] == [1, 2, 1, 2, 0, 0, 0, 0]


def test_heads_are_padded_one_by_one():
    w = np.arange(6 * 5, dtype=np.uint16).reshape(6, 5) + 1
    r = sequence.head_rows(w, 2, 3)
    assert r.shape == (128, 5) and np.array_equal(r[:3], w[:3]) and np.array_equal(r[64:67], w[3:]) and not r[3:64].any()
    c = sequence.head_columns(w.T.copy(), 2, 3)
    assert c.shape == (5, 128) and np.array_equal(c[:, 64:67], w.T[:, 3:]) and not c[:, 67:].any()


def test_bf16_rounds_to_nearest_even():
    x = np.array([1.0, 1.00390625, 1.01171875, -2.5, 3e-39, 65280.0], np.float32)
    torch = pytest.importorskip("torch")
    assert np.array_equal(sequence.bf16_bits(x), torch.from_numpy(x).to(torch.bfloat16).view(torch.uint16).numpy())


# ---- weight files ----------------------------------------------------------------------------------

def test_safetensors_round_trip_and_refusals(tmp_path):
    path = tmp_path / "m.safetensors"
    a, b = np.arange(12, dtype=np.uint16).reshape(3, 4), np.arange(3, dtype=np.int32)
    safetensors_io.write(path, {"a": a, "b": b})
    f = safetensors_io.SafeTensors(path)
    assert f.names() == ["a", "b"] and np.array_equal(f.bf16("a", (3, 4)), a) and np.array_equal(f.raw("b", "I32"), b)
    for bad in (lambda: f.bf16("a", (4, 3)), lambda: f.bf16("b", (3,)), lambda: f.raw("c")):
        with pytest.raises(safetensors_io.SafeTensorsError):
            bad()
    def rewrite(header, data=b"\0" * 8):
        text = header if isinstance(header, bytes) else json.dumps(header).encode()
        path.write_bytes(len(text).to_bytes(8, "little") + text + data)
        safetensors_io.SafeTensors(path)
    for header in (b"[1]", b"{", {"a": {"dtype": "BF16", "shape": [5], "data_offsets": [0, 10]}},
                   {"a": {"dtype": "BF16", "shape": [2], "data_offsets": [2, 8]}},
                   {"a": {"dtype": "BF16", "shape": [-1, -4], "data_offsets": [0, 8]}},
                   {"a": {"dtype": "Q4", "shape": [4], "data_offsets": [0, 8]}}, {"a": {"dtype": "BF16"}}):
        with pytest.raises(safetensors_io.SafeTensorsError):
            rewrite(header)
    path.write_bytes((1 << 40).to_bytes(8, "little") + b"{}")
    with pytest.raises(safetensors_io.SafeTensorsError):
        safetensors_io.SafeTensors(path)


# ---- configuration -----------------------------------------------------------------------------------

def test_registry_names_the_families(tmp_path):
    assert {"Kogilix", "Bosirax", "DenseQ4K"} <= set(models.families())
    assert [models.needs_sequence_library({"architecture": n}) for n in ("Bosirax", "Kogilix", "DenseQ4K")] == [True, True, False]
    (tmp_path / "config.json").write_text('{"architecture": "Nobody"}')
    with pytest.raises(models.ConfigError, match="Nobody"):
        models.load_model(tmp_path)
    (tmp_path / "config.json").write_text('{"layers": []}')
    with pytest.raises(models.ConfigError):
        models.read_config(tmp_path)


def build_layers(cfg, seed=0):
    return [make() for make in kogilix.weights(cfg, sm.random_weights(cfg, seed)).layers]


def test_every_branch_of_the_configuration_is_read():
    cfg = sm.config(sm.latent(), sm.mlstm(mlp=sm.dense()), sm.latent(kv_from=0, dim=16, vdim=8, heads=5, q_rank=20, mlp=sm.moe()),
                    sm.mlstm(mlp=sm.moe(shared=48)))
    a, b, c, d = build_layers(cfg)
    assert a.ffn is None and a.norm2 is None and a.mixer.kv_from is None and a.mixer.dkv.shape == (88, 136)
    assert b.mixer.gate_cap == 9.0 and b.ffn.gate.shape == (104, 136)
    assert c.mixer.kv_from == 0 and c.mixer.dkv is None and c.mixer.heads == 5
    assert len(c.ffn.up) == 7 and c.ffn.top == 2 and c.ffn.shared_up is None
    assert d.ffn.shared_up.shape == (48, 136) and d.ffn.shared_gate.shape == (1, 136)


@pytest.mark.parametrize("spoil", [
    lambda c: c["layers"][1]["mixer"].update(kv_from=1), lambda c: c["layers"][1]["mixer"].update(kv_from=2),
    lambda c: c["layers"][0]["mixer"].update(heads=0), lambda c: c["layers"][0]["mixer"].pop("scale"),
    lambda c: c["layers"][0].update(type="other"), lambda c: c["layers"][2].update(mlp={"kind": "odd"}),
    lambda c: c["layers"][2].update(mlp=sm.moe(experts=2, top=3)), lambda c: c["layers"][3]["mixer"].update(kv_from=2),
    lambda c: c["layers"][1]["mixer"].update(kv_rank=64)])
def test_faulty_configurations_are_refused(spoil):
    cfg = sm.config(sm.latent(), sm.latent(kv_from=0), sm.mlstm(mlp=sm.moe()), sm.latent(kv_from=0))
    tensors = sm.random_weights(cfg)
    spoil(cfg)
    with pytest.raises((models.ConfigError, AssertionError)) as e:
        [make() for make in kogilix.weights(cfg, tensors).layers]
    assert e.type is models.ConfigError


def test_every_branch_of_the_bosirax_configuration_is_read():
    cfg = sm.bosirax(sm.delta(mlp=sm.clamped(limit=1.25)), sm.attention(chunk=9, stretch=sm.scaling()), sm.attention(kv_from=1, heads=6, scale=0.5, mlp=sm.clamped(ff=50)),
                     sm.attention(rot=0))
    w = bosirax.weights(cfg, sm.random_bosirax(cfg))
    a, b, c, d = [make() for make in w.layers]
    assert w.embed_scale == 1.7 and (w.pairs.buckets, w.pairs.mul_prev, w.pairs.mul_cur, len(w.pairs.table)) == (97, 13, 5, 98)
    assert all(x.parallel for x in (a, b, c, d)) and a.norm1.dtype == np.float32 and abs(a.norm1.mean() - 1) < 0.2
    assert a.mixer.q_conv.shape == (80, 4) and a.mixer.v_conv.shape == (96, 4) and a.ffn.limit == 1.25 and a.mixer.head_norm.shape == (24,)
    assert b.ffn is None and b.norm2 is None and b.mixer.chunk == 9 and len(b.mixer.turns) == 6 and b.mixer.k.shape == (48, 136)
    assert c.mixer.k is None and c.mixer.v is None and c.mixer.kv_from == 1 and c.mixer.heads == 6 and c.mixer.chunk is None
    assert len(d.mixer.turns) == 0
    cfg["embedding"].pop("bigram")
    assert bosirax.weights(cfg, sm.random_bosirax(cfg)).pairs is None


@pytest.mark.parametrize("spoil", [
    lambda c: c["layers"][1]["mixer"].update(kv_from=1), lambda c: c["layers"][1]["mixer"].update(kv_from=3),
    lambda c: c["layers"][3]["mixer"].update(kv_from=2), lambda c: c["layers"][3]["mixer"].update(kv_from=1),
    lambda c: c["layers"][1]["mixer"].update(kv_heads=1), lambda c: c["layers"][0]["mixer"].update(kv_heads=3),
    lambda c: c["layers"][0]["mixer"]["rot"].update(dims=3), lambda c: c["layers"][0]["mixer"]["rot"].update(dims=26),
    lambda c: c["layers"][0]["mixer"]["rot"].update(scaling={"factor": 2.0}), lambda c: c["layers"][0]["mixer"].pop("rot"),
    lambda c: c["layers"][0]["mixer"].update(mask={"size": 0}), lambda c: c["layers"][2]["mixer"].update(conv=0),
    lambda c: c["layers"][2].update(mlp={"kind": "moe"}), lambda c: c["layers"][2]["mlp"].pop("limit"),
    lambda c: c["layers"][2].update(type="mlstm"), lambda c: c.pop("embedding"), lambda c: c["embedding"]["bigram"].update(buckets=0)])
def test_faulty_bosirax_configurations_are_refused(spoil):
    cfg = sm.bosirax(sm.attention(), sm.attention(kv_from=0), sm.delta(mlp=sm.clamped()), sm.attention(kv_from=0))
    tensors = sm.random_bosirax(cfg)
    spoil(cfg)
    with pytest.raises((models.ConfigError, AssertionError)) as e:
        [make() for make in bosirax.weights(cfg, tensors).layers]
    assert e.type is models.ConfigError


@pytest.mark.parametrize("stretch", [None, sm.scaling(), sm.scaling(8.0, 1.5, 6.0, 300)])
def test_rotary_turns_are_the_plain_frequencies(stretch):
    rot = dict(dims=46, base=700.0)
    if stretch:
        rot["scaling"] = stretch
        wave = 2 * np.pi / so.rotary_frequencies(46, 700.0)
        bands = {(w > stretch["original"] / stretch["low"]) - int(w < stretch["original"] / stretch["high"]) for w in wave}
        assert bands == {-1, 0, 1}
    assert np.allclose(bosirax.rotary_turns(rot) * 2 * np.pi, so.rotary_frequencies(46, 700.0, stretch), rtol=1e-13)


# ---- scheduler -----------------------------------------------------------------------------------------

class Counting:
    """A runner whose best token is (sum of the sequence so far) mod vocab; keeps its own copy of every slot."""

    vocab = 97

    def __init__(self, slots=3, cap=40, max_rows=8):
        self.slots, self.cap, self.max_rows = slots, cap, max_rows
        self.held = [[] for _ in range(slots)]
        self.steps = []

    def forward(self, entries, want=(), best=False):
        assert len({e[0] for e in entries}) == len(entries) and sum(len(e[2]) for e in entries) <= self.max_rows
        self.steps.append([len(e[2]) for e in entries])
        sums = []
        for slot, pos, ids in entries:
            if pos == 0:
                self.held[slot] = []
            assert len(self.held[slot]) == pos and pos + len(ids) <= self.cap
            for t in ids:
                self.held[slot].append(t)
                sums.append(sum(self.held[slot]) % self.vocab)
        chosen = [sums[w] for w in want]
        return chosen if best else np.eye(self.vocab)[chosen] if chosen else np.empty((0, self.vocab))

    def decode(self, slots, pos, ids, steps):
        out = np.empty((steps, len(slots)), np.int32)
        ids = list(ids)
        for s in range(steps):
            for b, slot in enumerate(slots):
                assert len(self.held[slot]) == pos[b] + s < self.cap
                self.held[slot].append(int(ids[b]))
                ids[b] = out[s, b] = sum(self.held[slot]) % self.vocab
        self.steps.append(("burst", len(slots), steps))
        return out

    def max_decode_steps(self, n):
        return 10


def expected(prompt, n):
    seq = list(prompt)
    for _ in range(n):
        seq.append(sum(seq) % Counting.vocab)
    return seq[len(prompt):]


def test_scheduler_serves_more_requests_than_slots():
    runner = Counting()
    e = engine.Engine(runner, portion=5, burst=4)
    prompts = [[7] * n for n in (1, 13, 6, 2, 9, 30, 3)]
    assert e.generate(prompts, 9) == [expected(p, 9) for p in prompts]
    assert len(e.sequences) == 0 and e.sequences.free() == 3
    mixed = [s for s in runner.steps if not isinstance(s, tuple) and 1 in s and max(s) > 1]
    assert mixed, "no step mixed decoding with a portion of a prompt"
    assert any(isinstance(s, tuple) and s[1] == 3 for s in runner.steps) or any(isinstance(s, tuple) for s in runner.steps)


def test_stop_tokens_and_limits():
    e = engine.Engine(Counting(), burst=8)
    full = expected([3, 4], 12)
    assert e.generate([[3, 4]], 12, stop=[full[4]]) == [full[:full.index(full[4]) + 1]]
    with pytest.raises(engine.CapacityError):
        e.submit("long", [1] * 35, 7)
    e.submit("fits", [1] * 35, 6)
    with pytest.raises(ValueError):
        e.submit("fits", [1], 1)
    with pytest.raises(ValueError):
        e.submit("bad", [97], 1)
    while e.pending():
        e.step()


def test_feed_cuts_what_exceeds_a_step_and_slots_are_used_again():
    runner = Counting(slots=2)
    e = engine.Engine(runner)
    tokens = list(range(1, 21))
    got = e.feed([("a", tokens, [0, 7, 8, 19])])
    assert [int(np.argmax(r)) for r in got[0]] == [sum(tokens[:k + 1]) % 97 for k in (0, 7, 8, 19)]
    e.feed([("b", [5], [])])
    with pytest.raises(engine.CapacityError):
        e.feed([("c", [1], [])])
    e.release("a")
    got = e.feed([("c", [1, 2], [1]), ("b", [6], [0])])
    assert [int(np.argmax(r[0])) for r in got] == [3, 11]
    with pytest.raises(engine.CapacityError):
        e.feed([("c", [1] * 39, [])])


def test_trace_replay_writes_wanted_rows(tmp_path):
    e = engine.Engine(Counting())
    said = []
    lines = [json.dumps({"step": 0, "entries": [{"id": "a", "tokens": [1, 2, 3], "want": [0, 2]}], "end": []}), "",
             json.dumps({"step": 4, "entries": [{"id": "a", "tokens": [4], "want": []}], "end": ["a"]}),
             json.dumps({"step": 5, "entries": [{"id": "a", "tokens": [9], "want": [0]}], "end": ["a", "nobody"]})]
    trace.replay(e, lines, tmp_path, said.append)
    assert said == ["done 0", "done 4", "done 5"] and sorted(p.name for p in tmp_path.iterdir()) == ["0.f32", "5.f32"]
    rows = np.fromfile(tmp_path / "0.f32", "<f4").reshape(2, 97)
    assert rows.argmax(axis=1).tolist() == [1, 6]
    assert np.fromfile(tmp_path / "5.f32", "<f4").argmax() == 9


# ---- the plain implementation itself -----------------------------------------------------------------

def test_recurrence_equals_its_unrolled_sum():
    rng = np.random.default_rng(3)
    T, d, v = 23, 6, 5
    q, k, val = rng.standard_normal((T, d)), rng.standard_normal((T, d)), rng.standard_normal((T, v))
    i, f = rng.standard_normal(T) * 3, -rng.uniform(0.01, 4, T)
    o, S, n, m = so.mlstm_recurrence(q, k, val, i, f)
    F = np.cumsum(f)
    for t in range(T):
        mt = max(F[t], max(F[t] - F[j] + i[j] for j in range(t + 1)))   # the running maximum starts at 0
        w = np.array([np.exp(F[t] - F[j] + i[j] - mt) * (k[j] @ q[t]) for j in range(t + 1)])
        want = (w @ val[:t + 1]) / (max(abs(w.sum()), np.exp(-mt)) + 1e-6)
        assert np.allclose(o[t], want, rtol=1e-10, atol=1e-12)
    assert abs(m - mt) < 1e-12


def test_routing_takes_the_largest_and_ties_go_low():
    ids, w = so.route(np.array([1.0, 3.0, 3.0, -1.0]), 3)
    assert ids == [1, 2, 0] and np.allclose(w, np.exp([3, 3, 1]) / np.exp([3, 3, 1]).sum())


def test_latent_attention_is_causal():
    cfg = sm.config(sm.latent())
    t = sm.random_weights(cfg, 5).plain()
    tokens = [5, 9, 100, 7, 3]
    a, b = so.kogilix(cfg, t, tokens), so.kogilix(cfg, t, tokens[:3] + [1, 2])
    assert np.array_equal(a[:3], b[:3]) and not np.allclose(a[3], b[3])


def test_rotation_keeps_lengths_and_sees_distances():
    rng = np.random.default_rng(4)
    freq = so.rotary_frequencies(6, 100.0)
    x = rng.standard_normal((2, 1, 8))
    y = so.rotate(x, [3, 3], freq)
    assert np.allclose(np.linalg.norm(y, axis=-1), np.linalg.norm(x, axis=-1)) and np.array_equal(y[..., 6:], x[..., 6:])
    dots = [so.rotate(x[:1], [p + 5], freq)[0, 0] @ so.rotate(x[1:], [p], freq)[0, 0] for p in (0, 7, 100)]
    assert np.allclose(dots, dots[0])


def test_delta_recurrence_equals_its_chunked_form():
    """The triangular system of a chunk, solved at once, against the recurrence token by token."""
    rng = np.random.default_rng(3)
    T, d, v = 19, 6, 5
    q, k, val = so.unit(rng.standard_normal((T, d))), so.unit(rng.standard_normal((T, d))), rng.standard_normal((T, v))
    decay, beta = rng.uniform(0.5, 1.0, T), rng.uniform(0.0, 1.0, T)
    o, S = so.delta_recurrence(q, k, val, decay, beta)
    G = np.cumsum(np.log(decay))
    f = np.tril(np.exp(G[:, None] - G[None]))
    u = np.linalg.solve(np.eye(T) + np.tril(beta[:, None] * f * (k @ k.T), -1), beta[:, None] * val)
    assert np.allclose((f * (q @ k.T)) @ u, o) and np.allclose((np.exp(G[-1] - G)[:, None] * k).T @ u, S)


def test_delta_rule_replaces_what_a_key_held():
    k = np.eye(3)[[0, 1, 0]]
    v = np.array([[1.0, 2.0], [3.0, 4.0], [5.0, 6.0]])
    o, S = so.delta_recurrence(k, k, v, np.ones(3), np.ones(3))
    assert np.allclose(S, [[5, 6], [3, 4], [0, 0]]) and np.allclose(o, v)


def test_chunked_attention_forgets_at_the_edge():
    rng = np.random.default_rng(8)
    q, k, v = (rng.standard_normal((9, 2, 4)) for _ in range(3))
    o = so.grouped_attention(q, k, v, 0.5, 4)
    assert np.allclose(o[4], v[4]) and np.allclose(o[8], v[8])
    assert np.allclose(o[4:8], so.grouped_attention(q[4:8], k[4:8], v[4:8], 0.5, None))


def test_short_convolution_and_pairs():
    x = np.arange(1.0, 6.0)[:, None]
    y = so.short_convolution(x, np.array([[100.0, 10.0, 1.0]]))
    z = np.array([1, 12, 123, 234, 345.0])[:, None]
    assert np.allclose(y, z * so.sigmoid(z))
    assert so.bigram_rows([3, 1, 4], 10, 1, 7) == [7, 31 % 7, 14 % 7]
