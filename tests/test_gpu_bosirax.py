"""Bosirax models on the GPU against the plain implementation (oracle/sequence_oracle.py): each mechanism alone, prompts,
portions, decoding, mixed batches, slots and ring rows used again, and generation through the engine."""
import ctypes
import json
import os
import subprocess
import sys
from pathlib import Path

import numpy as np
import pytest

from llaminar_amd import safetensors_io, sequence
from llaminar_amd.engine import Engine
from llaminar_amd.models import bosirax
from oracle import sequence_oracle as so
from tests import sequence_models as sm
from tests.sequence_models import check, run, tokens_of

pytestmark = pytest.mark.gpu
ROOT = Path(__file__).resolve().parent.parent


@pytest.fixture(scope="module", autouse=True)
def one_runtime(dev):
    """torch is imported (and with it the HIP runtime the process uses) before the library is loaded."""
    return dev


def load(cfg, tensors, dtype="float32", slots=4, cap=640, max_rows=640):
    return sequence.SequenceModel(bosirax.weights(cfg, tensors), slots, cap, max_rows, dtype)


# ---- operators -------------------------------------------------------------------------------------

def attend(dev, dtype, heads, groups, dim, vdim, ntok, chunk, pos, ring=None, n=1):
    """llam_seq_attention over a random cache, entry by entry against plain softmax in float32 on the CPU."""
    import torch

    L = sequence.load()
    td = torch.bfloat16 if dtype == "bfloat16" else torch.float32
    g = torch.Generator().manual_seed(heads * dim + ntok)
    S = pos + ntok
    ring = ring or -(-S // 128) * 128
    q = torch.randn(n * ntok, heads, dim, generator=g).to(td)
    keys, values = torch.randn(n, groups, S, dim, generator=g).to(td), torch.randn(n, groups, S, vdim, generator=g).to(td)
    k, v = torch.full((n, groups, ring, dim), 7.0).to(td), torch.full((n, groups, ring, vdim), 7.0).to(td)
    for p in range(max(0, S - ring), S):
        k[:, :, p % ring], v[:, :, p % ring] = keys[:, :, p], values[:, :, p]
    k, v, qd = k.to(dev), v.to(dev), q.to(dev)
    o = torch.zeros(n * ntok, heads * vdim, dtype=td, device=dev)
    floats = L.llam_seq_attention_scratch_floats(vdim)
    scratch = torch.zeros(floats, device=dev)
    entries = [torch.tensor(x, dtype=torch.int32, device=dev) for x in ([ntok * i for i in range(n)], [ntok] * n, list(range(n)), [pos] * n)]
    a = sequence.AttentionArgs(heads, groups, dim, vdim, ring, chunk, dim ** -0.5, k.data_ptr(), v.data_ptr())
    e = sequence.Entries(*[x.data_ptr() for x in entries])
    stream = torch.cuda.current_stream().cuda_stream
    assert L.llam_seq_attention(ctypes.byref(a), qd.data_ptr(), ctypes.byref(e), 0, n, ntok, S, o.data_ptr(), heads * vdim,
                                scratch.data_ptr(), floats, sequence.DTYPES[dtype], 0, stream), L.llam_ql_last_error()
    torch.cuda.synchronize()
    got = o.float().cpu().view(n, ntok, heads, vdim)
    i, j = torch.arange(pos, S)[:, None], torch.arange(S)[None]
    see = (j <= i) & ((i // chunk == j // chunk) if chunk else (j >= 0))
    per = heads // groups
    for b in range(n):
        for h in range(heads):
            s = q[b * ntok:(b + 1) * ntok, h].float() @ keys[b, h // per].float().T * dim ** -0.5
            want = s.masked_fill(~see, float("-inf")).softmax(-1) @ values[b, h // per].float()
            assert (got[b, :, h] - want).abs().max() < (2e-5 if dtype == "float32" else 0.02), (b, h)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("case", [
    (4, 4, 64, 64, 1, 0, 0), (6, 2, 64, 128, 1, 0, 700), (16, 2, 128, 128, 1, 1000, 2500), (40, 1, 64, 256, 3, 0, 500),
    (4, 2, 128, 64, 23, 0, 0), (8, 4, 128, 128, 300, 100, 0), (8, 4, 128, 64, 300, 100, 77), (4, 1, 64, 128, 30, 200, 399),
    (4, 4, 256, 256, 70, 64, 100), (4, 2, 128, 256, 200, 0, 1000), (24, 1, 256, 64, 33, 50, 20), (2, 1, 128, 128, 700, 1, 0),
    (2, 1, 256, 128, 129, 0, 64)], ids=str)
def test_attention_over_a_cache(dev, case, dtype):
    attend(dev, dtype, *case)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("vdim", [64, 128, 256])
@pytest.mark.parametrize("dim", [64, 128, 256])
def test_attention_at_every_padded_size(dev, dim, vdim, dtype):
    """Rows that the wavefronts share (decoding) and rows of their own (prompts), across a chunk's edge."""
    attend(dev, dtype, 4, 2, dim, vdim, 1, 0, 333)
    attend(dev, dtype, 6, 2, dim, vdim, 5, 90, 177)
    attend(dev, dtype, 6, 2, dim, vdim, 150, 90, 40)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("case", [(8, 2, 64, 64, 1, 100, 1000, 128), (4, 2, 128, 64, 60, 69, 1003, 128), (4, 4, 64, 128, 100, 150, 2040, 256)], ids=str)
def test_attention_over_a_ring_that_has_gone_round(dev, case, dtype):
    attend(dev, dtype, *case)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_attention_of_many_entries(dev, dtype):
    attend(dev, dtype, 8, 2, 64, 64, 1, 300, 900, None, 70)
    attend(dev, dtype, 4, 2, 64, 128, 9, 0, 120, None, 5)


def test_attention_refuses_what_the_cache_does_not_hold():
    L = sequence.load()
    a = sequence.AttentionArgs(4, 2, 64, 64, 128, 100, 1.0, 1 << 20, 1 << 20)
    e = sequence.Entries(1 << 20, 1 << 20, 1 << 20, 1 << 20)
    assert not L.llam_seq_attention(ctypes.byref(a), 1 << 20, ctypes.byref(e), 0, 1, 40, 1000, 1 << 20, 256, 1 << 20, 1 << 40, 0, 0, None)
    assert "139 positions" in L.llam_ql_last_error().decode()


# ---- mechanisms through the model --------------------------------------------------------------------

FULL = dict(dim=24, rot=24)
MECHANISMS = {
    "attention": [sm.attention()],
    "attention, every head its own": [sm.attention(heads=3, kv_heads=3, dim=8, vdim=72, rot=8)],
    "attention, one key head": [sm.attention(heads=20, kv_heads=1, dim=72, vdim=16, rot=34)],
    "attention, wide heads": [sm.attention(heads=2, kv_heads=1, dim=130, vdim=200, rot=130, scale=0.1)],
    "attention, widest heads": [sm.attention(heads=3, kv_heads=1, dim=250, vdim=70, rot=2, scale=0.1)],
    "attention, unrotated": [sm.attention(rot=0)],
    "attention, stretched": [sm.attention(**FULL, stretch=sm.scaling())],
    "attention, stretched otherwise": [sm.attention(dim=64, rot=64, base=20000.0, stretch=sm.scaling(8.0, 2.0, 3.0, 33))],
    "attention, chunk of one": [sm.attention(chunk=1)],
    "attention, chunk of 7": [sm.attention(chunk=7, heads=6, kv_heads=2)],
    "attention, chunk of 64": [sm.attention(chunk=64, **FULL)],
    "attention, chunk of 100": [sm.attention(chunk=100, **FULL)],
    "attention, long chunk": [sm.attention(chunk=1 << 20)],
    "attention, shared": [sm.attention(chunk=30, **FULL), sm.attention(chunk=110, kv_from=0, scale=0.9, **FULL), sm.attention(kv_from=0, **FULL)],
    "attention, shared by more heads": [sm.attention(vdim=66), sm.attention(kv_from=0, heads=10, vdim=66, chunk=11)],
    "delta": [sm.delta()],
    "delta, every head its own": [sm.delta(heads=3, kv_heads=3, dim=8, vdim=88)],
    "delta, one key head": [sm.delta(heads=5, kv_heads=1, dim=72, vdim=30)],
    "delta, one tap": [sm.delta(conv=1)],
    "delta, two taps": [sm.delta(conv=2, dim=64, vdim=64)],
    "delta, nine taps": [sm.delta(conv=9, heads=2, kv_heads=1)],
    "delta, dim 130": [sm.delta(heads=2, kv_heads=2, dim=130, vdim=33)],
    "delta, dim 250": [sm.delta(heads=2, kv_heads=1, dim=250, vdim=260)],
    "delta, dim 256": [sm.delta(heads=1, kv_heads=1, dim=256, vdim=128)],
    "feed-forward": [sm.delta(heads=1, kv_heads=1, dim=8, vdim=8, mlp=sm.clamped())],
    "feed-forward, tight": [sm.attention(mlp=sm.clamped(ff=40, limit=0.1))],
    "feed-forward, loose": [sm.attention(mlp=sm.clamped(ff=200, limit=7.0))],
}


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", MECHANISMS)
def test_each_mechanism_alone(name, dtype):
    """A prompt of 150 tokens at once, then the same one token after the other."""
    cfg = sm.bosirax(*MECHANISMS[name])
    t = sm.random_bosirax(cfg, seed=len(name))
    tokens = tokens_of(cfg, 150)
    want = so.bosirax(cfg, t.plain(), tokens)
    model = load(cfg, t, dtype)
    check(run(model, 1, tokens, [150]), want, dtype, note=name)
    check(run(model, 2, tokens, [1] * 150), want, dtype, note=name + ", decoded")
    model.close()


@pytest.mark.parametrize("pairs,scale", [(None, 1.0), (None, 0.25), ((1, 3, 4), 2.0), ((1009, 1000003, 77), 1.0), ((64, 1, 0), 3.0), ((200, 0, 1), 0.5)])
def test_embedding_of_tokens_and_pairs(pairs, scale):
    cfg = sm.bosirax(sm.attention(heads=1, kv_heads=1, dim=8, vdim=8, rot=0), pairs=pairs, scale=scale)
    t = sm.random_bosirax(cfg, 3)
    tokens = tokens_of(cfg, 60)
    want = so.bosirax(cfg, t.plain(), tokens)
    model = load(cfg, t)
    for slot, cuts in enumerate(([60], [1] * 60, [2] * 30, [7, 1, 1, 20, 31])):
        check(run(model, slot, tokens, cuts), want, "float32", note=f"pairs {pairs} {cuts[:3]}")
    model.close()


WHOLE = sm.bosirax(sm.delta(mlp=sm.clamped()), sm.attention(chunk=70, **FULL, stretch=sm.scaling(), mlp=sm.clamped(limit=2.0)),
                   sm.attention(kv_from=1, chunk=45, heads=8, scale=0.7, **FULL, stretch=sm.scaling()), sm.delta(heads=2, kv_heads=1, dim=72, vdim=100, conv=3),
                   sm.attention(heads=3, kv_heads=1, dim=20, vdim=68, rot=6, mlp=sm.clamped(ff=60)), sm.attention(kv_from=4, heads=3, kv_heads=1, dim=20, vdim=68, rot=6, chunk=128))


@pytest.fixture(scope="module")
def whole():
    t = sm.random_bosirax(WHOLE, 77)
    tokens = tokens_of(WHOLE, 330)
    return t, tokens, so.bosirax(WHOLE, t.plain(), tokens)


@pytest.fixture(scope="module")
def whole_f32(whole):
    model = load(WHOLE, whole[0], slots=6)
    yield model
    model.close()


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_residual_stream_after_every_layer(whole, dtype):
    t, tokens, _ = whole
    layers = []
    so.bosirax(WHOLE, t.plain(), tokens[:150], layers)
    model = load(WHOLE, t, dtype)
    got = model.trace_layers([(0, 0, tokens[:150])])
    for n, want in enumerate(layers):
        check(got[n], want, dtype, note=f"layer {n}")
    model.close()


CUTS = [[330], [2] * 165, [1] * 330, [3] * 110, [16] * 20 + [10], [17] * 19 + [7], [32] * 10 + [10], [63, 2, 65, 64, 136], [70, 70, 70, 70, 50],
        [69, 2, 68, 1, 1, 189], [100, 1, 1, 1, 2, 225], [1, 329], [2, 127, 1, 128, 72]]


@pytest.mark.parametrize("cuts", CUTS, ids=lambda c: "-".join(map(str, c[:5])))
def test_portions_of_a_prompt(whole, whole_f32, cuts):
    _, tokens, want = whole
    assert sum(cuts) == 330
    check(run(whole_f32, 3, tokens, cuts), want, "float32", note=str(cuts[:5]))


@pytest.mark.parametrize("cuts", [[330], [1] * 330, [37] * 8 + [34], [2] * 165])
def test_portions_of_a_prompt_in_bfloat16(whole, cuts):
    t, tokens, want = whole
    model = load(WHOLE, t, "bfloat16")
    check(run(model, 0, tokens, cuts), want, "bfloat16", note=str(cuts[:5]))
    model.close()


def test_first_tokens(whole, whole_f32):
    _, tokens, want = whole
    for n in (1, 2, 3, 4, 5):
        check(run(whole_f32, 0, tokens, [n]), want[:n], "float32", note=f"{n} tokens")


def test_unequal_requests_in_one_step(whole, whole_f32):
    """Portions of different sizes and single tokens of six sequences together, against each alone."""
    plain = whole[0].plain()
    seqs = [tokens_of(WHOLE, n, seed=n) for n in (90, 41, 7, 130, 64, 2)]
    want = [so.bosirax(WHOLE, plain, s) for s in seqs]
    got, at = [[] for _ in seqs], [0] * 6
    takes = [[70, 1, 2, 1, 16], [1, 1, 33, 5, 1], [1, 1, 1, 3, 1], [1, 65, 1, 1, 62], [17, 1, 1, 44, 1], [0, 0, 1, 0, 1]]
    for step in range(5):
        entries, places, rows = [], [], 0
        for b in np.random.default_rng(step).permutation(6):
            n = takes[b][step]
            if n:
                entries.append((int(b), at[b], seqs[b][at[b]:at[b] + n]))
                places.append((b, n))
                at[b] += n
                rows += n
        logits, row = whole_f32.forward(entries, range(rows)), 0
        for b, n in places:
            got[b].append(logits[row:row + n])
            row += n
    for b in range(6):
        assert at[b] == len(seqs[b])
        check(np.concatenate(got[b]), want[b], "float32", note=f"sequence {b}")


def test_a_slot_used_again_starts_afresh(whole, whole_f32):
    _, tokens, want = whole
    other = tokens_of(WHOLE, 200, seed=9)
    run(whole_f32, 2, other, [200])
    check(run(whole_f32, 2, tokens, [40, 1, 1, 30]), want[:72], "float32", note="prompt after another sequence")
    run(whole_f32, 2, other, [1] * 5)
    check(run(whole_f32, 2, tokens, [1] * 20), want[:20], "float32", note="decoding after another sequence")


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_long_sequences_in_a_ring(dtype):
    """The ring holds a chunk and a step: a sequence several times as long, in portions and decoded, in slots used twice."""
    cfg = sm.bosirax(sm.attention(chunk=90, **FULL), sm.attention(kv_from=0, chunk=50, **FULL), sm.attention(chunk=20, heads=2, dim=70, rot=8))
    t = sm.random_bosirax(cfg, 12)
    tokens = tokens_of(cfg, 700)
    want = so.bosirax(cfg, t.plain(), tokens)
    model = load(cfg, t, dtype, slots=2, cap=720, max_rows=39)
    assert model.slot_bytes() < 128 * 2 * (64 + 64 + 128 + 64) * 4 + 720 * 4 + 1
    for slot, cuts in ((0, [39] * 17 + [37]), (1, [1] * 700), (0, [38, 1] * 17 + [37]), (1, [2] * 350)):
        check(run(model, slot, tokens, cuts), want, dtype, note=f"ring {cuts[:3]}")
    model.close()


# ---- keys and writes that stand out ------------------------------------------------------------------

READER, TWIN = 202, 201


def twins(heads, kv_heads, chunk, scale=1.0):
    """Attention whose queries and keys are one map of half of the stream, in which READER and TWIN are alike, and whose
    values come from the other half: READER finds itself and, if the mask lets it, TWIN."""
    cfg = sm.bosirax(sm.attention(heads=heads, kv_heads=kv_heads, dim=32, vdim=32, rot=0, scale=scale, chunk=chunk), pairs=None)
    t = sm.random_bosirax(cfg, 4)
    plain, half = {n: x.astype(np.float32) for n, x in t.plain().items()}, cfg["width"] // 2
    plain["embed"][READER, :half] = plain["embed"][TWIN, :half]
    plain["embed"][TWIN, half:] = plain["embed"][READER, half:][::-1]   # (one length, so the norm treats them alike)
    k, v = 1.5 * plain["l0.mix.k"], 6 * plain["l0.mix.v"]
    k[:, half:], v[:, :half] = 0.0, 0.0
    t.put("embed", plain["embed"])
    t.put("l0.mix.k", k)
    t.put("l0.mix.q", np.repeat(k.reshape(kv_heads, 32, -1), heads // kv_heads, axis=0).reshape(heads * 32, -1))
    t.put("l0.mix.v", v)
    return cfg, t


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("heads,kv_heads", [(2, 2), (4, 1), (40, 2)])
def test_a_single_far_key_stands_out(heads, kv_heads, dtype):
    """At the borders of tiles and stretches, in a prompt and in decoding."""
    cfg, t = twins(heads, kv_heads, None)
    plain = t.plain()
    model = load(cfg, t, dtype)
    base = np.random.default_rng(2).integers(0, 200, 301).tolist()
    unmarked = so.bosirax(cfg, plain, base[:300] + [READER])[-1:]
    for where in (0, 1, 15, 16, 31, 32, 33, 63, 64, 65, 95, 96, 127, 128, 129, 191, 192, 255, 256, 257, 298, 299):
        tokens = base[:300] + [READER]
        tokens[where] = TWIN
        want = so.bosirax(cfg, plain, tokens)[-1:]
        for cuts in ([301], [300, 1], [299, 2], [where + 1, 300 - where]):
            check(run(model, 0, tokens, cuts)[-1:], want, dtype, f32=1e-4, bf16=0.06, note=f"twin at {where}")
        assert sm.row_errors(unmarked, want)[0] > 0.2   # the twin matters
    model.close()


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("chunk", [5, 64, 100, 128])
def test_the_edges_of_a_chunk(chunk, dtype):
    """A twin in the first place of the reader's chunk is seen, one place earlier it is not; the reader being the first, second
    and last of its chunk, in prompts cut around the edge and decoded."""
    cfg, t = twins(4, 2, chunk)
    plain = t.plain()
    model = load(cfg, t, dtype, cap=512, max_rows=400)
    edge = -(-140 // chunk) * chunk
    base = np.random.default_rng(6).integers(0, 200, edge + chunk).tolist()
    for reader in sorted({edge, edge + 1, edge + chunk - 1}):
        seen = {}
        for where in (edge - 1, edge):
            if where >= reader:
                continue
            tokens = base[:reader] + [READER]
            tokens[where] = TWIN
            want = seen[where] = so.bosirax(cfg, plain, tokens)[-1:]
            for cuts in ([reader + 1], [reader, 1], [edge - 1, reader + 2 - edge], [edge, reader + 1 - edge], [reader - 1, 2]):
                check(run(model, 1, tokens, [c for c in cuts if c])[-1:], want, dtype, f32=1e-4, bf16=0.06, note=f"chunk {chunk} reader {reader} twin {where}")
        if len(seen) == 2 and reader > edge:
            assert sm.row_errors(seen[edge - 1], seen[edge])[0] > 0.2
    model.close()


@pytest.mark.parametrize("a_log,dt_bias,gates", [(-8.0, -4.0, 0.1), (2.0, 4.0, 1.0), (0.0, 0.0, 8.0), (-3.0, -8.0, 6.0), (4.0, -3.0, 5.0)])
def test_delta_rule_with_extreme_gates(a_log, dt_bias, gates):
    """Nothing forgotten, all forgotten at once, writes that are whole or not at all, over many chunks."""
    cfg = sm.bosirax(sm.delta(), sm.delta(heads=2, kv_heads=1, dim=16, vdim=16))
    t = sm.random_bosirax(cfg, 8, a_log=a_log, dt_bias=dt_bias, gates=gates)
    tokens = tokens_of(cfg, 300)
    want = so.bosirax(cfg, t.plain(), tokens)
    model = load(cfg, t)
    for cuts in ([300], [1] * 300, [2, 64, 62, 1, 1, 33, 137]):
        check(run(model, 0, tokens, cuts), want, "float32", f32=5e-5, note=f"gates {a_log} {dt_bias} {gates} {cuts[:3]}")
    model.close()


def test_delta_rule_with_keys_that_repeat():
    """Few tokens, so the same keys are rewritten again and again within a chunk: the triangular system at its stiffest."""
    cfg = sm.bosirax(sm.delta(conv=1, heads=2, kv_heads=2, dim=16, vdim=40), vocab=5, pairs=None)
    t = sm.random_bosirax(cfg, 5, a_log=-6.0, gates=1.0)
    t.put("l0.mix.b", 40 * np.abs(sequence.bf16_to_f32(t.bits["l0.mix.b"])))
    tokens = tokens_of(cfg, 260)
    want = so.bosirax(cfg, t.plain(), tokens)
    model = load(cfg, t)
    for cuts in ([260], [1] * 260, [100, 160]):
        check(run(model, 0, tokens, cuts), want, "float32", f32=5e-5, note=f"repeats {cuts[:3]}")
    model.close()


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_delta_rule_keeps_an_early_token_for_long(dtype):
    """One token is written whole, the others hardly, nothing is forgotten: its value must still be read 400 tokens later."""
    cfg = sm.bosirax(sm.delta(heads=1, kv_heads=1, dim=32, vdim=32, conv=1), width=64, scale=1.0, pairs=None)
    t = sm.random_bosirax(cfg, 2)
    embed = sequence.bf16_to_f32(t.bits["embed"]).copy()
    embed[:, 0] = -8.0                     # one direction of the stream opens the gate, for the marker only
    embed[7, 0] = 8.0
    t.put("embed", embed)
    write = np.zeros((1, 64))
    write[0, 0], write[0, 1:] = 4.0, 0.0
    t.put("l0.mix.b", write)
    t.put("l0.mix.a", np.zeros((1, 64)))
    t.put("l0.mix.A_log", np.array([-9.0]))
    t.put("l0.mix.dt_bias", np.array([-9.0]))
    plain = t.plain()
    tokens = [8 if x == 7 else x for x in tokens_of(cfg, 420)]
    model = load(cfg, t, dtype)
    other = so.bosirax(cfg, plain, tokens)
    for where in (0, 1, 63, 64, 100):
        marked = tokens[:where] + [7] + tokens[where + 1:]
        want = so.bosirax(cfg, plain, marked)
        assert sm.row_errors(other[-1:], want[-1:])[0] > 0.05
        for cuts in ([420], [200] + [1] * 220, [50, 2, 65, 303]):
            # (before the marker there is nothing to read but what a closed gate lets through)
            check(run(model, 0, marked, cuts)[where:], want[where:], dtype, f32=5e-5, bf16=0.04, note=f"marker at {where}")
    model.close()


def test_the_convolution_over_portions():
    """One channel carries a token's mark; every cut falls once on every place of the taps behind it."""
    cfg = sm.bosirax(sm.delta(heads=1, kv_heads=1, dim=8, vdim=8, conv=5), pairs=None)
    t = sm.random_bosirax(cfg, 9)
    for name in ("q", "k", "v"):
        t.put(f"l0.mix.{name}.conv", 3 * sequence.bf16_to_f32(t.bits[f"l0.mix.{name}.conv"]))
    tokens = tokens_of(cfg, 40)
    want = so.bosirax(cfg, t.plain(), tokens)
    model = load(cfg, t)
    for first in range(1, 12):
        for second in (1, 2, 3, 4, 5, 6):
            check(run(model, 0, tokens, [first, second, 1, 40 - first - second - 1]), want, "float32", note=f"{first} {second}")
    model.close()


# ---- the engine -----------------------------------------------------------------------------------------

def test_generation_through_the_scheduler(whole, whole_f32):
    """More requests than slots, portions mixed with decoding, bursts on the device: the tokens of a plain loop."""
    t, _, _ = whole
    prompts = [tokens_of(WHOLE, n, seed=50 + n) for n in (5, 1, 60, 33, 2, 90, 17, 8)]
    got = Engine(whole_f32, portion=24, burst=16).generate(prompts, 40)
    for prompt, output in zip(prompts, got):
        assert len(output) == 40
        logits = so.bosirax(WHOLE, t.plain(), prompt + output)[len(prompt) - 1:-1]
        top = np.sort(logits, axis=1)
        close = top[:, -1] - top[:, -2] < 1e-3
        assert all(c or o == b for c, o, b in zip(close, output, logits.argmax(axis=1)))


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_replayed_decoding_equals_single_steps(whole, dtype):
    """Bursts (HIP graphs replayed, with eager work and host reads in between) against one step at a time."""
    t, tokens, _ = whole
    model = load(WHOLE, t, dtype, cap=600)
    twins_ = []
    for slot, n in ((0, 20), (2, 250), (3, 77)):
        first = ids = int(model.forward([(slot, 0, tokens[:n])], [n - 1], best=True)[0])
        model.forward([(1, 0, tokens[:n])])          # a twin of each, decoded one by one
        seq = []
        for pos in range(n, n + 60):
            ids = int(model.forward([(1, pos, [ids])], [0], best=True)[0])
            seq.append(ids)
        twins_.append((first, seq))
    pos, ids, out = np.array([20, 250, 77]), [f for f, _ in twins_], []
    for steps in (1, 7, 2, 30, 20):
        got = model.decode([0, 2, 3], pos, ids, steps)
        out.append(got)
        pos, ids = pos + steps, got[-1]
        model.forward([(1, 0, tokens[:9])], [8])     # eager work between replays
    out = np.concatenate(out)
    for b, (_, seq) in enumerate(twins_):
        same = np.mean(out[:, b] == np.array(seq))
        # greedy paths part for good at the first near-tie, which rounding may decide either way
        assert same == 1.0 or (dtype == "bfloat16" and out[:5, b].tolist() == seq[:5]), (b, same)
    model.close()


def test_pieces_agree_at_full_width():
    """Sizes at which the wide tiles of the linear layers and split positions run, with rows that do not fill them."""
    cfg = sm.bosirax(sm.attention(heads=16, kv_heads=4, dim=64, vdim=128, rot=64, scale=0.125, chunk=900, mlp=sm.clamped(ff=2500)),
                     sm.delta(heads=8, kv_heads=4, dim=128, vdim=192, mlp=sm.clamped(ff=500)), width=1000, vocab=3000)
    t = sm.random_bosirax(cfg, 6)
    tokens = tokens_of(cfg, 1500)
    model = load(cfg, t, "float32", slots=2, cap=1600, max_rows=1600)
    whole_ = run(model, 0, tokens, [1500])
    check(run(model, 1, tokens, [700, 1, 500, 16, 3, 250, 30]), whole_, "float32", note="pieces against the whole")
    check(whole_[:40], so.bosirax(cfg, t.plain(), tokens[:40]), "float32", note="whole against the plain implementation")
    model.close()
    model = load(cfg, t, "bfloat16", slots=2, cap=1600, max_rows=1600)
    check(run(model, 0, tokens, [1500]), whole_, "bfloat16", note="bfloat16 against 32-bit")
    model.close()


def test_a_model_with_latent_attention_and_memory_in_parallel_layers():
    """Parallel layers are not a matter of one family: the other mixers serve them too."""
    from llaminar_amd.models import kogilix

    cfg = sm.config(sm.latent(mlp=sm.dense()), sm.mlstm(mlp=sm.dense(ff=72)))
    t = sm.random_weights(cfg, 21)
    plain, tokens = t.plain(), tokens_of(cfg, 100)
    w = kogilix.weights(cfg, t)

    def parallel(make):
        def layer():
            out = make()
            out.parallel = True
            return out
        return layer
    w.layers = [parallel(make) for make in w.layers]
    x, eps = plain["embed"][tokens], cfg["norm"]["eps"]
    for n, layer in enumerate(cfg["layers"]):
        p = {k[len(f"l{n}."):]: v for k, v in plain.items() if k.startswith(f"l{n}.")}
        m, h = layer["mixer"], so.rms_norm(x, p["norm1"], eps)
        if layer["type"] == "latent_attention":
            y = so.latent_attention(h, so.latent_rows(h, p, eps), p, m["heads"], m["dim"], m["vdim"], m["scale"], eps)
        else:
            y = so.mlstm(h, p, m["heads"], m["dim"], m["vdim"], m["gate_cap"], eps)
        x = x + y + so.gated_ffn(so.rms_norm(x, p["norm2"], eps), p)
    want = so.rms_norm(x, plain["final.norm"], eps) @ plain["head"].T
    model = sequence.SequenceModel(w, 2, 128, 128, "float32")
    check(run(model, 0, tokens, [100]), want, "float32", note="parallel")
    check(run(model, 1, tokens, [1] * 100), want, "float32", note="parallel, decoded")
    model.close()


def test_programs_run_a_model_from_its_folder(tmp_path, whole):
    """bin/trace_run and the command line, as programs of their own."""
    t, tokens, want = whole
    (tmp_path / "config.json").write_text(json.dumps(WHOLE))
    safetensors_io.write(tmp_path / "model.safetensors", t.bits)
    out = tmp_path / "out"
    steps = [{"step": 0, "entries": [{"id": "a", "tokens": tokens[:50], "want": [0, 49]}], "end": []},
             {"step": 1, "entries": [{"id": "a", "tokens": tokens[50:52], "want": [1]}, {"id": "b", "tokens": tokens[:1], "want": [0]}], "end": ["a"]},
             {"step": 2, "entries": [{"id": "b", "tokens": tokens[1:3], "want": []}], "end": ["b"]}]
    p = subprocess.run([str(ROOT / "bin" / "trace_run"), "--model", str(tmp_path), "--dtype", "float32", "--out", str(out),
                        "--max-tokens", "64"], input="\n".join(map(json.dumps, steps)) + "\n", text=True, capture_output=True, timeout=100)
    assert p.returncode == 0, p.stderr
    assert [x for x in p.stdout.splitlines() if x.startswith("done")] == ["done 0", "done 1", "done 2"]
    assert sorted(x.name for x in out.iterdir()) == ["0.f32", "1.f32"]
    check(np.fromfile(out / "0.f32", "<f4").reshape(2, -1), want[[0, 49]], "float32")
    check(np.fromfile(out / "1.f32", "<f4").reshape(2, -1), want[[51, 0]], "float32")
    p = subprocess.run([sys.executable, "-m", "llaminar_amd", "generate", "--model", str(tmp_path), "--dtype", "float32",
                        "--prompt", ",".join(map(str, tokens[:10])), "--max-new", "4"], cwd=ROOT, text=True, capture_output=True,
                       timeout=100, env=dict(os.environ, PYTHONPATH=str(ROOT)))
    assert p.returncode == 0, p.stderr
    output = [int(x) for x in p.stdout.strip().split(",")]
    logits = so.bosirax(WHOLE, t.plain(), tokens[:10] + output)[9:-1]
    assert output == logits.argmax(axis=1).tolist()
