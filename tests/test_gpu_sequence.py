"""Sequence models on the GPU against the plain implementation (oracle/sequence_oracle.py): each mechanism alone,
prompts, portions, decoding, mixed batches, slots used again, and generation through the engine."""
import json
import os
import subprocess
import sys
from pathlib import Path

import numpy as np
import pytest

from llaminar_amd import safetensors_io, sequence
from llaminar_amd.engine import Engine
from llaminar_amd.models import kogilix
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
    return sequence.SequenceModel(kogilix.weights(cfg, tensors), slots, cap, max_rows, dtype)


MECHANISMS = {
    "latent": [sm.latent()],
    "latent sharp": [sm.latent(scale=2.0)],
    "latent one head": [sm.latent(heads=1, dim=8, vdim=72, q_rank=130, kv_rank=24)],
    "latent 20 heads": [sm.latent(heads=20, dim=12, vdim=4, q_rank=64, kv_rank=64)],
    "latent rank 200": [sm.latent(heads=18, kv_rank=200)],
    "latent rank 330": [sm.latent(kv_rank=330)],
    "latent rank 512": [sm.latent(heads=4, kv_rank=512)],
    "latent rank 150": [sm.latent(heads=9, kv_rank=150)],
    "latent rank 600": [sm.latent(heads=5, kv_rank=600)],
    "latent shared": [sm.latent(), sm.latent(kv_from=0, heads=7, dim=20, vdim=70, q_rank=90, scale=0.7)],
    "mlstm": [sm.mlstm()],
    "mlstm one head": [sm.mlstm(heads=1, dim=16, vdim=88, gate_cap=2.5)],
    "mlstm dim 130": [sm.mlstm(heads=2, dim=130, vdim=33)],
    "mlstm dim 300": [sm.mlstm(heads=2, dim=300, vdim=150, gate_cap=15.0)],
    "mlstm dim 256": [sm.mlstm(heads=1, dim=256, vdim=64, gate_cap=30.0)],
    "mlstm dim 512": [sm.mlstm(heads=1, dim=500, vdim=96)],
    "dense": [sm.mlstm(heads=1, dim=8, vdim=8, mlp=sm.dense())],
    "experts": [sm.mlstm(heads=1, dim=8, vdim=8, mlp=sm.moe())],
    "experts shared": [sm.latent(mlp=sm.moe(ff=40, experts=12, top=5, shared=136))],
    "one expert": [sm.mlstm(heads=1, dim=8, vdim=8, mlp=sm.moe(experts=1, top=1, shared=24))],
    "experts 100": [sm.mlstm(heads=1, dim=8, vdim=8, mlp=sm.moe(ff=16, experts=100, top=9))],
}


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", MECHANISMS)
def test_each_mechanism_alone(name, dtype):
    """A prompt of 150 tokens at once, then the same one token after the other."""
    cfg = sm.config(*MECHANISMS[name])
    t = sm.random_weights(cfg, seed=len(name))
    tokens = tokens_of(cfg, 150)
    want = so.kogilix(cfg, t.plain(), tokens)
    model = load(cfg, t, dtype)
    sharp = {"f32": 1e-4, "bf16": 0.08} if "sharp" in name else {}
    check(run(model, 1, tokens, [150]), want, dtype, note=name, **sharp)
    check(run(model, 2, tokens, [1] * 150), want, dtype, note=name + ", decoded", **sharp)
    model.close()


WHOLE = sm.config(sm.mlstm(mlp=sm.dense()), sm.latent(mlp=sm.moe(shared=48)), sm.mlstm(heads=2, dim=72, vdim=100),
                  sm.latent(kv_from=1, heads=5, dim=16, vdim=24, mlp=None), sm.latent(heads=4, kv_rank=64, mlp=sm.moe(experts=9, top=3)),
                  sm.mlstm(heads=4, dim=24, vdim=64, gate_cap=5.0, mlp=sm.moe(top=1)))


@pytest.fixture(scope="module")
def whole():
    t = sm.random_weights(WHOLE, 77)
    tokens = tokens_of(WHOLE, 330)
    return t, tokens, so.kogilix(WHOLE, t.plain(), tokens)


@pytest.fixture(scope="module")
def whole_f32(whole):
    model = load(WHOLE, whole[0], slots=6)
    yield model
    model.close()


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_residual_stream_after_every_layer(whole, dtype):
    t, tokens, _ = whole
    layers = []
    so.kogilix(WHOLE, t.plain(), tokens[:70], layers)
    model = load(WHOLE, t, dtype)
    got = model.trace_layers([(0, 0, tokens[:70])])
    for n, want in enumerate(layers):
        check(got[n], want, dtype, note=f"layer {n}")
    model.close()


@pytest.mark.parametrize("cuts", [[330], [2] * 165, [1] * 330, [3] * 110, [16] * 20 + [10], [17] * 19 + [7], [31] * 10 + [20],
                                  [32] * 10 + [10], [33] * 10, [63, 2, 65, 64, 136], [100, 1, 1, 1, 2, 225], [1, 329], [2, 127, 1, 128, 72]],
                         ids=lambda c: "-".join(map(str, c[:5])))
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
    for n in (1, 2, 3):
        check(run(whole_f32, 0, tokens, [n]), want[:n], "float32", note=f"{n} tokens")


def test_unequal_requests_in_one_step(whole, whole_f32):
    """Portions of different sizes and single tokens of six sequences together, against each alone."""
    t, _, _ = whole
    plain = t.plain()
    seqs = [tokens_of(WHOLE, n, seed=n) for n in (90, 41, 7, 130, 64, 2)]
    want = [so.kogilix(WHOLE, plain, s) for s in seqs]
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
    t, tokens, want = whole
    other = tokens_of(WHOLE, 200, seed=9)
    run(whole_f32, 2, other, [200])
    check(run(whole_f32, 2, tokens, [40, 1, 1, 30]), want[:72], "float32", note="prompt after another sequence")
    run(whole_f32, 2, other, [1] * 5)
    check(run(whole_f32, 2, tokens, [1] * 20), want[:20], "float32", note="decoding after another sequence")


MARKED = [0, 1, 15, 16, 30, 31, 32, 33, 62, 63, 64, 65, 95, 96, 126, 127, 128, 129, 255, 256, 257, 299]


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("heads", [2, 24, 40])
def test_a_single_far_key_stands_out(heads, dtype):
    """Queries and keys are the same map of the latent, so the last token finds its only twin among 300 tokens, wherever
    that lies: at the borders of the attention's tiles and stretches, in a prompt and in decoding."""
    cfg = sm.config(sm.latent(heads=heads, dim=32, vdim=32, q_rank=64, kv_rank=64, scale=1.5))
    t = sm.random_weights(cfg, 4)
    for a, b in (("dkv", "dq"), ("dkv.norm", "dq.norm"), ("uk", "uq")):
        t.bits["l0.mix." + a] = t.bits["l0.mix." + b]
    plain = t.plain()
    t.bits["l0.mix.uv"] = sequence.bf16_bits(4 * plain["l0.mix.uv"])
    plain = t.plain()
    model = load(cfg, t, dtype)
    rng = np.random.default_rng(2)
    base = rng.integers(0, 200, 301).tolist()
    unmarked = so.kogilix(cfg, plain, base[:300] + [202])[-1:]
    for where in MARKED:
        tokens = list(base[:300])
        tokens[where] = 202
        tokens.append(202)
        want = so.kogilix(cfg, plain, tokens)[-1:]
        for cuts in ([301], [300, 1], [299, 2]):
            got = run(model, 0, tokens, cuts)[-1:]
            check(got, want, dtype, f32=1e-4, bf16=0.06, note=f"twin at {where}")
    assert sm.row_errors(unmarked, want)[0] > 0.2 or where == 299   # the twin matters
    model.close()


@pytest.mark.parametrize("forget,inp", [(8.0, -4.0), (-6.0, 2.0), (0.0, 8.0), (8.0, 8.0)])
def test_memory_with_extreme_gates(forget, inp):
    """Long memory, quick forgetting, dominating inputs: the running maximum and its decay over many chunks."""
    cfg = sm.config(sm.mlstm(gate_cap=12.0), sm.mlstm(heads=2, dim=16, vdim=16, gate_cap=12.0))
    t = sm.random_weights(cfg, 8, forget_bias=forget, input_bias=inp)
    tokens = tokens_of(cfg, 300)
    want = so.kogilix(cfg, t.plain(), tokens)
    model = load(cfg, t)
    for cuts in ([300], [1] * 300, [2, 64, 62, 1, 1, 33, 137]):
        check(run(model, 0, tokens, cuts), want, "float32", f32=5e-5, note=f"gates {forget} {inp} {cuts[:3]}")
    model.close()


def test_memory_keeps_an_early_token_for_long():
    """One token opens the input gate wide, none forgets: its value must still be read 400 tokens later."""
    cfg = sm.config(sm.mlstm(heads=1, dim=32, vdim=32, gate_cap=20.0), width=64)
    t = sm.random_weights(cfg, 2)
    embed = sequence.bf16_to_f32(t.bits["embed"]).copy()
    embed[:, 0] = 0.0
    embed[7, 0] = 8.0                      # the marker's own direction opens the gate
    t.put("embed", embed)
    gate = np.zeros((1, 64))
    gate[0, 0] = 4.0
    t.put("l0.mix.i", gate)
    t.put("l0.mix.i.b", np.array([-6.0]))
    t.put("l0.mix.f", np.zeros((1, 64)))
    t.put("l0.mix.f.b", np.array([18.0]))
    tokens = [t_ if t_ != 7 else 8 for t_ in tokens_of(cfg, 420)]
    without = so.kogilix(cfg, t.plain(), tokens)
    model = load(cfg, t)
    for where in (0, 1, 31, 32, 63, 64, 100):
        marked = tokens[:where] + [7] + tokens[where + 1:]
        want = so.kogilix(cfg, t.plain(), marked)
        assert sm.row_errors(without[-1:], want[-1:])[0] > 0.1
        for cuts in ([420], [200] + [1] * 220, [50, 2, 65, 303]):
            check(run(model, 0, marked, cuts), want, "float32", f32=5e-5, note=f"marker at {where}")
    model.close()


def test_generation_through_the_scheduler(whole, whole_f32):
    """More requests than slots, portions mixed with decoding, bursts on the device: the tokens of a plain loop."""
    t, _, _ = whole
    prompts = [tokens_of(WHOLE, n, seed=50 + n) for n in (5, 1, 60, 33, 2, 90, 17, 8)]
    got = Engine(whole_f32, portion=24, burst=16).generate(prompts, 40)
    for prompt, output in zip(prompts, got):
        assert len(output) == 40
        logits = so.kogilix(WHOLE, t.plain(), prompt + output)[len(prompt) - 1:-1]
        top = np.sort(logits, axis=1)
        close = top[:, -1] - top[:, -2] < 1e-3
        assert all(c or o == b for c, o, b in zip(close, output, logits.argmax(axis=1)))


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_replayed_decoding_equals_single_steps(whole, dtype):
    """Bursts (HIP graphs replayed, with eager work and host reads in between) against one step at a time."""
    t, tokens, _ = whole
    model = load(WHOLE, t, dtype, cap=600)
    firsts = []
    for slot, n in ((0, 20), (2, 250), (3, 77)):
        firsts.append(int(model.forward([(slot, 0, tokens[:n])], [n - 1], best=True)[0]))
        model.forward([(1, 0, tokens[:n])])          # a twin of each, decoded one by one below
        ids, seq, pos = firsts[-1], [], n
        for _ in range(60):
            ids = int(model.forward([(1, pos, [ids])], [0], best=True)[0])
            seq.append(ids)
            pos += 1
        firsts[-1] = (firsts[-1], seq)
    pos, ids, out = np.array([20, 250, 77]), [f[0] for f in firsts], []
    for steps in (1, 7, 2, 30, 20):
        got = model.decode([0, 2, 3], pos, ids, steps)
        out.append(got)
        pos, ids = pos + steps, got[-1]
        model.forward([(1, 0, tokens[:9])], [8])     # eager work between replays
    out = np.concatenate(out)
    for b, (_, seq) in enumerate(firsts):
        same = np.mean(out[:, b] == np.array(seq))
        # greedy paths part for good at the first near-tie, which rounding may decide either way
        assert same == 1.0 or (dtype == "bfloat16" and out[:5, b].tolist() == seq[:5]), (b, same)
    model.close()


def test_logits_agree_between_row_and_tile_kernels_at_full_width():
    """Sizes at which the wide tiles of the linear layers run, with rows and columns that do not fill them."""
    cfg = sm.config(sm.latent(heads=16, dim=64, vdim=64, q_rank=300, kv_rank=256, mlp=sm.dense(ff=2500)),
                    sm.mlstm(heads=4, dim=128, vdim=192, mlp=sm.moe(ff=320, experts=6, top=2, shared=500)), width=1000, vocab=3000)
    t = sm.random_weights(cfg, 6)
    tokens = tokens_of(cfg, 1500)
    model = load(cfg, t, "float32", slots=2, cap=1600, max_rows=1600)
    whole_ = run(model, 0, tokens, [1500])
    pieces = run(model, 1, tokens, [700, 1, 500, 16, 3, 250, 30])
    check(pieces, whole_, "float32", note="pieces against the whole")
    short = so.kogilix(cfg, t.plain(), tokens[:40])
    check(whole_[:40], short, "float32", note="whole against the plain implementation")
    model.close()
    model = load(cfg, t, "bfloat16", slots=2, cap=1600, max_rows=1600)
    check(run(model, 0, tokens, [1500]), whole_, "bfloat16", note="bfloat16 against 32-bit")
    model.close()


def test_limits_are_reported(whole_f32):
    with pytest.raises(sequence.SequenceError, match="slot 6"):
        whole_f32.forward([(6, 0, [1])])
    with pytest.raises(sequence.SequenceError, match="do not fit"):
        whole_f32.forward([(0, 639, [1, 2])])
    with pytest.raises(sequence.SequenceError, match="twice"):
        whole_f32.forward([(0, 0, [1]), (0, 1, [1])])
    with pytest.raises(sequence.SequenceError, match="at most"):
        whole_f32.forward([(0, 0, [1] * 400), (1, 0, [1] * 300)])
    with pytest.raises(sequence.SequenceError, match="outside the step"):
        whole_f32.forward([(0, 0, [1])], [1])


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
    logits = so.kogilix(WHOLE, t.plain(), tokens[:10] + output)[9:-1]
    assert output == logits.argmax(axis=1).tolist()


def test_the_dense_family_behind_the_same_engine(tmp_path, dev):
    """The quantized dense decoder served by the scheduler: the tokens of its own step driver fed by hand."""
    from llaminar_amd import decoder, models

    (tmp_path / "config.json").write_text(json.dumps({"architecture": "DenseQ4K", "hidden": 512, "n_heads": 4, "n_kv": 2,
                                                      "ffn": 768, "vocab": 1000, "n_layers": 2, "seed": 3}))
    prompts = [[5, 9, 11], [7], [100, 200, 300, 400, 500, 600]]
    runner = models.load_model(tmp_path, slots=2, cap=40)
    got = Engine(runner, portion=2).generate(prompts, 6)
    runner.close()
    for prompt, output in zip(prompts, got):
        dec = decoder.DenseDecoder(decoder.Shape(512, 4, 2, 128, 768, 1000, 2), 2, 64, dev, seed=3)
        want, tokens = [], list(prompt)
        for n in range(len(prompt) + 5):
            dec.set_state([tokens[n], 0], [n, 0])
            dec.step()
            chosen = int(dec.buffer("ids").cpu()[0])
            if n >= len(prompt) - 1:
                want.append(chosen)
                tokens.append(chosen)
        dec.close()
        assert output == want
