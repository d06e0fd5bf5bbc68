"""Serving loop: sequences in slots, and a scheduler that mixes portions of prompts with decoding.

``Engine`` owns the runner of a model (llaminar_amd.models).  Below it is the state of the live
sequences (slot, length); above it two ways to drive a step:

  feed / release   given tokens of chosen sequences, logits where asked for (scoring, replaying traces)
  submit / step    requests that are generated greedily: every step takes one token of each decoding
                   sequence and, with what is left of ``max_rows``, portions of waiting prompts; while
                   no prompt waits, decoding runs in bursts on the device
"""
from __future__ import annotations

from collections import deque
from dataclasses import dataclass, field


class CapacityError(RuntimeError):
    """No slot is free, or a sequence is longer than a slot."""


@dataclass
class Sequence:
    slot: int
    length: int = 0   # tokens in the cache or state


class Sequences:
    """Live sequences and the slots of a runner they occupy."""

    def __init__(self, slots: int, cap: int):
        self.cap = cap
        self._free = list(range(slots - 1, -1, -1))
        self._live: dict = {}

    def __contains__(self, name) -> bool:
        return name in self._live

    def __len__(self) -> int:
        return len(self._live)

    def free(self) -> int:
        return len(self._free)

    def get(self, name) -> Sequence:
        return self._live[name]

    def open(self, name) -> Sequence:
        if not self._free:
            raise CapacityError(f"no free slot for sequence {name!r} ({len(self._live)} are live)")
        self._live[name] = Sequence(self._free.pop())
        return self._live[name]

    def close(self, name):
        self._free.append(self._live.pop(name).slot)


@dataclass
class Request:
    name: object
    prompt: list
    max_new: int
    stop: frozenset = frozenset()
    output: list = field(default_factory=list)
    fed: int = 0   # tokens of the prompt that have run

    def finished(self) -> bool:
        return len(self.output) >= self.max_new or bool(self.output and self.output[-1] in self.stop)


class Engine:
    def __init__(self, runner, portion: int = 512, burst: int = 64):
        self.runner = runner
        self.portion = max(1, min(portion, runner.max_rows))
        self.burst = burst
        self.sequences = Sequences(runner.slots, runner.cap)
        self._waiting: deque[Request] = deque()
        self._running: list[Request] = []

    # ---- given tokens
    def feed(self, entries, best: bool = False):
        """Run the next tokens of some sequences: (name, tokens, places among them that are wanted).  A new name
        opens a sequence.  Returns one array per entry: logits [wanted, vocab], or the best tokens.  Longer
        than max_rows in all, the tokens run in several steps."""
        for name, tokens, want in entries:
            seq = self.sequences.get(name) if name in self.sequences else self.sequences.open(name)
            if seq.length + len(tokens) > self.runner.cap:
                raise CapacityError(f"sequence {name!r}: {seq.length + len(tokens)} tokens, a slot holds {self.runner.cap}")
        results = [[] for _ in entries]
        todo = [(n, 0) for n, e in enumerate(entries) if e[1]]
        while todo:
            batch, want, owner, row, rest = [], [], [], 0, []
            for n, at in todo:
                name, tokens, wanted = entries[n]
                take = min(len(tokens) - at, self.runner.max_rows - row)
                if take > 0:
                    seq = self.sequences.get(name)
                    batch.append((seq.slot, seq.length, tokens[at:at + take]))
                    here = [k for k in wanted if at <= k < at + take]
                    want += [row + k - at for k in here]
                    owner += [(n, k) for k in here]
                    seq.length += take
                    row += take
                if at + take < len(tokens):
                    rest.append((n, at + take))
            got = self.runner.forward(batch, want, best)
            for (n, k), row_result in zip(owner, got):
                results[n].append((k, row_result))
            todo = rest
        out = []
        for (_, _, wanted), rows in zip(entries, results):
            by_place = dict(rows)
            out.append([by_place[k] for k in wanted])
        return out

    def release(self, name):
        """A sequence is finished: its slot is free again."""
        self.sequences.close(name)

    # ---- requests
    def submit(self, name, prompt, max_new: int, stop=()):
        prompt = [int(t) for t in prompt]
        if not prompt or max_new < 1:
            raise ValueError("a request needs a prompt and at least one token to generate")
        bad = [t for t in prompt if not 0 <= t < self.runner.vocab]
        if bad:
            raise ValueError(f"token {bad[0]} is outside the vocabulary of {self.runner.vocab}")
        if len(prompt) + max_new - 1 > self.runner.cap:
            raise CapacityError(f"request {name!r}: {len(prompt)} + {max_new} tokens, a slot holds {self.runner.cap}")
        if name in self.sequences or any(r.name == name for r in self._waiting):
            raise ValueError(f"request {name!r} is already there")
        self._waiting.append(Request(name, prompt, max_new, frozenset(stop)))

    def pending(self) -> bool:
        return bool(self._waiting or self._running)

    def step(self) -> list[Request]:
        """One turn of the scheduler; returns the requests that finished in it."""
        while self._waiting and self.sequences.free():
            request = self._waiting.popleft()
            self.sequences.open(request.name)
            self._running.append(request)
        decoding = [r for r in self._running if r.output]
        prompts = [r for r in self._running if not r.output]
        if decoding and not prompts:
            self._burst(decoding)
        else:
            entries, owners, room = [], [], self.runner.max_rows
            for r in decoding[:room]:
                entries.append((r.name, [r.output[-1]], [0]))
                owners.append(r)
            room -= len(entries)
            for r in prompts:
                take = min(self.portion, room, len(r.prompt) - r.fed)
                if take < 1:
                    break
                last = r.fed + take == len(r.prompt)
                entries.append((r.name, r.prompt[r.fed:r.fed + take], [take - 1] if last else []))
                owners.append(r)
                r.fed += take
                room -= take
            for r, chosen in zip(owners, self.feed(entries, best=True)):
                if chosen:
                    r.output.append(int(chosen[0]))
        return self._retire()

    def _burst(self, decoding: list[Request]):
        seqs = [self.sequences.get(r.name) for r in decoding]
        left = min(r.max_new - len(r.output) for r in decoding)
        steps = max(1, min(self.burst, left, self.runner.max_decode_steps(len(decoding))))
        out = self.runner.decode([s.slot for s in seqs], [s.length for s in seqs], [r.output[-1] for r in decoding], steps)
        for b, (r, s) in enumerate(zip(decoding, seqs)):
            s.length += steps
            for t in out[:, b]:
                r.output.append(int(t))
                if r.finished():
                    break   # what the burst added after a stop token is dropped with the sequence

    def _retire(self) -> list[Request]:
        done = [r for r in self._running if r.finished()]
        for r in done:
            self._running.remove(r)
            self.release(r.name)
        return done

    def generate(self, prompts, max_new: int, stop=()) -> list[list[int]]:
        """Greedy continuations of several prompts, in their order."""
        names = [("generate", n) for n in range(len(prompts))]
        for name, prompt in zip(names, prompts):
            self.submit(name, prompt, max_new, stop)
        done = {}
        while self.pending():
            for r in self.step():
                done[r.name] = r.output
        return [done[n] for n in names]
