"""The dense quantized family behind the engine: llaminar_amd.decoder's step driver as a runner.

config.json: {"architecture": "DenseQ4K", and any of decoder.Shape's fields, "seed"}.  The weights are
random (seeded), as everywhere that driver is used.  Its step takes one token of every slot, so a portion
of a prompt runs token by token; slots an entry does not name repeat their newest position, where the
next real token of that slot overwrites what the step leaves.
"""
from __future__ import annotations

from dataclasses import fields
from pathlib import Path

import numpy as np

from . import ConfigError, register


class DenseRunner:
    max_rows = 1 << 30

    def __init__(self, shape, slots: int, cap: int, device_id: int, seed: int):
        import torch

        from .. import decoder

        self.torch = torch
        cap = -(-(cap + 1) // 32) * 32   # one position more: where idle slots of a full length write
        self.slots, self.cap, self.vocab = slots, cap - 1, shape.vocab
        self.dec = decoder.DenseDecoder(shape, slots, cap, torch.device("cuda", device_id), seed=seed)
        self.pos = np.zeros(slots, np.int32)

    def _tick(self, tokens: dict[int, tuple[int, int]]):
        """One token of some slots: slot -> (position, token)."""
        ids, pos = np.zeros(self.slots, np.int32), self.pos.copy()
        for slot, (p, t) in tokens.items():
            pos[slot], ids[slot] = p, t
            self.pos[slot] = p + 1
        self.dec.set_state(ids, pos)
        self.dec.step()

    def forward(self, entries, want=(), best: bool = False):
        rows, row = {}, 0
        for slot, _, ids in entries:
            for k in range(len(ids)):
                rows[row + k] = (slot, k)
            row += len(ids)
        logits = np.empty((len(want), self.vocab), np.float32)
        for k in range(max(len(e[2]) for e in entries)):
            self._tick({slot: (pos + k, ids[k]) for slot, pos, ids in entries if k < len(ids)})
            wanted = [(j, rows[w][0]) for j, w in enumerate(want) if rows[w][1] == k]
            if wanted:
                self.torch.cuda.synchronize()
                got = self.dec.buffer("logits").cpu().numpy()
                for j, slot in wanted:
                    logits[j] = got[slot]
        return logits.argmax(axis=1).astype(np.int32) if best else logits

    def decode(self, slots, pos, ids, steps: int) -> np.ndarray:
        out = np.empty((steps, len(slots)), np.int32)
        ids = list(ids)
        for s in range(steps):
            self._tick({slot: (p + s, t) for slot, p, t in zip(slots, pos, ids)})
            self.torch.cuda.synchronize()
            chosen = self.dec.buffer("ids").cpu().numpy()
            ids = [int(chosen[slot]) for slot in slots]
            out[s] = ids
        return out

    def max_decode_steps(self, n: int) -> int:
        return self.cap

    def close(self):
        self.dec.close()


@register("DenseQ4K")
def load(config: dict, model_dir: Path, slots: int = 8, cap: int = 4096, max_rows: int = 0, dtype: str = "bfloat16",
         device_id: int = 0) -> DenseRunner:
    from .. import decoder

    if dtype != "bfloat16":
        raise ConfigError("the quantized dense family has one number format")
    if not 1 <= slots <= 8:
        raise ConfigError(f"{slots} slots: the dense step driver takes 1 to 8 sequences")
    shape = decoder.Shape(**{f.name: config[f.name] for f in fields(decoder.Shape) if f.name in config})
    return DenseRunner(shape, slots, cap, device_id, int(config.get("seed", 0)))
