"""The W4A16 / Q8-KV transformer (decode_step.py, prefill_step.py) as a served model.

A folder holds config.json - "architecture": "W4A16Transformer" and the fields of `DecodeConfig` - and
weights.llmopt with the tensors `tensor_names` lists.  A sequence owns a slot of the Q8 pool; a prompt's
first portion runs through a `PrefillStep`, everything behind it token by token through the slot's retained
plan (the prefill entries start at position 0).  Activations are fp16, whatever type is asked for, except
that float32 is refused.
"""
from __future__ import annotations

import dataclasses
import os
from typing import Sequence as Tokens

import numpy as np

from .decode_step import DecodeConfig, DecodeStep, u32s
from .native import Prebaked, Runtime
from .prefill_step import PrefillStep
from .sequence_state import Sequence, StatePool
from .weight_archive import WeightArchive

_MATRICES = ("q", "k", "v", "o", "gate", "up", "down")
_NORMS = ("attn_norm", "ffn_norm")


def archive_tensors(weights: dict) -> dict[str, np.ndarray]:
    """A weight dictionary (decode_step.random_weights) under the names of a weights.llmopt archive."""
    out = {"embedding": weights["embedding"], "final_norm": weights["final_norm"],
           "lm_head.weight": weights["lm_head"][0], "lm_head.scale": weights["lm_head"][1]}
    for index, layer in enumerate(weights["layers"]):
        for key in _NORMS:
            out[f"layers.{index}.{key}"] = layer[key]
        for key in _MATRICES:
            out[f"layers.{index}.{key}.weight"], out[f"layers.{index}.{key}.scale"] = layer[key]
    return out


class W4a16Model:
    def __init__(self, runtime: Runtime, config: DecodeConfig, device: dict, slots: int = 8, max_context: int = 32768):
        self.runtime, self.config, self.device = runtime, config, device
        self.vocabulary = config.vocabulary
        self.state = StatePool(runtime, [], slots, max_context, 1)
        self._slot_bytes = max_context * config.token_stride
        self._pool = runtime.create_buffer(slots * self._slot_bytes)
        self._slots_host = np.arange(max_context + 1, dtype=np.uint32)
        self._slots = runtime.buffer_of_bytes(self._slots_host)
        self._steps: dict[int, tuple] = {}
        self._last = runtime.create_buffer(config.vocabulary * 2)

    @staticmethod
    def load(runtime: Runtime, directory: str, config: dict, activations: str = "bfloat16", **options) -> "W4a16Model":
        if activations == "float32":
            raise ValueError("the W4A16 transformer runs in fp16")
        fields = {f.name for f in dataclasses.fields(DecodeConfig)}
        parsed = DecodeConfig(**{key: value for key, value in config.items() if key in fields})
        archive = WeightArchive(runtime, os.path.join(directory, "weights.llmopt"))
        pair = lambda name: archive.w4a16_pair(name + ".weight", name + ".scale")
        device = {"embedding": archive.buffer("embedding"), "final_norm": archive.buffer("final_norm"),
                  "lm_head": pair("lm_head"),
                  "layers": [{**{key: archive.buffer(f"layers.{i}.{key}") for key in _NORMS},
                              **{key: pair(f"layers.{i}.{key}") for key in _MATRICES}} for i in range(parsed.layers)]}
        return W4a16Model(runtime, parsed, device, **options)

    def open(self) -> Sequence:
        return self.state.open()

    def close(self, sequence: Sequence) -> None:
        self.state.close(sequence)

    def _slot_pool(self, slot: int):
        return self._pool.view(slot * self._slot_bytes, self._slot_bytes)

    def _lm_head(self, row, logits, token) -> tuple:
        c = self.config
        return ("llmopt_w4a16_lm_head_argmax_extra_f16", [row, self.device["final_norm"], *self.device["lm_head"], token, logits],
                u32s(1, c.vocabulary, c.hidden) + np.float32(c.epsilon).tobytes(), (256, 1, 1), (256, 1, 1))

    def _decode_plan(self, slot: int) -> tuple:
        """The slot's decode step and its plan, with the logits beside the argmax."""
        if slot not in self._steps:
            step = DecodeStep(self.runtime, self.config, {}, 1, self._slot_pool(slot), self._slots, [0], [0], [0], [0],
                              max_context=self.state.max_context, slots_host=self._slots_host,
                              device_weights=self.device)
            step.dispatches[-1] = self._lm_head(step.work["x"][0], self._last, step.token_ids)
            self._steps[slot] = (step, Prebaked(self.runtime, step.dispatches, step.tokens, step.token_ids))
        return self._steps[slot]

    def decode(self, sequence: Sequence, token: int) -> int:
        self.state.reserve(sequence, 1)
        step, plan = self._decode_plan(sequence.slot)
        step.seek([sequence.position], [sequence.position])
        out = plan.execute(int(token), sequence.position)
        sequence.position += 1
        return out

    def logits_row(self) -> np.ndarray:
        return self._last.numpy(np.float16, (self.vocabulary,)).astype(np.float32)

    def step(self, sequence: Sequence, tokens: Tokens[int], want: Tokens[int] = ()) -> np.ndarray:
        tokens, want = [int(t) for t in tokens], [int(w) for w in want]
        if not tokens or any(not 0 <= t < self.vocabulary for t in tokens) or any(not 0 <= w < len(tokens) for w in want):
            raise ValueError("a step has at least one token, all inside the vocabulary, and wants places among them")
        self.state.reserve(sequence, len(tokens))
        rows = np.zeros((len(want), self.vocabulary), dtype=np.float32)
        if sequence.position == 0 and len(tokens) > 1:
            c = self.config
            prefill = PrefillStep(self.runtime, c, {}, len(tokens), self._slot_pool(sequence.slot), self._slots,
                                  device_weights=self.device)
            prefill.tokens.write(np.asarray(tokens, dtype=np.int64))
            batch = self.runtime.begin_batch()
            prefill.record(batch)
            logits = [self.runtime.create_buffer(self.vocabulary * 2) for _ in want]
            for place, out in zip(want, logits):
                batch.dispatch(*self._lm_head(prefill.work["x"][0].view(place * c.hidden * 2, c.hidden * 2), out,
                                              prefill.token_id))
            batch.commit()
            sequence.position += len(tokens)
            for index, out in enumerate(logits):
                rows[index] = out.numpy(np.float16, (self.vocabulary,))
            return rows
        for place, token in enumerate(tokens):
            self.decode(sequence, token)
            if place in want:
                row = self.logits_row()
                rows[[index for index, w in enumerate(want) if w == place]] = row
        return rows
