"""Replays a trace of token ids through a served model, step by step, and writes logits.

Standard input has one JSON object a line:

    {"step": 0, "entries": [{"id": "a", "tokens": [5, 17, 3], "want": [0, 2]}], "end": []}

`entries` are the next tokens of requests and the places among them whose logits are wanted; `end` lists
requests that are over after the step.  A step in which something is wanted leaves OUT/<step>.f32: float32
rows [wanted, vocabulary] in the order of the entries.  Every step is answered with a line `done <step>`.
"""
from __future__ import annotations

import json
import os
import sys

import numpy as np


def replay(model, lines, out_directory: str, answer) -> None:
    live = {}
    for line in lines:
        if not line.strip():
            continue
        step = json.loads(line)
        rows = []
        for entry in step["entries"]:
            if entry["id"] not in live:
                live[entry["id"]] = model.open()
            logits = model.step(live[entry["id"]], entry["tokens"], entry["want"])
            if len(entry["want"]):
                rows.append(logits)
        for name in step["end"]:
            model.close(live.pop(name))
        if rows:
            path = os.path.join(out_directory, f"{step['step']}.f32")
            np.concatenate(rows).astype("<f4").tofile(path)
        answer(f"done {step['step']}")


def answer_on_stdout(text: str) -> None:
    sys.stdout.write(text + "\n")
    sys.stdout.flush()
