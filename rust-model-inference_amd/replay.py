"""Replays a trace: given token ids through a model's session, step by step, the wanted logits to files.

Steps are read as JSON objects, one a line:

    {"step": 0, "entries": [{"id": "a", "tokens": [5, 17, 3], "want": [0, 2]}], "end": ["a"]}

For a step in which something is wanted OUT/<step>.f32 gets the logits of the wanted places, little-endian f32,
[wanted, vocab]; then "done <step>" is printed.  A request keeps its cache and state between steps; `end` gives them
back.  The session holds one sequence, so requests come one after the other.
"""
import json
import os
import sys

import numpy as np

from . import models


class Replay:
    def __init__(self, session, out_dir):
        self.session, self.out_dir, self.live = session, out_dir, None

    def run(self, step):
        logits = []
        for entry in step["entries"]:
            if self.live is None:
                self.session.reset()
                self.live = entry["id"]
            elif self.live != entry["id"]:
                raise ValueError(f"request {entry['id']!r} begins before {self.live!r} has ended")
            logits.append(self.session.step(entry["tokens"], entry.get("want", ())))
        if sum(len(x) for x in logits):
            path = os.path.join(self.out_dir, f"{step['step']}.f32")
            np.concatenate(logits).astype("<f4").tofile(path)
        for name in step.get("end", ()):
            if name == self.live:
                self.live = None


def main(model, dtype, out_dir, max_tokens, lines=sys.stdin, done=sys.stdout):
    session = models.open_session(model, max(int(max_tokens), 1), dtype)
    replay = Replay(session, out_dir)
    for line in lines:
        if not line.strip():
            continue
        step = json.loads(line)
        replay.run(step)
        done.write(f"done {step['step']}\n")
        done.flush()
    session.close()
    return 0
