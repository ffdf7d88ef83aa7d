"""Replays recorded traffic through a model's session and writes the logits asked for.

Every input line is a JSON object: ``step`` (a number), ``entries`` (each the ``id`` of a sequence, its next
``tokens``, and ``want``, indices into them) and ``end`` (ids of sequences that are over).  The wanted rows of a step
go to OUT/<step>.f32 as little-endian f32, in order, and "done <step>" follows on standard output.  A sequence keeps
its cache and state from step to step until `end` names it; the session holds one, so the next begins after that.
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
