"""Replays a trace of token ids through a model, step by step, and writes the logits asked for.  Nothing is sampled: the model's step, its slots and its kernels are the ones
that generation uses (runtime.XcdReplicas.run).

Every line of standard input is a step, a JSON object such as
    {"step": 7, "entries": [{"id": "q1", "tokens": [11], "want": [0]}, {"id": "q2", "tokens": [40], "want": []}], "end": ["q1"]}
All entries form one batch.  `want` holds offsets into an entry's tokens: the logits of those rows go to OUT/<step>.f32, fp32 little-endian, one row of vocab floats after the
other in the order the step names them (no file for a step that wants none).  Requests named in `end` leave their slots free.  The answer to a line is `done <step>`.
"""
import json
import os
import sys

import numpy as np


class Trace:
    def __init__(self, model, make_slots):
        self.model, self.make_slots = model, make_slots
        self.slots, self.n_slots, self.live = None, 0, {}   # live: id -> [slot, tokens so far]

    def step(self, entries, end):
        """logits fp32 [wanted, vocab] of one step (None when nothing is wanted)"""
        fresh = [e["id"] for e in entries if e["id"] not in self.live]
        need = len(self.live) + len(fresh)
        if need > self.n_slots:
            if self.live:
                raise ValueError("%d requests live at once: the batch was opened for %d" % (need, self.n_slots))
            if self.slots is not None:
                self.slots.close()
            self.slots, self.n_slots = self.make_slots(self.model, need), need
        for i in fresh:
            self.live[i] = [self.slots.acquire(), 0]
        spans, want = [], []
        for k, e in enumerate(entries):
            slot, at = self.live[e["id"]]
            spans.append((slot, at, e["tokens"]))
            want += [(k, w) for w in e["want"]]
        out = self.slots.run(spans, want)
        for e in entries:
            self.live[e["id"]][1] += len(e["tokens"])
        for i in end:
            self.slots.release(self.live.pop(i)[0])
        return out if want else None


def replay(model, make_slots, out_dir, lines=sys.stdin, say=print):
    t = Trace(model, make_slots)
    for line in lines:
        if not line.strip():
            continue
        s = json.loads(line)
        logits = t.step(s["entries"], s.get("end", []))
        if logits is not None:
            path = os.path.join(out_dir, "%d.f32" % s["step"])
            with open(path + ".part", "wb") as f:
                f.write(np.ascontiguousarray(logits, dtype="<f4").tobytes())
            os.replace(path + ".part", path)
        say("done %d" % s["step"], flush=True)
    if t.slots is not None:
        t.slots.close()
