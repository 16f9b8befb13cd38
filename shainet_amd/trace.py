"""Replays a trace of token ids through a model, step by step, and writes the logits it is asked for.

Steps come as JSON lines on standard input:

    {"step": 4, "entries": [{"id": "chat-7", "tokens": [81, 2, 2, 640], "want": [3]}], "end": ["chat-7"]}

An entry holds a request's next tokens and the places among them whose logits are wanted; "end" lists the
requests that are finished after the step.  OUT/<step>.f32 receives the wanted rows as little-endian
float32 [wanted, vocab] (no file where nothing is wanted); "done <step>" is printed after every step.
A model serves one sequence at a time, so a request has to end before the next one begins."""
import argparse
import json
import os
import sys


class Replay:
    """The model's one sequence, and the request it belongs to."""

    def __init__(self, model):
        self.model, self.active = model, None

    def entry(self, request, tokens, want):
        if self.active is None:
            self.active = request
        elif self.active != request:
            raise ValueError(f"request {request!r} begins before {self.active!r} has ended")
        if not tokens:
            raise ValueError(f"request {request!r} brings no tokens")
        return self.model.run_rows(tokens, want)

    def end(self, request):
        if request == self.active:
            self.model.clear_cache()
            self.active = None


def main(argv=None):
    ap = argparse.ArgumentParser(prog="trace_run", description=__doc__.split("\n\n")[0])
    ap.add_argument("--model", required=True, help="folder with config.json and model.safetensors")
    ap.add_argument("--dtype", required=True, choices=("bfloat16", "float32"),
                    help="the models here compute in 32-bit throughout: both name the same kernels, "
                         "whatever type the weights are stored in")
    ap.add_argument("--out", required=True, help="folder for the logits")
    ap.add_argument("--max-tokens", type=int, default=0, help="most tokens a live request holds: room made ahead")
    a = ap.parse_args(argv)

    from . import HFLoader, build_library, library_path

    if not os.path.exists(library_path()):
        build_library(force=False)
    model = HFLoader.load_model(a.model)
    if a.max_tokens > 0:
        model.reserve(a.max_tokens)
    replay = Replay(model)
    for line in sys.stdin:
        if not line.strip():
            continue
        step = json.loads(line)
        rows = [replay.entry(e["id"], e["tokens"], e.get("want", [])) for e in step["entries"]]
        if sum(len(r) for r in rows):
            with open(os.path.join(a.out, f"{step['step']}.f32"), "wb") as f:
                for r in rows:
                    f.write(r.astype("<f4", copy=False).tobytes())
        for request in step.get("end", []):
            replay.end(request)
        print(f"done {step['step']}", flush=True)
    model.close()
    return 0
