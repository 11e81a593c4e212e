"""Replays a trace: given tokens, step by step, through a model's own passes; nothing is sampled.

Standard input, one JSON object a line:
    {"step": 0, "entries": [{"id": "a", "tokens": [5, 17, 3], "want": [0, 2]}], "end": ["b"]}
All entries of a step are one batch.  The logits at the wanted places go to OUT/<step>.f32 (little-endian f32, [wanted,
vocab], in the order of the entries), then "done <step>" is printed.  Requests named in "end" give back what they hold.
"""
import json
import os
import sys

LIVE_REQUESTS = 4                                         # rows and recurrent states of the decoder


def add_arguments(ap):
    ap.add_argument("--model", required=True, help="folder with config.json and model.safetensors")
    ap.add_argument("--dtype", choices=("bfloat16", "float32"), default="bfloat16")
    ap.add_argument("--out", required=True, help="existing folder for <step>.f32")
    ap.add_argument("--max-tokens", type=int, required=True, help="tokens that live requests hold at most (sizes the cache pool)")
    ap.add_argument("--device", type=int, default=0)


def run(a, lines=None):
    import fandhe_ai_amd as fa
    from fandhe_ai_amd import models, scheduler

    ops = fa.tape_for(fa.Device.Rocm(a.device))
    decoder = models.load_model(ops, a.model, a.dtype, models.Capacity(a.max_tokens, LIVE_REQUESTS, LIVE_REQUESTS))
    batcher = scheduler.PortionBatcher(decoder)
    for line in sys.stdin if lines is None else lines:
        if not line.strip():
            continue
        step = json.loads(line)
        entries = [(e["id"], e["tokens"], e.get("want", [])) for e in step.get("entries", [])]
        if entries:
            logits = batcher.feed(entries)
            if len(logits):
                logits.astype("<f4").tofile(os.path.join(a.out, "%d.f32" % step["step"]))
        for rid in step.get("end", []):
            batcher.release(rid)
        print("done %d" % step["step"], flush=True)
    decoder.close()
    ops.close()
    return 0
