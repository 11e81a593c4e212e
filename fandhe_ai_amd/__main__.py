"""Command line: ``python -m fandhe_ai_amd generate`` and ``python -m fandhe_ai_amd trace``.

generate: continues prompts of token ids with a model folder, through the batch scheduler.
trace: feeds given tokens through a model, step by step, and writes the logits asked for (trace.py).
"""
import argparse
import json
import sys


def _generate(a):
    import numpy as np
    import fandhe_ai_amd as fa
    from fandhe_ai_amd import models, scheduler

    prompts = [[int(t) for t in p.replace(",", " ").split()] for p in a.prompt]
    if a.top_k:
        strategy = scheduler.SamplingStrategy.TopK(a.top_k)
    elif a.temperature:
        strategy = scheduler.SamplingStrategy.Temperature(a.temperature)
    else:
        strategy = scheduler.SamplingStrategy.Greedy()
    longest = max(len(p) for p in prompts) + a.new_tokens
    ops = fa.tape_for(fa.Device.Rocm(a.device))
    capacity = models.Capacity(a.max_tokens or len(prompts) * (longest + 16), min(len(prompts), 32))
    decoder = models.load_model(ops, a.model, a.dtype, capacity)
    sched = scheduler.BatchScheduler(decoder, scheduler.SchedulerLimits(capacity.max_batch, len(prompts), longest))
    for i, p in enumerate(prompts):
        sched.submit(np.array(p, dtype=np.int32), scheduler.GenerateConfig(len(p) + a.new_tokens, strategy, a.seed + i))
    out, failed = {}, 0
    while len(out) + failed < len(prompts):
        sched.step()
        out.update(sched.take_finished())
        for rid, error in sched.take_failed():
            failed += 1
            print("request %d: %s" % (rid, error), file=sys.stderr)
    for rid in sorted(out):
        print(json.dumps({"id": rid, "tokens": [int(t) for t in out[rid]]}))
    decoder.close()
    ops.close()
    return 1 if failed else 0


def main(argv=None):
    ap = argparse.ArgumentParser(prog="python -m fandhe_ai_amd")
    sub = ap.add_subparsers(dest="command", required=True)
    g = sub.add_parser("generate", help="continue prompts of token ids")
    g.add_argument("--model", required=True, help="folder with config.json and model.safetensors")
    g.add_argument("--prompt", action="append", required=True, help="token ids, separated by commas or spaces (may be repeated)")
    g.add_argument("--new-tokens", type=int, default=32)
    g.add_argument("--dtype", choices=("bfloat16", "float32"), default="bfloat16")
    g.add_argument("--temperature", type=float, default=0.0, help="0: greedy")
    g.add_argument("--top-k", type=int, default=0)
    g.add_argument("--seed", type=int, default=0)
    g.add_argument("--max-tokens", type=int, default=0, help="size of the cache pool (default: what the prompts need)")
    g.add_argument("--device", type=int, default=0)
    from fandhe_ai_amd import trace
    trace.add_arguments(sub.add_parser("trace", help="feed given tokens, write logits"))
    a = ap.parse_args(argv)
    return trace.run(a) if a.command == "trace" else _generate(a)


if __name__ == "__main__":
    sys.exit(main())
