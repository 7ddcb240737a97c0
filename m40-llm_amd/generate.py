"""Generates from a model folder (config.json + model.safetensors) through the continuous-batching scheduler.

    python m40-llm_amd/generate.py --model DIR --prompt 1,5,9 [--prompt 7,7 ...] [--max-tokens N] [--temperature T --top-k K --top-p P --seed S]
                                   [--stop ID ...] [--dtype bfloat16|float32] [--cache-tokens N] [--slots N]

Prompts are token ids (tokenizers are outside this package).  Prints one JSON line a prompt: {"prompt": [...], "generated": [...]}.
"""
from __future__ import annotations

import argparse
import importlib
import json
import os
import sys

ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
if ROOT not in sys.path:
    sys.path.insert(0, ROOT)
m40 = importlib.import_module("m40-llm_amd")
layered = importlib.import_module("m40-llm_amd.layered")
scheduler = importlib.import_module("m40-llm_amd.scheduler")


def generate(model, prompts, max_tokens, stop_ids=(), temperature=1.0, top_k=1, top_p=0.0, seed=42, slots=0):
    """Generated ids of every prompt; more prompts than slots take turns."""
    s = scheduler.Scheduler.for_model(model, slots)
    rids, waiting, out = {}, list(enumerate(prompts)), [None] * len(prompts)
    while waiting or s.active():
        while waiting and s.available_slots():
            i, p = waiting.pop(0)
            rids[i] = s.submit(p, max_tokens=max_tokens, stop_ids=stop_ids, temperature=temperature, top_k=top_k, top_p=top_p, seed=seed)
        s.tick()
    for i, rid in rids.items():
        if s.state(rid) != "complete":
            raise RuntimeError("prompt %d: %s" % (i, s.error(rid)))
        out[i] = s.generated(rid)
    s.close()
    return out


def main(argv=None):
    ap = argparse.ArgumentParser(description=__doc__, formatter_class=argparse.RawDescriptionHelpFormatter)
    ap.add_argument("--model", required=True)
    ap.add_argument("--prompt", action="append", required=True, type=lambda t: [int(x) for x in t.split(",")])
    ap.add_argument("--max-tokens", type=int, default=32)
    ap.add_argument("--stop", type=int, action="append", default=[])
    ap.add_argument("--temperature", type=float, default=1.0)
    ap.add_argument("--top-k", type=int, default=1)
    ap.add_argument("--top-p", type=float, default=0.0)
    ap.add_argument("--seed", type=int, default=42)
    ap.add_argument("--dtype", default="bfloat16", choices=["bfloat16", "float32"])
    ap.add_argument("--cache-tokens", type=int, default=0, help="tokens the cache pool holds; 0 = what the prompts need")
    ap.add_argument("--slots", type=int, default=4)
    a = ap.parse_args(argv)
    need = sum((len(p) + a.max_tokens + 63) // 64 * 64 for p in a.prompt)
    if not (os.path.exists(m40.NATIVE_LIB) and os.path.exists(m40.HOST_LIB)):
        m40.build()
    model = layered.LayeredModel.open(m40.Context(0), a.model, a.dtype, a.cache_tokens or need, a.slots)
    for p, g in zip(a.prompt, generate(model, a.prompt, a.max_tokens, a.stop, a.temperature, a.top_k, a.top_p, a.seed)):
        print(json.dumps({"prompt": p, "generated": g}), flush=True)
    model.close()


if __name__ == "__main__":
    main()
