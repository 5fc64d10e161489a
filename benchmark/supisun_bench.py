"""Prompt and decode throughput of the Supisun design on the ragged engine at sizes that resemble a real model's layers
(random weights), beside the closest model of the framework at equal size: Dimelix on the same engine (attention, a delta rule
with a matrix state and a dense feed-forward are its parts too), with the same width, number of layer executions, vocabulary,
feed-forward, attention heads and delta-rule states.

    python bench.py --bench supisun [--steps K] [--warmup W] [--in-len S]

Prints one JSON line: tokens/s of a prompt of S tokens in one step and of single-token steps behind it (batch 1 and
batch 8), for both designs and every size.  BIGDL_SUPISUN_SIZES=a,b picks sizes, BIGDL_SUPISUN_ONLY=prefill|decode and
BIGDL_SUPISUN_DESIGNS=supisun,dimelix narrow a run down for a profiler.
"""
import json
import os

import torch

from merusun_bench import engine_numbers

SIZES = {
    "a": dict(width=2048, layers=6, heads=16, kv_heads=4, dim=128, ff=5632, vocab=32000, chunk=1024, rot_dims=64, delta_heads=16,
              delta_kv_heads=8, delta_dim=64, delta_vdim=64, inner=4096, state=16, dt_rank=128),
    "b": dict(width=3072, layers=12, heads=24, kv_heads=8, dim=128, ff=8192, vocab=32000, chunk=2048, rot_dims=64, delta_heads=24,
              delta_kv_heads=12, delta_dim=64, delta_vdim=64, inner=6144, state=16, dt_rank=192),
}


def supisun_engine(size, device):
    from bigdl_amd.models import supisun
    return supisun.build_random(supisun.example_config(**SIZES[size]), torch.bfloat16, device, seed=1)


def dimelix_engine(size, device):
    from bigdl_amd.models import dimelix
    s = SIZES[size]
    cfg = dimelix.example_config(width=s["width"], layers=s["layers"], loop=None, heads=s["heads"], kv_heads=s["kv_heads"], dim=s["dim"],
                                 ff=s["ff"], vocab=s["vocab"], window=s["chunk"], rank=512, latent_dim=s["dim"],
                                 delta_heads=s["delta_heads"], delta_dim=s["delta_dim"], rot_dims=s["rot_dims"], streams=0)
    return dimelix.build_random(cfg, torch.bfloat16, device, seed=1)


def main(args):
    device = torch.device("cuda", 0)
    in_len = args.in_len if args.in_len != 1024 else 2048
    only = os.environ.get("BIGDL_SUPISUN_ONLY", "")
    designs = (os.environ.get("BIGDL_SUPISUN_DESIGNS") or "supisun,dimelix").split(",")
    res = {}
    for size in (os.environ.get("BIGDL_SUPISUN_SIZES") or ",".join(SIZES)).split(","):
        res[size] = {}
        for name, make in (("supisun", supisun_engine), ("dimelix", dimelix_engine)):
            if name in designs:
                eng = make(size, device)
                res[size][name] = engine_numbers(eng, SIZES[size]["vocab"], in_len, args.warmup, args.steps, only)
                res[size][name]["layer_executions"] = len(eng.runs)
                del eng
                torch.cuda.empty_cache()
    print(json.dumps({"bench": "supisun", "prompt_tokens": in_len, "dtype": "bf16", "data": "synthetic",
                      "sizes": {k: dict(v) for k, v in SIZES.items()}, "results": res}), flush=True)
