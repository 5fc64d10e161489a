"""Prompt and decode throughput of the Lifenex design on the ragged engine at sizes that resemble a real model's layers (random
weights), beside the closest models of the framework at equal size on the same engine: Supisun (attention, a gated delta rule and a
selective scan) and Filanex (parallel blocks with dense and routed gated feed-forwards), with the same width, number of layer
executions, vocabulary and attention heads, and feed-forwards of as many multiply-adds per token.

    python bench.py --bench lifenex [--steps K] [--warmup W] [--in-len S]

Prints one JSON line: tokens/s of a prompt of S tokens in one step and of single-token steps behind it (batch 1 and batch 8), for
the designs and every size.  BIGDL_LIFENEX_SIZES=a,b picks sizes, BIGDL_LIFENEX_ONLY=prefill|decode and
BIGDL_LIFENEX_DESIGNS=lifenex,supisun,filanex narrow a run down for a profiler.
"""
import json
import os

import torch

from merusun_bench import engine_numbers

SIZES = {
    "a": dict(width=2048, layers=6, heads=16, kv_heads=4, dim=128, ff=5632, vocab=32000, bias_max=1024, delta_heads=16, delta_kv_heads=8,
              delta_dim=64, delta_vdim=64, ssm_heads=64, ssm_vdim=64, ssm_state=128, ssm_groups=8, norm_groups=8, expert_ff=1024, experts=32,
              top=4, groups=4, keep=2, shared_ff=1536),
    "b": dict(width=3072, layers=12, heads=24, kv_heads=8, dim=128, ff=8192, vocab=32000, bias_max=2048, delta_heads=24, delta_kv_heads=12,
              delta_dim=64, delta_vdim=64, ssm_heads=96, ssm_vdim=64, ssm_state=128, ssm_groups=8, norm_groups=8, expert_ff=1024, experts=64,
              top=6, groups=8, keep=4, shared_ff=2048),
}


def lifenex_engine(size, device):
    from bigdl_amd.models import lifenex
    return lifenex.build_random(lifenex.example_config(**SIZES[size]), torch.bfloat16, device, seed=1)


def supisun_engine(size, device):
    from bigdl_amd.models import supisun
    s = SIZES[size]
    ff = 3 * (s["top"] * s["expert_ff"] + s["shared_ff"]) // 2             # two matrices instead of three
    cfg = supisun.example_config(width=s["width"], layers=s["layers"], heads=s["heads"], kv_heads=s["kv_heads"], dim=s["dim"], ff=ff,
                                 vocab=s["vocab"], chunk=8192, rot_dims=64, delta_heads=s["delta_heads"], delta_kv_heads=s["delta_kv_heads"],
                                 delta_dim=s["delta_dim"], delta_vdim=s["delta_vdim"], inner=s["ssm_heads"] * s["ssm_vdim"], state=16,
                                 dt_rank=s["width"] // 16)
    return supisun.build_random(cfg, torch.bfloat16, device, seed=1)


def filanex_engine(size, device):
    from bigdl_amd.models import filanex
    s = SIZES[size]
    cfg = filanex.example_config(width=s["width"], layers=s["layers"], heads=s["heads"], kv_heads=s["kv_heads"], dim=s["dim"], vdim=s["dim"],
                                 ff=s["ff"], expert_ff=s["expert_ff"], experts=s["experts"], top=s["top"], groups=s["groups"], keep=s["keep"],
                                 vocab=s["vocab"], block=8192, rot_dims=64, loop=None)
    return filanex.build_random(cfg, torch.bfloat16, device, seed=1)


def main(args):
    device = torch.device("cuda", 0)
    in_len = args.in_len if args.in_len != 1024 else 2048
    only = os.environ.get("BIGDL_LIFENEX_ONLY", "")
    designs = (os.environ.get("BIGDL_LIFENEX_DESIGNS") or "lifenex,supisun,filanex").split(",")
    res = {}
    for size in (os.environ.get("BIGDL_LIFENEX_SIZES") or ",".join(SIZES)).split(","):
        res[size] = {}
        for name, make in (("lifenex", lifenex_engine), ("supisun", supisun_engine), ("filanex", filanex_engine)):
            if name in designs:
                eng = make(size, device)
                res[size][name] = engine_numbers(eng, SIZES[size]["vocab"], in_len, args.warmup, args.steps, only)
                res[size][name]["layer_executions"] = len(eng.runs)
                del eng
                torch.cuda.empty_cache()
    print(json.dumps({"bench": "lifenex", "prompt_tokens": in_len, "dtype": "bf16", "data": "synthetic",
                      "sizes": {k: dict(v) for k, v in SIZES.items()}, "results": res}), flush=True)
