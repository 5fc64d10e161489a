"""The Lifenex design on the ragged engine against the plain float64 statement in ``lifenex_oracle.py``.

Every test runs twice: on the CPU (the engine's bookkeeping over the unfused statements of ``ops/ragged.py``) and,
marked ``gpu``, on the device (the HIP kernels of ``libbigdl_ragged.so``).  Models are small and random; where random
weights would hide a fault (one key among many, a step of the distance bias, a sink, a decayed state) the inputs are made so
that it shows.
"""
import json
import math
import os
import random

import pytest
import torch

import lifenex_oracle as O
from bigdl_amd.models import lifenex
from bigdl_amd.models.paged import PagedStatePool
from bigdl_amd.ops import ragged as R

DEVICES = ["cpu", pytest.param("cuda", marks=pytest.mark.gpu)]
F32_TOL = 3e-4
MOE = (8, 2, 4, 2, 24)         # experts, top, groups, kept groups, inner size of the shared expert


def engine_for(config, W, dtype, device):
    return lifenex.build_engine(lifenex.read_config(O.plain_config(config)), W, dtype, device)


def full_model():
    """both kinds of layers with every kind of feed-forward"""
    return O.make_config([O.parallel_layer(), O.mamba2_layer(ff=16, moe=MOE), O.parallel_layer(heads=3, kv_heads=3, dim=10, vdim=6, bias_max=70,
                          rel_rows=9, temp=(0.7, 5), d_heads=3, d_kv=1, d_dim=9, d_vdim=7, conv=5, ff=None),
                          O.mamba2_layer(heads=4, vdim=9, state=7, groups=4, norm_groups=1, conv=2, ff=None),
                          O.parallel_layer(heads=6, kv_heads=2, dim=12, vdim=8, bias_max=20, rel_rows=8, ff=16, moe=(6, 3, 3, 2, None)),
                          O.mamba2_layer(ff=40)])


def run_schedule(engine, prompts, schedule, max_tokens, slots=4, seen=None):
    """schedule: steps of [(request, count)]; returns {request: logits of all its positions [T, V]} (float64, host)"""
    engine.pool = None
    pool = engine.ensure_pool(max_tokens, slots)
    at, slot, got = {}, {}, {k: [] for k in prompts}
    for step in schedule:
        entries, want = [], []
        for rid, n in step:
            if rid not in slot:
                slot[rid] = pool.admit()
            lo = at.get(rid, 0)
            entries.append((slot[rid], prompts[rid][lo:lo + n]))
            want.append(list(range(n)))
            at[rid] = lo + n
        logits = engine.step(entries, want).double().cpu()
        row = 0
        for rid, n in step:
            got[rid].append(logits[row:row + n])
            row += n
            if seen is not None:
                seen.setdefault(rid, (set(), set()))[0].update(pool.pages_of[slot[rid]])
                seen[rid][1].add(slot[rid])
            if at[rid] == len(prompts[rid]):
                pool.release(slot.pop(rid))
    return {k: torch.cat(v) for k, v in got.items() if v}


def close(a, b, tol=F32_TOL):
    assert a.shape == b.shape
    err = float((a - b).abs().max())
    assert err <= tol, f"max difference {err}"


# ------------------------------------------------------------------------------------------------ whole models
@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("layers,more", [
    ([O.parallel_layer()], {}),
    ([O.mamba2_layer()], {}),
    ([O.parallel_layer(ff=16, moe=MOE)], {}),
    ([O.parallel_layer(heads=1, kv_heads=1, dim=8, vdim=12, bias_max=2, rel_rows=2, temp=(0.0, 1), d_heads=1, d_kv=1, d_dim=24, d_vdim=24,
                       conv=1, ff=None)], {"logit_scale": 1.0, "low_rank": (1, 1)}),
    ([O.parallel_layer(heads=6, kv_heads=6, dim=12, vdim=10, bias_max=64, rel_rows=16, temp=(1.5, 1), d_heads=6, d_kv=6, d_dim=40, d_vdim=7,
                       conv=4)], {"low_rank": (8, 16)}),
    ([O.parallel_layer(heads=8, kv_heads=1, dim=32, vdim=136, bias_max=300, rel_rows=31, temp=(0.2, 64), d_heads=4, d_kv=1, d_dim=5, d_vdim=33,
                       conv=2)], {"eps": 1e-3}),                                # values wider than keys, an odd number of bias rows
    ([O.parallel_layer(heads=5, kv_heads=5, dim=7, vdim=3, bias_max=11, rel_rows=6, scale=0.9, d_heads=2, d_kv=1, d_dim=70, d_vdim=130,
                       conv=4)], {"width": 33}),                                # odd sizes
    ([O.parallel_layer(ff=8, moe=(6, 1, 6, 3, 8))], {}),                        # groups of one expert
    ([O.parallel_layer(ff=8, moe=(5, 5, 1, 1, None))], {}),                     # one group, every expert, no shared one
    ([O.mamba2_layer(heads=1, vdim=24, state=1, groups=1, norm_groups=1, conv=1, ff=None)], {}),
    ([O.mamba2_layer(heads=8, vdim=6, state=16, groups=1, norm_groups=8, conv=2)] * 2, {}),
    ([O.mamba2_layer(heads=3, vdim=11, state=37, groups=3, norm_groups=3, conv=6, ff=16, moe=MOE)], {"width": 37}),
    ([O.mamba2_layer(heads=2, vdim=70, state=130, groups=1, norm_groups=2)], {}),
])
def test_each_layer_kind_alone(device, layers, more):
    cfg = O.make_config(layers, **more)
    W = O.random_weights(cfg, seed=1)
    toks = O.random_tokens(90, cfg["vocab"], 2)
    want = O.forward(toks, W, cfg)
    eng = engine_for(cfg, W, torch.float32, device)
    close(run_schedule(eng, {"a": toks}, [[("a", 60)], [("a", 2)]] + [[("a", 1)] for _ in range(28)], 128)["a"], want)


@pytest.mark.parametrize("device", DEVICES)
def test_layer_outputs_one_by_one(device):
    cfg = full_model()
    W = O.random_weights(cfg, seed=3)
    toks = O.random_tokens(40, cfg["vocab"], 4)
    want = []
    O.forward(toks, W, cfg, layers_out=want)
    eng = engine_for(cfg, W, torch.float32, device)
    pool = eng.ensure_pool(64, 1)
    slot, got, rows = pool.admit(), [], []
    eng.step([(slot, toks[:30])], collect=got)
    for t in range(30, 40):
        rows.append([])
        eng.step([(slot, toks[t:t + 1])], collect=rows[-1])
    assert len(got) == len(want) == len(cfg["layers"])
    for i, b in enumerate(want):
        a = torch.cat([got[i]] + [r[i] for r in rows])
        err = float((a.double().cpu() - b).abs().max()) / max(1.0, float(b.abs().max()))
        assert err < 2e-5, f"layer {i}: {err}"


@pytest.mark.parametrize("device", DEVICES)
def test_prompt_against_token_by_token_and_portions(device):
    cfg = full_model()
    W = O.random_weights(cfg, seed=5)
    toks = O.random_tokens(150, cfg["vocab"], 6)
    want = O.forward(toks, W, cfg)
    eng = engine_for(cfg, W, torch.float32, device)
    close(run_schedule(eng, {"a": toks}, [[("a", 150)]], 192)["a"], want)
    close(run_schedule(eng, {"a": toks}, [[("a", 1)] for _ in range(150)], 192)["a"], want)
    for sizes in ([2] * 75, [64, 2, 62, 3, 1, 1, 17], [63, 1, 1, 63, 2, 20], [1, 2, 3, 4, 5, 64, 65, 6], [9, 1, 8, 2, 70, 60]):
        assert sum(sizes) == 150
        close(run_schedule(eng, {"a": toks}, [[("a", n)] for n in sizes], 192)["a"], want)


@pytest.mark.parametrize("device", DEVICES)
def test_unequal_requests_in_one_batch_and_reuse_of_pages_and_slots(device):
    cfg = full_model()
    W = O.random_weights(cfg, seed=7)
    lens = {"a": 130, "b": 7, "c": 70, "d": 1, "e": 66, "f": 90}
    prompts = {k: O.random_tokens(n, cfg["vocab"], 10 + i) for i, (k, n) in enumerate(lens.items())}
    want = {k: O.forward(p, W, cfg) for k, p in prompts.items()}
    # three slots, pool of 5 pages (320 tokens) for 364 tokens in total: d, e, f run in what a, b, c gave back
    schedule = [[("a", 60), ("b", 2), ("c", 1)], [("a", 1), ("b", 5), ("c", 63)], [("a", 5), ("c", 6)],
                [("a", 64), ("d", 1)], [("e", 1), ("f", 1)], [("e", 1), ("f", 29)], [("e", 64), ("f", 1)], [("f", 59)]]
    eng = engine_for(cfg, W, torch.float32, device)
    seen = {}
    got = run_schedule(eng, prompts, schedule, 320, slots=3, seen=seen)
    for k in prompts:
        close(got[k], want[k])
    old, new = ("a", "b", "c"), ("d", "e", "f")
    assert set().union(*(seen[k][0] for k in new)) & set().union(*(seen[k][0] for k in old)), "no page was used twice"
    assert set().union(*(seen[k][1] for k in new)) & set().union(*(seen[k][1] for k in old)), "no slot was used twice"
    alone = run_schedule(eng, {"c": prompts["c"]}, [[("c", 70)]], 128)["c"]
    close(alone, got["c"], 2e-4)


@pytest.mark.parametrize("device", DEVICES)
def test_long_decoding_past_pages_and_the_farthest_bucket(device):
    cfg = O.make_config([O.parallel_layer(bias_max=100), O.mamba2_layer(), O.parallel_layer(bias_max=30, temp=(0.5, 64), ff=8, moe=MOE)])
    W = O.random_weights(cfg, seed=9)
    for li in (0, 2):                                        # slow decays: early tokens still weigh at the end
        W[f"l{li}.mix.right.dt_bias"] = W[f"l{li}.mix.right.dt_bias"] - 4.0
    W["l1.mix.dt_bias"] = W["l1.mix.dt_bias"] - 4.0
    toks = O.random_tokens(200, cfg["vocab"], 11)
    want = O.forward(toks, W, cfg)
    eng = engine_for(cfg, W, torch.float32, device)
    got = run_schedule(eng, {"a": toks}, [[("a", 5)]] + [[("a", 1)] for _ in range(195)], 256)["a"]
    close(got, want)


@pytest.mark.parametrize("device", DEVICES)
def test_long_portions_run_the_recurrences_in_chunks(device):
    """portions of several hundred tokens (the delta rule is cut into chunks that are scanned side by side and chained) beside a
    short one and a single token, into states that earlier portions have left"""
    cfg = O.make_config([O.mamba2_layer(state=20, ff=None), O.parallel_layer(heads=2, kv_heads=1, d_heads=4, d_kv=2, d_dim=24, d_vdim=40, ff=None)])
    W = O.random_weights(cfg, seed=15)
    for name in ("l0.mix.dt_bias", "l1.mix.right.dt_bias"):  # slow decays: what an early chunk wrote reaches the last one
        W[name] = W[name] - 4.0
    prompts = {"a": O.random_tokens(420, cfg["vocab"], 16), "b": O.random_tokens(300, cfg["vocab"], 17), "c": O.random_tokens(9, cfg["vocab"], 18)}
    want = {k: O.forward(p, W, cfg) for k, p in prompts.items()}
    eng = engine_for(cfg, W, torch.float32, device)
    got = run_schedule(eng, prompts, [[("a", 30), ("c", 3)], [("a", 390), ("b", 257), ("c", 1)], [("b", 43), ("c", 5)]], 832)
    for k in prompts:
        close(got[k], want[k], 5e-4)


def _relative(got, want):
    d = got - want
    d = d - d.mean(-1, keepdim=True)
    return d.pow(2).mean(-1).sqrt() / (want - want.mean(-1, keepdim=True)).pow(2).mean().sqrt()


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("odd", [False, True])
def test_bfloat16_stays_near_the_exact_result(device, odd):
    if odd:          # sizes that take none of the vector or matrix-core paths
        layers = [O.parallel_layer(heads=3, kv_heads=1, dim=18, vdim=14, d_heads=3, d_kv=1, d_dim=17, d_vdim=9),
                  O.mamba2_layer(heads=5, vdim=7, state=11, groups=5, norm_groups=5), O.parallel_layer(heads=6, kv_heads=1, dim=10, vdim=14, conv=2)]
    else:            # sizes that the vector and matrix-core paths serve
        layers = [O.parallel_layer(heads=4, kv_heads=2, dim=32, vdim=32, d_heads=4, d_kv=2, d_dim=32, d_vdim=32, conv=4),
                  O.mamba2_layer(heads=8, vdim=16, state=32, groups=2, norm_groups=4), O.parallel_layer(heads=8, kv_heads=2, dim=64, vdim=32, bias_max=50),
                  O.mamba2_layer(heads=2, vdim=80, state=40, groups=1, norm_groups=1)]
    cfg = O.make_config(layers, width=64)
    W = O.random_weights(cfg, seed=13)
    toks = O.random_tokens(100, cfg["vocab"], 14)
    want = O.forward(toks, W, cfg)
    eng = engine_for(cfg, W, torch.bfloat16, device)
    rel = _relative(run_schedule(eng, {"a": toks}, [[("a", 70)], [("a", 2)]] + [[("a", 1)] for _ in range(28)], 128)["a"], want)
    assert float(rel.median()) < 0.05 and float(rel.max()) < 0.15, (float(rel.median()), float(rel.max()))


def _random_design(seed):
    """a model of the design with everything drawn at random: kinds and order of layers, sizes, constants"""
    rnd = random.Random(seed)

    def feed_forward():
        kind = rnd.choice(["none", "dense", "moe", "moe"])
        if kind != "moe":
            return dict(ff=rnd.choice([24, 56]) if kind == "dense" else None)
        groups, size = rnd.choice([(1, 5), (2, 3), (3, 2), (4, 1), (4, 4)])
        keep = rnd.randint(1, groups)
        return dict(ff=rnd.choice([8, 12, 16]), moe=(groups * size, rnd.randint(1, min(4, keep * size)), groups, keep, rnd.choice([None, 8, 20])))

    layers = []
    for _ in range(rnd.randint(2, 4)):
        if rnd.random() < 0.6:
            kv, dkv, dim = rnd.choice([1, 2, 3]), rnd.choice([1, 2, 3]), rnd.choice([8, 12, 16, 24, 40, 64])
            rows = rnd.choice([2, 5, 8, 16, 32])
            layers.append(O.parallel_layer(
                heads=kv * rnd.choice([1, 2, 4]), kv_heads=kv, dim=dim, vdim=rnd.choice([8, 12, 16, 48, 80]), rel_rows=rows,
                scale=rnd.choice([0.5, 1.0, 2.0]) * dim ** -0.5, bias_max=rows // 2 + rnd.choice([1, 7, 50, 128, 400]),
                temp=(rnd.choice([0.0, 0.2, 1.0]), rnd.choice([1, 7, 64, 100])), d_heads=dkv * rnd.choice([1, 2, 3]), d_kv=dkv,
                d_dim=rnd.choice([8, 16, 32, 40, 72]), d_vdim=rnd.choice([8, 20, 48, 64, 96]), conv=rnd.choice([1, 2, 3, 4, 5]), **feed_forward()))
        else:
            groups, per = rnd.choice([1, 2, 4]), rnd.choice([1, 2, 3])
            layers.append(O.mamba2_layer(heads=groups * per, vdim=rnd.choice([4, 12, 16, 40, 64]), state=rnd.choice([1, 8, 16, 24, 64]), groups=groups,
                                         norm_groups=rnd.choice([1, groups, groups * per]), conv=rnd.choice([1, 2, 4, 5]), **feed_forward()))
    return O.make_config(layers, width=rnd.choice([24, 40, 64]), vocab=rnd.choice([50, 67, 128]), eps=rnd.choice([1e-5, 1e-6, 1e-3]),
                         logit_scale=rnd.choice([0.1, 1.0, 2.5]), low_rank=(rnd.choice([1, 4, 8, 13]), rnd.choice([1, 6, 16])))


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("seed", range(10))
def test_random_models_of_the_design(device, seed):
    """three unequal requests in mixed steps (two slots, pages used again) against the plain statement, in float32; in
    bfloat16 the same steps stay near it"""
    cfg = _random_design(seed)
    W = O.random_weights(cfg, seed=100 + seed)
    prompts = {"a": O.random_tokens(140, cfg["vocab"], 200 + seed), "b": O.random_tokens(30, cfg["vocab"], 300 + seed),
               "c": O.random_tokens(75, cfg["vocab"], 400 + seed)}
    want = {k: O.forward(p, W, cfg) for k, p in prompts.items()}
    schedule = [[("a", 66), ("b", 3)], [("a", 1), ("b", 27)], [("a", 2), ("c", 70)], [("a", 70), ("c", 1)], [("a", 1), ("c", 4)]]
    got = run_schedule(engine_for(cfg, W, torch.float32, device), prompts, schedule, 320, slots=2)
    for k in prompts:
        scale = max(1.0, float(want[k].abs().max()))
        close(got[k] / scale, want[k] / scale)
    got = run_schedule(engine_for(cfg, W, torch.bfloat16, device), prompts, schedule, 320, slots=2)
    for k in prompts:                                        # (a row whose experts change places under rounding is far off)
        rel = _relative(got[k], want[k])
        assert float(rel.median()) < 0.06 and float(rel.quantile(0.9)) < 0.3, (k, float(rel.median()), float(rel.quantile(0.9)))


# ------------------------------------------------------------------------------------------------ attention alone
def test_steps_of_the_distance_bias():
    """every distance's row against the formula in exact comparisons: distance n has row half + m when (n / half)^R lies in
    [(far / half)^m, (far / half)^(m + 1)), R rows for the far half"""
    for rows, far in ((16, 130), (32, 128), (8, 64), (16, 8 * 256), (9, 70), (2, 2), (2, 5), (31, 300), (12, 40), (64, 1000), (4, 3), (32, 4096)):
        half, R_ = rows // 2, rows - rows // 2
        last = -1
        for n in list(range(0, min(far, 700) + 3)) + [far - 1, far, far + 1]:
            got = lifenex.distance_bucket(n, rows, far)
            if n < half:
                assert got == n
            elif n >= far:
                assert got == rows - 1
            else:
                m = got - half                               # n^R half^m >= far^m half^R, in integers
                assert n ** R_ * half ** m >= far ** m * half ** R_
                assert n ** R_ * half ** (m + 1) < far ** (m + 1) * half ** R_ or got == rows - 1
            if n <= far and n > 0:
                assert got == O.bucket(n, rows, far) if n < far else True
            assert got >= last or n == far - 1
            last = got
    rel = torch.arange(12.0).view(6, 2)
    tab = lifenex.distance_bias(rel, 20)
    assert tab.shape == (2, 21) and [int(v) // 2 for v in tab[0]] == [lifenex.distance_bucket(n, 6, 20) for n in range(21)]
    assert bool((tab[1] == tab[0] + 1).all())


def _attend_through_pages(device, q, k, v, portions, *, scale, bias, sink=None, page_order=None, dtype=torch.float32):
    """q [T, H, d], k [T, G, d], v [T, G, e] (float64), bias [H, n], through the paged attention op in the given portions"""
    T, H, d = q.shape
    G, e = k.shape[1], v.shape[2]
    ops = R.ops_for(device)
    pool = PagedStatePool({0: [("kv", G, d, e)]}, 64 * ((T + 63) // 64 + 2), 2, dtype, device)
    if page_order:
        pool.free_pages = list(page_order)
    slot = pool.admit()
    out, at = [], 0
    for n in portions:
        pages = list(pool.reserve(slot, n))
        meta = R.BatchMeta([(slot, at, n, pages)], torch.device(device))
        pos = torch.arange(at, at + n)
        pg = torch.tensor(pages)[pos // 64].to(device)
        pool.k[0][pg, :, (pos % 64).to(device)] = k[at:at + n].to(dtype).to(device)
        pool.v[0][pg, :, (pos % 64).to(device)] = v[at:at + n].to(dtype).to(device)
        out.append(ops.paged_attn(q[at:at + n].reshape(n, H * d).float().to(device).contiguous(), pool.k[0], pool.v[0], meta, maps=1, H=H,
                                  G=G, d=d, vd=e, window=0, keep_first=0, scale=scale, lam=0.0, out_scale=1.0, out_norm=False, eps=1e-6,
                                  sinks=None if sink is None else sink.float().to(device), dist_bias=bias.float().to(device).contiguous()))
        pool.commit(slot, n)
        at += n
    return torch.cat(out).double().cpu().view(T, H, e)


def _one_query(q, k, v, i, scale, bias, sink):
    """[H, e]: query i of every head over the keys 0 .. i, the bias read at min(i - j, last)"""
    out = []
    for h in range(q.shape[1]):
        b = torch.stack([bias[h, min(i - j, bias.shape[1] - 1)] for j in range(i + 1)])
        s = torch.cat([k[:i + 1, 0] @ q[i, h] * scale + b, sink[h:h + 1]])
        out.append(torch.softmax(s, 0)[:-1] @ v[:i + 1, 0])
    return torch.stack(out)


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("decoded", [False, True])
@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
def test_far_keys_page_borders_and_bias_steps_stand_out(device, decoded, dtype):
    """Query i and key j are made parallel and long, so key j takes all of the weight; its value is a marker.  A bias of -60 that
    begins one distance later (or ends one earlier) takes the marker away or brings it back.  Queries are part of a prompt's portion or
    decoded alone; heads disagree about the bias."""
    g = torch.Generator().manual_seed(21)
    T, H, G, d, e = 210, 2, 1, 16, 16
    sink = torch.tensor([1.0, -3.0], dtype=O.F64)
    cases = [(100, 63), (100, 64), (130, 127), (130, 128), (64, 63), (64, 64), (0, 0), (1, 0), (15, 0), (209, 0), (209, 1), (191, 64), (192, 64),
             (193, 128), (128, 0), (127, 127)]
    for i, j in cases:
        q = torch.randn(T, H, d, generator=g).bfloat16().double() * 0.25
        k = torch.randn(T, G, d, generator=g).bfloat16().double() * 0.25
        v = torch.randn(T, G, e, generator=g).bfloat16().double()
        direction = torch.randn(d, generator=g).double()
        direction /= direction.norm()
        q[i, :] = (6.0 * direction).bfloat16().double()
        k[j, 0] = (6.0 * direction).bfloat16().double()
        v[j, 0] = 100.0
        n = i - j
        last = max(n + 1, 2)                                 # table entries 0 .. last; everything farther takes the last one
        bias = torch.zeros(H, last + 1, dtype=O.F64)
        bias[0, n] = -60.0                                   # head 0: this distance alone is pushed out
        bias[1, n + 1:] = -60.0                              # head 1: the next farther ones are
        if n > 0:
            bias[1, n - 1] = -60.0
        portions = [m for m in ([i, 1, T - i - 1] if decoded else [i // 2, i + 1 - i // 2, T - i - 1]) if m]
        got = _attend_through_pages(device, q, k, v, portions, scale=1.0, bias=bias, sink=sink, page_order=[5, 0, 3, 1, 4, 2], dtype=dtype)
        want = _one_query(q, k, v, i, 1.0, bias, sink)
        close(got[i] / 100, want / 100, 2e-5 if dtype == torch.float32 else 4e-3)
        assert float(want[1, 0]) > 50.0 and (float(want[0, 0]) < 50.0 or n == 0 and i == 0)      # (the marker does decide)


@pytest.mark.parametrize("device", DEVICES)
def test_sinks_are_not_scaled_and_count_once(device):
    """a sink far above the scores takes nearly everything, one far below nothing; the first token alone against its closed form"""
    g = torch.Generator().manual_seed(23)
    T, d, e = 70, 8, 4
    q, k, v = (torch.randn(T, n, w, generator=g).double() for n, w in ((3, d), (1, d), (1, e)))
    sink = torch.tensor([12.0, -40.0, 0.7], dtype=O.F64)
    bias = torch.randn(3, 5, generator=g).double()
    got = _attend_through_pages(device, q, k, v, [1, 66, 1, 2], scale=0.1, bias=bias, sink=sink)
    for i in (0, 1, 5, 64, 66, 69):
        close(got[i], _one_query(q, k, v, i, 0.1, bias, sink), 1e-5)
    s = 0.1 * (q[0] @ k[0, 0]) + bias[:, 0]
    close(got[0], (torch.exp(s) / (torch.exp(s) + torch.exp(sink)))[:, None] * v[0], 1e-5)
    assert float(got[69, 0].abs().max()) < 0.05


@pytest.mark.gpu
@pytest.mark.parametrize("H,G,d,e,nb", [(4, 2, 64, 128, 90), (2, 2, 48, 48, 1), (3, 1, 16, 32, 64), (8, 2, 128, 64, 300), (8, 1, 40, 16, 5000),
                                        (2, 1, 96, 80, 2)])
def test_matrix_core_attention_with_distance_bias_and_sinks(H, G, d, e, nb):
    """bfloat16 prompt portions (the MFMA kernel; the table in LDS or too long for it) and single tokens (the row-wise kernel)
    against the plain statement on the same bfloat16-rounded keys and values"""
    g = torch.Generator().manual_seed(71)
    T = 200
    q = torch.randn(T, H, d, generator=g).double()
    k = torch.randn(T, G, d, generator=g).bfloat16().double()
    v = torch.randn(T, G, e, generator=g).bfloat16().double()
    bias, sink = 2 * torch.randn(H, nb, generator=g).double(), torch.randn(H, generator=g).double()
    qr = q.clone()
    qr[:190] = q[:190].bfloat16().double()                   # the MFMA kernel rounds its queries
    i, j = torch.arange(T)[:, None], torch.arange(T)[None]
    got = _attend_through_pages("cuda", q, k, v, [120, 64, 3, 3] + [1] * 10, scale=2.0 * d ** -0.5, bias=bias, sink=sink, dtype=torch.bfloat16)
    for h in range(H):
        s = qr[:, h] @ k[:, h // (H // G)].T * (2.0 * d ** -0.5) + bias[h][(i - j).clamp(0, nb - 1)]
        s = torch.cat([s.masked_fill(j > i, float("-inf")), sink[h].expand(T, 1)], 1)
        want = torch.softmax(s, -1)[:, :-1] @ v[:, h // (H // G)]
        assert float((got[:, h] - want).abs().max()) < 0.03, (h, float((got[:, h] - want).abs().max()))


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("H,G,d,e,temp", [(4, 2, 16, 24, (0.4, 9)), (3, 3, 10, 6, (1.0, 1)), (8, 1, 64, 136, None), (1, 1, 5, 1, (0.3, 64)),
                                          (6, 2, 128, 64, (2.0, 70))])
def test_normed_heads_and_query_temperature(device, H, G, d, e, temp):
    """per-head norms with shared weights and the temperature of the query's position, against the statement; what the pages hold is
    what the scores and the sum see"""
    g = torch.Generator().manual_seed(25)
    ops, T, past, eps = R.ops_for(device), 21, 60, 1e-5
    P = torch.randn(T, (H + G) * d + G * e, generator=g) * torch.tensor([0.2, 4.0])[torch.randint(0, 2, (T, 1), generator=g)]
    qw, kw = 1 + torch.randn(d, generator=g), 1 + torch.randn(d, generator=g)
    pool = PagedStatePool({0: [("kv", G, d, e)]}, 192, 1, torch.float32, device)
    pool.free_pages = [1, 2, 0]
    slot = pool.admit()
    pool.reserve(slot, past)
    pool.commit(slot, past)
    pages = list(pool.reserve(slot, T))
    meta = R.BatchMeta([(slot, past, T, pages)], torch.device(device))
    got, _ = ops.qkv_rows(P.to(device), qw.to(device), kw.to(device), eps, 0, None, pool.k[0], pool.v[0], meta, H=H, G=G, d=d, vd=e,
                          head_norms=True, q_temp=temp)
    pd, nq, nk = P.double(), H * d, G * d
    q, k = O.rms(pd[:, :nq].view(T, H, d), eps, qw.double()), O.rms(pd[:, nq:nq + nk].reshape(T, G, d), eps, kw.double())
    if temp:
        q = torch.stack([q[t] * O.query_temperature(past + t, *temp) for t in range(T)])
    close(got.double().cpu().view(T, H, d), q, 1e-4)
    for t in range(T):
        pg, at = pages[(past + t) // 64], (past + t) % 64
        close(pool.k[0][pg, :, at].double().cpu(), k[t], 1e-4)
        close(pool.v[0][pg, :, at].double().cpu(), pd[t, nq + nk:].view(G, e), 1e-6)


# ------------------------------------------------------------------------------------------------ recurrences alone
@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("H,G,d,e,taps", [(4, 2, 16, 24, 4), (1, 1, 48, 8, 1), (3, 1, 40, 64, 3), (2, 2, 130, 33, 4), (6, 3, 5, 7, 2),
                                          (2, 1, 300, 20, 3), (2, 1, 128, 128, 4), (2, 2, 64, 64, 4), (1, 1, 24, 160, 5)])
def test_channel_decays_across_portions_and_in_a_used_slot(device, H, G, d, e, taps):
    """preparation (convolutions, unit vectors, gates, decays per key channel) and scan against the token-by-token statement: portions
    of 1, 2 and many tokens, a second sequence in the first one's slot, long portions in chunks, decays near one"""
    g = torch.Generator().manual_seed(33)
    ops, T = R.ops_for(device), 330
    C, b0 = 2 * G * d + H * e, 2 * G * d + H * e + 3
    P, wl = torch.randn(T, C + H + 5, generator=g), torch.randn(T, H * d, generator=g)
    cw = torch.randn(C, taps, generator=g) * 0.6
    rate, dtb = torch.exp(torch.randn(H, generator=g) - 2.0), torch.randn(H * d, generator=g) - 3.0
    decay = torch.exp(-rate.double().repeat_interleave(d) * O.softplus(wl.double() + dtb.double())).view(T, H, d)

    def statement(lo, hi):
        u = O.silu(O.causal_conv(P[lo:hi, :C].double(), cw.double()))
        n = hi - lo
        q, k = O.unit(u[:, :G * d].view(n, G, d)) * d ** -0.5, O.unit(u[:, G * d:2 * G * d].reshape(n, G, d))
        v, beta = u[:, 2 * G * d:].reshape(n, H, e), torch.sigmoid(P[lo:hi, b0:b0 + H].double())
        return torch.stack([O.channel_delta(q[:, h // (H // G)], k[:, h // (H // G)], v[:, h], decay[lo:hi, h], beta[:, h])[0] for h in range(H)], 1)

    def scan(pool, slot, lo, hi):
        meta = R.BatchMeta([(slot, pool.len_of[slot], hi - lo, [])], torch.device(device))
        qf, kf, v, gb, wf = ops.gated_delta_prep(P[lo:hi].to(device).contiguous(), cw.to(device), taps, pool.tail.get(0), b0, 0, rate.to(device),
                                                 dtb.to(device), O.UNIT_EPS, H, G, d, e, meta, wl=wl[lo:hi].to(device).contiguous())
        close(wf.double().cpu().view(hi - lo, H, d), decay[lo:hi], 1e-5)
        out = ops.gated_delta_scan(qf, kf, gb, G, v, pool.matrix[0], H, d, e, meta, wf=wf)
        pool.commit(slot, hi - lo)
        return out.double().cpu().view(hi - lo, H, e)

    specs = [("matrix", H, d, e)] + ([("tail", taps - 1, C)] if taps > 1 else [])
    pool = PagedStatePool({0: specs}, 64, 1, torch.float32, device)
    want, other = statement(0, T), statement(100, 160)
    scale = float(want.abs().max())
    for cuts in ([0, 1, 3, 40, 41, 43, 330], [0, 200, 201, 202, 330], [0, 330]):
        slot = pool.admit()
        got = torch.cat([scan(pool, slot, lo, hi) for lo, hi in zip(cuts, cuts[1:])])
        close(got / scale, want / scale, 5e-5)
        pool.release(slot)
        slot = pool.admit()                                  # the same slot: neither its state nor its inputs may leak
        close(scan(pool, slot, 100, 160) / scale, other / scale, 5e-5)
        pool.release(slot)
    if device == "cuda":                                     # the walk over the chunks as library products (very tall states)
        ops.delta_chain = False
        slot = pool.admit()
        close(torch.cat([scan(pool, slot, 0, 20), scan(pool, slot, 20, 330)]) / scale, want / scale, 5e-5)


@pytest.mark.parametrize("device", DEVICES)
def test_a_channel_forgets_by_its_own_decay_before_the_write(device):
    """two orthogonal keys written with strength 1; then one key channel is wiped: only what was stored under it is gone, and a
    rewrite in the same step reads the wiped state"""
    ops, d, e = R.ops_for(device), 8, 5
    k = torch.zeros(4, d)
    k[0, 3] = k[1, 6] = 1.0
    k[2, 3] = k[3, 6] = 1.0
    q = k.clone()
    v = torch.stack([torch.arange(1.0, e + 1), -2 * torch.arange(1.0, e + 1), torch.zeros(e), torch.zeros(e)])
    gb = torch.tensor([[[1.0, 1.0]], [[1.0, 1.0]], [[1.0, 0.0]], [[1.0, 0.5]]])       # (strength 0: read only; 0.5: half way to the value)
    wf = torch.ones(4, d)
    wf[2, 3] = 0.0
    wf[3, 6] = 0.25
    pool = PagedStatePool({0: [("matrix", 1, d, e)]}, 64, 1, torch.float32, device)
    slot = pool.admit()
    meta = R.BatchMeta([(slot, 0, 4, [])], torch.device(device))
    dev = lambda t: t.to(device)                             # noqa: E731
    out = ops.gated_delta_scan(dev(q), dev(k), dev(gb), 1, dev(v), pool.matrix[0], 1, d, e, meta, wf=dev(wf)).cpu()
    close(out, torch.stack([v[0], v[1], torch.zeros(e), 0.125 * v[1]]), 1e-6)


def _space_inputs(H, G, N, e, T, g, dtype):
    X = torch.randn(T, H * e + 2 * G * N + 8, generator=g).to(dtype)
    P = torch.randn(T, 16 + H, generator=g).to(dtype)
    return X, P, torch.randn(H, generator=g) - 4.0, torch.exp(torch.randn(H, generator=g)), torch.randn(H, generator=g)


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("H,G,N,e", [(4, 2, 16, 24), (1, 1, 1, 5), (3, 3, 37, 11), (2, 1, 130, 64), (8, 2, 128, 64), (2, 2, 32, 100), (4, 1, 72, 16),
                                     (1, 1, 256, 48), (2, 1, 96, 130)])
def test_state_space_scan_across_portions_and_in_a_used_slot(device, dtype, H, G, N, e):
    """the scan op alone against the token-by-token statement on the same (rounded) inputs: portions of 1, 2 and many tokens, a second
    sequence in a slot that the first has left, portions beside each other.  Steps are small, so that the first tokens still weigh
    at the end.  bfloat16: long portions run in blocks of 64 on the matrix cores, the longest in segments side by side."""
    g = torch.Generator().manual_seed(31)
    ops, T = R.ops_for(device), 330
    X, P, dtb, rate, D = _space_inputs(H, G, N, e, T, g, dtype)
    b0, c0, dt0 = H * e + (8 if H * e % 8 == 0 else 0), H * e + 8 + G * N, 8
    if b0 + G * N > c0:
        c0 = b0 + G * N
    xd, pd = X.double(), P.double()
    step = O.softplus(pd[:, dt0:dt0 + H] + dtb.double())

    def statement(lo, hi):
        return torch.stack([O.state_space(xd[lo:hi, h * e:(h + 1) * e], xd[lo:hi, b0 + h // (H // G) * N:][:, :N], xd[lo:hi, c0 + h // (H // G) * N:][:, :N],
                                          step[lo:hi, h], rate[h].double(), D[h].double())[0] for h in range(H)], 1)

    def scan(pool, parts):
        """parts: (slot, lo, hi) side by side in one batch"""
        meta = R.BatchMeta([(s, pool.len_of[s], hi - lo, []) for s, lo, hi in parts], torch.device(device))
        rows = torch.cat([torch.arange(lo, hi) for _, lo, hi in parts])
        y = ops.state_space_scan(X[rows].to(device).contiguous(), b0, c0, P[rows].to(device).contiguous(), dt0, dtb.to(device), rate.to(device),
                                 D.to(device), pool.matrix[0], H, G, N, e, meta).double().cpu().view(len(rows), H, e)
        for s, lo, hi in parts:
            pool.commit(s, hi - lo)
        return y

    pool = PagedStatePool({0: [("matrix", H, N, e)]}, 64, 2, dtype, device)
    want, other = statement(0, T), statement(100, 160)
    scale, tol = float(want.abs().max()), 2e-5 if dtype == torch.float32 or device == "cpu" else 1e-4
    for cuts in ([0, 1, 3, 40, 41, 43, 330], [0, 200, 201, 330], [0, 64, 192, 330], [0, 330], [0, 5, 330]):
        slot = pool.admit()
        got = torch.cat([scan(pool, [(slot, lo, hi)]) for lo, hi in zip(cuts, cuts[1:])])
        close(got / scale, want / scale, tol)
        pool.release(slot)
        slot = pool.admit()                                  # the same slot: its old state must not leak into a new sequence
        close(scan(pool, [(slot, 100, 160)]) / scale, other / scale, tol)
        pool.release(slot)
    a, b = pool.admit(), pool.admit()
    got = torch.cat([scan(pool, [(a, 0, 40), (b, 100, 101)])[:40], scan(pool, [(b, 101, 160), (a, 40, 330)])[59:]])
    close(got / scale, want / scale, tol)


@pytest.mark.parametrize("device", DEVICES)
def test_state_space_with_strong_decays_and_large_steps(device):
    """steps so large that a token's decay is nothing, next to tiny ones: no factor overflows, nothing leaks past a wiped state"""
    g = torch.Generator().manual_seed(35)
    ops, T, H, N, e = R.ops_for(device), 140, 2, 16, 32
    X, P, dtb, rate, D = _space_inputs(H, 1, N, e, T, g, torch.bfloat16)
    P[:, 8:8 + H] = torch.where(torch.rand(T, H, generator=g) < 0.15, torch.tensor(90.0), torch.tensor(-3.0)).to(torch.bfloat16)
    rate[:] = torch.tensor([3.0, 0.01])
    b0, c0 = H * e, H * e + N
    xd, step = X.double(), O.softplus(P[:, 8:8 + H].double() + dtb.double())
    want = torch.stack([O.state_space(xd[:, h * e:(h + 1) * e], xd[:, b0:b0 + N], xd[:, c0:c0 + N], step[:, h], rate[h].double(), D[h].double())[0]
                        for h in range(H)], 1)
    pool = PagedStatePool({0: [("matrix", H, N, e)]}, 64, 1, torch.bfloat16, device)
    meta = R.BatchMeta([(pool.admit(), 0, T, [])], torch.device(device))
    got = ops.state_space_scan(X.to(device), b0, c0, P.to(device), 8, dtb.to(device), rate.to(device), D.to(device), pool.matrix[0], H, 1, N, e,
                               meta).double().cpu().view(T, H, e)
    assert bool(torch.isfinite(got).all())
    for h in range(H):
        close(got[:, h] / want[:, h].abs().max(), want[:, h] / want[:, h].abs().max(), 1e-4)


# ------------------------------------------------------------------------------------------------ norms, router, experts
@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("D", [48, 50, 1000, 1026, 2000, 4000, 4100])
def test_joined_outputs_and_the_two_norms(device, D):
    """the stream's update from one mixer's output, from two normed ones, with and without a feed-forward, and both operands, at every
    width's code path"""
    g = torch.Generator().manual_seed(43)
    ops, eps, rows = R.ops_for(device), 1e-4, 5
    x, y, y2, ya, yb = (torch.randn(rows, D, generator=g) * s for s in (2.0, 3.0, 0.5, 0.01, 40.0))
    wa, wb, w1, w2 = (1 + torch.randn(D, generator=g) for _ in range(4))
    dev = lambda t: None if t is None else t.clone().to(device)          # noqa: E731
    for first, second, side in ((None, None, False), (y, None, False), (y, y2, False), (None, y2, True), (None, None, True)):
        new = x.double()
        for t in (first, second):
            new = new if t is None else new + t.double()
        if side:
            new = new + 0.5 * (O.rms(ya.double(), eps, wa.double()) + O.rms(yb.double(), eps, wb.double()))
        for wn1, wn2 in ((w1, w2), (w1, None), (None, None)):
            xs = dev(x)
            u1, u2 = ops.join_norms(xs, dev(first), dev(second), (dev(ya), dev(yb), dev(wa), dev(wb), 0.5) if side else None, dev(wn1), dev(wn2), eps,
                                    torch.float32)
            close(xs.double().cpu(), new, 1e-4)
            for u, w in ((u1, wn1), (u2, wn2)):
                assert (u is None) == (w is None)
                if w is not None:
                    close(u.double().cpu(), O.rms(new, eps, w.double()), 1e-4)


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("n,groups", [(48, 1), (48, 4), (90, 6), (2048, 2), (4096, 1), (9000, 2), (5001, 1)])
def test_gate_before_the_grouped_norm(device, n, groups):
    g = torch.Generator().manual_seed(45)
    ops, eps, rows, z0 = R.ops_for(device), 1e-4, 4, 4
    y, P, w = torch.randn(rows, n, generator=g), torch.randn(rows, n + 4, generator=g) * 3, 1 + torch.randn(n, generator=g)
    y[:, : n // groups] *= 30.0                              # a part of its own size: its neighbours must not feel it
    want = O.grouped_norm(y.double() * O.silu(P[:, z0:].double()), groups, eps, w.double())
    close(ops.gate_group_norm(y.to(device), P.to(device), z0, w.to(device), groups, eps, torch.float32).double().cpu(), want, 1e-4)


@pytest.mark.parametrize("device", DEVICES)
def test_normed_embedding_rows(device):
    g = torch.Generator().manual_seed(47)
    ops = R.ops_for(device)
    table, w = torch.randn(9, 300, generator=g) * 5, 1 + torch.randn(300, generator=g)
    ids = torch.tensor([0, 8, 3, 3])
    got = ops.embed_rows(ids.to(device), table.to(device), norm=w.to(device), eps=1e-3)
    close(got.double().cpu(), O.rms(table[ids].double(), 1e-3, w.double()), 1e-5)


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("E,groups,keep,top", [(12, 3, 2, 4), (8, 1, 1, 2), (6, 6, 2, 2), (6, 2, 1, 3), (96, 8, 2, 7), (5, 1, 1, 5), (130, 13, 4, 9)])
def test_choice_by_corrected_scores(device, E, groups, keep, top):
    """corrections of either sign decide who is chosen -- with all corrected scores negative too, where the experts of dropped groups
    must still lose -- but not the weights; the row of the shared expert's gate"""
    g = torch.Generator().manual_seed(49)
    ops, T, D = R.ops_for(device), 300 if E == 12 else 40, 36     # (many rows and few rows are different launches)
    x, wr, wg = torch.randn(T, D, generator=g), torch.randn(E, D, generator=g) / 6, torch.randn(D, generator=g) / 6
    for shift in (-3.0, 0.0, 0.4):
        corr = shift + 0.5 * torch.randn(E, generator=g)
        idx, wts, gate = ops.moe_route(x.to(device), wr.to(device), groups, keep, top, 1.0, "sigmoid", 2, False, correction=corr.to(device),
                                       w_gate=wg.to(device))
        s = O.sigmoid(x.double() @ wr.double().T)
        close(gate.double().cpu(), O.sigmoid(x.double() @ wg.double()), 1e-6)
        for t in range(T):
            want = O.choose(s[t], corr.double(), top, groups, keep)
            got = idx[t].tolist()
            assert sorted(got) == sorted(want), (t, got, want)
            close(wts[t].double().cpu(), s[t, got], 1e-6)
    plain = ops.moe_route(x.to(device), wr.to(device), groups, keep, top, 1.0, "sigmoid", 2)
    zero = ops.moe_route(x.to(device), wr.to(device), groups, keep, top, 1.0, "sigmoid", 2, correction=torch.zeros(E, device=device))
    assert len(plain) == len(zero) == 2 and torch.equal(plain[0], zero[0]) and torch.equal(plain[1], zero[1])


@pytest.mark.parametrize("device", DEVICES)
def test_a_dropped_group_loses_even_with_the_best_expert(device):
    """one group has the single best expert, another the best pair: pairs decide, and the dropped group's expert is out although every
    score that stays is negative"""
    ops = R.ops_for(device)
    z = torch.tensor([[3.0, -9.0, 1.0, 0.9, 0.2, 0.1]])      # groups (0, 1), (2, 3), (4, 5)
    corr = torch.full((6,), -5.0)
    idx, wts = ops.moe_route(z.to(device), torch.eye(6).to(device), 3, 1, 2, 1.0, "sigmoid", 2, correction=corr.to(device))
    assert sorted(idx[0].tolist()) == [2, 3]
    close(wts.sort().values.double().cpu(), O.sigmoid(torch.tensor([[0.9, 1.0]], dtype=O.F64)), 1e-6)
    corr[0] = 4.0                                            # a correction can bring it back; the weight stays the score
    idx, wts = ops.moe_route(z.to(device), torch.eye(6).to(device), 3, 1, 1, 1.0, "sigmoid", 2, correction=corr.to(device))
    assert idx.tolist() == [[0]]
    close(wts.double().cpu(), O.sigmoid(torch.tensor([[3.0]], dtype=O.F64)), 1e-6)


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
def test_experts_of_short_and_long_portions(device, dtype):
    """rows served one by one, experts as products over sorted rows and (bfloat16) as grouped products, with the gated shared expert,
    against the statement"""
    cfg = O.make_config([O.parallel_layer(ff=16, moe=MOE)], width=48)
    W = O.random_weights(cfg, seed=51)
    eng = engine_for(cfg, W, dtype, device)
    f, lt = eng.cfg.mlps[0], eng.layers[0]
    g = torch.Generator().manual_seed(53)
    for T in (1, 3, 40, 100):
        x = torch.randn(T, 48, generator=g).to(dtype)
        want = O.experts_ff(x.double(), W, "l0.mlp.", cfg["layers"][0]["mlp"])
        got = eng._experts(f, lt, x.to(device), R.BatchMeta([(0, 0, T, [0, 1])], torch.device(device))).double().cpu()
        tol = 1e-4 if dtype == torch.float32 else 0.03
        close(got / want.abs().max(), want / want.abs().max(), tol)


# ------------------------------------------------------------------------------------------------ configuration
def test_what_every_layer_keeps_and_what_is_refused():
    cfg = full_model()
    eng = engine_for(cfg, O.random_weights(cfg, 1), torch.float32, "cpu")
    kinds = [sorted(s[0] for s in v) for v in eng.state_specs().values()]
    assert kinds == [["kv", "matrix", "tail"], ["matrix", "tail"]] * 3
    one = O.make_config([O.parallel_layer(conv=1), O.mamba2_layer(conv=1)])
    eng = engine_for(one, O.random_weights(one, 1), torch.float32, "cpu")
    assert [sorted(s[0] for s in v) for v in eng.state_specs().values()] == [["kv", "matrix"], ["matrix"]]
    assert eng.weight_bytes() > 0 and eng.cfg.logit_scale == 0.3
    with pytest.raises(ValueError):
        lifenex.read_config(dict(O.plain_config(cfg), layers=[dict(cfg["layers"][0], type="conv")]))
    with pytest.raises(ValueError):
        lifenex.read_config(dict(O.plain_config(cfg), layers=[dict(cfg["layers"][0], mlp={"kind": "wide"})]))


@pytest.mark.parametrize("device", DEVICES)
def test_example_model_steps(device):
    cfg = lifenex.example_config(width=64, layers=3, heads=4, kv_heads=2, dim=16, ff=96, vocab=70, bias_max=50, temp=(0.2, 16), delta_heads=4,
                                 delta_kv_heads=2, delta_dim=16, delta_vdim=24, ssm_heads=4, ssm_vdim=16, ssm_state=16, ssm_groups=2, norm_groups=2,
                                 expert_ff=16, experts=8, top=2, groups=4, keep=2, shared_ff=24)
    sd = lifenex.random_state_dict(cfg, device, seed=3, rel_rows=10, low_rank=12)
    eng = lifenex.build_engine(lifenex.read_config(cfg), sd, torch.float32, device)
    W = {k: v.double().cpu() for k, v in sd.items()}
    toks = O.random_tokens(70, 70, 4)
    close(run_schedule(eng, {"a": toks}, [[("a", 68)], [("a", 1)], [("a", 1)]], 128)["a"], O.forward(toks, W, cfg))


# ------------------------------------------------------------------------------------------------ entry points
def _save_checkpoint(tmp_path, cfg, W):
    from safetensors.torch import save_file
    path = str(tmp_path / "model")
    os.makedirs(path, exist_ok=True)
    with open(os.path.join(path, "config.json"), "w") as f:
        json.dump(O.plain_config(cfg), f)
    save_file({k: v.to(torch.bfloat16).contiguous() for k, v in W.items()}, os.path.join(path, "model.safetensors"))
    return path


def _greedy_is_consistent(cfg, W, sequence, n_prompt):
    """every generated token is the oracle's argmax given what came before it, or within a rounding-sized gap of it"""
    logits = O.forward(sequence[:-1], W, cfg)
    for t in range(n_prompt, len(sequence)):
        row = logits[t - 1]
        assert float(row.max() - row[sequence[t]]) < 1e-3, f"token {t}"


@pytest.mark.parametrize("device", DEVICES)
def test_greedy_generation_through_the_auto_class_and_the_scheduler(device, tmp_path):
    from bigdl_amd.serving.continuous import ContinuousBatcher, SeqRequest
    from bigdl_amd.transformers import AutoModelForCausalLM
    cfg = full_model()
    W = O.random_weights(cfg, seed=61)
    path = _save_checkpoint(tmp_path, cfg, W)
    model = AutoModelForCausalLM.from_pretrained(path).to(device, torch.float32)
    prompts = torch.tensor([O.random_tokens(9, cfg["vocab"], 62), O.random_tokens(9, cfg["vocab"], 63)])
    out = model.generate(prompts, max_new_tokens=10)
    assert out.shape == (2, 19) and bool((out[:, :9] == prompts).all())
    for row in out.tolist():
        _greedy_is_consistent(cfg, W, row, 9)
    # more requests than slots, a pool that cannot hold them all at once, prompts longer than the per-step budget
    cb = ContinuousBatcher(model.engine, max_num_seqs=2, max_seq_len=128, max_prefill_tokens=24, max_live_tokens=192)
    reqs = [cb.submit(SeqRequest(str(i), O.random_tokens(n, cfg["vocab"], 70 + i), max_new_tokens=m))
            for i, (n, m) in enumerate([(70, 6), (3, 12), (30, 4), (1, 9), (50, 5)])]
    cb.run_until_done(500)
    assert all(r.finished and len(r.output_ids) == r.max_new_tokens for r in reqs)
    assert cb.mixed_steps > 0 and not cb.pool.len_of and len(cb.pool.free_pages) == cb.pool.num_pages
    for r in reqs:
        _greedy_is_consistent(cfg, W, r.input_ids + r.output_ids, len(r.input_ids))


def test_command_line_and_sampling(tmp_path, capsys):
    """``llm-cli --prompt-ids`` on a checkpoint without a tokenizer (greedy), and sampled generation through the same
    scheduler: with a fixed seed it repeats itself, and top_k = 1 is the greedy answer"""
    from bigdl_amd.cli import llm_cli
    from bigdl_amd.transformers import AutoModelForCausalLM
    cfg = O.make_config([O.parallel_layer(ff=16, moe=MOE), O.mamba2_layer()])
    W = O.random_weights(cfg, seed=91)
    path = _save_checkpoint(tmp_path, cfg, W)
    prompt = O.random_tokens(11, cfg["vocab"], 92)
    model = AutoModelForCausalLM.from_pretrained(path).to("cpu", torch.float32)
    greedy = model.generate(torch.tensor([prompt]), max_new_tokens=7)[0].tolist()
    _greedy_is_consistent(cfg, W, greedy, len(prompt))
    assert model.generate(torch.tensor([prompt]), max_new_tokens=7, do_sample=True, top_k=1)[0].tolist() == greedy
    torch.manual_seed(3)
    a = model.generate(torch.tensor([prompt]), max_new_tokens=7, do_sample=True, temperature=1.5)[0].tolist()
    torch.manual_seed(3)
    assert model.generate(torch.tensor([prompt]), max_new_tokens=7, do_sample=True, temperature=1.5)[0].tolist() == a
    if torch.cuda.is_available():
        return                                               # (the command line would take the GPU: covered by the gpu tests)
    served = AutoModelForCausalLM.from_pretrained(path).to("cpu").generate(torch.tensor([prompt]), max_new_tokens=7)[0].tolist()
    llm_cli.main(["-m", path, "--prompt-ids", " ".join(map(str, prompt)), "-n", "7"])     # (the default type: bfloat16)
    assert capsys.readouterr().out.split()[-7:] == [str(t) for t in served[len(prompt):]]


def test_trace_runner_replays_steps(tmp_path):
    import subprocess
    import sys
    import numpy as np
    cfg = full_model()
    W = O.random_weights(cfg, seed=81)
    path = _save_checkpoint(tmp_path, cfg, W)
    toks = O.random_tokens(20, cfg["vocab"], 82)
    steps = [{"step": 0, "entries": [{"id": "x", "tokens": toks[:13], "want": [0, 12]}], "end": []},
             {"step": 1, "entries": [{"id": "x", "tokens": toks[13:15], "want": []}, {"id": "y", "tokens": toks[:3], "want": [2]}],
              "end": ["y"]},
             {"step": 2, "entries": [{"id": "x", "tokens": toks[15:], "want": [4]}], "end": ["x"]}]
    root = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
    out = str(tmp_path / "out")
    r = subprocess.run([sys.executable, os.path.join(root, "bin", "trace_run"), "--model", path, "--dtype", "float32", "--out", out,
                        "--max-tokens", "128", "--device", "cpu"], input="\n".join(json.dumps(s) for s in steps) + "\n",
                       capture_output=True, text=True, timeout=300)
    assert r.returncode == 0, r.stderr
    assert [l for l in r.stdout.splitlines() if l.startswith("done")] == ["done 0", "done 1", "done 2"]
    want = O.forward(toks, W, cfg)
    for step, rows in ((0, [0, 12]), (1, [2]), (2, [19])):
        got = torch.from_numpy(np.fromfile(os.path.join(out, f"{step}.f32"), dtype="<f4")).view(len(rows), -1).double()
        close(got, want[rows])
