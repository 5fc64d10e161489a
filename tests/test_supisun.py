"""The Supisun design on the ragged engine against the plain float64 statement in ``supisun_oracle.py``.

Every test runs twice: on the CPU (the engine's bookkeeping over the unfused statements of ``ops/ragged.py``) and,
marked ``gpu``, on the device (the HIP kernels of ``libbigdl_ragged.so``).  Models are small and random; where random
weights would hide a fault (one key among many, a block's edge, a page's border, a decayed state) the inputs are made so
that it shows.
"""
import json
import math
import os
import random

import pytest
import torch

import supisun_oracle as O
from bigdl_amd.models import supisun
from bigdl_amd.models.paged import PagedStatePool
from bigdl_amd.ops import ragged as R

DEVICES = ["cpu", pytest.param("cuda", marks=pytest.mark.gpu)]
F32_TOL = 3e-4


def engine_for(config, W, dtype, device):
    return supisun.build_engine(supisun.read_config(config), W, dtype, device)


def full_model():
    """all three kinds of layers, two without a feed-forward; the first mixing layer is not the first attention layer, and an
    attention layer between the mixing ones keeps its values to itself"""
    return O.make_config([O.delta_layer(), O.attention_layer(heads=3, kv_heads=3, dim=10, vdim=6, chunk=20, rot=(10, 50.0), v_mix=False, ff=None),
                          O.attention_layer(chunk=9), O.mamba_layer(), O.attention_layer(heads=2, kv_heads=1, dim=8, vdim=24, chunk=70, v_mix=False),
                          O.delta_layer(heads=3, kv_heads=1, dim=10, vdim=6, conv=5, ff=None),
                          O.attention_layer(heads=4, kv_heads=2, dim=12, vdim=24, chunk=33, rot=(6, 1000.0))])


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
@pytest.mark.parametrize("layers,taps", [
    ([O.attention_layer()], 4),
    ([O.mamba_layer()], 4),
    ([O.delta_layer()], 4),
    ([O.attention_layer(heads=1, kv_heads=1, dim=8, vdim=12, chunk=1, rot=(8, 7.0), ff=None)], 1),        # blocks of one position
    ([O.attention_layer(heads=6, kv_heads=6, dim=12, vdim=10, chunk=64, rot=None, v_mix=False)], 2),      # blocks that are pages
    ([O.attention_layer(heads=8, kv_heads=1, dim=32, vdim=136, chunk=65, rot=(2, 1e4))], 3),              # values wider than keys
    ([O.attention_layer(heads=2, kv_heads=2, dim=16, vdim=16, chunk=None)] * 3, 4),                       # no blocks, mixed twice
    ([O.attention_layer(heads=5, kv_heads=5, dim=7, vdim=3, chunk=11, rot=(4, 30.0), scale=0.9)] * 2, 7), # odd sizes
    ([O.mamba_layer(inner=24, state=1, dt_rank=1, conv=1, ff=None)], 4),
    ([O.mamba_layer(inner=70, state=16, dt_rank=5, conv=2)] * 2, 2),
    ([O.mamba_layer(inner=33, state=37, dt_rank=2, conv=6)], 5),
    ([O.delta_layer(heads=1, kv_heads=1, dim=24, vdim=24, conv=1, ff=None)], 4),
    ([O.delta_layer(heads=6, kv_heads=6, dim=40, vdim=7, conv=4)], 1),
    ([O.delta_layer(heads=4, kv_heads=1, dim=5, vdim=33, conv=2), O.delta_layer(heads=1, kv_heads=1, dim=70, vdim=130, conv=4)], 4),
])
def test_each_layer_kind_alone(device, layers, taps):
    cfg = O.make_config(layers, taps=taps)
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
    for t in range(30, 40):                                  # a step of single tokens joins the norm with the next convolution
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
    for sizes in ([2] * 75, [64, 2, 62, 3, 1, 1, 17], [63, 1, 1, 63, 2, 20], [5, 128, 2, 2, 13], [1, 2, 3, 4, 5, 64, 65, 6],
                  [9, 1, 8, 2, 70, 60]):
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
def test_long_decoding_past_blocks_and_pages(device):
    cfg = O.make_config([O.attention_layer(chunk=16), O.mamba_layer(), O.attention_layer(chunk=70, ff=None), O.delta_layer()])
    W = O.random_weights(cfg, seed=9)
    toks = O.random_tokens(200, cfg["vocab"], 11)
    want = O.forward(toks, W, cfg)
    eng = engine_for(cfg, W, torch.float32, device)
    got = run_schedule(eng, {"a": toks}, [[("a", 5)]] + [[("a", 1)] for _ in range(195)], 256)["a"]
    close(got, want)


@pytest.mark.parametrize("device", DEVICES)
def test_long_portions_run_the_recurrences_in_chunks(device):
    """portions of several hundred tokens (both recurrences are cut into chunks that are scanned side by side and chained)
    beside a short one and a single token, into states that earlier portions have left"""
    cfg = O.make_config([O.mamba_layer(inner=48, state=20), O.delta_layer(heads=4, kv_heads=2, dim=24, vdim=40, ff=None),
                         O.attention_layer(chunk=150, ff=None)])
    W = O.random_weights(cfg, seed=15)
    for li, name in ((0, "dt.b"), (1, "dt_bias")):           # slow decays: what an early chunk wrote reaches the last one
        W[f"l{li}.mix.{name}"] = W[f"l{li}.mix.{name}"] - 4.0
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
        layers = [O.attention_layer(heads=3, kv_heads=1, dim=18, vdim=14, chunk=30, rot=(6, 90.0)), O.mamba_layer(inner=35, state=5, dt_rank=3),
                  O.attention_layer(heads=6, kv_heads=1, dim=10, vdim=14, chunk=17), O.delta_layer(heads=3, kv_heads=1, dim=17, vdim=9)]
    else:            # sizes that the vector and matrix-core paths serve
        layers = [O.attention_layer(heads=4, kv_heads=2, dim=32, vdim=32, chunk=40, rot=(16, 1e4)), O.mamba_layer(inner=128, state=16, dt_rank=8),
                  O.attention_layer(heads=8, kv_heads=2, dim=64, vdim=32, chunk=64), O.delta_layer(heads=4, kv_heads=2, dim=32, vdim=32, conv=4)]
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
    layers = []
    mix_kv, mix_vdim = rnd.choice([1, 2, 3]), rnd.choice([8, 16, 20, 48, 80])
    for _ in range(rnd.randint(3, 5)):
        kind = rnd.choice(["attention", "attention", "mamba1", "delta"])
        ff = rnd.choice([None, 24, 56])
        if kind == "attention":
            mix = rnd.random() < 0.7
            kv = mix_kv if mix else rnd.choice([1, 2])
            dim = rnd.choice([8, 12, 16, 24, 40, 48, 64])
            rot = rnd.choice([None, (rnd.choice([2, 4, 8]), rnd.choice([100.0, 1e4, 5e5])), (dim, 77.0)])
            layers.append(O.attention_layer(heads=kv * rnd.choice([1, 2, 4]), kv_heads=kv, dim=dim, vdim=mix_vdim if mix else 12,
                                            chunk=rnd.choice([1, 5, 33, 64, 100, 150]), rot=rot, v_mix=mix, ff=ff,
                                            scale=rnd.choice([0.5, 1.0, 2.0]) * dim ** -0.5))
        elif kind == "mamba1":
            layers.append(O.mamba_layer(inner=rnd.choice([24, 50, 128]), state=rnd.choice([1, 4, 8, 16, 24, 32]), dt_rank=rnd.randint(1, 9),
                                        conv=rnd.choice([1, 2, 4, 5]), ff=ff))
        else:
            kv = rnd.choice([1, 2, 3])
            layers.append(O.delta_layer(heads=kv * rnd.choice([1, 2, 3]), kv_heads=kv, dim=rnd.choice([8, 16, 32, 40, 72]),
                                        vdim=rnd.choice([8, 20, 48, 64, 96]), conv=rnd.choice([1, 2, 4, 5]), ff=ff))
    return O.make_config(layers, width=rnd.choice([24, 40, 64]), vocab=rnd.choice([50, 67, 128]), taps=rnd.choice([1, 2, 3, 4, 6]),
                         eps=rnd.choice([1e-5, 1e-6, 1e-3]), max_positions=rnd.choice([140, 200]))


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
    for k in prompts:
        rel = _relative(got[k], want[k])                     # (a head or row that is nearly zero in front of its norm is ill-conditioned)
        assert float(rel.median()) < 0.06 and float(rel.quantile(0.95)) < 0.25, (k, float(rel.median()), float(rel.quantile(0.95)))


# ------------------------------------------------------------------------------------------------ mechanisms alone
def _attend_through_pages(device, q, k, v, portions, *, scale, chunk, page_order=None, dtype=torch.float32):
    """q [T, H, d], k [T, G, d], v [T, G, e] (float64) through the paged attention op in the given portions"""
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
                                  chunk=chunk or 0))
        pool.commit(slot, n)
        at += n
    return torch.cat(out).double().cpu().view(T, H, e)


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("decoded", [False, True])
@pytest.mark.parametrize("chunk", [70, 64, 16, 128, 1, 129, 37, None])
def test_block_edges_far_keys_and_page_borders_stand_out(device, decoded, chunk):
    """Query i and key j are made parallel and long, so key j takes all of the weight when it is visible; its value is a
    marker.  One position off at a block's edge or at a page's border swaps the marker in or out.  Queries are part of a
    prompt's portion or decoded alone."""
    g = torch.Generator().manual_seed(21)
    T, H, G, d, e = 210, 2, 1, 12, 4
    cases = [(100, 63), (100, 64), (130, 127), (130, 128), (64, 63), (64, 64), (0, 0), (1, 0), (15, 0), (16, 0), (16, 15), (209, 0)]
    for i in (140, 191, 192, 193, 209, 69, 70, 127, 128):
        lo = i // chunk * chunk if chunk else 0              # the first key that i sees
        cases += [(i, lo), (i, lo - 1), (i, lo + 1), (i, i), (i, i - 1)]
    cases = sorted({(i, j) for i, j in cases if 0 <= j <= i})
    for i, j in cases:
        q = torch.randn(T, H, d, generator=g).double() * 0.3
        k = torch.randn(T, G, d, generator=g).double() * 0.3
        v = torch.randn(T, G, e, generator=g).double()
        direction = torch.randn(d, generator=g).double()
        direction /= direction.norm()
        q[i, :] = 9.0 * direction
        k[j, 0] = 9.0 * direction
        v[j, 0] = torch.tensor([100.0, -100.0, 50.0, 25.0], dtype=O.F64)
        portions = [n for n in ([i, 1, T - i - 1] if decoded else [i // 2, i + 1 - i // 2, T - i - 1]) if n]
        got = _attend_through_pages(device, q, k, v, portions, scale=1.0, chunk=chunk, page_order=[5, 0, 3, 1, 4, 2])
        want = _one_query(q, k, v, i, chunk)
        close(got[i], want, 2e-3)
        seen = j // chunk == i // chunk if chunk else True
        assert (float(want[0, 0]) > 50.0) == seen            # (the marker does decide)


def _one_query(q, k, v, i, chunk):
    js = [j for j in range(i + 1) if not chunk or j // chunk == i // chunk]
    return torch.stack([torch.softmax(k[js, 0] @ q[i, h], -1) @ v[js, 0] for h in range(q.shape[1])])


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("H,G,d,e,rot", [(4, 2, 16, 24, 8), (3, 3, 10, 6, 10), (8, 1, 64, 136, 0), (1, 1, 5, 1, 2), (6, 2, 128, 64, 128)])
def test_queries_keys_and_values_of_a_row(device, H, G, d, e, rot):
    """norms over whole projections, rotation, normed and mixed values, against the statement; what the pages hold is what the
    scores and the sum see"""
    g = torch.Generator().manual_seed(25)
    ops, T, past, eps, lam = R.ops_for(device), 21, 60, 1e-5, 0.37
    P = torch.randn(T, (H + G) * d + G * e, generator=g) * torch.tensor([0.2, 4.0])[torch.randint(0, 2, (T, 1), generator=g)]
    qw, kw = 1 + torch.randn(H * d, generator=g), 1 + torch.randn(G * d, generator=g)
    first = torch.randn(T, G * e, generator=g)
    pool = PagedStatePool({0: [("kv", G, d, e)]}, 192, 1, torch.float32, device)
    pool.free_pages = [1, 2, 0]
    slot = pool.admit()
    pool.reserve(slot, past)
    pool.commit(slot, past)
    pages = list(pool.reserve(slot, T))
    meta = R.BatchMeta([(slot, past, T, pages)], torch.device(device))
    from bigdl_amd.models.ragged_engine import rotary_inv_freq
    freq = rotary_inv_freq(rot, 50.0, 1.0).to(device) if rot else None
    pd = P.double()
    nq, nk = H * d, G * d
    q = (O.rms(pd[:, :nq], eps) * qw.double()).view(T, H, d)
    k = (O.rms(pd[:, nq:nq + nk], eps) * kw.double()).view(T, G, d)
    v = O.rms(pd[:, nq + nk:].view(T, G, e), eps)
    if rot:
        q, k = (torch.stack([O.turn_halves(u[t], past + t, rot, 50.0) for t in range(T)]) for u in (q, k))
    for mixed in (False, True):
        got, vals = ops.qkv_rows(P.to(device), qw.to(device), kw.to(device), eps, rot, freq, pool.k[0], pool.v[0], meta, H=H, G=G, d=d, vd=e,
                                 v_norm=True, first_in=first.to(device) if mixed else None, lam=lam, want_first=True)
        want_v = O.mix_values(v, first.double().view(T, G, e), lam) if mixed else v
        close(got.double().cpu().view(T, H, d), q, 1e-4)
        close(vals.double().cpu().view(T, G, e), want_v, 1e-5)
        for t in range(T):
            pg, at = pages[(past + t) // 64], (past + t) % 64
            close(pool.k[0][pg, :, at].double().cpu(), k[t], 1e-4)
            close(pool.v[0][pg, :, at].double().cpu(), want_v[t], 1e-5)
    ops.qkv_rows(P.to(device), qw.to(device), kw.to(device), eps, rot, freq, pool.k[0], pool.v[0], meta, H=H, G=G, d=d, vd=e)
    close(pool.v[0][pages[0], :, 63].double().cpu(), pd[3, nq + nk:].view(G, e), 1e-6)           # values as they came


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("D,taps", [(48, 4), (1000, 3), (2000, 4), (4000, 4), (3000, 1), (5000, 4), (4100, 6)])
def test_output_norm_and_the_convolved_stream(device, D, taps):
    """x + LN(y), alone and joined with the convolution of the stream for single tokens, every width's code path; sequences
    younger than the taps, in slots that older sequences have left full"""
    g = torch.Generator().manual_seed(43)
    ops, eps, slots = R.ops_for(device), 1e-4, 4
    w, b, cw = torch.randn(D, generator=g), torch.randn(D, generator=g), torch.randn(D, taps, generator=g)
    dev = lambda t: t.clone().to(device)                     # noqa: E731
    stream = {0: [], 2: [], 3: []}                           # slot -> its rows so far
    tail = dev(torch.randn(slots, taps - 1, D, generator=g)) if taps > 1 else None      # (left by sequences that are gone)
    starts = {0: 0, 2: 1, 3: 3}                              # the step in which a slot's sequence begins
    for step in range(7):
        rows = [s for s in stream if starts[s] <= step]
        x, y = torch.randn(len(rows), D, generator=g) * 2, 0.5 + torch.randn(len(rows), D, generator=g) * 3
        new = x.double() + O.layer_norm(y.double(), w.double(), b.double(), eps)
        meta = R.BatchMeta([(s, len(stream[s]), 1, [0]) for s in rows], torch.device(device))
        xs = dev(x)
        got = ops.ln_add(xs, dev(y), dev(w), dev(b), eps, torch.float32, cw=dev(cw), tail=tail, meta=meta)
        close(xs.double().cpu(), new, 1e-4)
        for i, s in enumerate(rows):
            stream[s].append(new[i])
            h = torch.stack(stream[s])
            close(got[i].double().cpu(), (h + O.causal_conv(h, cw.double()))[-1], 2e-4)
        xs = dev(x)
        close(ops.ln_add(xs, dev(y), dev(w), dev(b), eps, torch.float32).double().cpu(), new, 1e-4)
        close(xs.double().cpu(), new, 1e-4)
        xs = dev(x)
        close(ops.ln_add(xs, None, dev(w), dev(b), eps, torch.float32).double().cpu(), O.layer_norm(x.double(), w.double(), b.double(), eps), 1e-4)
        close(xs.cpu(), x, 0.0)
        xs = dev(x)
        assert ops.ln_add(xs, dev(y), dev(w), dev(b), eps, torch.float32, want=False) is None
        close(xs.double().cpu(), new, 1e-4)


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("taps", [1, 2, 3, 4, 7])
def test_convolution_of_rows_across_portions(device, taps):
    """column ranges behind a convolution with bias and silu, and plain sums with their input, in portions of 1, 2 and many rows
    of two sequences side by side, in slots with old contents"""
    g = torch.Generator().manual_seed(45)
    ops, C, c0, T = R.ops_for(device), 300, 5, 75
    cw, bias = torch.randn(C, taps, generator=g), torch.randn(C, generator=g)
    data = {0: torch.randn(T, C + 9, generator=g), 1: torch.randn(T, C + 9, generator=g)}
    tails = [torch.randn(3, taps - 1, C, generator=g).to(device) if taps > 1 else None for _ in range(2)]
    slot, at = {0: 2, 1: 0}, {0: 0, 1: 0}
    out = {0: [[], []], 1: [[], []]}
    for step in ([(0, 1)], [(0, 1), (1, 1)], [(0, 2), (1, 1)], [(1, 33), (0, 1)], [(0, 1), (1, 1)], [(0, 40), (1, 2)], [(0, 29), (1, 37)]):
        meta = R.BatchMeta([(slot[s], at[s], n, [0, 1]) for s, n in step], torch.device(device))
        rows = torch.cat([data[s][at[s]:at[s] + n] for s, n in step]).to(device)
        a = ops.conv_rows(rows, c0, cw.to(device), bias.to(device), tails[0], meta, torch.float32, silu=True).double().cpu()
        b = ops.conv_rows(rows, c0, cw.to(device), None, tails[1], meta, torch.float32, add=True).double().cpu()
        r = 0
        for s, n in step:
            out[s][0].append(a[r:r + n])
            out[s][1].append(b[r:r + n])
            r += n
            at[s] += n
    for s in (0, 1):
        assert at[s] == T
        u = data[s][:, c0:c0 + C].double()
        close(torch.cat(out[s][0]), O.silu(O.causal_conv(u, cw.double(), bias.double())), 1e-4)
        close(torch.cat(out[s][1]), u + O.causal_conv(u, cw.double()), 1e-4)


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("C,N", [(40, 6), (300, 16), (17, 1), (64, 33), (5, 70), (9, 300)])
def test_selective_scan_across_portions_and_in_a_used_slot(device, C, N):
    """the scan op alone against the token-by-token statement: portions of 1, 2 and many tokens, a second sequence in a slot that
    the first has left, and long portions that are scanned in chunks.  Steps are small, so that the first tokens still weigh at
    the end."""
    g = torch.Generator().manual_seed(31)
    ops, T = R.ops_for(device), 330
    x, z, M = torch.randn(T, C, generator=g), torch.randn(T, C + 3, generator=g), torch.randn(T, 2 * N + 4, generator=g)
    dt, dtb, D = torch.randn(T, C, generator=g), torch.randn(C, generator=g) - 5.0, torch.randn(C, generator=g)
    A = -torch.exp(0.5 * torch.randn(C, N, generator=g))
    A2 = (A.double() / math.log(2.0)).float().to(device)
    step = O.softplus(dt.double() + dtb.double())
    f64 = lambda t: t.double()                               # noqa: E731

    def statement(lo, hi):
        y, _ = O.selective_scan(f64(x[lo:hi]), step[lo:hi], f64(A), f64(M[lo:hi, 3:3 + N]), f64(M[lo:hi, 4 + N:]), f64(D))
        return y * O.silu(f64(z[lo:hi, 3:]))

    def scan(pool, slot, lo, hi):
        meta = R.BatchMeta([(slot, pool.len_of[slot], hi - lo, [])], torch.device(device))
        y = ops.selective_scan(x[lo:hi].to(device).contiguous(), dt[lo:hi].to(device).contiguous(), dtb.to(device), M[lo:hi].to(device), 3,
                               4 + N, A2, D.to(device), z[lo:hi].to(device), 3, pool.matrix[0], meta)
        pool.commit(slot, hi - lo)
        return y.double().cpu()

    pool = PagedStatePool({0: [("matrix", 1, C, N)]}, 64, 1, torch.float32, device)
    want = statement(0, T)
    scale = float(want.abs().max())
    for cuts in ([0, 1, 3, 40, 41, 43, 330], [0, 200, 201, 330], [0, 330], [0, 5, 133, 135, 300, 330]):
        slot = pool.admit()
        got = torch.cat([scan(pool, slot, lo, hi) for lo, hi in zip(cuts, cuts[1:])])
        close(got / scale, want / scale, 2e-5)
        pool.release(slot)
        slot = pool.admit()                                  # the same slot: its old state must not leak into a new sequence
        close(scan(pool, slot, 100, 160) / scale, statement(100, 160) / scale, 2e-5)
        pool.release(slot)


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("H,G,d,e,taps", [(4, 2, 16, 24, 4), (1, 1, 48, 8, 1), (3, 1, 40, 64, 3), (2, 2, 130, 33, 4), (6, 3, 5, 7, 2),
                                          (2, 1, 300, 20, 4), (2, 1, 128, 128, 4), (1, 1, 117, 16, 4), (2, 2, 64, 64, 4)])
def test_gated_delta_rule_across_portions_and_in_a_used_slot(device, H, G, d, e, taps):
    """preparation (convolutions, unit vectors, gates) and scan against the token-by-token statement: portions of 1, 2 and many
    tokens, a second sequence in the first one's slot, long portions in chunks, decays near one"""
    g = torch.Generator().manual_seed(33)
    ops, T = R.ops_for(device), 330
    C = 2 * G * d + H * e
    P = torch.randn(T, C + 2 * H + 3, generator=g)
    cw = torch.randn(C, taps, generator=g) * 0.6
    rate, dtb = torch.exp(torch.randn(H, generator=g) - 2.0), torch.randn(H, generator=g) - 3.0
    b0, a0 = C + 1, C + 2 + H

    def statement(lo, hi):
        u = O.silu(O.causal_conv(P[lo:hi, :C].double(), cw.double()))
        n = hi - lo
        q, k = O.unit(u[:, :G * d].view(n, G, d)) * d ** -0.5, O.unit(u[:, G * d:2 * G * d].reshape(n, G, d))
        v = u[:, 2 * G * d:].reshape(n, H, e)
        gd = torch.exp(-rate.double() * O.softplus(P[lo:hi, a0:a0 + H].double() + dtb.double()))
        beta = torch.sigmoid(P[lo:hi, b0:b0 + H].double())
        return torch.stack([O.gated_delta(q[:, h // (H // G)], k[:, h // (H // G)], v[:, h], gd[:, h], beta[:, h])[0] for h in range(H)], 1)

    def scan(pool, slot, lo, hi):
        meta = R.BatchMeta([(slot, pool.len_of[slot], hi - lo, [])], torch.device(device))
        qf, kf, v, gb = ops.gated_delta_prep(P[lo:hi].to(device).contiguous(), cw.to(device), taps, pool.tail.get(0), b0, a0, rate.to(device),
                                             dtb.to(device), O.UNIT_EPS, H, G, d, e, meta)
        out = ops.gated_delta_scan(qf, kf, gb, G, v, pool.matrix[0], H, d, e, meta)
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
def test_delta_rule_replaces_what_a_key_held(device):
    """write strength 1 and no decay: the second value under the same unit key replaces the first, and the read-out of a token
    sees that token's own write; half a decay scales what is left"""
    ops, d, e = R.ops_for(device), 8, 5
    k = torch.zeros(3, d)
    k[:, 3] = 1.0
    v = torch.stack([torch.arange(1.0, e + 1), -2 * torch.arange(1.0, e + 1), torch.zeros(e)])
    gb = torch.tensor([[[1.0, 1.0]], [[1.0, 1.0]], [[0.5, 0.0]]])
    pool = PagedStatePool({0: [("matrix", 1, d, e)]}, 64, 1, torch.float32, device)
    slot = pool.admit()
    meta = R.BatchMeta([(slot, 0, 3, [])], torch.device(device))
    out = ops.gated_delta_scan(k.to(device), k.to(device), gb.to(device), 1, v.to(device), pool.matrix[0], 1, d, e, meta).cpu()
    close(out, torch.stack([v[0], v[1], 0.5 * v[1]]), 1e-6)


@pytest.mark.parametrize("device", DEVICES)
def test_head_norm_with_a_silu_gate(device):
    g = torch.Generator().manual_seed(37)
    ops, T, H, e = R.ops_for(device), 7, 3, 70
    o, w, P = torch.randn(T, H * e, generator=g), torch.randn(e, generator=g), torch.randn(T, 4 + H * e, generator=g) * 3
    want = O.rms(o.double().view(T, H, e), 1e-5) * w.double() * O.silu(P[:, 4:].double()).view(T, H, e)
    got = ops.head_norm_gate(o.to(device), w.repeat(H).to(device), P.to(device), 4, H, e, 1e-5, torch.float32, gate="silu")
    close(got.double().cpu(), want.reshape(T, -1), 1e-4)


def test_what_every_layer_keeps_and_which_values_are_shared():
    cfg = full_model()
    eng = engine_for(cfg, O.random_weights(cfg, 1), torch.float32, "cpu")
    specs = eng.state_specs()
    kinds = [sorted(s[0] for s in specs[i]) for i in range(len(cfg["layers"]))]
    assert kinds == [["matrix", "stream_tail", "tail"], ["kv", "stream_tail"], ["kv", "stream_tail"], ["matrix", "stream_tail", "tail"],
                     ["kv", "stream_tail"], ["matrix", "stream_tail", "tail"], ["kv", "stream_tail"]]
    assert eng._v_first == 2
    one = O.make_config([O.delta_layer(conv=1), O.mamba_layer(conv=1)], taps=1)
    eng = engine_for(one, O.random_weights(one, 1), torch.float32, "cpu")
    assert [[s[0] for s in v] for v in eng.state_specs().values()] == [["matrix"], ["matrix"]] and eng._v_first is None
    bad = O.make_config([O.attention_layer(vdim=24), O.attention_layer(vdim=12)])
    with pytest.raises(ValueError):
        engine_for(bad, O.random_weights(bad, 1), torch.float32, "cpu")
    with pytest.raises(ValueError):
        supisun.read_config(dict(cfg, layers=[dict(cfg["layers"][0], type="conv")]))


@pytest.mark.parametrize("device", DEVICES)
def test_sequences_end_with_the_position_table(device):
    from bigdl_amd.serving.continuous import ContinuousBatcher, SeqRequest
    cfg = O.make_config([O.attention_layer(chunk=7), O.mamba_layer()], max_positions=30)
    W = O.random_weights(cfg, seed=51)
    eng = engine_for(cfg, W, torch.float32, device)
    toks = O.random_tokens(31, cfg["vocab"], 52)
    close(run_schedule(eng, {"a": toks[:30]}, [[("a", 20)], [("a", 9)], [("a", 1)]], 64)["a"], O.forward(toks[:30], W, cfg))
    eng.pool = None
    pool = eng.ensure_pool(64, 2)
    slot = pool.admit()
    with pytest.raises(ValueError):
        eng.step([(slot, toks)])
    assert not pool.pages_of[slot] and pool.len_of[slot] == 0          # nothing was taken or written
    eng.step([(slot, toks[:30])])
    with pytest.raises(ValueError):
        eng.step([(slot, toks[:1])])
    eng.pool = None
    cb = ContinuousBatcher(eng, max_num_seqs=2, max_seq_len=64)
    with pytest.raises(ValueError):
        cb.submit(SeqRequest("x", toks[:20], max_new_tokens=12))
    req = cb.submit(SeqRequest("y", toks[:20], max_new_tokens=11))
    cb.run_until_done(50)
    assert len(req.output_ids) == 11


# ------------------------------------------------------------------------------------------------ entry points
def _save_checkpoint(tmp_path, cfg, W):
    from safetensors.torch import save_file
    path = str(tmp_path / "model")
    os.makedirs(path, exist_ok=True)
    with open(os.path.join(path, "config.json"), "w") as f:
        json.dump(cfg, f)
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
    cfg = O.make_config([O.attention_layer(), O.mamba_layer(), O.delta_layer()])
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


# ------------------------------------------------------------------------------------------------ kernels of long bfloat16 portions
@pytest.mark.gpu
@pytest.mark.parametrize("H,G,d,e,chunk", [(4, 2, 64, 128, 100), (2, 2, 48, 48, 70), (3, 1, 16, 32, 64), (8, 2, 128, 64, 1), (8, 1, 40, 16, 33)])
def test_matrix_core_attention_in_blocks(H, G, d, e, chunk):
    """bfloat16 prompt portions (the MFMA kernel) and single tokens (the row-wise kernel) against the plain statement on
    the same bfloat16-rounded keys and values"""
    g = torch.Generator().manual_seed(71)
    T = 200
    q = torch.randn(T, H, d, generator=g).double()
    k = torch.randn(T, G, d, generator=g).bfloat16().double()
    v = torch.randn(T, G, e, generator=g).bfloat16().double()
    qr = q.clone()
    qr[:190] = q[:190].bfloat16().double()                   # the MFMA kernel rounds its queries
    want = O.attend(qr, k, v, 2.0 * d ** -0.5, chunk=chunk)
    got = _attend_through_pages("cuda", q, k, v, [120, 64, 3, 3] + [1] * 10, scale=2.0 * d ** -0.5, chunk=chunk, dtype=torch.bfloat16)
    assert float((got - want).abs().max()) < 0.03, float((got - want).abs().max())
