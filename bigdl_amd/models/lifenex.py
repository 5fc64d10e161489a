"""Lifenex on the ragged engine: reader of its ``config.json`` and the map from checkpoint tensor names to ``LayerTensors``.

The design: x = rms(embed[token]); per layer x <- x + mixer(rms1(x)) + ff(rms2(x)), both sublayers reading the same x through a norm
of their own; logits = logit_scale * embed rms(x), the embedding table itself being the output matrix.

Mixers (``type`` of a layer):

* ``mamba2``: state space layer with one decay per head (``StateSpace``);
* ``parallel``: two mixers side by side, half the sum of their outputs, each RMS-normed over the width with a weight.  Left: full causal
  attention with grouped key/value heads, queries and keys RMS-normed per head, no rotation; queries grow with the position
  (``q_temp``), a learned bias per head by distance joins the scores -- the table's first half of rows for the distances one by one, the
  others in logarithmic steps that end at ``bias_max`` -- and the normaliser holds exp(sink) of a learned number per head.  Right: a
  gated delta rule with one decay per head and key channel and a sigmoid gate, both through low-rank pairs (``GatedDelta``).

Feed-forward of a layer: W_down relu(W_up u)^2, a mixture of gated experts (sigmoid scores, choice in groups by corrected scores,
weights of the uncorrected ones as they are) with a gated shared expert, or none.
"""
from __future__ import annotations

import json
import math
import os

import torch

from .ragged_engine import (DenseMlp, GatedDelta, LayerTensors, RaggedConfig, RaggedDecoder, RoutedExperts, SideBySide, StateSpace,
                            WindowAttention)

ARCHITECTURE = "Lifenex"
UNIT_EPS = 1e-6                # fixed by the design: inside the root of a unit vector's length
GROUP_TOP = 2                  # a group of experts is worth the sum of its two best corrected scores
BRANCH_MIX = 0.5               # half the sum of the two normed outputs


def is_lifenex(config: dict) -> bool:
    return config.get("architecture") == ARCHITECTURE


def _side_by_side(m: dict) -> SideBySide:
    a, b = m["left"], m["right"]
    temp = a.get("q_temp")
    left = WindowAttention(heads=int(a["heads"]), kv_heads=int(a["kv_heads"]), dim=int(a["dim"]), vdim=int(a["vdim"]),
                           scale=float(a["scale"]), qk_norm=True, one_pass=True, head_sinks=True, dist_far=int(a["bias_max"]),
                           q_temp=(float(temp["coef"]), int(temp["every"])) if temp else None)
    right = GatedDelta(heads=int(b["heads"]), kv_heads=int(b["kv_heads"]), dim=int(b["dim"]), vdim=int(b["vdim"]),
                       conv_taps=int(b["conv"]), unit_eps=UNIT_EPS)
    return SideBySide(left, right, out_norms=True, mix=BRANCH_MIX)


def _feed_forward(f):
    if f is None:
        return None
    if f.get("kind") == "dense":
        return DenseMlp(ff=int(f["ff"]), act="relu2", bias=False)
    if f.get("kind") != "moe":
        raise ValueError(f"unknown feed-forward kind {f.get('kind')!r}")
    r, shared = f["router"], f.get("shared") or {}
    groups = r.get("groups") or {}
    count = int(groups.get("count", 1))
    return RoutedExperts(experts=int(r["experts"]), top=int(r["top"]), ff=int(f["expert"]["ff"]), groups=count,
                         keep=int(groups.get("keep", count)), score="sigmoid", group_top=GROUP_TOP, act="swiglu", correction=True,
                         shared_ff=int(shared.get("ff") or 0), shared_gate=bool(shared.get("ff")))


def read_config(config: dict) -> RaggedConfig:
    """(the ranks of the right mixer's low-rank pairs are tensor shapes, not config entries: ``build_engine`` fills them in)"""
    mixers, mlps = [], []
    for layer in config["layers"]:
        m, kind = layer["mixer"], layer["type"]
        if kind == "mamba2":
            mixers.append(StateSpace(heads=int(m["heads"]), vdim=int(m["vdim"]), state=int(m["state"]), groups=int(m["groups"]),
                                     norm_groups=int(m["norm_groups"]), conv_taps=int(m["conv"])))
        elif kind == "parallel":
            mixers.append(_side_by_side(m))
        else:
            raise ValueError(f"unknown layer type {kind!r}")
        mlps.append(_feed_forward(layer.get("mlp")))
    return RaggedConfig(vocab=int(config["vocab"]), width=int(config["width"]), mixers=mixers, mlps=mlps,
                        norm_eps=float((config.get("norm") or {}).get("eps", 1e-6)), name=ARCHITECTURE, block="parallel", two_norms=True,
                        embed_norm=True, logit_scale=float(config.get("logit_scale", 1.0)))


def distance_bucket(n: int, rows: int, far: int) -> int:
    """row of a bias table for distance ``n``: rows 0 .. rows // 2 - 1 belong to one distance each, the others to logarithmic steps
    up to ``far``; everything from ``far`` on has the last row"""
    half = rows // 2
    if n < half:
        return n
    if n >= far or half == 0:
        return rows - 1
    step = math.log(n / half) / math.log(far / half) * (rows - half)
    whole = round(step)                              # (a step that is a whole number must not fall below it by rounding)
    return min(rows - 1, half + (whole if abs(step - whole) < 1e-9 else math.floor(step)))


def distance_bias(rel: torch.Tensor, far: int) -> torch.Tensor:
    """float [heads, far + 1] by distance from the bias table [rows, heads]"""
    idx = torch.tensor([distance_bucket(n, rel.shape[0], far) for n in range(far + 1)], device=rel.device)
    return rel.float()[idx].t().contiguous()


def build_engine(cfg: RaggedConfig, sd: dict, dtype=torch.bfloat16, device="cuda") -> RaggedDecoder:
    """``sd``: checkpoint tensors by name ('l<i>.mix.left.q', 'l<i>.mlp.e<j>.gate', ...).  Projection and expert weights take the
    activation type; norm weights, router rows, sinks, distance biases, convolution taps and everything of the recurrences become
    float32 (what reads them computes in 32 bits)."""
    dev = torch.device(device)

    def act(*names):
        return torch.cat([sd[n] for n in names], 0).to(dev, dtype).contiguous()

    def f32(name):
        return sd[name].float().reshape(-1).to(dev).contiguous()

    def taps(*names):
        return torch.cat([sd[n].float() for n in names], 0).to(dev).contiguous()

    def padded(t, rows):                             # zero rows at the end
        return torch.cat([t, torch.zeros(rows - t.shape[0], t.shape[1], dtype=t.dtype, device=t.device)], 0).contiguous()

    def up8(n):
        return (n + 7) // 8 * 8

    def low_rank(first, second):
        """(first [rank, width], second [n, rank]) with the rank filled up by zeros to a multiple of eight: rows of 16 bytes"""
        a, b = act(first), act(second)
        r = up8(a.shape[0])
        return padded(a, r), padded(b.t().contiguous(), r).t().contiguous()

    def gate_up(p):                                  # gate and up rows of an inner channel next to each other
        return torch.stack([sd[p + "gate"], sd[p + "up"]], 1).reshape(-1, cfg.width)

    layers = []
    for li, (m, mlp) in enumerate(zip(cfg.mixers, cfg.mlps)):
        l, p, q = f"l{li}.", f"l{li}.mix.", f"l{li}.mlp."
        if isinstance(m, StateSpace):
            w_in = act(p + "in")
            lt = LayerTensors(w_in=padded(w_in, up8(w_in.shape[0])), w_out=act(p + "o"), norm1=None, conv_w=taps(p + "conv"),
                              conv_b=f32(p + "conv.b"), dt_bias=f32(p + "dt_bias"), decay_rate=torch.exp(f32(p + "A_log")),
                              ssm_d=f32(p + "D"), o_norm=f32(p + "norm"))
        else:
            a, b = p + "left.", p + "right."
            w_in = act(a + "q", a + "k", a + "v")
            left = LayerTensors(w_in=padded(w_in, up8(w_in.shape[0])), w_out=act(a + "o"), norm1=None, q_norm=f32(a + "q.norm"),
                                k_norm=f32(a + "k.norm"), sinks=f32(a + "sink"),
                                dist_bias=distance_bias(sd[a + "rel"].to(dev), m.left.dist_far), out_norm=f32(a + "out"))
            (a1, a2), (g1, g2) = low_rank(b + "a1", b + "a2"), low_rank(b + "g1", b + "g2")
            m.right.decay_rank, m.right.gate_rank = a1.shape[0], g1.shape[0]
            w_in = torch.cat([act(b + "q", b + "k", b + "v"), a1, g1, act(b + "b")], 0)
            right = LayerTensors(w_in=padded(w_in, up8(w_in.shape[0])), w_out=act(b + "o"), norm1=None,
                                 conv_w=taps(*[b + n + ".conv" for n in ("q", "k", "v")]), decay_rate=torch.exp(f32(b + "A_log")),
                                 decay_bias=f32(b + "dt_bias"), w_decay=a2, w_gate=g2,
                                 o_norm=f32(b + "norm").repeat(m.right.heads).contiguous(), out_norm=f32(b + "out"))
            lt = LayerTensors(w_in=torch.cat([left.w_in, right.w_in], 0).contiguous(), w_out=None, norm1=None, left=left, right=right)
        lt.norm1 = f32(l + "norm1")
        if mlp is not None:
            lt.norm2 = f32(l + "norm2")
        if isinstance(mlp, DenseMlp):
            lt.w_ff, lt.w_down = act(q + "up"), act(q + "down")
        elif isinstance(mlp, RoutedExperts):
            lt.w_router, lt.correction = sd[q + "router"].float().to(dev).contiguous(), f32(q + "correction")
            lt.w_up = torch.stack([gate_up(q + f"e{e}.") for e in range(mlp.experts)]).to(dev, dtype).contiguous()
            lt.w_dn = torch.stack([sd[q + f"e{e}.down"] for e in range(mlp.experts)]).to(dev, dtype).contiguous()
            if mlp.shared_ff:
                lt.w_sup, lt.w_sdn = gate_up(q + "shared.").to(dev, dtype).contiguous(), act(q + "shared.down")
                lt.w_sgate = f32(q + "shared.sg")
        layers.append(lt)
    embed = act("embed")
    return RaggedDecoder(cfg, embed, layers, f32("final.norm"), embed, act_dtype=dtype, device=dev, embed_norm=f32("embed.norm"))


def load(path: str, dtype=torch.bfloat16, device="cuda") -> RaggedDecoder:
    """Engine for the checkpoint directory ``path`` (config.json + model.safetensors)."""
    from .arch import load_checkpoint_tensors
    with open(os.path.join(path, "config.json")) as f:
        config = json.load(f)
    if not is_lifenex(config):
        raise ValueError(f"{path}: not a {ARCHITECTURE} checkpoint")
    return build_engine(read_config(config), load_checkpoint_tensors(path), dtype, device)


def example_config(width=2048, layers=6, heads=16, kv_heads=4, dim=128, ff=5632, vocab=32000, bias_max=1024, temp=(0.1, 1024), delta_heads=16,
                   delta_kv_heads=8, delta_dim=64, delta_vdim=64, conv=4, ssm_heads=64, ssm_vdim=64, ssm_state=128, ssm_groups=8,
                   norm_groups=8, expert_ff=1024, experts=32, top=4, groups=4, keep=2, shared_ff=1536, logit_scale=0.25) -> dict:
    """A config.json of this design at the proportions of a real model: two side-by-side layers and a state space layer in turn, the
    first layer with a dense feed-forward, the others with experts.  For benchmarks and smoke tests (random weights)."""
    side = {"left": {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": dim, "scale": dim ** -0.5, "bias_max": bias_max,
                     "q_temp": {"coef": temp[0], "every": temp[1]}},
            "right": {"heads": delta_heads, "kv_heads": delta_kv_heads, "dim": delta_dim, "vdim": delta_vdim, "conv": conv}}
    space = {"heads": ssm_heads, "vdim": ssm_vdim, "state": ssm_state, "groups": ssm_groups, "norm_groups": norm_groups, "conv": conv}
    moe = {"kind": "moe", "expert": {"ff": expert_ff}, "shared": {"ff": shared_ff},
           "router": {"experts": experts, "top": top, "groups": {"count": groups, "keep": keep}}}
    out = []
    for i in range(layers):
        kind, mixer = ("mamba2", space) if i % 3 == 2 else ("parallel", side)
        out.append({"type": kind, "mixer": json.loads(json.dumps(mixer)), "mlp": json.loads(json.dumps(moe)) if i else {"kind": "dense", "ff": ff}})
    return {"architecture": ARCHITECTURE, "layers": out, "norm": {"eps": 1e-5}, "vocab": vocab, "width": width, "logit_scale": logit_scale}


def random_state_dict(config: dict, device="cuda", seed: int = 0, rel_rows: int = 32, low_rank: int = 64) -> dict:
    """Random checkpoint tensors (bfloat16, created on ``device``) with the names and shapes the design gives them."""
    dev = torch.device(device)
    g = torch.Generator(device=dev).manual_seed(seed)
    D = config["width"]

    def mat(n, k, s=1.0):
        return (torch.randn(n, k, device=dev, generator=g) * (s / math.sqrt(k))).to(torch.bfloat16)

    def vec(n, mean=0.0, s=0.1):
        return (mean + s * torch.randn(n, device=dev, generator=g)).to(torch.bfloat16)

    def expert(p, ff):
        return {p + "gate": mat(ff, D), p + "up": mat(ff, D), p + "down": mat(D, ff)}

    sd = {"embed": mat(config["vocab"], D, math.sqrt(D)), "embed.norm": vec(D, 1.0), "final.norm": vec(D, 1.0)}
    for li, layer in enumerate(config["layers"]):
        l, p, m = f"l{li}.", f"l{li}.mix.", layer["mixer"]
        sd[l + "norm1"] = vec(D, 1.0)
        if layer["type"] == "mamba2":
            H, inner, gn = m["heads"], m["heads"] * m["vdim"], m["groups"] * m["state"]
            sd.update({p + "in": mat(2 * inner + 2 * gn + H, D), p + "conv": mat(inner + 2 * gn, m["conv"]), p + "conv.b": vec(inner + 2 * gn),
                       p + "dt_bias": vec(H, -3.0, 1.0), p + "A_log": vec(H, 1.0, 0.7), p + "D": vec(H, 1.0), p + "norm": vec(inner, 1.0),
                       p + "o": mat(D, inner)})
        else:
            a, b = p + "left.", p + "right."
            H, G, d, e = (m["left"][n] for n in ("heads", "kv_heads", "dim", "vdim"))
            sd.update({a + "q": mat(H * d, D), a + "k": mat(G * d, D), a + "v": mat(G * e, D), a + "q.norm": vec(d, 1.0), a + "k.norm": vec(d, 1.0),
                       a + "rel": mat(rel_rows, H, math.sqrt(H)), a + "sink": vec(H, 0.0, 1.0), a + "o": mat(D, H * e), a + "out": vec(D, 1.0)})
            H, G, d, e = (m["right"][n] for n in ("heads", "kv_heads", "dim", "vdim"))
            for n, rows in (("q", G * d), ("k", G * d), ("v", H * e)):
                sd.update({b + n: mat(rows, D), b + n + ".conv": mat(rows, m["right"]["conv"])})
            sd.update({b + "b": mat(H, D), b + "A_log": vec(H, -2.0, 1.0), b + "dt_bias": vec(H * d, -3.0, 0.5), b + "norm": vec(e, 1.0),
                       b + "a1": mat(low_rank, D), b + "a2": mat(H * d, low_rank), b + "g1": mat(low_rank, D), b + "g2": mat(H * e, low_rank),
                       b + "o": mat(D, H * e), b + "out": vec(D, 1.0)})
        f, q = layer.get("mlp"), l + "mlp."
        if f is None:
            continue
        sd[l + "norm2"] = vec(D, 1.0)
        if f["kind"] == "dense":
            sd.update({q + "up": mat(f["ff"], D), q + "down": mat(D, f["ff"])})
            continue
        n = f["router"]["experts"]
        sd.update({q + "router": mat(n, D, 0.5), q + "correction": vec(n, 0.0, 0.05)})
        for e in range(n):
            sd.update(expert(q + f"e{e}.", f["expert"]["ff"]))
        if f.get("shared"):
            sd.update(expert(q + "shared.", f["shared"]["ff"]))
            sd[q + "shared.sg"] = mat(1, D)
    return sd


def build_random(config: dict, dtype=torch.bfloat16, device="cuda", seed: int = 0, rel_rows: int = 32, low_rank: int = 64) -> RaggedDecoder:
    return build_engine(read_config(config), random_state_dict(config, device, seed, rel_rows, low_rank), dtype, device)
