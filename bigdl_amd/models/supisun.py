"""Supisun on the ragged engine: reader of its ``config.json`` and the map from checkpoint tensor names to ``LayerTensors``.

The design: x = embed[token] + pos[position]; per layer x <- x + LN1(mixer(h)) and x <- x + LN2(ff(x)), LayerNorms with weight
and bias on the sublayers' outputs only, where the mixer reads h = x + conv(x), a causal convolution of ``canon.taps`` taps per
channel of the stream; a last LayerNorm and an output projection of its own.

Mixers (``type`` of a layer):

* ``attention``: grouped key/value heads; queries and keys RMS-normed over the whole projection with a weight per channel, the
  first ``rot.dims`` channels of every head turned in pairs (i, i + dims / 2); values RMS-normed per head without a weight;
  with ``v_mix`` the values of the first such layer are mixed in, v <- (1 - lambda) v + lambda v_first; softmax inside blocks of
  ``mask.size`` positions counted from the sequence's start;
* ``mamba1``: selective scan (``SelectiveScan``);
* ``delta``: gated delta rule (``GatedDelta``).

Feed-forward: W_down gelu(W_up x), the exact gelu.
"""
from __future__ import annotations

import json
import math
import os

import torch

from .ragged_engine import (DenseMlp, GatedDelta, LayerTensors, RaggedConfig, RaggedDecoder, SelectiveScan, WindowAttention,
                            rotary_inv_freq)

ARCHITECTURE = "Supisun"
UNIT_EPS = 1e-6                # fixed by the design: inside the root of a unit vector's length


def is_supisun(config: dict) -> bool:
    return config.get("architecture") == ARCHITECTURE


def _mixer(kind: str, m: dict):
    if kind == "attention":
        rot = m.get("rot") or {}
        return WindowAttention(heads=int(m["heads"]), kv_heads=int(m["kv_heads"]), dim=int(m["dim"]), vdim=int(m["vdim"]),
                               scale=float(m["scale"]), qk_norm_rows=True, rot_dims=int(rot.get("dims") or 0),
                               rot_base=float(rot.get("base", 10000.0)), chunk=int((m.get("mask") or {}).get("size") or 0), v_norm=True,
                               v_mix=bool(m.get("v_mix")))
    if kind == "mamba1":
        return SelectiveScan(inner=int(m["inner"]), state=int(m["state"]), dt_rank=int(m["dt_rank"]), conv_taps=int(m["conv"]))
    if kind == "delta":
        return GatedDelta(heads=int(m["heads"]), kv_heads=int(m["kv_heads"]), dim=int(m["dim"]), vdim=int(m["vdim"]),
                          conv_taps=int(m["conv"]), unit_eps=UNIT_EPS)
    raise ValueError(f"unknown layer type {kind!r}")


def read_config(config: dict) -> RaggedConfig:
    mixers, mlps = [], []
    for layer in config["layers"]:
        mixers.append(_mixer(layer["type"], layer["mixer"]))
        f = layer.get("mlp")
        if f is None:
            mlps.append(None)
        elif f.get("kind", "dense") == "dense":
            mlps.append(DenseMlp(ff=int(f["ff"]), act="gelu_erf", bias=False))
        else:
            raise ValueError(f"unknown feed-forward kind {f.get('kind')!r}")
    return RaggedConfig(vocab=int(config["vocab"]), width=int(config["width"]), mixers=mixers, mlps=mlps,
                        norm_eps=float((config.get("norm") or {}).get("eps", 1e-5)), name=ARCHITECTURE, block="output_norm",
                        positions=int(config["max_positions"]), stream_conv=int(config["canon"]["taps"]))


def build_engine(cfg: RaggedConfig, sd: dict, dtype=torch.bfloat16, device="cuda") -> RaggedDecoder:
    """``sd``: checkpoint tensors by name ('l<i>.mix.q', 'l<i>.mlp.up', ...).  Projection weights and the embedding tables take
    the activation type; norm weights and biases, convolution taps and everything of the recurrences become float32."""
    dev = torch.device(device)

    def act(*names):
        return torch.cat([sd[n] for n in names], 0).to(dev, dtype).contiguous()

    def f32(name):
        return sd[name].float().to(dev).contiguous()

    layers = []
    for li, (m, mlp) in enumerate(zip(cfg.mixers, cfg.mlps)):
        l, p = f"l{li}.", f"l{li}.mix."
        lt = LayerTensors(w_in=None, w_out=act(p + "o"), norm1=f32(l + "norm1"), norm1_bias=f32(l + "norm1.b"), stream_conv=f32(l + "canon1"))
        if isinstance(m, WindowAttention):
            lt.w_in = act(p + "q", p + "k", p + "v")
            lt.q_norm, lt.k_norm = f32(p + "q.norm").view(-1), f32(p + "k.norm").view(-1)
            if m.rot_dims:
                lt.inv_freq = rotary_inv_freq(m.rot_dims, m.rot_base, 1.0).to(dev)
            if m.v_mix:
                lt.v_lam = float(sd[p + "vmix"].float().reshape(()))
        elif isinstance(m, SelectiveScan):
            lt.w_in, lt.conv_w, lt.conv_b = act(p + "in"), f32(p + "conv"), f32(p + "conv.b")
            lt.w_low, lt.w_dt, lt.dt_bias = act(p + "x"), act(p + "dt"), f32(p + "dt.b")
            lt.ssm_a = (-torch.exp(sd[p + "A_log"].double()) * math.log2(math.e)).float().to(dev).contiguous()
            lt.ssm_d = f32(p + "D")
        else:
            lt.w_in = act(*[p + n for n in ("q", "k", "v", "g", "b", "a")])
            lt.conv_w = torch.cat([f32(p + n + ".conv") for n in ("q", "k", "v")], 0).contiguous()
            lt.decay_rate, lt.decay_bias = torch.exp(f32(p + "A_log")), f32(p + "dt_bias")
            lt.o_norm = f32(p + "norm").repeat(m.heads).contiguous()
        if mlp is not None:
            lt.norm2, lt.norm2_bias = f32(l + "norm2"), f32(l + "norm2.b")
            lt.w_ff, lt.w_down = act(l + "mlp.up"), act(l + "mlp.down")
        layers.append(lt)
    return RaggedDecoder(cfg, act("embed"), layers, f32("final.norm"), act("head"), act_dtype=dtype, device=dev, pos_table=act("pos"),
                         final_norm_bias=f32("final.norm.b"))


def load(path: str, dtype=torch.bfloat16, device="cuda") -> RaggedDecoder:
    """Engine for the checkpoint directory ``path`` (config.json + model.safetensors)."""
    from .arch import load_checkpoint_tensors
    with open(os.path.join(path, "config.json")) as f:
        config = json.load(f)
    if not is_supisun(config):
        raise ValueError(f"{path}: not a {ARCHITECTURE} checkpoint")
    return build_engine(read_config(config), load_checkpoint_tensors(path), dtype, device)


def example_config(width=2048, layers=6, heads=16, kv_heads=4, dim=128, ff=5632, vocab=32000, chunk=1024, rot_dims=64, delta_heads=16,
                   delta_kv_heads=8, delta_dim=64, delta_vdim=64, inner=4096, state=16, dt_rank=128, conv=4, taps=4,
                   max_positions=8192) -> dict:
    """A config.json of this design at the proportions of a real model: the three kinds of layers in turn.  For benchmarks and
    smoke tests (random weights)."""
    attn = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": dim, "scale": dim ** -0.5, "v_mix": True, "mask": {"size": chunk},
            "rot": {"dims": rot_dims, "base": 10000.0}}
    delta = {"heads": delta_heads, "kv_heads": delta_kv_heads, "dim": delta_dim, "vdim": delta_vdim, "conv": conv}
    mamba = {"inner": inner, "state": state, "dt_rank": dt_rank, "conv": conv}
    kinds = [("attention", attn), ("delta", delta), ("mamba1", mamba)]
    out = [{"type": kinds[i % 3][0], "mixer": json.loads(json.dumps(kinds[i % 3][1])), "mlp": {"kind": "dense", "ff": ff}} for i in range(layers)]
    return {"architecture": ARCHITECTURE, "canon": {"taps": taps}, "layers": out, "max_positions": max_positions, "norm": {"eps": 1e-5},
            "vocab": vocab, "width": width}


def random_state_dict(config: dict, device="cuda", seed: int = 0) -> dict:
    """Random checkpoint tensors (bfloat16, created on ``device``) with the names and shapes the design gives them."""
    dev = torch.device(device)
    g = torch.Generator(device=dev).manual_seed(seed)
    D, taps = config["width"], config["canon"]["taps"]

    def mat(n, k, s=1.0):
        return (torch.randn(n, k, device=dev, generator=g) * (s / math.sqrt(k))).to(torch.bfloat16)

    def vec(n, mean=0.0, s=0.1):
        return (mean + s * torch.randn(n, device=dev, generator=g)).to(torch.bfloat16)

    sd = {"embed": mat(config["vocab"], D, math.sqrt(D)), "pos": mat(config["max_positions"], D, 0.3 * math.sqrt(D)),
          "final.norm": vec(D, 1.0), "final.norm.b": vec(D), "head": mat(config["vocab"], D)}
    for li, layer in enumerate(config["layers"]):
        l, p, m = f"l{li}.", f"l{li}.mix.", layer["mixer"]
        sd.update({l + "norm1": vec(D, 1.0), l + "norm1.b": vec(D), l + "canon1": mat(D, taps, 0.5)})
        if layer["type"] == "mamba1":
            c, n, r = m["inner"], m["state"], m["dt_rank"]
            a_log = torch.arange(1, n + 1, device=dev).float().log()[None].repeat(c, 1).to(torch.bfloat16)
            sd.update({p + "in": mat(2 * c, D), p + "conv": mat(c, m["conv"]), p + "conv.b": vec(c), p + "x": mat(r + 2 * n, c),
                       p + "dt": mat(c, r), p + "dt.b": vec(c, -3.0, 1.0), p + "A_log": a_log, p + "D": vec(c, 1.0), p + "o": mat(D, c)})
        else:
            H, G, d, e = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
            sd[p + "o"] = mat(D, H * e)
            if layer["type"] == "attention":
                sd.update({p + "q": mat(H * d, D), p + "k": mat(G * d, D), p + "v": mat(G * e, D), p + "q.norm": vec(H * d, 1.0),
                           p + "k.norm": vec(G * d, 1.0), p + "vmix": vec(1, 0.5).reshape(())})
            else:
                for n, rows in (("q", G * d), ("k", G * d), ("v", H * e)):
                    sd.update({p + n: mat(rows, D), p + n + ".conv": mat(rows, m["conv"])})
                sd.update({p + "b": mat(H, D), p + "a": mat(H, D), p + "A_log": vec(H, -2.0, 1.0), p + "dt_bias": vec(H, -3.0, 0.5),
                           p + "norm": vec(e, 1.0), p + "g": mat(H * e, D)})
        f = layer.get("mlp")
        if f is not None:
            sd.update({l + "norm2": vec(D, 1.0), l + "norm2.b": vec(D), l + "mlp.up": mat(f["ff"], D), l + "mlp.down": mat(D, f["ff"])})
    return sd


def build_random(config: dict, dtype=torch.bfloat16, device="cuda", seed: int = 0) -> RaggedDecoder:
    return build_engine(read_config(config), random_state_dict(config, device, seed), dtype, device)
