"""Plain, slow float64 statement of the Supisun design: one function per mechanism, whole sequences, token by token where
there is a recurrence, nothing shared with ``bigdl_amd``.  Weights are a dict of float64 tensors by checkpoint name;
``config`` is the parsed ``config.json``.

Notation: LN(u) = (u - mean u) / sqrt(var u + eps) * w + b;  rms(u) = u / sqrt(mean u^2 + eps);  per layer
x <- x + LN1(mixer(h)) with h = x + causal_conv(x), then x <- x + LN2(ff(x)).
"""
import math
import random

import torch

F64 = torch.float64
UNIT_EPS = 1e-6


def rms(u, eps):
    return u / torch.sqrt(u.pow(2).mean(-1, keepdim=True) + eps)


def layer_norm(u, w, b, eps):
    mu = u.mean(-1, keepdim=True)
    return (u - mu) / torch.sqrt((u - mu).pow(2).mean(-1, keepdim=True) + eps) * w + b


def silu(z):
    return z / (1.0 + torch.exp(-z))


def softplus(z):
    return torch.clamp(z, min=0.0) + torch.log1p(torch.exp(-z.abs()))


def gelu_erf(z):
    return 0.5 * z * (1.0 + torch.erf(z / math.sqrt(2.0)))


def causal_conv(u, w, bias=None):
    """u [T, C], w [C, taps]: out[t, c] = sum_j w[c, j] u[t - taps + 1 + j, c] (+ bias[c]), nothing before the start"""
    T, taps = u.shape[0], w.shape[1]
    out = torch.zeros_like(u)
    for t in range(T):
        for j in range(taps):
            s = t - taps + 1 + j
            if s >= 0:
                out[t] = out[t] + w[:, j] * u[s]
    return out if bias is None else out + bias


# ---------------------------------------------------------------------------------------- attention
def turn_halves(u, pos, dims, base):
    """channel pairs (i, i + dims / 2), i < dims / 2, of u [..., n] turned by pos * base^(-2 i / dims)"""
    out, half = u.clone(), dims // 2
    for i in range(half):
        ang = pos * base ** (-2.0 * i / dims)
        c, s = math.cos(ang), math.sin(ang)
        a, b = u[..., i], u[..., i + half]
        out[..., i], out[..., i + half] = a * c - b * s, b * c + a * s
    return out


def attend(q, k, v, scale, chunk=None):
    """q [T, H, d], k [T, G, d], v [T, G, e] -> [T, H, e].  Query i sees key j <= i of its own block of ``chunk`` positions."""
    T, H, G = q.shape[0], q.shape[1], k.shape[1]
    out = torch.zeros(T, H, v.shape[2], dtype=F64)
    for i in range(T):
        js = [j for j in range(i + 1) if not chunk or j // chunk == i // chunk]
        for h in range(H):
            g = h // (H // G)
            out[i, h] = torch.softmax((k[js, g] @ q[i, h]) * scale, -1) @ v[js, g]
    return out


def mix_values(v, first, lam):
    return (1.0 - lam) * v + lam * first


def qkv(h, W, p, m, eps, first=None):
    """queries, keys and values as the scores and the sum see them; ``first``: the values of the first mixing layer (None in
    that layer itself and without mixing)"""
    T = h.shape[0]
    H, G, d, e = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q = (rms(h @ W[p + "q"].T, eps) * W[p + "q.norm"]).view(T, H, d)
    k = (rms(h @ W[p + "k"].T, eps) * W[p + "k.norm"]).view(T, G, d)
    v = rms((h @ W[p + "v"].T).view(T, G, e), eps)
    rot = m.get("rot")
    if rot and rot.get("dims"):
        q = torch.stack([turn_halves(q[t], t, rot["dims"], rot["base"]) for t in range(T)])
        k = torch.stack([turn_halves(k[t], t, rot["dims"], rot["base"]) for t in range(T)])
    if first is not None:
        v = mix_values(v, first, W[p + "vmix"])
    return q, k, v


def attention_mixer(h, W, p, m, eps, carry):
    """``carry["v"]``: the values of the first layer with ``v_mix``, left there by that layer"""
    mixes = bool(m.get("v_mix"))
    q, k, v = qkv(h, W, p, m, eps, carry.get("v") if mixes else None)
    if mixes:
        carry.setdefault("v", v)
    o = attend(q, k, v, m["scale"], (m.get("mask") or {}).get("size"))
    return o.reshape(h.shape[0], -1) @ W[p + "o"].T


# ---------------------------------------------------------------------------------------- selective scan
def selective_scan(x, dt, A, B, C, D, S0=None):
    """x, dt [T, c]; A [c, n]; B, C [T, n]; D [c]: S <- exp(dt A) S + dt x B, y = S C + D x.  Returns (y [T, c], last S)."""
    S = torch.zeros_like(A) if S0 is None else S0.clone()
    y = torch.zeros_like(x)
    for t in range(x.shape[0]):
        S = torch.exp(dt[t][:, None] * A) * S + (dt[t] * x[t])[:, None] * B[t][None, :]
        y[t] = S @ C[t] + D * x[t]
    return y, S


def mamba1_mixer(h, W, p, m):
    inner, n, r = m["inner"], m["state"], m["dt_rank"]
    xz = h @ W[p + "in"].T
    x = silu(causal_conv(xz[:, :inner], W[p + "conv"], W[p + "conv.b"]))
    low = x @ W[p + "x"].T
    dt = softplus(low[:, :r] @ W[p + "dt"].T + W[p + "dt.b"])
    y, _ = selective_scan(x, dt, -torch.exp(W[p + "A_log"]), low[:, r:r + n], low[:, r + n:], W[p + "D"])
    return (y * silu(xz[:, inner:])) @ W[p + "o"].T


# ---------------------------------------------------------------------------------------- gated delta rule
def unit(u):
    return u / torch.sqrt(u.pow(2).sum(-1, keepdim=True) + UNIT_EPS)


def gated_delta(q, k, v, g, beta, S0=None):
    """one head: q, k [T, d], v [T, e], g, beta [T]: S <- g S; u = beta (v - S^T k); S <- S + k u^T; o = S^T q"""
    S = torch.zeros(k.shape[1], v.shape[1], dtype=F64) if S0 is None else S0.clone()
    out = torch.zeros(q.shape[0], v.shape[1], dtype=F64)
    for t in range(q.shape[0]):
        S = g[t] * S
        S = S + torch.outer(k[t], beta[t] * (v[t] - S.T @ k[t]))
        out[t] = S.T @ q[t]
    return out, S


def delta_gates(h, W, p):
    beta = 1.0 / (1.0 + torch.exp(-(h @ W[p + "b"].T)))
    return torch.exp(-torch.exp(W[p + "A_log"]) * softplus(h @ W[p + "a"].T + W[p + "dt_bias"])), beta


def delta_mixer(h, W, p, m, eps):
    T = h.shape[0]
    H, G, d, e = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q, k, v = (silu(causal_conv(h @ W[p + n].T, W[p + n + ".conv"])) for n in "qkv")
    q, k, v = unit(q.view(T, G, d)) * d ** -0.5, unit(k.view(T, G, d)), v.view(T, H, e)
    g, beta = delta_gates(h, W, p)
    o = torch.stack([gated_delta(q[:, i // (H // G)], k[:, i // (H // G)], v[:, i], g[:, i], beta[:, i])[0] for i in range(H)], 1)
    o = rms(o, eps) * W[p + "norm"] * silu(h @ W[p + "g"].T).view(T, H, e)
    return o.reshape(T, H * e) @ W[p + "o"].T


# ---------------------------------------------------------------------------------------- whole model
def mixer(h, W, p, layer, eps, carry):
    kind, m = layer["type"], layer["mixer"]
    if kind == "attention":
        return attention_mixer(h, W, p, m, eps, carry)
    if kind == "mamba1":
        return mamba1_mixer(h, W, p, m)
    if kind == "delta":
        return delta_mixer(h, W, p, m, eps)
    raise ValueError(kind)


def forward(tokens, W, config, layers_out=None):
    """logits [T, vocab] of one sequence; ``layers_out`` collects the stream behind every layer"""
    eps = config["norm"]["eps"]
    x = W["embed"][torch.tensor(tokens)] + W["pos"][:len(tokens)]
    carry = {}
    for li, layer in enumerate(config["layers"]):
        p = f"l{li}."
        h = x + causal_conv(x, W[p + "canon1"])
        x = x + layer_norm(mixer(h, W, p + "mix.", layer, eps, carry), W[p + "norm1"], W[p + "norm1.b"], eps)
        if layer.get("mlp") is not None:
            f = gelu_erf(x @ W[p + "mlp.up"].T) @ W[p + "mlp.down"].T
            x = x + layer_norm(f, W[p + "norm2"], W[p + "norm2.b"], eps)
        if layers_out is not None:
            layers_out.append(x.clone())
    return layer_norm(x, W["final.norm"], W["final.norm.b"], eps) @ W["head"].T


# ---------------------------------------------------------------------------------------- small random models
def attention_layer(heads=4, kv_heads=2, dim=16, vdim=24, chunk=9, rot=(8, 100.0), v_mix=True, ff=48, scale=None):
    m = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale or dim ** -0.5, "v_mix": v_mix}
    if chunk:
        m["mask"] = {"size": chunk}
    if rot:
        m["rot"] = {"dims": rot[0], "base": rot[1]}
    return {"type": "attention", "mixer": m, "mlp": {"kind": "dense", "ff": ff} if ff else None}


def mamba_layer(inner=40, state=6, dt_rank=3, conv=4, ff=48):
    return {"type": "mamba1", "mixer": {"inner": inner, "state": state, "dt_rank": dt_rank, "conv": conv},
            "mlp": {"kind": "dense", "ff": ff} if ff else None}


def delta_layer(heads=4, kv_heads=2, dim=12, vdim=20, conv=3, ff=48):
    return {"type": "delta", "mixer": {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "conv": conv},
            "mlp": {"kind": "dense", "ff": ff} if ff else None}


def make_config(layers, width=40, vocab=67, taps=4, eps=1e-5, max_positions=512):
    return {"architecture": "Supisun", "canon": {"taps": taps}, "layers": layers, "max_positions": max_positions,
            "norm": {"eps": eps}, "vocab": vocab, "width": width}


def tensor_shapes(config):
    """name -> shape of every checkpoint tensor of ``config``"""
    D, V = config["width"], config["vocab"]
    out = {"embed": (V, D), "pos": (config["max_positions"], D), "final.norm": (D,), "final.norm.b": (D,), "head": (V, D)}
    for li, layer in enumerate(config["layers"]):
        p, m = f"l{li}.mix.", layer["mixer"]
        out.update({f"l{li}.norm1": (D,), f"l{li}.norm1.b": (D,), f"l{li}.canon1": (D, config["canon"]["taps"])})
        if layer["type"] == "mamba1":
            c, n, r = m["inner"], m["state"], m["dt_rank"]
            out.update({p + "in": (2 * c, D), p + "conv": (c, m["conv"]), p + "conv.b": (c,), p + "x": (r + 2 * n, c), p + "dt": (c, r),
                        p + "dt.b": (c,), p + "A_log": (c, n), p + "D": (c,), p + "o": (D, c)})
        else:
            H, G, d, e = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
            o = D, H * e
            if layer["type"] == "attention":
                out.update({p + "q": (H * d, D), p + "k": (G * d, D), p + "v": (G * e, D), p + "q.norm": (H * d,), p + "k.norm": (G * d,),
                            p + "vmix": (), p + "o": o})
            else:
                for n, rows in (("q", G * d), ("k", G * d), ("v", H * e)):
                    out.update({p + n: (rows, D), p + n + ".conv": (rows, m["conv"])})
                out.update({p + "b": (H, D), p + "a": (H, D), p + "A_log": (H,), p + "dt_bias": (H,), p + "norm": (e,), p + "g": (H * e, D),
                            p + "o": o})
        if layer.get("mlp") is not None:
            f = layer["mlp"]["ff"]
            out.update({f"l{li}.norm2": (D,), f"l{li}.norm2.b": (D,), f"l{li}.mlp.up": (f, D), f"l{li}.mlp.down": (D, f)})
    return out


def random_weights(config, seed=0):
    """bfloat16-representable random tensors by name (so that an engine that stores bfloat16 reads the same numbers)"""
    g = torch.Generator().manual_seed(seed)
    W = {}
    for name, shape in tensor_shapes(config).items():
        leaf = name.split(".")[-1]
        n = torch.randn(shape, generator=g)
        if leaf in ("conv", "canon1"):
            t = 0.5 * n
        elif name in ("embed", "pos"):
            t = n if name == "embed" else 0.5 * n
        elif leaf == "A_log" and len(shape) == 2:
            t = torch.log(torch.arange(1, shape[1] + 1).float())[None] + 0.2 * n
        elif leaf == "A_log":
            t = -1.0 + n
        elif leaf == "b" and len(shape) == 1:                  # biases of norms, of the convolution and of the step size
            t = -1.0 + 0.5 * n if name.endswith("dt.b") else 0.3 * n
        elif leaf == "dt_bias":
            t = -1.0 + 0.5 * n
        elif leaf == "vmix":
            t = 0.45 + 0.2 * n
        elif leaf in ("norm", "norm1", "norm2", "D"):
            t = 1.0 + 0.2 * n
        elif len(shape) == 2:
            t = n * (1.5 / math.sqrt(shape[1]))
        else:
            raise ValueError(name)
        W[name] = t.to(torch.bfloat16).to(F64)
    return W


def random_tokens(n, vocab, seed):
    rnd = random.Random(seed)
    return [rnd.randrange(vocab) for _ in range(n)]
