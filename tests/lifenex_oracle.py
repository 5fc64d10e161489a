"""Plain, slow float64 statement of the Lifenex design: one function per mechanism, whole sequences, token by token where there is
a recurrence, nothing shared with ``bigdl_amd``.  Weights are a dict of float64 tensors by checkpoint name; ``config`` is the
parsed ``config.json``.

Notation: rms(u, w) = u / sqrt(mean u^2 + eps) * w.  x = rms(embed[token]); per layer x <- x + mixer(rms1(x)) + ff(rms2(x)), both of
the same x; logits = logit_scale * embed rms(x).
"""
import math
import random

import torch

F64 = torch.float64
UNIT_EPS = 1e-6


def rms(u, eps, w=None):
    v = u / torch.sqrt(u.pow(2).mean(-1, keepdim=True) + eps)
    return v if w is None else v * w


def sigmoid(z):
    return 1.0 / (1.0 + torch.exp(-z))


def silu(z):
    return z * sigmoid(z)


def softplus(z):
    return torch.clamp(z, min=0.0) + torch.log1p(torch.exp(-z.abs()))


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


# ---------------------------------------------------------------------------------------- attention with a distance bias
def bucket(n, rows, far):
    """row of the bias table for distance n: the first half of the rows one by one, the others in logarithmic steps that end at
    distance ``far``"""
    half = rows // 2
    if n < half:
        return n
    step = math.log(n / half) / math.log(far / half) * (rows - half)
    near = round(step)
    return min(rows - 1, half + (near if abs(step - near) < 1e-9 else math.floor(step)))     # (an integer that rounding missed)


def query_temperature(pos, coef, every):
    return 1.0 + coef * math.log((pos + 1) // every + 1)


def attend(q, k, v, scale, rel, far, sink):
    """q [T, H, d], k [T, G, d], v [T, G, e] -> [T, H, e]; score = scale q . k + rel[bucket(i - j), h], exp(sink[h]) joins the sum
    of the exponentials"""
    T, H, G = q.shape[0], q.shape[1], k.shape[1]
    out = torch.zeros(T, H, v.shape[2], dtype=F64)
    rows = torch.tensor([bucket(n, rel.shape[0], far) for n in range(T)])
    for i in range(T):
        bias = rel[rows[:i + 1].flip(0)]                     # [i + 1, H]
        for h in range(H):
            g = h // (H // G)
            s = (k[:i + 1, g] @ q[i, h]) * scale + bias[:, h]
            top = torch.maximum(s.max(), sink[h])
            w = torch.exp(s - top)
            out[i, h] = (w / (w.sum() + torch.exp(sink[h] - top))) @ v[:i + 1, g]
    return out


def attention_qkv(h, W, p, m, eps):
    T, H, G, d, e = h.shape[0], m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q = rms((h @ W[p + "q"].T).view(T, H, d), eps, W[p + "q.norm"])
    k = rms((h @ W[p + "k"].T).view(T, G, d), eps, W[p + "k.norm"])
    if m.get("q_temp"):
        q = torch.stack([q[t] * query_temperature(t, m["q_temp"]["coef"], m["q_temp"]["every"]) for t in range(T)])
    return q, k, (h @ W[p + "v"].T).view(T, G, e)


def left_mixer(h, W, p, m, eps):
    q, k, v = attention_qkv(h, W, p, m, eps)
    return attend(q, k, v, m["scale"], W[p + "rel"], m["bias_max"], W[p + "sink"]).reshape(h.shape[0], -1) @ W[p + "o"].T


# ---------------------------------------------------------------------------------------- delta rule, a decay per key channel
def unit(u):
    return u / torch.sqrt(u.pow(2).sum(-1, keepdim=True) + UNIT_EPS)


def channel_delta(q, k, v, g, beta, S0=None):
    """one head: q, k, g [T, d], v [T, e], beta [T]: S <- diag(g) S; u = beta (v - S^T k); S <- S + k u^T; o = S^T q"""
    S = torch.zeros(k.shape[1], v.shape[1], dtype=F64) if S0 is None else S0.clone()
    out = torch.zeros(q.shape[0], v.shape[1], dtype=F64)
    for t in range(q.shape[0]):
        S = g[t][:, None] * S
        S = S + torch.outer(k[t], beta[t] * (v[t] - S.T @ k[t]))
        out[t] = S.T @ q[t]
    return out, S


def delta_inputs(h, W, p, m):
    T, H, G, d, e = h.shape[0], m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q, k, v = (silu(causal_conv(h @ W[p + n].T, W[p + n + ".conv"])) for n in "qkv")
    rate = torch.exp(W[p + "A_log"]).repeat_interleave(d)
    g = torch.exp(-rate * softplus((h @ W[p + "a1"].T) @ W[p + "a2"].T + W[p + "dt_bias"]))
    return unit(q.view(T, G, d)) * d ** -0.5, unit(k.view(T, G, d)), v.view(T, H, e), g.view(T, H, d), sigmoid(h @ W[p + "b"].T)


def right_mixer(h, W, p, m, eps):
    T, H, G, e = h.shape[0], m["heads"], m["kv_heads"], m["vdim"]
    q, k, v, g, beta = delta_inputs(h, W, p, m)
    o = torch.stack([channel_delta(q[:, i // (H // G)], k[:, i // (H // G)], v[:, i], g[:, i], beta[:, i])[0] for i in range(H)], 1)
    gate = sigmoid((h @ W[p + "g1"].T) @ W[p + "g2"].T).view(T, H, e)
    return (rms(o, eps, W[p + "norm"]) * gate).reshape(T, H * e) @ W[p + "o"].T


def parallel_mixer(h, W, p, m, eps):
    left = rms(left_mixer(h, W, p + "left.", m["left"], eps), eps, W[p + "left.out"])
    right = rms(right_mixer(h, W, p + "right.", m["right"], eps), eps, W[p + "right.out"])
    return 0.5 * (left + right)


# ---------------------------------------------------------------------------------------- Mamba-2
def state_space(x, B, C, dt, rate, D, S0=None):
    """one head: x [T, e], B, C [T, N], dt [T]: S <- exp(-rate dt) S + dt B x^T, y = S^T C + D x"""
    S = torch.zeros(B.shape[1], x.shape[1], dtype=F64) if S0 is None else S0.clone()
    y = torch.zeros_like(x)
    for t in range(x.shape[0]):
        S = torch.exp(-rate * dt[t]) * S + dt[t] * torch.outer(B[t], x[t])
        y[t] = S.T @ C[t] + D * x[t]
    return y, S


def grouped_norm(y, groups, eps, w):
    T = y.shape[0]
    return rms(y.view(T, groups, -1), eps).reshape(T, -1) * w


def mamba2_mixer(h, W, p, m, eps):
    T, H, e, N, G = h.shape[0], m["heads"], m["vdim"], m["state"], m["groups"]
    inner = H * e
    P = h @ W[p + "in"].T
    z, dt = P[:, :inner], softplus(P[:, 2 * inner + 2 * G * N:] + W[p + "dt_bias"])
    u = silu(causal_conv(P[:, inner:2 * inner + 2 * G * N], W[p + "conv"], W[p + "conv.b"]))
    x, B, C = u[:, :inner].reshape(T, H, e), u[:, inner:inner + G * N].reshape(T, G, N), u[:, inner + G * N:].reshape(T, G, N)
    rate = torch.exp(W[p + "A_log"])
    y = torch.stack([state_space(x[:, i], B[:, i // (H // G)], C[:, i // (H // G)], dt[:, i], rate[i], W[p + "D"][i])[0] for i in range(H)], 1)
    y = grouped_norm(y.reshape(T, inner) * silu(z), m["norm_groups"], eps, W[p + "norm"])
    return y @ W[p + "o"].T


# ---------------------------------------------------------------------------------------- feed-forward
def gated_expert(h, W, p):
    return (silu(h @ W[p + "gate"].T) * (h @ W[p + "up"].T)) @ W[p + "down"].T


def choose(scores, correction, top, groups, keep):
    """indices of the ``top`` experts with the best corrected scores inside the ``keep`` best groups; a group is worth the sum of its
    two best corrected scores"""
    c = scores + correction
    size = len(c) // groups
    worth = [sum(sorted(c[g * size:(g + 1) * size].tolist(), reverse=True)[:2]) for g in range(groups)]
    best = sorted(range(groups), key=lambda g: -worth[g])[:keep]
    allowed = [e for e in range(len(c)) if e // size in best]
    return sorted(allowed, key=lambda e: -float(c[e]))[:top]


def experts_ff(h, W, p, f):
    r = f["router"]
    scores = sigmoid(h @ W[p + "router"].T)
    gr = r.get("groups") or {"count": 1, "keep": 1}
    out = torch.zeros_like(h)
    for t in range(h.shape[0]):
        for e in choose(scores[t], W[p + "correction"], r["top"], gr["count"], gr["keep"]):
            out[t] = out[t] + scores[t, e] * gated_expert(h[t:t + 1], W, f"{p}e{e}.")[0]
    if f.get("shared"):
        out = out + gated_expert(h, W, p + "shared.") * sigmoid(h @ W[p + "shared.sg"].T)
    return out


def feed_forward(h, W, p, f):
    if f["kind"] == "dense":
        return torch.relu(h @ W[p + "up"].T).pow(2) @ W[p + "down"].T
    return experts_ff(h, W, p, f)


# ---------------------------------------------------------------------------------------- whole model
def mixer(h, W, p, layer, eps):
    return {"parallel": parallel_mixer, "mamba2": mamba2_mixer}[layer["type"]](h, W, p, layer["mixer"], eps)


def forward(tokens, W, config, layers_out=None):
    """logits [T, vocab] of one sequence; ``layers_out`` collects the stream behind every layer"""
    eps = config["norm"]["eps"]
    x = rms(W["embed"][torch.tensor(tokens)], eps, W["embed.norm"])
    for li, layer in enumerate(config["layers"]):
        l = f"l{li}."
        u = mixer(rms(x, eps, W[l + "norm1"]), W, l + "mix.", layer, eps)
        if layer.get("mlp") is not None:
            u = u + feed_forward(rms(x, eps, W[l + "norm2"]), W, l + "mlp.", layer["mlp"])
        x = x + u
        if layers_out is not None:
            layers_out.append(x.clone())
    return rms(x, eps, W["final.norm"]) @ W["embed"].T * config["logit_scale"]


# ---------------------------------------------------------------------------------------- small random models
def _mlp(ff, moe):
    """``ff``: inner size of a dense feed-forward (None: none), or with ``moe`` = (experts, top, groups, keep, shared ff) of an expert"""
    if ff is None:
        return None
    if moe is None:
        return {"kind": "dense", "ff": ff}
    experts, top, groups, keep, shared = moe
    f = {"kind": "moe", "expert": {"ff": ff}, "router": {"experts": experts, "top": top, "groups": {"count": groups, "keep": keep}}}
    if shared:
        f["shared"] = {"ff": shared}
    return f


def parallel_layer(heads=4, kv_heads=2, dim=16, vdim=24, scale=None, bias_max=40, rel_rows=12, temp=(0.4, 9), d_heads=4, d_kv=2, d_dim=12,
                   d_vdim=20, conv=3, ff=48, moe=None):
    """(``rel_rows``, the number of rows of the bias table, is a tensor's shape in a checkpoint: ``tensor_shapes`` reads it here)"""
    left = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale or dim ** -0.5, "bias_max": bias_max,
            "q_temp": {"coef": temp[0], "every": temp[1]}}
    right = {"heads": d_heads, "kv_heads": d_kv, "dim": d_dim, "vdim": d_vdim, "conv": conv}
    return {"type": "parallel", "mixer": {"left": left, "right": right}, "mlp": _mlp(ff, moe), "_rel_rows": rel_rows}


def mamba2_layer(heads=6, vdim=12, state=10, groups=2, norm_groups=3, conv=4, ff=48, moe=None):
    return {"type": "mamba2", "mixer": {"heads": heads, "vdim": vdim, "state": state, "groups": groups, "norm_groups": norm_groups,
                                        "conv": conv}, "mlp": _mlp(ff, moe)}


def make_config(layers, width=40, vocab=67, eps=1e-5, logit_scale=0.3, low_rank=(7, 5)):
    return {"architecture": "Lifenex", "layers": layers, "norm": {"eps": eps}, "vocab": vocab, "width": width, "logit_scale": logit_scale,
            "_low_rank": low_rank}


def plain_config(config):
    """``config`` without what only the random weights need (entries that start with an underscore)"""
    out = {k: v for k, v in config.items() if not k.startswith("_")}
    out["layers"] = [{k: v for k, v in layer.items() if not k.startswith("_")} for layer in config["layers"]]
    return out


def tensor_shapes(config):
    """name -> shape of every checkpoint tensor of ``config``"""
    D, V = config["width"], config["vocab"]
    ra, rg = config["_low_rank"]
    out = {"embed": (V, D), "embed.norm": (D,), "final.norm": (D,)}
    for li, layer in enumerate(config["layers"]):
        p, m = f"l{li}.mix.", layer["mixer"]
        out[f"l{li}.norm1"] = (D,)
        if layer["type"] == "mamba2":
            inner, gn = m["heads"] * m["vdim"], m["groups"] * m["state"]
            out.update({p + "in": (2 * inner + 2 * gn + m["heads"], D), p + "conv": (inner + 2 * gn, m["conv"]), p + "conv.b": (inner + 2 * gn,),
                        p + "dt_bias": (m["heads"],), p + "A_log": (m["heads"],), p + "D": (m["heads"],), p + "norm": (inner,), p + "o": (D, inner)})
        else:
            a, H, G, d, e = p + "left.", *(m["left"][n] for n in ("heads", "kv_heads", "dim", "vdim"))
            out.update({a + "q": (H * d, D), a + "k": (G * d, D), a + "v": (G * e, D), a + "q.norm": (d,), a + "k.norm": (d,),
                        a + "rel": (layer["_rel_rows"], H), a + "sink": (H,), a + "o": (D, H * e), a + "out": (D,)})
            b, H, G, d, e = p + "right.", *(m["right"][n] for n in ("heads", "kv_heads", "dim", "vdim"))
            for n, rows in (("q", G * d), ("k", G * d), ("v", H * e)):
                out.update({b + n: (rows, D), b + n + ".conv": (rows, m["right"]["conv"])})
            out.update({b + "b": (H, D), b + "A_log": (H,), b + "norm": (e,), b + "a1": (ra, D), b + "a2": (H * d, ra), b + "dt_bias": (H * d,),
                        b + "g1": (rg, D), b + "g2": (H * e, rg), b + "o": (D, H * e), b + "out": (D,)})
        f, q = layer.get("mlp"), f"l{li}.mlp."
        if f is None:
            continue
        out[f"l{li}.norm2"] = (D,)
        if f["kind"] == "dense":
            out.update({q + "up": (f["ff"], D), q + "down": (D, f["ff"])})
            continue
        n = f["router"]["experts"]
        out.update({q + "router": (n, D), q + "correction": (n,)})
        parts = [(f"e{e}.", f["expert"]["ff"]) for e in range(n)]
        if f.get("shared"):
            out[q + "shared.sg"] = (1, D)
            parts.append(("shared.", f["shared"]["ff"]))
        for name, ff in parts:
            out.update({q + name + "gate": (ff, D), q + name + "up": (ff, D), q + name + "down": (D, ff)})
    return out


def random_weights(config, seed=0):
    """bfloat16-representable random tensors by name (so that an engine that stores bfloat16 reads the same numbers)"""
    g = torch.Generator().manual_seed(seed)
    W = {}
    for name, shape in tensor_shapes(config).items():
        leaf = name.split(".")[-1]
        n = torch.randn(shape, generator=g)
        if leaf == "conv":
            t = 0.5 * n
        elif leaf in ("embed", "rel"):
            t = n
        elif leaf == "A_log":
            t = -1.0 + n
        elif leaf == "b" and len(shape) == 1:                  # bias of a convolution
            t = 0.3 * n
        elif leaf == "dt_bias":
            t = -1.0 + 0.5 * n
        elif leaf == "sink":
            t = 1.5 * n
        elif leaf == "correction":
            t = -0.6 + 0.4 * n                                 # (most corrected scores are negative, some are not)
        elif leaf in ("norm", "norm1", "norm2", "out", "D"):
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
