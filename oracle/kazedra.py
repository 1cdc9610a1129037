"""TEST INFRASTRUCTURE ONLY: a plain, slow restatement of the Kazedra decoder, one function per mechanism.

One sequence at a time, whole prompt, no cache, no batching: every function takes the rows of one sequence and returns
the rows of one sequence.  Runs in the dtype of its inputs (the tests use float64).  Shares no code with the package.
"""
from __future__ import annotations

import math

import torch


def rms(x, eps):
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def norm_one_plus(x, w, eps):
    return rms(x, eps) * (1 + w)


def silu(z):
    return z * torch.sigmoid(z)


def temperature(p, coef, every):
    """Factor on the query at position p."""
    return 1 + coef * math.log(math.floor((p + 1) / every) + 1)


def distance_bucket(n, buckets, longest):
    """Distances below half the buckets have one each, longer ones share logarithmic buckets up to `longest`."""
    half = buckets // 2
    if n < half:
        return n
    return min(buckets - 1, half + math.floor(math.log(n / half) / math.log(longest / half) * (buckets - half) + 1e-9))


def tied_attention(q, k, v, scale, rel, longest, sink):
    """q [T, H, d], k and v [T, G, d]; rel [buckets, H]; sink [H].  Causal softmax whose denominator has one more term."""
    T, H, d = q.shape
    share = H // k.shape[1]
    out = torch.zeros_like(q)
    bucket = torch.tensor([distance_bucket(n, rel.shape[0], longest) for n in range(T)])
    for h in range(H):
        s = (q[:, h] @ k[:, h // share].T) * scale
        n = torch.arange(T)[:, None] - torch.arange(T)[None, :]
        s = s + rel[bucket[n.clamp(min=0)], h]
        s = s.masked_fill(n < 0, -math.inf)
        top = torch.maximum(s.max(-1).values, sink[h])
        e = torch.exp(s - top[:, None])
        out[:, h] = (e / (e.sum(-1) + torch.exp(sink[h] - top))[:, None]) @ v[:, h // share]
    return out


def attention(h, w, c, eps):
    """w: tensors by their names below the mixer; c: the mixer's sizes."""
    T, H, G, d = h.shape[0], c["heads"], c["kv_heads"], c["dim"]
    q = h @ w["q"].T + w["q.b"]
    k = h @ w["k"].T + w["k.b"]
    v = k
    q = rms(q, eps) * w["q.norm"]
    k = rms(k, eps) * w["k.norm"]
    t = c["q_temp"]
    q = q * torch.tensor([temperature(p, t["coef"], t["every"]) for p in range(T)], dtype=q.dtype)[:, None]
    o = tied_attention(q.view(T, H, d), k.view(T, G, d), v.view(T, G, d), c["scale"], w["rel"], c["bias_max"], w["sink"])
    return o.reshape(T, H * d) @ w["o"].T + w["o.b"]


def causal_conv(x, w):
    """x [T, C], w [C, taps] (last column: the token itself)."""
    T, taps = x.shape[0], w.shape[1]
    padded = torch.cat([x.new_zeros(taps - 1, x.shape[1]), x])
    return sum(padded[t: t + T] * w[:, t] for t in range(taps))


def unit(x):
    return x / torch.sqrt((x * x).sum(-1, keepdim=True) + 1e-6)


def delta_rule(q, k, v, g, beta):
    """q, k [T, H, d], v [T, H, e], g and beta [T, H]: o [T, H, e] and the last state [H, d, e]."""
    T, H, d = q.shape
    S = q.new_zeros(H, d, v.shape[2])
    out = []
    for t in range(T):
        S = g[t][:, None, None] * S
        u = beta[t][:, None] * (v[t] - (S * k[t][:, :, None]).sum(1))
        S = S + k[t][:, :, None] * u[:, None, :]
        out.append((S * q[t][:, :, None]).sum(1))
    return torch.stack(out), S


def gated_delta(h, w, c, eps):
    T, H, K, d, e = h.shape[0], c["heads"], c["kv_heads"], c["dim"], c["vdim"]
    q, k, v = (silu(causal_conv(h @ w[n].T, w[n + ".conv"])) for n in "qkv")
    q, k = unit(q.view(T, K, d)) * d ** -0.5, unit(k.view(T, K, d))
    q, k = (x.repeat_interleave(H // K, dim=1) for x in (q, k))
    beta = torch.sigmoid(h @ w["b"].T)
    g = torch.exp(-torch.exp(w["A_log"]) * torch.nn.functional.softplus(h @ w["a"].T + w["dt_bias"]))
    o, _ = delta_rule(q, k, v.view(T, H, e), g, beta)
    o = rms(o, eps) * w["norm"] * silu(h @ w["g"].T).view(T, H, e)
    return o.reshape(T, H * e) @ w["o"].T


def feed_forward(h, w):
    return (silu(h @ w["gate"].T) * (h @ w["up"].T)) @ w["down"].T


def _below(weights, prefix):
    return {k[len(prefix):]: v for k, v in weights.items() if k.startswith(prefix)}


def mixer(h, w, c, eps):
    return (c["left_scale"] * attention(h, _below(w, "left."), c["left"], eps)
            + c["right_scale"] * gated_delta(h, _below(w, "right."), c["right"], eps))


def forward(cfg, weights, tokens, dtype=torch.float64):
    """Returns (logits [T, vocab], list of the residual stream after every layer)."""
    w = {k: v.to(dtype) for k, v in weights.items()}
    eps = cfg["norm"]["eps"]
    x = w["embed"][torch.as_tensor(tokens, dtype=torch.long)]
    stream = []
    for i, L in enumerate(cfg["layers"]):
        lw = _below(w, f"l{i}.")
        x = x + mixer(norm_one_plus(x, lw["norm1"], eps), _below(lw, "mix."), L["mixer"], eps)
        if L["mlp"]:
            x = x + feed_forward(norm_one_plus(x, lw["norm2"], eps), _below(lw, "mlp."))
        stream.append(x)
    return norm_one_plus(x, w["final.norm"], eps) @ w["head"].T * cfg["logit_scale"], stream
