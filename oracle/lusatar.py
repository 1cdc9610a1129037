"""TEST INFRASTRUCTURE ONLY: a plain, slow restatement of the Lusatar decoder, one function per mechanism.

One sequence at a time, whole prompt, no cache, no batching: every function takes the rows of one sequence and returns
the rows of one sequence.  Runs in the dtype of its inputs (the tests use float64).  Shares no code with the package.
"""
from __future__ import annotations

import math

import torch


def rms_norm(x, w, eps):
    y = x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)
    return y if w is None else y * w


def gelu_tanh(z):
    return 0.5 * z * (1 + torch.tanh(math.sqrt(2 / math.pi) * (z + 0.044715 * z ** 3)))


def relu2(z):
    return torch.clamp(z, min=0) ** 2


def softcap(z, cap):
    return z if not cap else cap * torch.tanh(z / cap)


def rotary_frequencies(base, dims, scaling):
    """(dims / 2 frequencies, factor on cos and sin): plain rotation, or the blend of the plain and the stretched
    frequencies that YaRN prescribes."""
    f = [base ** (-2.0 * i / dims) for i in range(dims // 2)]
    if not scaling:
        return f, 1.0

    def dim_of_turns(t):
        return dims * math.log(scaling["original"] / (2 * math.pi * t)) / (2 * math.log(base))

    lo = max(math.floor(dim_of_turns(scaling["fast"])), 0)
    hi = min(math.ceil(dim_of_turns(scaling["slow"])), dims - 1)
    out = []
    for i, fi in enumerate(f):
        ramp = min(max((i - lo) / max(hi - lo, 0.001), 0.0), 1.0)
        out.append(fi / scaling["factor"] * ramp + fi * (1 - ramp))
    return out, 0.1 * math.log(scaling["factor"]) + 1


def rotate(v, positions, base, dims, scaling):
    """v [T, ..., d]: element i < dims/2 turns together with element i + dims/2; elements from dims on stay."""
    freqs, mag = rotary_frequencies(base, dims, scaling)
    out = v.clone()
    shape = [-1] + [1] * (v.dim() - 2)
    for i, f in enumerate(freqs):
        a = positions.to(v.dtype) * f
        c, s = (mag * torch.cos(a)).view(shape), (mag * torch.sin(a)).view(shape)
        x, y = v[..., i], v[..., i + dims // 2]
        out[..., i] = x * c - y * s
        out[..., i + dims // 2] = y * c + x * s
    return out


def window_attention(q, k, v, scale, window):
    """q, k [T, H, d], v [T, H, dv]: softmax over the keys j with 0 <= i - j < window (all j <= i without one)."""
    T = q.shape[0]
    i = torch.arange(T)[:, None]
    j = torch.arange(T)[None, :]
    seen = (j <= i) if not window else (j <= i) & (i - j < window)
    s = torch.einsum("ihd,jhd->hij", q, k) * scale
    s = s.masked_fill(~seen, -math.inf)
    return torch.einsum("hij,jhd->ihd", torch.softmax(s, -1), v)


def latent_attention(h, w, c, eps):
    """w: tensors by their names below the mixer; c: the mixer's sizes."""
    T, H, R = h.shape[0], c["heads"], c["kv_rank"]
    pos = torch.arange(T)
    rot = c["rot"]
    cq = rms_norm(h @ w["dq"].T, w["dq.norm"], eps)
    q = (cq @ w["uq"].T).view(T, H, c["dim"] + c["rot_dim"])
    down = h @ w["dkv"].T
    lat = rms_norm(down[:, :R], w["dkv.norm"], eps)
    k_rot = rotate(down[:, R:], pos, rot["base"], rot["dims"], rot.get("scaling"))
    q_rot = rotate(q[..., c["dim"]:], pos, rot["base"], rot["dims"], rot.get("scaling"))
    k = torch.cat([(lat @ w["uk"].T).view(T, H, c["dim"]), k_rot[:, None, :].expand(T, H, c["rot_dim"])], -1)
    v = (lat @ w["uv"].T).view(T, H, c["vdim"])
    q = torch.cat([q[..., :c["dim"]], q_rot], -1)
    window = c["mask"]["size"] if c.get("mask") else None
    o = window_attention(q, k, v, c["scale"], window)
    return o.reshape(T, H * c["vdim"]) @ w["o"].T


def causal_conv(x, w, b):
    """x [T, C], w [C, taps] (last column: the token itself)."""
    T, taps = x.shape[0], w.shape[1]
    padded = torch.cat([x.new_zeros(taps - 1, x.shape[1]), x])
    y = sum(padded[t: t + T] * w[:, t] for t in range(taps))
    return y + b


def gated_linear_recurrence(u, w, c):
    """The real-gated linear recurrent unit over u [T, width]: returns the states S_1 .. S_T."""
    T, nb = u.shape[0], c["blocks"]
    ub = u.view(T, nb, -1)
    r = torch.sigmoid(torch.einsum("tbi,boi->tbo", ub, w["ra"]) + w["ra.b"]).reshape(T, -1)
    i = torch.sigmoid(torch.einsum("tbi,boi->tbo", ub, w["ri"]) + w["ri.b"]).reshape(T, -1)
    a = torch.exp(-8.0 * r * torch.nn.functional.softplus(w["lam"]))
    S = torch.zeros_like(u[0])
    out = []
    for t in range(T):
        S = a[t] * S + torch.sqrt(1 - a[t] ** 2) * i[t] * u[t]
        out.append(S)
    return torch.stack(out)


def rglru(h, w, c):
    y = gelu_tanh(h @ w["y"].T + w["y.b"])
    u = causal_conv(h @ w["x"].T + w["x.b"], w["conv"], w["conv.b"])
    return (gated_linear_recurrence(u, w, c) * y) @ w["o"].T


def feed_forward(h, w):
    return relu2(h @ w["up"].T) @ w["down"].T


def _below(weights, prefix):
    return {k[len(prefix):]: v for k, v in weights.items() if k.startswith(prefix)}


def forward(cfg, weights, tokens, dtype=torch.float64):
    """Returns (logits [T, vocab], list of the residual stream after every layer run)."""
    w = {k: v.to(dtype) for k, v in weights.items()}
    eps = cfg["norm"]["eps"]
    x0 = w["embed"][torch.as_tensor(tokens, dtype=torch.long)] * cfg["embedding"]["scale"]
    x = x0
    loop = cfg.get("loop")
    order = []                                        # (layer, pass it opens or None)
    i = 0
    while i < len(cfg["layers"]):
        if loop and i == loop["start"] and loop["stop"] > loop["start"]:
            for t in range(loop["times"]):
                order += [(j, t if j == loop["start"] else None) for j in range(loop["start"], loop["stop"])]
            i = loop["stop"]
        else:
            order.append((i, None))
            i += 1
    stream = []
    for li, opens in order:
        if opens is not None:
            if opens > 0:
                x = x + x0
            x = x + w["loop.step"][opens]
        L = cfg["layers"][li]
        lw = _below(w, f"l{li}.")
        mixer = latent_attention if L["type"] == "latent_attention" else rglru
        args = (eps,) if L["type"] == "latent_attention" else ()
        x = x + rms_norm(mixer(rms_norm(x, lw["norm1"], eps), _below(lw, "mix."), L["mixer"], *args), lw["norm1b"], eps)
        if L["mlp"]:
            x = x + rms_norm(feed_forward(rms_norm(x, lw["norm2"], eps), _below(lw, "mlp.")), lw["norm2b"], eps)
        stream.append(x)
    logits = rms_norm(x, w["final.norm"], eps) @ w["embed"].T
    return softcap(logits, cfg.get("logit_softcap")), stream
