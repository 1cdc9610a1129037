"""Small random Lusatar configurations and weights for the tests, and comparison helpers."""
import json
import math
import os
import struct

import torch

YARN = {"factor": 4.0, "original": 96, "fast": 8.0, "slow": 0.5}


def attention(heads=3, dim=24, rot_dim=8, vdim=20, q_rank=28, kv_rank=36, size=21, ff=72, scaling=YARN, base=1000.0, scale=None):
    return {"type": "latent_attention",
            "mixer": {"heads": heads, "dim": dim, "rot_dim": rot_dim, "vdim": vdim, "q_rank": q_rank, "kv_rank": kv_rank,
                      "mask": {"size": size} if size else None, "rot": {"base": base, "dims": rot_dim, "scaling": scaling},
                      "scale": scale if scale is not None else 1.7 / math.sqrt(dim + rot_dim)},
            "mlp": {"kind": "dense", "ff": ff} if ff else None}


def recurrent(width=60, blocks=3, conv=4, ff=0):
    return {"type": "rglru", "mixer": {"width": width, "blocks": blocks, "conv": conv},
            "mlp": {"kind": "dense", "ff": ff} if ff else None}


def config(layers, width=84, vocab=131, loop=None, cap=9.0, eps=1e-5, embed_scale=3.1):
    return {"architecture": "Lusatar", "embedding": {"scale": embed_scale}, "layers": layers, "logit_softcap": cap, "loop": loop,
            "norm": {"eps": eps}, "vocab": vocab, "width": width}


CONFIGS = {
    # recurrent and attention layers with and without feed-forwards, different windows, a loop over the middle
    "mixed": config([recurrent(ff=40), attention(), attention(size=5, ff=0, heads=2, vdim=12), recurrent(width=44, blocks=1, conv=3)],
                    loop={"start": 1, "stop": 3, "times": 3}),
    # no loop, no cap, plain rotation, no window, one head, convolution of one and two taps
    "plain": config([attention(heads=1, size=None, scaling=None, dim=16, rot_dim=16, vdim=40), recurrent(conv=1, blocks=4, width=64),
                     recurrent(conv=2, blocks=2, width=128, ff=64)], width=128, vocab=64, cap=None),
    # everything runs twice; windows of one token and beyond the prompts; more heads than a tile
    "looped": config([attention(heads=18, size=1, kv_rank=70, dim=10, vdim=70), attention(size=300, q_rank=130, ff=130),
                      recurrent(width=96, blocks=2, conv=6)], width=100, vocab=257, loop={"start": 0, "stop": 3, "times": 2}),
    # one pass of a loop at the end, wide heads
    "tail": config([recurrent(width=72, blocks=6), attention(heads=2, dim=72, rot_dim=40, vdim=136, kv_rank=150, size=40)],
                   width=64, vocab=100, loop={"start": 1, "stop": 2, "times": 1}, cap=30.0, eps=1e-3),
    # sizes no tile kernel takes, odd widths, a loop that runs nothing extra
    "large": config([attention(heads=2, dim=260, rot_dim=72, vdim=300, kv_rank=530, size=33, ff=33), recurrent(width=1056, blocks=1)],
                    width=50, vocab=77, loop={"start": 1, "stop": 1, "times": 2}),
}


def tensor_shapes(cfg):
    D, out = cfg["width"], {"embed": (cfg["vocab"], cfg["width"]), "final.norm": (cfg["width"],)}
    if cfg.get("loop"):
        out["loop.step"] = (cfg["loop"]["times"], D)
    for i, L in enumerate(cfg["layers"]):
        m, mix = L["mixer"], {}
        if L["type"] == "latent_attention":
            H = m["heads"]
            mix = {"dq": (m["q_rank"], D), "dq.norm": (m["q_rank"],), "uq": (H * (m["dim"] + m["rot_dim"]), m["q_rank"]),
                   "dkv": (m["kv_rank"] + m["rot_dim"], D), "dkv.norm": (m["kv_rank"],), "uk": (H * m["dim"], m["kv_rank"]),
                   "uv": (H * m["vdim"], m["kv_rank"]), "o": (D, H * m["vdim"])}
        else:
            W, nb = m["width"], m["blocks"]
            mix = {"y": (W, D), "y.b": (W,), "x": (W, D), "x.b": (W,), "conv": (W, m["conv"]), "conv.b": (W,),
                   "ra": (nb, W // nb, W // nb), "ra.b": (nb, W // nb), "ri": (nb, W // nb, W // nb), "ri.b": (nb, W // nb),
                   "lam": (W,), "o": (D, W)}
        for k, s in mix.items():
            out[f"l{i}.mix.{k}"] = s
        norms = ["norm1", "norm1b"]
        if L["mlp"]:
            norms += ["norm2", "norm2b"]
            out[f"l{i}.mlp.up"], out[f"l{i}.mlp.down"] = (L["mlp"]["ff"], D), (D, L["mlp"]["ff"])
        for n in norms:
            out[f"l{i}.{n}"] = (D,)
    return out


def weights(cfg, seed=0):
    g = torch.Generator().manual_seed(seed)
    w = {}
    for name, shape in tensor_shapes(cfg).items():
        t = torch.randn(shape, generator=g)
        leaf = name.split(".")[-1]
        if "norm" in leaf:
            t = 1 + 0.3 * t
        elif leaf == "lam":
            t = t * 1.5 - 1.0
        elif leaf == "b" or name == "loop.step":
            t = 0.4 * t
        elif leaf == "conv":
            t = 0.6 * t
        elif name == "embed":
            t = t / math.sqrt(shape[1]) * 1.5
        else:
            t = t / math.sqrt(shape[-1]) * 1.4
        w[name] = t.to(torch.bfloat16)
    return w


def tokens(cfg, n, seed=0):
    return torch.randint(0, cfg["vocab"], (n,), generator=torch.Generator().manual_seed(1000 + seed)).tolist()


def save(folder, cfg, w):
    """config.json and model.safetensors as a checkpoint folder holds them."""
    os.makedirs(folder, exist_ok=True)
    with open(os.path.join(folder, "config.json"), "w") as f:
        json.dump(cfg, f)
    header, blob, at = {"__metadata__": {"format": "pt"}}, b"", 0
    for name, t in w.items():
        raw = t.contiguous().view(torch.uint8).numpy().tobytes() if t.dtype != torch.bfloat16 else \
            t.contiguous().view(torch.int16).numpy().tobytes()
        header[name] = {"dtype": {"torch.bfloat16": "BF16", "torch.float32": "F32", "torch.int32": "I32"}[str(t.dtype)],
                        "shape": list(t.shape), "data_offsets": [at, at + len(raw)]}
        blob += raw
        at += len(raw)
    head = json.dumps(header).encode()
    with open(os.path.join(folder, "model.safetensors"), "wb") as f:
        f.write(struct.pack("<Q", len(head)) + head + blob)
    return folder


def rel_rms(got, want):
    """Per row: root mean square of the difference over that of all of `want`."""
    d = got.double().cpu() - want.double()
    return (d ** 2).mean(-1).sqrt() / (want.double() ** 2).mean().sqrt()
