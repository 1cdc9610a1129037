"""Small random Kazedra configurations and weights for the tests."""
import math

import torch


def layer(heads=6, kv_heads=2, dim=24, bias_max=40, buckets=10, temp=(0.3, 7), scale=None, r_heads=6, r_kv=3, r_dim=20, r_vdim=12, conv=4,
          ff=72, scales=(0.7, 1.3)):
    return {"type": "parallel",
            "mixer": {"left": {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": dim, "bias_max": bias_max,
                               "q_temp": {"coef": temp[0], "every": temp[1]}, "scale": scale or 1.3 / math.sqrt(dim)},
                      "right": {"heads": r_heads, "kv_heads": r_kv, "dim": r_dim, "vdim": r_vdim, "conv": conv},
                      "left_scale": scales[0], "right_scale": scales[1]},
            "mlp": {"kind": "dense", "ff": ff} if ff else None, "buckets": buckets}


def config(layers, width=84, vocab=131, eps=1e-5, logit_scale=1.7):
    return {"architecture": "Kazedra", "layers": layers, "norm": {"eps": eps}, "vocab": vocab, "width": width, "logit_scale": logit_scale}


CONFIGS = {
    # grouped heads, layers of different sizes, one without a feed-forward; heads padded for the tiles
    "mixed": config([layer(), layer(heads=4, kv_heads=4, dim=40, bias_max=90, buckets=7, r_heads=3, r_kv=3, r_dim=33, r_vdim=40, conv=3, ff=0),
                     layer(heads=5, kv_heads=1, dim=32, buckets=2, temp=(1.1, 64), r_heads=4, r_kv=1, r_dim=32, r_vdim=16)]),
    # more query heads than a tile, one and two taps, a bias that reaches beyond the prompts, everything scaled by one
    "wide": config([layer(heads=18, kv_heads=1, dim=64, bias_max=1000, buckets=32, r_heads=2, r_kv=1, r_dim=64, r_vdim=64, conv=1, scales=(1.0, 1.0)),
                    layer(heads=40, kv_heads=2, dim=16, bias_max=33, buckets=16, temp=(0.0, 1), conv=2)], width=128, vocab=64, logit_scale=1.0),
    # full-size heads, as many key heads as value heads, long filters
    "full": config([layer(heads=2, kv_heads=1, dim=128, r_heads=2, r_kv=2, r_dim=128, r_vdim=128, conv=6, ff=130),
                    layer(heads=2, kv_heads=2, dim=192, r_heads=3, r_kv=1, r_dim=96, r_vdim=80, buckets=64, bias_max=256)],
                   width=100, vocab=257, eps=1e-3, logit_scale=0.4),
    # sizes no tile kernel takes
    "large": config([layer(heads=2, kv_heads=1, dim=260, r_heads=2, r_kv=1, r_dim=150, r_vdim=300, ff=33)], width=50, vocab=77),
}


def weights(cfg, seed=0):
    g = torch.Generator().manual_seed(seed)
    D, w = cfg["width"], {}

    def put(name, *shape, by=None, mean=0.0):
        t = torch.randn(shape, generator=g) * (by if by is not None else 1.4 / math.sqrt(shape[-1])) + mean
        w[name] = t.to(torch.bfloat16)

    put("embed", cfg["vocab"], D, by=1.0)
    put("head", cfg["vocab"], D)
    put("final.norm", D, by=0.3)
    for i, L in enumerate(cfg["layers"]):
        a, r, p = L["mixer"]["left"], L["mixer"]["right"], f"l{i}."
        put(p + "norm1", D, by=0.3)
        m = p + "mix.left."
        for n, rows in (("q", a["heads"] * a["dim"]), ("k", a["kv_heads"] * a["dim"])):
            put(m + n, rows, D)
            put(m + n + ".b", rows, by=0.4)
            put(m + n + ".norm", rows, by=0.3, mean=1.0)
        put(m + "rel", L["buckets"], a["heads"], by=1.5)
        put(m + "sink", a["heads"], by=1.0, mean=1.0)
        put(m + "o", D, a["heads"] * a["dim"])
        put(m + "o.b", D, by=0.3)
        m = p + "mix.right."
        for n, rows in (("q", r["kv_heads"] * r["dim"]), ("k", r["kv_heads"] * r["dim"]), ("v", r["heads"] * r["vdim"])):
            put(m + n, rows, D)
            put(m + n + ".conv", rows, r["conv"], by=0.6)
        put(m + "b", r["heads"], D)
        put(m + "a", r["heads"], D)
        put(m + "A_log", r["heads"], by=1.0, mean=-1.5)
        put(m + "dt_bias", r["heads"], by=1.0, mean=-1.0)
        put(m + "norm", r["vdim"], by=0.3, mean=1.0)
        put(m + "g", r["heads"] * r["vdim"], D)
        put(m + "o", D, r["heads"] * r["vdim"])
        if L["mlp"]:
            put(p + "norm2", D, by=0.3)
            ff = L["mlp"]["ff"]
            put(p + "mlp.gate", ff, D)
            put(p + "mlp.up", ff, D)
            put(p + "mlp.down", D, ff)
    return w
