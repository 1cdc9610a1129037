"""Kazedra: a pre-norm decoder whose layers run attention and a gated delta rule side by side.

Attention uses its keys (before their norm) as values, knows positions by a learned bias over distances and a temperature
on the query, and has a sink; feed-forwards are gated (silu) and may be missing.  Norm weights are stored around zero.
The residual stream is fp32.  All sizes and constants come from config.json.
"""
from __future__ import annotations

from typing import Optional

import torch

from .. import ops_hybrid as hops
from ..layers.feed_forward import GatedFeedForward
from ..layers.gated_delta import GatedDelta
from ..layers.linear import Linear, pad, padded, vector
from ..layers.parallel import Parallel
from ..layers.position_bias import temperature
from ..layers.tied_attention import TiedAttention
from .output import output_logits


def tensor_shapes(config: dict) -> dict:
    """Shape of every tensor of a checkpoint with this configuration, by name (None: the tensor gives the size)."""
    D, V = config["width"], config["vocab"]
    out = {"embed": (V, D), "head": (V, D), "final.norm": (D,)}
    for i, c in enumerate(config["layers"]):
        if c["type"] != "parallel":
            raise ValueError(f"layer {i}: unknown mixer {c['type']!r}")
        a, r = c["mixer"]["left"], c["mixer"]["right"]
        if a.get("vdim", a["dim"]) != a["dim"]:
            raise ValueError(f"layer {i}: values of {a['vdim']} elements cannot be keys of {a['dim']}")
        nq, nk = a["heads"] * a["dim"], a["kv_heads"] * a["dim"]
        mix = {"left.q": (nq, D), "left.q.b": (nq,), "left.k": (nk, D), "left.k.b": (nk,), "left.q.norm": (nq,), "left.k.norm": (nk,),
               "left.rel": (None, a["heads"]), "left.sink": (a["heads"],), "left.o": (D, nq), "left.o.b": (D,)}
        H, taps = r["heads"], r["conv"]
        for name, n in (("q", r["kv_heads"] * r["dim"]), ("k", r["kv_heads"] * r["dim"]), ("v", H * r["vdim"])):
            mix["right." + name], mix[f"right.{name}.conv"] = (n, D), (n, taps)
        mix.update({"right.b": (H, D), "right.a": (H, D), "right.A_log": (H,), "right.dt_bias": (H,), "right.norm": (r["vdim"],),
                    "right.g": (H * r["vdim"], D), "right.o": (D, H * r["vdim"])})
        out.update({f"l{i}.mix.{k}": s for k, s in mix.items()})
        out[f"l{i}.norm1"] = (D,)
        if c.get("mlp"):
            if c["mlp"]["kind"] != "dense":
                raise ValueError(f"layer {i}: unknown feed-forward {c['mlp']['kind']!r}")
            ff = c["mlp"]["ff"]
            out.update({f"l{i}.norm2": (D,), f"l{i}.mlp.gate": (ff, D), f"l{i}.mlp.up": (ff, D), f"l{i}.mlp.down": (D, ff)})
    return out


class _Layer:
    """Weights of one layer."""

    def __init__(self, model: "Kazedra", i: int, c: dict, get):
        m, pitch = c["mixer"], model.pitch
        below = lambda side: lambda name, dt=None: get(f"l{i}.mix.{side}.{name}", dt)
        self.norm1 = model.norm_weight(get(f"l{i}.norm1", torch.float32))
        self.mixer = Parallel([
            TiedAttention(m["left"], below("left"), pitch, model.eps, model.dtype, model.temperature(m["left"].get("q_temp")),
                          model.max_context, m["left_scale"]),
            GatedDelta(m["right"], below("right"), pitch, model.eps, model.dtype, m["right_scale"])], pitch, model.dtype)
        self.mlp = None
        if c.get("mlp"):
            self.norm2 = model.norm_weight(get(f"l{i}.norm2", torch.float32))
            self.mlp = GatedFeedForward(*(get(f"l{i}.mlp.{n}") for n in ("gate", "up", "down")), pitch)


class Kazedra:
    tensor_shapes = staticmethod(tensor_shapes)

    def __init__(self, config: dict, weights, dtype: torch.dtype, device, max_context: int):
        if dtype not in (torch.bfloat16, torch.float32):
            raise ValueError("Kazedra runs in bfloat16 or float32")
        self.config, self.dtype, self.device, self.max_context = config, dtype, device, max_context
        self.width, self.vocab, self.eps = config["width"], config["vocab"], config["norm"]["eps"]
        self.pitch = pad(self.width, 128)
        self._tables = {}
        shapes = tensor_shapes(config)
        get = lambda name, dt=None: weights.get(name, shapes[name], dt)
        self.embed = padded(get("embed"), self.vocab, self.pitch)
        self.head = Linear(padded(get("head"), pad(self.vocab, 16), self.pitch))
        self.layers = [_Layer(self, i, c, get) for i, c in enumerate(config["layers"])]
        # the factor on the logits joins the last norm's weight, in fp32
        self.final_norm = self.norm_weight(get("final.norm", torch.float32)) * config["logit_scale"]
        self._tables.clear()

    def norm_weight(self, w: torch.Tensor) -> torch.Tensor:
        return vector(1 + w, self.pitch)

    def temperature(self, c: Optional[dict]) -> torch.Tensor:
        key = (c["coef"], c["every"]) if c else None
        if key not in self._tables:
            self._tables[key] = temperature(c, self.max_context, self.device)
        return self._tables[key]

    def cache_layers(self):
        """Per layer, what it keeps between steps (mem_cache.HybridCache)."""
        return [L.mixer.cache_spec for L in self.layers]

    def weight_bytes(self) -> int:
        """Bytes of matrix weights a step reads."""
        return sum(L.mixer.bytes() + (L.mlp.bytes() if L.mlp else 0) for L in self.layers) + self.head.bytes()

    def forward(self, batch, cache, collect: Optional[list] = None):
        """One step over the rows of `batch`: the caches and states advance, returns fp32 logits [wanted rows, vocab]
        (None if no row is wanted).  collect: receives the residual stream after every layer."""
        T, dev, D = batch.T, self.device, self.width
        x = torch.empty(T, self.pitch, dtype=torch.float32, device=dev)
        h = torch.empty(T, self.pitch, dtype=self.dtype, device=dev)
        norm = lambda **kw: hops.residual_norm(x, D, self.eps, dtype=self.dtype, **kw)
        pending = dict(embed=self.embed, ids=batch.ids)           # joins x at the next norm
        for n, (L, pools) in enumerate(zip(self.layers, cache.layers)):
            norm(**pending, h=h, w_next=L.norm1)
            if collect is not None and n:
                collect.append(x[:, :D].clone())
            pending = dict(src=L.mixer.forward(h, batch, pools), step=L.mixer.bias)
            if L.mlp is not None:
                norm(**pending, h=h, w_next=L.norm2)
                pending = dict(src=L.mlp.forward(h))
        if collect is not None:
            norm(**pending)
            collect.append(x[:, :D].clone())
            pending = {}
        if batch.wanted == 0:
            return None
        norm(**pending, h=h, w_next=self.final_norm, rows=batch.logit_rows, store_x=False)
        return output_logits(self.head, h, batch.wanted, self.vocab)
