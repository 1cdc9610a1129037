"""Lusatar: a decoder that mixes windowed latent attention and gated linear recurrences.

Every sublayer is normalised on both sides, x += norm_b(sublayer(norm_a(x))), over an fp32 residual stream; feed-forwards
are un-gated (square of relu) and may be missing; a range of layers can run several times in a row with the same weights,
each run with a cache or state of its own, the embedding output and a learned vector added in front; the embedding table
is also the output matrix, behind a tanh cap.  All sizes and constants come from config.json.
"""
from __future__ import annotations

import dataclasses
from typing import List, Optional

import torch

from .. import ops_hybrid as hops
from ..layers.feed_forward import FeedForward
from ..layers.latent_attention import LatentAttention
from ..layers.linear import Linear, pad, padded, vector
from ..layers.rglru import Rglru
from ..layers.rotary import rotary_table
from .output import output_logits


@dataclasses.dataclass
class LayerRun:
    """One run of a layer: which one, and the pass of the repeated range it opens (None: none)."""
    layer: int
    opens: Optional[int]


def layer_runs(layers: int, loop: Optional[dict]) -> List[LayerRun]:
    """The order in which the layers run; `loop`: layers start .. stop - 1 run `times` times in a row."""
    runs, i = [], 0
    start, stop, times = (loop["start"], loop["stop"], loop["times"]) if loop else (layers, layers, 0)
    if not 0 <= start <= stop <= layers:
        raise ValueError(f"loop over layers {start} .. {stop} of {layers}")
    while i < layers:
        if i == start and stop > start:
            runs += [LayerRun(j, t if j == start else None) for t in range(times) for j in range(start, stop)]
            i = stop
        else:
            runs.append(LayerRun(i, None))
            i += 1
    if not runs:
        raise ValueError("the configuration runs no layer")
    return runs


def tensor_shapes(config: dict) -> dict:
    """Shape of every tensor of a checkpoint with this configuration, by name."""
    D, loop = config["width"], config.get("loop")
    out = {"embed": (config["vocab"], D), "final.norm": (D,)}
    if loop:
        out["loop.step"] = (loop["times"], D)
    for i, c in enumerate(config["layers"]):
        m = c["mixer"]
        if c["type"] == "latent_attention":
            H, R = m["heads"], m["kv_rank"]
            mix = {"dq": (m["q_rank"], D), "dq.norm": (m["q_rank"],), "uq": (H * (m["dim"] + m["rot_dim"]), m["q_rank"]),
                   "dkv": (R + m["rot_dim"], D), "dkv.norm": (R,), "uk": (H * m["dim"], R), "uv": (H * m["vdim"], R),
                   "o": (D, H * m["vdim"])}
        elif c["type"] == "rglru":
            W, nb = m["width"], m["blocks"]
            if W % nb:
                raise ValueError(f"layer {i}: {W} channels in {nb} blocks")
            bw = W // nb
            mix = {"y": (W, D), "y.b": (W,), "x": (W, D), "x.b": (W,), "conv": (W, m["conv"]), "conv.b": (W,), "ra": (nb, bw, bw),
                   "ra.b": (nb, bw), "ri": (nb, bw, bw), "ri.b": (nb, bw), "lam": (W,), "o": (D, W)}
        else:
            raise ValueError(f"layer {i}: unknown mixer {c['type']!r}")
        out.update({f"l{i}.mix.{k}": s for k, s in mix.items()})
        norms = ["norm1", "norm1b"]
        if c.get("mlp"):
            if c["mlp"]["kind"] != "dense":
                raise ValueError(f"layer {i}: unknown feed-forward {c['mlp']['kind']!r}")
            ff = c["mlp"]["ff"]
            out[f"l{i}.mlp.up"], out[f"l{i}.mlp.down"] = (ff, D), (D, ff)
            norms += ["norm2", "norm2b"]
        out.update({f"l{i}.{n}": (D,) for n in norms})
    return out


class _Layer:
    """Weights of one layer."""

    def __init__(self, model: "Lusatar", i: int, c: dict, get):
        pitch, m = model.pitch, c["mixer"]
        norm = lambda n: vector(get(f"l{i}.{n}", torch.float32), pitch)
        mix = lambda n: get(f"l{i}.mix.{n}")
        self.kind = c["type"]
        self.norm1, self.norm1b = norm("norm1"), norm("norm1b")
        if self.kind == "latent_attention":
            rot = m["rot"]
            self.mixer = LatentAttention(m, mix, pitch, model.eps, model.dtype, model.device,
                                         model.rotary(rot["dims"], rot["base"], rot.get("scaling")))
        else:
            self.mixer = Rglru(m, mix, pitch, model.dtype)
        self.mlp = None
        if c.get("mlp"):
            self.norm2, self.norm2b = norm("norm2"), norm("norm2b")
            self.mlp = FeedForward(get(f"l{i}.mlp.up"), get(f"l{i}.mlp.down"), pitch)

    def cache_spec(self):
        if self.kind == "latent_attention":
            return ("latent", *self.mixer.cache_row)
        return ("recurrent", self.mixer.W, self.mixer.w.taps)


class Lusatar:
    tensor_shapes = staticmethod(tensor_shapes)

    def __init__(self, config: dict, weights, dtype: torch.dtype, device, max_context: int):
        if dtype not in (torch.bfloat16, torch.float32):
            raise ValueError("Lusatar runs in bfloat16 or float32")
        self.config, self.dtype, self.device, self.max_context = config, dtype, device, max_context
        self.width, self.vocab, self.eps = config["width"], config["vocab"], config["norm"]["eps"]
        self.pitch = pad(self.width, 128)
        self.embed_scale = config["embedding"]["scale"]
        self.logit_cap = config.get("logit_softcap")
        self._tables = {}
        shapes = tensor_shapes(config)
        get = lambda name, dt=None: weights.get(name, shapes[name], dt)
        table = padded(get("embed"), pad(self.vocab, 16), self.pitch)
        self.head = Linear(table)                         # the row-major copy is also the embedding table
        self.layers = [_Layer(self, i, c, get) for i, c in enumerate(config["layers"])]
        loop = config.get("loop")
        self.runs = layer_runs(len(self.layers), loop)
        self.loop_step = None
        if loop:
            steps = get("loop.step", torch.float32)
            self.loop_step = [vector(s, self.pitch) for s in steps]
        self.repeats = any(r.opens for r in self.runs)    # a pass after the first: the embedding output is kept
        self.final_norm = vector(get("final.norm", torch.float32), self.pitch)
        self._tables.clear()

    def rotary(self, dims, base, scaling):
        key = (dims, base, tuple(sorted(scaling.items())) if scaling else None)
        if key not in self._tables:
            self._tables[key] = rotary_table(dims, base, self.max_context, self.device, scaling)
        return self._tables[key]

    def cache_layers(self):
        """Per layer run, what it keeps between steps (mem_cache.HybridCache)."""
        return [self.layers[r.layer].cache_spec() for r in self.runs]

    def weight_bytes(self) -> int:
        """Bytes of matrix weights a step over all layer runs reads."""
        per = [L.mixer.bytes() + (L.mlp.bytes() if L.mlp else 0) for L in self.layers]
        return sum(per[r.layer] for r in self.runs) + self.head.bytes()

    def forward(self, batch, cache, collect: Optional[list] = None):
        """One step over the rows of `batch`: the cache and states advance, returns fp32 logits [wanted rows, vocab]
        (None if no row is wanted).  collect: receives the residual stream after every layer run."""
        T, dev, D = batch.T, self.device, self.width
        x = torch.empty(T, self.pitch, dtype=torch.float32, device=dev)
        x0 = torch.empty_like(x) if self.repeats else None
        h = torch.empty(T, self.pitch, dtype=self.dtype, device=dev)
        norm = lambda **kw: hops.residual_norm(x, D, self.eps, dtype=self.dtype, **kw)
        pending = dict(embed=self.head.weight, ids=batch.ids, embed_scale=self.embed_scale, x0=x0)  # joins x at the next norm

        def opening(r):
            add = {}
            if r.opens is not None:
                add["step"] = self.loop_step[r.opens]
                if r.opens > 0:
                    add.update(x0=x0, add_x0=True)
            return add

        for n, r in enumerate(self.runs):
            L, pool = self.layers[r.layer], cache.layers[n]
            if collect is not None:
                norm(**pending)
                if n:
                    collect.append(x[:, :D].clone())
                pending = {}
            norm(**{**pending, **opening(r)}, h=h, w_next=L.norm1)
            if L.kind == "latent_attention":
                src = L.mixer.forward(h, batch, pool.get_key_buffer(0)[:, 0])
            else:
                src = L.mixer.forward(h, batch, pool)
            if L.mlp is not None:
                norm(src=src, w_post=L.norm1b, h=h, w_next=L.norm2)
                pending = dict(src=L.mlp.forward(h), w_post=L.norm2b)
            else:
                pending = dict(src=src, w_post=L.norm1b)
        if collect is not None:
            norm(**pending)
            collect.append(x[:, :D].clone())
            pending = {}
        W = batch.wanted
        if W == 0:
            return None
        norm(**pending, h=h, w_next=self.final_norm, rows=batch.logit_rows, store_x=False)
        return output_logits(self.head, h, W, self.vocab, self.logit_cap)
