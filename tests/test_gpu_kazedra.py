"""GPU: every mechanism of the Kazedra layers alone and the whole model through the engine, against the plain oracle
(oracle/kazedra.py, float64)."""
import functools
import json
import math
import subprocess
import sys

import pytest
import torch

import kazedra_models as K
import lusatar_models as M
from oracle import kazedra as O
from test_gpu_lusatar import _Batch, _root, close, cut, gen, i32, rnd, source

pytestmark = pytest.mark.gpu
DEV = "cuda"
BF16, F32 = torch.bfloat16, torch.float32
TOL = {BF16: 1e-2, F32: 3e-6}


# ---- row kernels --------------------------------------------------------------------------------------------------------
@pytest.mark.parametrize("dtype,splits", [(BF16, 0), (BF16, 5), (F32, 1)])
def test_gated_activation(dtype, splits):
    from sglang_security_amd import ops_hybrid as H

    src, sv = source(rnd(gen(splits), 7, 2 * 48) * 3, splits, dtype)
    out = torch.empty(7, 48, dtype=dtype, device=DEV)
    close(H.source_gated_act(src, out, H.ACT_SILU), O.silu(sv[:, :48]) * sv[:, 48:], TOL[dtype], "gated")


@pytest.mark.parametrize("dtype,splits", [(BF16, 0), (BF16, 3), (F32, 1)])
@pytest.mark.parametrize("H_,G,dim,D", [(6, 2, 24, 32), (1, 1, 128, 128), (18, 1, 64, 64), (5, 5, 100, 128), (64, 8, 128, 128)])
def test_tied_prep(dtype, splits, H_, G, dim, D):
    """Norms over whole projections, temperature and weight on the queries, plain rows and their factors into the pool."""
    from sglang_security_amd import ops_hybrid as H

    g, rows, eps = gen(H_ + splits), 5, 1e-3
    s = torch.zeros(rows, H_ + G, D)
    s[..., :dim] = rnd(g, rows, H_ + G, dim)
    bias, wq = torch.zeros(H_ + G, D), torch.zeros(H_, D)
    bias[:, :dim], wq[:, :dim] = rnd(g, H_ + G, dim), rnd(g, H_, dim)
    src, sv = source(s.view(rows, -1), splits, dtype)
    factor = rnd(g, 40).abs() + 0.5
    pos, loc = torch.tensor([0, 39, 7, 8, 20]), i32(8, 1, 3, 2, 7)
    pool, rms = torch.full((10, G * D), 5.0, dtype=dtype, device=DEV), torch.full((10,), 9.0, device=DEV)
    q = torch.empty(rows, H_ * D, dtype=dtype, device=DEV)
    H.tied_prep(src, bias.view(-1).to(DEV), wq.view(-1).to(DEV), factor.to(DEV), q, pool, rms, loc, pos.int().to(DEV), H_ * dim, G * dim, eps)
    x = sv + bias.view(-1).double()
    xq, xk = (t.view(rows, -1, D)[..., :dim].reshape(rows, -1) for t in (x[:, : H_ * D], x[:, H_ * D:]))
    want = O.rms(xq, eps) * wq[:, :dim].reshape(-1).double() * factor[pos].double()[:, None]
    close(q.view(rows, H_, D)[..., :dim].reshape(rows, -1), want, TOL[dtype], "queries")
    close(pool[loc.long()].view(rows, G, D)[..., :dim].reshape(rows, -1), xk, TOL[dtype], "rows")
    close(rms[loc.long()], 1 / torch.sqrt((xk ** 2).mean(-1) + eps), 3e-6, "factors")
    assert not q.view(rows, H_, D)[..., dim:].any() and not pool[loc.long()].view(rows, G, D)[..., dim:].any()
    assert bool((pool[[0, 4, 5, 6, 9]] == 5.0).all()) and bool((rms[[0, 4, 5, 6, 9]] == 9.0).all())


# ---- attention ------------------------------------------------------------------------------------------------------------
def _tied_case(g, lengths, H_, G, D, dim, buckets, longest, dtype, loud=()):
    """Requests with scattered slots: (request table, pool, factors, weights, rel, sink); loud: (request, position) whose key
    stands out."""
    from sglang_security_amd import ops_hybrid as H
    from sglang_security_amd.layers.position_bias import LOG2E, distance_table

    total = sum(lengths)
    slots = torch.randperm(total + 7, generator=g)[:total] + 1
    r2t = torch.zeros(len(lengths) + 1, max(lengths) + 3, dtype=torch.int32)
    pool, rms = torch.zeros(total + 9, G, D), rnd(g, total + 9).abs() + 0.5
    at = 0
    for b, n in enumerate(lengths):
        r2t[b + 1, :n] = slots[at: at + n].int()          # request row b + 1: row 0 is nobody's
        pool[slots[at: at + n].long(), :, :dim] = 0.5 * rnd(g, n, G, dim)
        at += n
    for b, p in loud:
        pool[int(r2t[b + 1, p])] *= 5.0
    rel, sink = 2.0 * rnd(g, buckets, H_), rnd(g, H_) + 1.0
    w = H.TiedWeights(bias=distance_table(rel, longest, max(lengths) + 3).to(DEV), sink=(sink * LOG2E).to(DEV), heads=H_, kv_heads=G, D=D)
    return r2t, pool.to(dtype), rms, w, rel, sink


def _tied_want(q, pool, rms, r2t, b, n, rel, longest, sink, first):
    """Rows first .. n - 1 of request b; q [n - first, H, D] in natural units."""
    v = pool[r2t[b + 1, :n].long()].double()
    k = v * rms[r2t[b + 1, :n].long()].double()[:, None, None]
    full = torch.cat([q.new_zeros(first, *q.shape[1:]).double(), q.double()])
    return O.tied_attention(full, k, v, 1.0, rel.double(), longest, sink.double())[first:]


TIED = [(6, 2, 32, 24, 10, 40), (7, 1, 64, 64, 14, 100), (2, 2, 96, 80, 4, 9), (40, 2, 128, 128, 32, 300), (3, 1, 192, 192, 2, 40),
        (18, 1, 64, 50, 64, 128), (2, 1, 256, 256, 12, 64)]


@pytest.mark.parametrize("H_,G,D,dim,buckets,longest", TIED)
def test_tied_decode(H_, G, D, dim, buckets, longest):
    """Rows at every kind of length; a key far back, the first one, and the row's own stand out."""
    from sglang_security_amd import ops_hybrid as H
    from sglang_security_amd.layers.position_bias import LOG2E

    g = gen(D + H_)
    lengths = [1, 2, 31, 32, 33, 64, 130, 401, longest, longest + 1, longest + 33]
    loud = [(6, 0), (7, 1), (7, 399), (8, 0), (9, 0), (10, 0), (4, 32), (5, 31)]
    r2t, pool, rms, w, rel, sink = _tied_case(g, lengths, H_, G, D, dim, buckets, longest, BF16, loud)
    q = torch.zeros(len(lengths), H_, D)
    q[..., :dim] = rnd(g, len(lengths), H_, dim) / math.sqrt(dim)
    for b, p in loud:
        q[b] += 1.5 * pool[int(r2t[b + 1, p])].float().repeat_interleave(H_ // G, 0) / dim
    q = (q * LOG2E).to(BF16)
    want = torch.stack([_tied_want(q[b: b + 1].double() / LOG2E, pool, rms, r2t, b, n, rel, longest, sink, n - 1)[0]
                        for b, n in enumerate(lengths)]) * 0.75
    n = len(lengths)
    req, pos = i32(*range(1, n + 1)), i32(*[x - 1 for x in lengths])
    pd = pool.view(pool.shape[0], -1).to(DEV)
    args = (rms.to(DEV), r2t.to(DEV), req, pos, w)
    for S in (1, 3, 8):
        part, lse = torch.full((n, H_, S, D), math.nan, device=DEV), torch.full((n, H_, S), math.nan, device=DEV)
        H.tied_decode(q.view(n, -1).to(DEV), pd, *args, part, lse)
        out = torch.full((n, H_ * D + 8), 3.0, dtype=BF16, device=DEV)
        H.tied_merge(part, lse, w, out[:, : H_ * D], 0.75)
        close(out[:, : H_ * D].view(n, H_, D), want, 1e-2, f"{S} splits")
        assert bool((out[:, H_ * D:] == 3.0).all())
    out = torch.full((n, H_ * D + 8), 3.0, dtype=BF16, device=DEV)
    H.tied_decode(q.view(n, -1).to(DEV), pd, *args, out=out[:, : H_ * D], out_scale=0.75)
    close(out[:, : H_ * D].view(n, H_, D), want, 1e-2, "finished")
    assert bool((out[:, H_ * D:] == 3.0).all())
    for dt, tol in ((BF16, 1e-2), (F32, 1e-5)):
        out = torch.empty(n, H_ * D, dtype=dt, device=DEV)
        H.tied_rows(q.view(n, -1).to(dt).to(DEV), pd.to(dt), *args, out, 0.75)
        close(out.view(n, H_, D), want, tol, f"rows {dt}")


@pytest.mark.parametrize("H_,G,D,dim,buckets,longest", TIED)
@pytest.mark.parametrize("many", [False, True])
def test_tied_prefill(H_, G, D, dim, buckets, longest, many):
    """Portions of unequal length behind prefixes of unequal length; loud keys near and far."""
    from sglang_security_amd import ops_hybrid as H
    from sglang_security_amd.layers.position_bias import LOG2E

    g = gen(D + H_ + 1)
    seqs = [(0, 2), (0, 131), (70, 64), (33, 65), (1, 17), (200, 3), (longest - 1, 4), (0, 1)]     # (tokens before the portion, rows)
    if many:                                                                    # enough blocks for two tiles of rows per wave
        seqs += [(5, 30)] * (256 // H_)
    lengths = [s + n for s, n in seqs]
    loud = [(1, 0), (1, 100), (2, 0), (3, 33), (5, 1), (6, 0)]
    r2t, pool, rms, w, rel, sink = _tied_case(g, lengths, H_, G, D, dim, buckets, longest, BF16, loud)
    row0 = [4]                                                                  # rows in front belong to somebody else
    for _, n in seqs:
        row0.append(row0[-1] + n)
    T = row0[-1]
    q = torch.zeros(T, H_, D)
    q[..., :dim] = rnd(g, T, H_, dim) / math.sqrt(dim)
    for b, p in loud:
        q[row0[b]: row0[b + 1]: 3] += 1.5 * pool[int(r2t[b + 1, p])].float().repeat_interleave(H_ // G, 0) / dim
    q = (q * LOG2E).to(BF16)
    out = torch.full((T, H_ * D + 8), 3.0, dtype=BF16, device=DEV)
    pd = pool.view(pool.shape[0], -1).to(DEV)
    H.tied_prefill(q.view(T, -1).to(DEV), pd, rms.to(DEV), r2t.to(DEV), i32(*row0[:-1]), i32(*[n for _, n in seqs]),
                   i32(*[s for s, _ in seqs]), i32(*range(1, len(seqs) + 1)), max(n for _, n in seqs), w, out[:, : H_ * D], 1.25)
    for b, (s, n) in enumerate(seqs[:10]):
        want = _tied_want(q[row0[b]: row0[b + 1]].double() / LOG2E, pool, rms, r2t, b, s + n, rel, longest, sink, s) * 1.25
        close(out[row0[b]: row0[b + 1], : H_ * D].view(n, H_, D), want, 1.2e-2, f"sequence {b}")
    assert bool((out[:4] == 3.0).all()) and bool((out[:, H_ * D:] == 3.0).all())


def test_tied_prefill_with_a_bias_table_beyond_the_lds():
    from sglang_security_amd.layers.position_bias import bucket_starts

    assert bucket_starts(64, 3000)[-1] > 2048
    for D, many in ((64, False), (128, True), (192, False)):
        test_tied_prefill(2, 1, D, D, 64, 3000, many)


# ---- gated delta rule -----------------------------------------------------------------------------------------------------
def _delta(c, dtype, seed=0, change=None):
    from sglang_security_amd.layers.gated_delta import GatedDelta
    from sglang_security_amd.layers.linear import Linear, pad, padded
    from sglang_security_amd.mem_cache.memory_pool import RecurrentStatePool

    cfg = K.config([K.layer(r_heads=c["heads"], r_kv=c["kv_heads"], r_dim=c["dim"], r_vdim=c["vdim"], conv=c["conv"])], width=64)
    p = "l0.mix.right."
    w = {k[len(p):]: v for k, v in K.weights(cfg, seed).items() if k.startswith(p)}
    if change:
        change(w)
    m = GatedDelta(c, lambda n, dt=None: w[n].to(dt or dtype).to(DEV), 128, 1e-5, dtype, 0.6)
    _, channels, taps, shape = m.cache_spec
    lin = Linear(padded(m.w_in, pad(m.w_in.shape[0], 128), 128))

    def forward(h, batch, pool):
        out = torch.empty(h.shape[0], m.w_out.shape[1], dtype=dtype, device=DEV)
        m.mix(lin.source(h).columns(0, m.w_in.shape[0]), batch, pool, out)
        return out.double().cpu() @ m.w_out.double().cpu().t()[:, :64]

    return forward, RecurrentStatePool(5, channels, taps, dtype, DEV, shape), w


DELTA = [dict(heads=6, kv_heads=3, dim=20, vdim=12, conv=4), dict(heads=2, kv_heads=2, dim=128, vdim=128, conv=4),
         dict(heads=4, kv_heads=1, dim=64, vdim=48, conv=2), dict(heads=3, kv_heads=3, dim=96, vdim=80, conv=1),
         dict(heads=2, kv_heads=1, dim=32, vdim=256, conv=7), dict(heads=1, kv_heads=1, dim=256, vdim=64, conv=3),
         dict(heads=2, kv_heads=1, dim=150, vdim=300, conv=4)]


@pytest.mark.parametrize("dtype", [F32, BF16])
@pytest.mark.parametrize("c", DELTA, ids=lambda c: "-".join(map(str, c.values())))
def test_delta_portions_and_slots(dtype, c):
    """Four sequences of which pieces of every length run together, slots reused for later sequences."""
    forward, pool, w = _delta(c, dtype)
    pool.state.fill_(1e3)                                                      # what an earlier owner left
    pool.conv.fill_(1e3)
    g = gen(c["dim"])
    seqs = [rnd(g, n, 64, dtype=dtype) for n in (260, 70, 66, 5)]
    w64 = {k: v.double() for k, v in w.items()}
    want = [O.gated_delta(x.double(), w64, c, 1e-5) * 0.6 for x in seqs]
    slot, at, got = [3, 0, 4, 1], [0] * 4, [[] for _ in seqs]
    plan = [{0: 64, 1: 2}, {0: 1, 1: 1, 2: 1, 3: 2}, {0: 67, 2: 63, 1: 3}, {0: 2, 1: 1, 3: 1, 2: 2}, {3: 2, 1: 63, 0: 1}, {0: 125}]
    for step in plan:
        order = sorted(step, key=lambda s: step[s] > 1)
        b = _Batch([(slot[s], at[s], step[s]) for s in order])
        h = torch.zeros(sum(step.values()), 128, dtype=dtype)
        h[:, :64] = torch.cat([seqs[s][at[s]: at[s] + step[s]] for s in order])
        out, r = forward(h.to(DEV), b, pool), 0
        for s in order:
            got[s].append(out[r: r + step[s]])
            at[s] += step[s]
            r += step[s]
    tol = 2e-5 if dtype == F32 else 3e-2
    for s in range(4):
        close(torch.cat(got[s]), want[s][: at[s]], tol, f"sequence {s}")
    b = _Batch([(3, 0, 5)])                                                    # as if the slot had been cleared
    h = torch.zeros(5, 128, dtype=dtype)
    h[:, :64] = seqs[3]
    close(forward(h.to(DEV), b, pool), want[3], tol, "reused slot")


@pytest.mark.parametrize("dtype", [F32, BF16])
def test_delta_memory_reaches_far_back(dtype):
    """Hardly any decay: what the first tokens wrote still shows after a thousand, however the rows were cut, and what a
    repeated key held has been replaced."""
    c = dict(heads=2, kv_heads=1, dim=128, vdim=64, conv=4)

    def change(w):
        w["A_log"].fill_(-12.0)
        w["b"] *= 0.5

    forward, pool, w = _delta(c, dtype, change=change)
    g = gen(3)
    x = 0.05 * rnd(g, 1000, 64)
    x[:3] = 5.0 * rnd(g, 3, 64)
    x[997:] = x[:3]                                                            # asks with the first keys again
    w64 = {k: v.double() for k, v in w.items()}
    x = x.to(dtype)
    want = O.gated_delta(x.double(), w64, c, 1e-5) * 0.6
    quiet = x.double().clone()
    quiet[:3] = 0
    lost = O.gated_delta(quiet, w64, c, 1e-5) * 0.6
    assert (want[-1] - lost[-1]).abs().max() > 0.1 * want[-1].abs().max()
    h = torch.zeros(1000, 128, dtype=dtype)
    h[:, :64] = x
    for cuts in ((0, 1000), (0, 130, 998, 999, 1000), (0, 2, 64, 129, 700, 1000)):
        out = torch.cat([forward(h[a:b].to(DEV), _Batch([(2, a, b - a)]), pool) for a, b in zip(cuts, cuts[1:])])
        close(out, want, 2e-4 if dtype == F32 else 3e-2, f"cut at {cuts}")


# ---- the whole model through the engine ------------------------------------------------------------------------------------
@functools.lru_cache(None)
def oracle_logits(name, seed, n):
    cfg = K.CONFIGS[name]
    return O.forward(cfg, K.weights(cfg), M.tokens(cfg, n, seed))


@functools.lru_cache(None)
def oracle_noise(name, seed, n):
    """Largest relative change of each logits row over three runs with norm outputs disturbed by 2^-9."""
    cfg, plain = K.CONFIGS[name], O.rms
    want, worst = oracle_logits(name, seed, n)[0], torch.zeros(n, dtype=torch.float64)
    try:
        for k in range(3):
            g = gen(k)
            O.rms = lambda x, e: plain(x, e) * (1 + 2 ** -9 * torch.randn(x.shape, generator=g, dtype=torch.float64))
            worst = torch.maximum(worst, M.rel_rms(O.forward(cfg, K.weights(cfg), M.tokens(cfg, n, seed))[0], want))
    finally:
        O.rms = plain
    return worst


@pytest.fixture(scope="module")
def engines():
    from sglang_security_amd.engine import Engine
    from sglang_security_amd.model_loader import Weights
    from sglang_security_amd.models import model_class

    made = {}

    def get(name, dtype, max_tokens=640, max_requests=4, **kw):
        key = (name, dtype)
        if key not in made:
            cfg = K.CONFIGS[name]
            ws = Weights(K.weights(cfg), dtype, torch.device(DEV, 0))
            made[key] = model_class(cfg)(cfg, ws, dtype, torch.device(DEV, 0), 640)
            ws.check_all_used()
        return Engine(made[key], max_tokens, max_requests, **kw)

    return get


CASES = [(n, d) for n in K.CONFIGS for d in (F32, BF16)]


def agrees(err, dtype, noise, what):
    """Relative errors per row; bf16 against what a small disturbance of the oracle does to each row."""
    limit = torch.full_like(err, 1e-4) if dtype == F32 else 0.02 + 5 * noise[: len(err)]
    at = int((err / limit).argmax())
    says = f"{what}: {float(err[at]):.4g} at row {at} of {len(err)}, limit {float(limit[at]):.4g}, mean {float(err.mean()):.4g}"
    assert bool((err <= limit).all()) and float(err.mean()) <= (1e-4 if dtype == F32 else 0.035), says


def run(engine, name, plan):
    """plan: steps of {sequence id: (seed, total length, rows now)}; a sequence closes when its tokens are through.
    Compares every row's logits with the oracle and returns {id: logits}."""
    from sglang_security_amd.engine import Entry

    cfg, live, got, meta = K.CONFIGS[name], {}, {}, {}
    for step in plan:
        entries, ids = [], []
        for sid, (seed, total, n) in step.items():
            if sid not in live:
                live[sid] = engine.open()
                got[sid], meta[sid] = [], (seed, total)
            at = live[sid].length
            entries.append(Entry(live[sid], M.tokens(cfg, total, seed)[at: at + n], range(n)))
            ids.append(sid)
        out, r = engine.step(entries).cpu(), 0
        for sid, e in zip(ids, entries):
            got[sid].append(out[r: r + len(e.tokens)])
            r += len(e.tokens)
            if live[sid].length == meta[sid][1]:
                engine.close(live.pop(sid))
    got = {sid: torch.cat(v) for sid, v in got.items()}
    for sid, (seed, total) in meta.items():
        err = M.rel_rms(got[sid], oracle_logits(name, seed, total)[0][: len(got[sid])])
        agrees(err, engine.model.dtype, oracle_noise(name, seed, total), f"{name} {sid}")
    return got


@pytest.mark.parametrize("name,dtype", CASES)
def test_whole_prompts_and_residual_stream(engines, name, dtype):
    from sglang_security_amd.engine import Entry

    e = engines(name, dtype)
    for seed, n in enumerate((1, 2, 3, 150, 300)):
        run(e, name, [{0: (seed, n, n)}])
    s, col = e.open(), []
    e.step([Entry(s, M.tokens(K.CONFIGS[name], 150, 3), [149])], collect=col)
    stream = oracle_logits(name, 3, 150)[1]
    assert len(col) == len(stream)
    for i, (a, b) in enumerate(zip(col, stream)):
        agrees(M.rel_rms(a, b), dtype, oracle_noise(name, 3, 150), f"layer {i}")
    e.close(s)


@pytest.mark.parametrize("name,dtype", CASES)
def test_token_by_token_equals_the_prompt(engines, name, dtype):
    e = engines(name, dtype)
    run(e, name, [{0: p} for p in cut(3, 150, [1])])                      # graph replays from the third step on
    run(e, name, [{0: p} for p in cut(4, 300, [180] + [1] * 120)])


@pytest.mark.parametrize("name", list(K.CONFIGS))
def test_contexts_too_short_to_split(engines, name):
    run(engines(name, BF16, max_context=100), name, [{0: a, 1: b} for a, b in zip(cut(5, 90, [1]), cut(6, 97, [7] + [1] * 90))])


@pytest.mark.parametrize("name,dtype", CASES)
@pytest.mark.parametrize("parts", [[2], [3, 2, 37], [64, 1, 63, 65], [5, 40, 2, 130]])
def test_portions(engines, name, dtype, parts):
    run(engines(name, dtype), name, [{0: p} for p in cut(3, 150, parts)])


@pytest.mark.parametrize("name,dtype", CASES)
def test_mixed_batches_with_reused_slots(engines, name, dtype):
    """Unequal requests come and go; portions beside single tokens; some are left out of steps; 640 slots serve more
    than a thousand tokens."""
    e = engines(name, dtype)
    queue = [(i, cut(seed, n, parts)) for i, (seed, n, parts) in enumerate(
        [(4, 300, [100, 1, 1, 1, 50, 2]), (0, 1, [1]), (3, 150, [37, 3, 24, 2]), (5, 90, [60] + [1] * 30), (6, 97, [97]),
         (7, 66, [64, 2]), (8, 120, [1, 2, 40, 1]), (9, 200, [150] + [1] * 50), (3, 150, [149, 1]), (2, 3, [2, 1])])]
    live, plan, t = [], [], 0
    while queue or live:
        while queue and len(live) < 4:
            live.append(queue.pop(0))
        step = {}
        for k, (sid, parts) in enumerate(live):
            if len(live) > 1 and (t + k) % 5 == 4:
                continue
            step[sid] = parts.pop(0)
        live = [x for x in live if x[1]]
        plan.append(step)
        t += 1
    run(e, name, plan)
    assert e.free_tokens() == 640 and e.cache.req_pool.available_size() == 4


@pytest.mark.parametrize("name", list(K.CONFIGS))
def test_batches_equal_each_alone(engines, name):
    """bf16: the same requests alone, together, and on other slots differ by rounding only."""
    e = engines(name, BF16)
    alone = {s: run(e, name, [{s: p} for p in cut(s, n, [n - 4, 1, 1, 1, 1])])[s] for s, n in ((3, 150), (5, 90), (6, 97))}
    steps = [dict(zip((3, 5, 6), ps)) for ps in zip(*[cut(s, n, [n - 4, 1, 1, 1, 1]) for s, n in ((3, 150), (5, 90), (6, 97))])]
    both = run(e, name, steps)
    for s, n in ((3, 150), (5, 90), (6, 97)):
        agrees(M.rel_rms(both[s], alone[s].double()), BF16, oracle_noise(name, s, n), f"{name} {s}")


def test_graph_replays_equal_eager_steps(engines):
    from sglang_security_amd.engine import Entry

    name = "mixed"
    a, b = engines(name, BF16), engines(name, BF16, use_graph=False)
    sa, sb = [a.open() for _ in range(3)], [b.open() for _ in range(3)]
    t = M.tokens(K.CONFIGS[name], 120, 1)
    for e, s in ((a, sa), (b, sb)):
        e.step([Entry(q, t[:n]) for q, n in zip(s, (40, 1, 9))])
    for i in range(24):
        want = [[0], [], [0]] if i % 3 else [[0]] * 3
        n = 3 if i % 4 else 2
        la, lb = (e.step([Entry(q, [t[50 + i + j]], w) for j, (q, w) in enumerate(zip(s[:n], want))]) for e, s in ((a, sa), (b, sb)))
        assert torch.equal(la, lb), f"step {i}"
        torch.randn(1000, device=DEV).sum().item()                        # the program's own work between the replays
    assert set(a.graphs) == {2, 3} and not b.graphs


@pytest.mark.parametrize("name", ["mixed", "full"])
def test_greedy_generation_through_the_scheduler(engines, name):
    from sglang_security_amd.engine import SamplingParams, Scheduler

    cfg = K.CONFIGS[name]
    prompts = [M.tokens(cfg, n, 50 + n) for n in (3, 41, 70, 1, 25, 9)]
    outs = Scheduler(engines(name, F32), prefill_budget=32).generate(prompts, SamplingParams(max_new_tokens=12))
    for p, o in zip(prompts, outs):
        lg, _ = O.forward(cfg, K.weights(cfg), p + o)
        for i, t in enumerate(o):
            row = lg[len(p) - 1 + i]
            assert float(row[t]) >= float(row.max()) - 1e-3, f"token {i}"      # the arg-max, ties aside
    sched = Scheduler(engines(name, BF16), prefill_budget=32)
    outs = sched.generate(prompts, SamplingParams(max_new_tokens=12))
    for p, o in zip(prompts, outs):
        lg, _ = O.forward(cfg, K.weights(cfg), p + o)
        spread = float((lg ** 2).mean().sqrt())
        for i, t in enumerate(o):
            row = lg[len(p) - 1 + i]
            assert float(row[t]) >= float(row.max()) - 0.3 * spread
    assert sched.generate(prompts, SamplingParams(max_new_tokens=12)) == outs


def test_command_line_and_trace(tmp_path):
    """generate and trace from a checkpoint folder, in processes of their own."""
    import numpy as np

    name = "mixed"
    cfg = K.CONFIGS[name]
    folder = M.save(str(tmp_path / "model"), cfg, K.weights(cfg))
    t = M.tokens(cfg, 90, 5)
    r = subprocess.run([sys.executable, "-m", "sglang_security_amd.cli", "generate", "--model", folder, "--dtype", "float32",
                        "--prompt-ids", ",".join(map(str, t[:30])), "--max-new-tokens", "5"], capture_output=True, text=True, timeout=100,
                       cwd=_root())
    assert r.returncode == 0, r.stderr[-2000:]
    out = json.loads(r.stdout.strip().splitlines()[-1])["output_ids"]
    lg, _ = O.forward(cfg, K.weights(cfg), t[:30] + out)
    assert len(out) == 5 and all(float(lg[29 + i].max() - lg[29 + i][v]) < 1e-3 for i, v in enumerate(out))
    steps = [{"step": 0, "entries": [{"id": "a", "tokens": t[:50], "want": [49, 0]}, {"id": "b", "tokens": t[:1], "want": []}], "end": []},
             {"step": 1, "entries": [{"id": "b", "tokens": t[1:4], "want": []}], "end": ["b"]},
             {"step": 2, "entries": [{"id": "c", "tokens": t[:2], "want": [1]}, {"id": "a", "tokens": t[50:51], "want": [0]}], "end": ["a", "c"]}]
    p = subprocess.run(["bin/trace_run", "--model", folder, "--dtype", "float32", "--out", str(tmp_path), "--max-tokens", "128"],
                       input="\n".join(map(json.dumps, steps)) + "\n", capture_output=True, text=True, timeout=100, cwd=_root())
    assert p.returncode == 0, p.stderr[-2000:]
    assert [l for l in p.stdout.splitlines() if l.startswith("done")] == ["done 0", "done 1", "done 2"]
    lg = oracle_logits(name, 5, 90)[0]
    read = lambda n: torch.from_numpy(np.fromfile(tmp_path / f"{n}.f32", "<f4")).view(-1, cfg["vocab"])
    assert float(M.rel_rms(read(0), lg[[49, 0]]).max()) < 1e-4 and not (tmp_path / "1.f32").exists()
    assert float(M.rel_rms(read(2), lg[[1, 50]]).max()) < 1e-4
