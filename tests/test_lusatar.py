"""CPU: the Lusatar oracle against hand-worked facts, how sensitive the test models are, and the host side of the
engine (registry, checkpoint files, layer order, step layout, scheduling)."""
import json
import math
import types

import numpy as np
import pytest
import torch

import lusatar_models as M
from oracle import lusatar as O


# ---- oracle -------------------------------------------------------------------------------------------------------------
def test_rotation_keeps_relative_scores_and_the_untouched_part():
    g = torch.Generator().manual_seed(0)
    q, k = torch.randn(1, 12, generator=g).double(), torch.randn(1, 12, generator=g).double()
    at = lambda v, p: O.rotate(v, torch.tensor([p]), 100.0, 8, None)
    s = [float((at(q, p + 5)[..., :8] * at(k, p)[..., :8]).sum()) for p in (0, 3, 40)]
    assert max(s) - min(s) < 1e-9
    assert torch.equal(at(q, 7)[..., 8:], q[..., 8:])
    a = torch.tensor(7 * 100.0 ** (-2 * 1 / 8))
    assert abs(float(at(q, 7)[0, 1]) - float(q[0, 1] * torch.cos(a) - q[0, 5] * torch.sin(a))) < 1e-6


def test_yarn_frequencies_blend_between_plain_and_stretched():
    sc = {"factor": 8.0, "original": 256, "fast": 16.0, "slow": 1.0}
    plain, _ = O.rotary_frequencies(500.0, 32, None)
    f, mag = O.rotary_frequencies(500.0, 32, sc)
    assert abs(mag - (0.1 * math.log(8.0) + 1)) < 1e-12
    assert f[0] == plain[0] and abs(f[-1] - plain[-1] / 8.0) < 1e-12
    assert all(p / 8.0 - 1e-12 <= x <= p + 1e-12 for x, p in zip(f, plain))


def test_window_counts_the_token_itself():
    T, w = 9, 4
    q = torch.zeros(T, 1, 2).double()
    v = torch.eye(T).view(T, 1, T).double()
    o = O.window_attention(q, q, v, 1.0, w)[:, 0]
    for i in range(T):
        seen = {j for j in range(T) if o[i, j] > 0}
        assert seen == set(range(max(0, i - w + 1), i + 1))


def test_convolution_last_tap_is_the_token_itself():
    x = torch.arange(1.0, 6.0).view(5, 1).double()
    y = O.causal_conv(x, torch.tensor([[100.0, 10.0, 1.0]]).double(), torch.zeros(1).double())
    assert y[:, 0].tolist() == [1.0, 12.0, 123.0, 234.0, 345.0]


def test_recurrence_first_state_has_no_special_case():
    w = {"ra": torch.zeros(1, 1, 1), "ra.b": torch.zeros(1, 1), "ri": torch.zeros(1, 1, 1), "ri.b": torch.zeros(1, 1),
         "lam": torch.zeros(1)}
    w = {k: v.double() for k, v in w.items()}
    u = torch.tensor([[2.0], [0.0]]).double()
    a = math.exp(-8 * 0.5 * math.log(2.0))
    S = O.gated_linear_recurrence(u, w, {"blocks": 1})[:, 0].tolist()
    assert abs(S[0] - math.sqrt(1 - a * a) * 0.5 * 2.0) < 1e-12 and abs(S[1] - a * S[0]) < 1e-12


def _spoilt(name, cfg, w):
    """The same model with one mistake, planted in what the oracle is given."""
    c, v = json.loads(json.dumps(cfg)), dict(w)
    att = next(L for L in c["layers"] if L["type"] == "latent_attention")
    if name == "window":
        att["mixer"]["mask"]["size"] += 1
    elif name == "yarn":
        att["mixer"]["rot"]["scaling"] = None
    elif name == "step":
        v["loop.step"] = w["loop.step"].flip(0)
    elif name == "cap":
        c["logit_softcap"] = None
    elif name == "taps":
        v["l0.mix.conv"] = w["l0.mix.conv"].flip(1)
    return c, v


@pytest.mark.parametrize("name", ["window", "yarn", "step", "cap", "taps"])
def test_test_models_show_a_mistake(name):
    cfg = M.CONFIGS["mixed"]
    w, t = M.weights(cfg), M.tokens(cfg, 48)
    want, _ = O.forward(cfg, w, t)
    got, _ = O.forward(*_spoilt(name, cfg, w), t)
    assert float(M.rel_rms(got, want).max()) > 0.02      # against 1e-4 that the fp32 comparisons allow


# ---- product host side ---------------------------------------------------------------------------------------------------
def test_rotary_table_matches_the_plain_frequencies():
    from sglang_security_amd.layers.rotary import rotary_table

    for dims, base, sc in ((8, 1000.0, None), (16, 50.0, {"factor": 4.0, "original": 64, "fast": 4.0, "slow": 1.0}),
                           (64, 1e5, {"factor": 32.0, "original": 4096, "fast": 32.0, "slow": 1.0}),
                           (6, 10.0, {"factor": 2.0, "original": 8, "fast": 1.0, "slow": 1.0})):
        f, mag = O.rotary_frequencies(base, dims, sc)
        a = torch.arange(700.0, dtype=torch.float64)[:, None] * torch.tensor(f, dtype=torch.float64)
        want = torch.cat([a.cos(), a.sin()], -1) * mag
        assert float((rotary_table(dims, base, 700, "cpu", sc).double() - want).abs().max()) < 1e-7 * mag + 1e-7


def test_layer_runs():
    from sglang_security_amd.models.lusatar import layer_runs

    flat = lambda n, loop: [(r.layer, r.opens) for r in layer_runs(n, loop)]
    assert flat(2, None) == [(0, None), (1, None)]
    assert flat(4, {"start": 1, "stop": 3, "times": 2}) == [(0, None), (1, 0), (2, None), (1, 1), (2, None), (3, None)]
    assert flat(2, {"start": 0, "stop": 2, "times": 1}) == [(0, 0), (1, None)]
    assert flat(2, {"start": 1, "stop": 1, "times": 3}) == [(0, None), (1, None)]
    with pytest.raises(ValueError):
        layer_runs(2, {"start": 1, "stop": 3, "times": 1})


def test_registry_and_command_line(capsys):
    from sglang_security_amd import cli, models
    from sglang_security_amd.models.lusatar import Lusatar

    assert models.model_class({"architecture": "Lusatar"}) is Lusatar
    assert models.model_class({"architectures": ["Lusatar"]}) is Lusatar
    with pytest.raises(ValueError, match="unknown architecture"):
        models.model_class({"architecture": "Nothing"})
    assert models.synthetic_config("llama3-8b", "bf16").hidden == 4096
    assert cli.main(["models"]) == 0
    assert "Lusatar" in capsys.readouterr().out


def test_checkpoint_files(tmp_path):
    from safetensors.torch import load_file
    from sglang_security_amd.model_loader import load_config, load_weights

    cfg = M.CONFIGS["tail"]
    w = M.weights(cfg)
    w["extra"] = torch.arange(6, dtype=torch.int32).view(2, 3)
    folder = M.save(str(tmp_path / "m"), cfg, w)
    assert load_config(folder) == cfg
    ws = load_weights(folder, torch.float32, "cpu")
    theirs = load_file(folder + "/model.safetensors")
    for name, t in w.items():
        assert torch.equal(ws.get(name, tuple(t.shape), t.dtype), t) and torch.equal(theirs[name], t)
    ws = load_weights(folder, torch.float32, "cpu")
    for name, t in M.weights(cfg).items():
        ws.get(name, tuple(t.shape))
    with pytest.raises(ValueError, match="extra"):
        ws.check_all_used()
    with pytest.raises(ValueError, match="shape"):
        ws.get("embed", (1, 2))
    with pytest.raises(ValueError, match="no tensor"):
        ws.get("nothing", (1,))
    broken = tmp_path / "b"
    broken.mkdir()
    (broken / "model.safetensors").write_bytes((1 << 40).to_bytes(8, "little") + b"{}")
    with pytest.raises(ValueError, match="header"):
        load_weights(str(broken), torch.float32, "cpu")


class _Model:
    """Stands in for a model on the CPU: the next token is the last one plus one."""
    vocab, max_context, dtype, device = 50, 64, torch.float32, torch.device("cpu")

    def cache_layers(self):
        return []


def _engine(max_tokens=64, max_requests=3):
    from sglang_security_amd.engine import Engine

    e = Engine(_Model(), max_tokens, max_requests)
    e.log = []

    def forward(batch, collect=None):
        h = batch.host
        e.log.append({k: v.copy() for k, v in h.items()} | {"singles": batch.singles})
        for t, s in enumerate(h["row_seq"]):
            e.req_to_token[h["slot"][s], h["positions"][t]] = int(h["loc"][t])
        out = torch.zeros(len(h["logit_rows"]), 50)
        out[torch.arange(len(out)), torch.tensor((h["ids"][h["logit_rows"]] + 1) % 50).long()] = 1.0
        return out if len(out) else None

    e._forward = forward
    return e


def _scheduler(e, budget):
    from sglang_security_amd.engine import Scheduler

    s = Scheduler(e, budget)
    s.sampler = lambda logits, params: logits.argmax(-1).tolist()
    return s


def test_step_layout_orders_single_rows_first_and_keeps_the_answers_in_entry_order():
    from sglang_security_amd.engine import Entry

    e = _engine(max_tokens=300, max_requests=3)
    e.max_context = 300
    e.req_to_token = torch.zeros(3, 300, dtype=torch.int32)
    a, b, c = e.open(), e.open(), e.open()
    e.step([Entry(b, [7])])
    out = e.step([Entry(a, list(range(40)) * 2, [79, 0]), Entry(b, [9], [0]), Entry(c, [3, 4], [1])])
    assert out.argmax(-1).tolist() == [40, 1, 10, 5]
    h = e.log[-1]
    assert h["singles"] == 1 and h["rows"].tolist() == [1, 80, 2] and h["start"].tolist() == [1, 0, 0]
    assert h["slot"].tolist() == [b.slot, a.slot, c.slot] and h["row0"].tolist() == [0, 1, 81]
    assert h["tile0"].tolist() == [0, 0, 2] and h["tile_row"].tolist() == [1, 65, 81] and h["tile_rows"].tolist() == [64, 16, 2]
    assert h["positions"].tolist() == [1] + list(range(80)) + [0, 1]
    assert len(set(h["loc"].tolist())) == 83 and 0 not in h["loc"]


def test_expansion_lists_what_a_window_can_see():
    from sglang_security_amd.engine import Entry, StepBatch

    e = _engine(max_tokens=64)
    a, b = e.open(), e.open()
    e.step([Entry(a, [1] * 10), Entry(b, [2] * 3)])
    e.step([Entry(a, [1] * 4), Entry(b, [2] * 5)])
    h = {k: v for k, v in e.log[-1].items() if k != "singles"}
    batch = StepBatch(h, 0, e.req_to_token, 64)
    x = batch.expansion(6)
    assert x.rows.tolist() == [4, 5] and x.ahead.tolist() == [5, 3] and x.tok0.tolist() == [0, 9] and x.max_rows == 5
    slots = e.req_to_token.view(-1)[x.table_index.long()].tolist()
    want = [t for s in a.locs for t in s.tolist()][5:] + [t for s in b.locs for t in s.tolist()]
    assert slots == want
    assert batch.expansion(0).ahead.tolist() == [10, 3]


def test_engine_refuses_what_does_not_fit():
    from sglang_security_amd.engine import Entry

    e = _engine(max_tokens=8, max_requests=1)
    s = e.open()
    with pytest.raises(RuntimeError):
        e.open()
    for bad in ([Entry(s, [])], [Entry(s, [50])], [Entry(s, [1], [1])], [Entry(s, [1]), Entry(s, [2])], [Entry(s, [1] * 65)]):
        with pytest.raises(ValueError):
            e.step(bad)
    with pytest.raises(RuntimeError, match="exhausted"):
        e.step([Entry(s, [1] * 9)])
    assert s.length == 0 and e.free_tokens() == 8
    e.step([Entry(s, [1] * 8)])
    assert e.free_tokens() == 0
    e.close(s)
    assert e.free_tokens() == 8
    with pytest.raises(ValueError):
        e.step([Entry(s, [1])])


def test_scheduler_portions_admission_and_reuse():
    from sglang_security_amd.engine import SamplingParams

    e = _engine(max_tokens=40, max_requests=2)
    s = _scheduler(e, budget=6)
    outs = s.generate([[10] * 15, [20], [30] * 9, [48]], SamplingParams(max_new_tokens=4))
    assert outs == [[11, 12, 13, 14], [21, 22, 23, 24], [31, 32, 33, 34], [49, 0, 1, 2]]
    assert e.free_tokens() == 40 and e.cache.req_pool.available_size() == 2
    assert all(len(h["ids"]) <= 6 + 2 for h in e.log) and any(h["singles"] and h["singles"] < len(h["rows"]) for h in e.log)
    assert max(len(h["rows"]) for h in e.log) == 2
    r = s.add([5], SamplingParams(max_new_tokens=9, stop_token_ids=(8,)))
    s.run()
    assert r.output == [6, 7, 8]
    with pytest.raises(ValueError):
        s.add([1] * 60, SamplingParams())


def test_a_partial_library_is_enough_for_the_engine_only(monkeypatch, tmp_path):
    from sglang_security_amd import _lib, build, models

    monkeypatch.setattr(_lib, "_lib", None)
    monkeypatch.setattr(_lib, "_partial", True)
    lib = _lib.lib()
    assert lib.sglk_residual_norm(*([None] * 2 + [None, 0, 1.0, None, 0, 1, 0, 0, None, None, 0, None, None, None, 0, None, 0, 1, 8, 8,
                                                  1e-5, 2, None])) == -1
    here = {p.split("/")[-1] for p in build._sources()}
    for name in models.ARCHITECTURES:
        assert set(models.kernel_sources({"architecture": name}) + models.SAMPLING_SOURCES) <= here
