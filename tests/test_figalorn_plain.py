"""The plain formulas of the Figalorn decoder checked against independent ones on the CPU, the configuration, and the
model as data."""
import json
import math

import pytest
import torch

import herbert_rs_amd as hb
from herbert_rs_amd.config import FigalornConfig
from herbert_rs_amd.config.registry import resolve_architecture
from herbert_rs_amd.engine.model import Model
from herbert_rs_amd.errors import ConfigError
from herbert_rs_amd.kernels.heads import HeadsLayout
from herbert_rs_amd.parts import PartSpec, build
from herbert_rs_amd.parts.position import RotaryHalves, RotaryPairs

from .figalorn_tiny import CONFIGS, make_folder, random_tokens
from .plain import figalorn as plain


def rand(*shape, seed=0, scale=1.0):
    return torch.randn(*shape, generator=torch.Generator().manual_seed(seed), dtype=torch.float64) * scale


def test_norms_and_the_exact_gelu():
    x, w = rand(5, 12, seed=1), rand(12, seed=2)
    want = torch.stack([r / math.sqrt(float((r ** 2).sum()) / 12 + 0.01) * (w + 1) for r in x])
    assert torch.allclose(plain.norm_around_one(x, w, 0.01), want)
    z = torch.linspace(-9, 9, 400, dtype=torch.float64)
    assert torch.allclose(plain.gelu_erf(z), torch.nn.functional.gelu(z), atol=1e-12)
    assert not torch.allclose(plain.gelu_erf(z), torch.nn.functional.gelu(z, approximate="tanh"), atol=1e-5)


def test_rates_by_wavelength():
    rot = {"dims": 8, "base": 100.0, "scaling": {"factor": 5.0, "low": 1.0, "high": 4.0, "original": 64}}
    base, got = plain.base_rates(rot), plain.rates_by_wavelength(rot)
    kinds = set()
    for f, r in zip(base.tolist(), got.tolist()):
        turns = 64 * f / (2 * math.pi)                      # in the original length
        if turns > 4:
            kinds.add("kept")
            assert r == f
        elif turns < 1:
            kinds.add("slowed")
            assert abs(r - f / 5) < 1e-15
        else:
            kinds.add("between")
            s = (turns - 1) / 3
            assert abs(r - f * (s + (1 - s) / 5)) < 1e-12
    assert kinds == {"kept", "slowed", "between"}
    part = RotaryPairs(100.0, 8, (5.0, 1.0, 4.0, 64))
    assert torch.allclose(torch.tensor(part.pair_rates_host(), dtype=torch.float64), got, rtol=1e-14) and part.amplitude == 1.0


def test_rates_by_ramp():
    rot = {"dims": 32, "base": 1000.0, "scaling": {"factor": 6.0, "original": 512, "fast": 20.0, "slow": 1.5}}
    base = plain.base_rates(rot)
    got, grow = plain.rates_by_ramp(rot)
    share = got / base                                      # 1 where a rate is kept, 1/6 where it is slowed
    first, last = share[0], share[-1]
    assert first == 1.0 and abs(float(last) - 1 / 6) < 1e-12
    assert all(a >= b - 1e-15 for a, b in zip(share.tolist(), share.tolist()[1:]))
    turns = 512 * base / (2 * math.pi)
    for t, s in zip(turns.tolist(), share.tolist()):       # outside the (rounded) stretch between fast and slow turns
        assert t < 20.0 * 1.3 or s > 0.83
        assert s == 1.0 if t > 20.0 * 1.3 else True
    steps = [a - b for a, b in zip(share.tolist(), share.tolist()[1:]) if 1 / 6 + 1e-9 < b and a < 1 - 1e-9]
    assert max(steps) - min(steps) < 1e-12                 # a straight line over the pairs
    assert abs(grow - (1 + math.log(6.0) / 10)) < 1e-15
    part = RotaryHalves(1000.0, 32, (6.0, 512, 20.0, 1.5))
    assert torch.allclose(torch.tensor(part.pair_rates_host(), dtype=torch.float64), got, rtol=1e-14) and part.amplitude == grow
    assert RotaryHalves(1000.0, 32).amplitude == 1.0
    # a stretch of no length: the pair at its start keeps its rate, the next is slowed
    rot["scaling"].update(fast=1e9, slow=1e9)
    got, _ = plain.rates_by_ramp(rot)
    assert got[0] == base[0] and torch.allclose(got[1:] * 6.0, base[1:])
    assert RotaryHalves(1000.0, 32, (6.0, 512, 1e9, 1e9)).pair_rates_host() == got.tolist()


def test_rotations_turn_the_right_pairs():
    x, p = rand(3, 2, 10, seed=3), torch.tensor([0, 7, 1000])
    rot = {"dims": 6, "base": 50.0}
    for turn, pairs in ((plain.rotate_pairs, [(0, 1), (2, 3), (4, 5)]), (plain.rotate_halves, [(0, 3), (1, 4), (2, 5)])):
        y = turn(x, p, rot)
        assert torch.equal(y[0], x[0]) and torch.equal(y[..., 6:], x[..., 6:])
        for i, (a, b) in enumerate(pairs):
            ang = p.double() * 50.0 ** (-2 * i / 6)
            z = torch.complex(x[..., a], x[..., b]) * torch.exp(1j * ang)[:, None]
            assert torch.allclose(torch.view_as_real(z), torch.stack([y[..., a], y[..., b]], -1), atol=1e-12)
    rot["scaling"] = {"factor": 3.0, "original": 100, "fast": 8.0, "slow": 1.0}
    y = plain.rotate_halves(x, p, rot)
    assert torch.allclose(y[0, :, :6], x[0, :, :6] * (1 + math.log(3.0) / 10))


def test_chunks_and_windows():
    chunk, window = plain.visible_chunk(torch.arange(30), 7), plain.visible_window(torch.arange(30), 7)
    for i in range(30):
        for j in range(30):
            assert bool(chunk[i, j]) == (j <= i and j >= i - i % 7)
            assert bool(window[i, j]) == (i - 7 < j <= i)
    for see in (plain.visible_chunk(torch.arange(9), None), plain.visible_window(torch.arange(9), None)):
        assert torch.equal(see, torch.ones(9, 9).tril().bool())


def test_a_difference_of_two_maps_written_out():
    T, W = 6, 10
    m = {"heads": 4, "kv_heads": 2, "dim": 3, "vdim": 5, "scale": 0.7, "diff": 0.4, "mask": {"size": 4}}
    w = {"q": rand(24, W, seed=1), "q.b": rand(24, seed=2), "k": rand(12, W, seed=3), "k.b": rand(12, seed=4), "v": rand(10, W, seed=5),
         "v.b": rand(10, seed=6), "g": rand(20, W, seed=7), "o": rand(W, 20, seed=8),
         **{k: rand(3, seed=9 + i, scale=0.4) for i, k in enumerate(("lq1", "lk1", "lq2", "lk2"))}}
    h = rand(T, W, seed=20)
    lam = math.exp(float(w["lq1"] @ w["lk1"])) - math.exp(float(w["lq2"] @ w["lk2"])) + 0.4
    want = torch.zeros(T, 20, dtype=torch.float64)
    for i in range(T):
        for a in range(4):
            g = a // 2
            sums = []
            for j in range(2):
                r = slice((2 * a + j) * 3, (2 * a + j) * 3 + 3)
                q = w["q"][r] @ h[i] + w["q.b"][r]
                r = slice((2 * g + j) * 3, (2 * g + j) * 3 + 3)
                e = {t: math.exp(0.7 * float(q @ (w["k"][r] @ h[t] + w["k.b"][r]))) for t in range(4 * (i // 4), i + 1)}
                r = slice(5 * g, 5 * g + 5)
                sums.append(sum(p / sum(e.values()) * (w["v"][r] @ h[t] + w["v.b"][r]) for t, p in e.items()))
            o = sums[0] - lam * sums[1]
            o = o / math.sqrt(float((o * o).mean()) + 1e-3) * 0.6
            want[i, 5 * a:5 * a + 5] = o / (1 + torch.exp(-(w["g"][5 * a:5 * a + 5] @ h[i])))
    assert torch.allclose(plain.difference_mixer(h, w, m, 1e-3, torch.arange(T)), want @ w["o"].T)


def test_values_that_are_keys_written_out():
    T, W = 6, 10
    m = {"heads": 4, "kv_heads": 2, "dim": 6, "vdim": 6, "scale": 0.9, "softcap": 1.5, "mask": {"size": 3}, "rot": {"dims": 4, "base": 20.0}}
    w = {"q": rand(24, W, seed=1), "k": rand(12, W, seed=2), "q.norm": rand(6, seed=3), "k.norm": rand(6, seed=4), "o": rand(W, 24, seed=5)}
    h = rand(T, W, seed=20)

    def turned(v, weight, p):
        v = v / math.sqrt(float((v * v).mean()) + 1e-3) * weight
        out = v.clone()
        for i in range(2):
            c, s = math.cos(p * 20.0 ** (-i / 2)), math.sin(p * 20.0 ** (-i / 2))
            out[i], out[i + 2] = v[i] * c - v[i + 2] * s, v[i + 2] * c + v[i] * s
        return out
    want = torch.zeros(T, 24, dtype=torch.float64)
    for i in range(T):
        for a in range(4):
            r = slice(6 * (a // 2), 6 * (a // 2) + 6)
            q = turned(w["q"][6 * a:6 * a + 6] @ h[i], w["q.norm"], i)
            e = {t: math.exp(1.5 * math.tanh(0.9 * float(q @ turned(w["k"][r] @ h[t], w["k.norm"], t)) / 1.5))
                 for t in range(max(0, i - 2), i + 1)}
            want[i, 6 * a:6 * a + 6] = sum(p / sum(e.values()) * (w["k"][r] @ h[t]) for t, p in e.items())
    assert torch.allclose(plain.key_value_mixer(h, w, m, 1e-3, torch.arange(T)), want @ w["o"].T)


def test_the_order_of_runs_and_where_a_pass_starts():
    cfg = {"layers": [0] * 5, "loop": {"start": 1, "stop": 3, "times": 3}}
    assert plain.runs(cfg) == [(0, False), (1, True), (2, False), (1, True), (2, False), (1, True), (2, False), (3, False), (4, False)]
    for name in "PQRS":
        raw = CONFIGS[name][0]
        spec = resolve_architecture(raw).build_spec(FigalornConfig.from_dict(raw))
        assert [(e.layer, e.starts_pass is not None) for e in spec.schedule] == plain.runs(raw)
        m = Model(spec)
        assert len(m.cache_needs()) == len(spec.schedule)          # every run has a cache of its own
        assert m.graph_safe
    raw = json.loads(json.dumps(CONFIGS["P"][0]))
    del raw["loop"]
    m = Model(resolve_architecture(raw).build_spec(FigalornConfig.from_dict(raw)))
    assert len(m.cache_needs()) == 4 and "loop.in" not in m.tensor_needs() and m.pass_input is None


def test_what_a_pass_starts_from():
    x, x0, w = rand(4, 6, seed=1), rand(4, 6, seed=2), rand(6, 12, seed=3)
    assert torch.allclose(plain.loop_input(x, x0, w), x @ w[:, :6].T + x0 @ w[:, 6:].T)


def test_windows_are_the_caches_and_chunks_are_not():
    raw = CONFIGS["P"][0]
    needs = Model(resolve_architecture(raw).build_spec(FigalornConfig.from_dict(raw))).cache_needs()
    assert [n.window for n in needs.values()] == [None, 50, None, 50, None, 50, None, 9]


def test_portions_do_not_change_the_plain_model(tmp_path):
    """The first rows of a longer sequence are those of the shorter one."""
    cfg, w = plain.load_folder(make_folder(tmp_path, "P"))
    tokens = random_tokens(cfg["vocab"], 80, 1)
    assert torch.allclose(plain.forward(cfg, w, tokens)[:33], plain.forward(cfg, w, tokens[:33]), atol=1e-5)


@pytest.mark.parametrize("name", sorted(CONFIGS))
def test_configuration_round_trip_and_tensors(name, tmp_path):
    raw = CONFIGS[name][0]
    cfg = FigalornConfig.from_dict(raw)
    assert FigalornConfig.from_dict(json.loads(json.dumps(cfg.to_dict()))) == cfg
    folder = make_folder(tmp_path, name)
    needs = Model(resolve_architecture(raw).build_spec(cfg)).tensor_needs()
    got = hb.weights.read_tensors(folder, needs, strict=True)
    assert set(got) == set(needs) and ("loop.in" in needs) == ("loop" in raw)
    for i, layer in enumerate(raw["layers"]):
        m, two = layer["mixer"], layer["type"] == "attention"
        assert (f"l{i}.norm2" in needs) == (layer["mlp"] is not None) == (f"l{i}.mlp.up" in needs)
        assert (f"l{i}.mix.v" in needs) == (f"l{i}.mix.g" in needs) == (f"l{i}.mix.q.b" in needs) == (f"l{i}.mix.lq1" in needs) == two
        assert (f"l{i}.mix.q.norm" in needs) != two and f"l{i}.mix.o.b" not in needs
        assert got[f"l{i}.mix.q"].shape == (m["heads"] * (2 if two else 1) * m["dim"], raw["width"])
        assert got[f"l{i}.mix.k"].shape == (m["kv_heads"] * (2 if two else 1) * m["dim"], raw["width"])
        assert got[f"l{i}.mix.o"].shape == (raw["width"], m["heads"] * m["vdim"])


def test_values_have_the_keys_size_where_they_are_the_keys():
    raw = json.loads(json.dumps(CONFIGS["Q"][0]))
    del raw["layers"][0]["mixer"]["vdim"]
    assert FigalornConfig.from_dict(raw) == FigalornConfig.from_dict(CONFIGS["Q"][0])


@pytest.mark.parametrize("change,word", [
    (lambda r: r["layers"][0].update(type="mamba2"), "unknown layer type"),
    (lambda r: r["layers"][0].update(mlp={"kind": "moe"}), "unknown feed-forward"),
    (lambda r: r["layers"][1]["mixer"].update(kv_heads=4), "multiple of kv_heads"),
    (lambda r: r["layers"][1]["mixer"].update(vdim=24), "vdim must be dim"),
    (lambda r: r["layers"][1]["mixer"].update(softcap=0.0), "softcap"),
    (lambda r: r["layers"][0]["mixer"].pop("diff"), "diff"),
    (lambda r: r["layers"][0]["mixer"].pop("scale"), "scale"),
    (lambda r: r["layers"][0]["mixer"]["mask"].update(size=0), "mask.size"),
    (lambda r: r["layers"][0]["mixer"]["rot"].update(dims=7), "even"),
    (lambda r: r["layers"][0]["mixer"]["rot"].update(dims=14), "at most 12"),
    (lambda r: r["layers"][0]["mixer"]["rot"]["scaling"].pop("high"), "high"),
    (lambda r: r["layers"][1]["mixer"]["rot"]["scaling"].pop("fast"), "fast"),
    (lambda r: r.update(loop={"start": 2, "stop": 2, "times": 2}), "loop"),
    (lambda r: r.update(loop={"start": 0, "stop": 9, "times": 2}), "loop"),
    (lambda r: r.update(loop={"start": 0, "stop": 2, "times": 0}), "loop"),
    (lambda r: r.pop("norm"), "norm"),
    (lambda r: r.update(width=0), "width"),
])
def test_what_a_configuration_may_not_say(change, word):
    raw = json.loads(json.dumps(CONFIGS["P"][0]))
    change(raw)
    with pytest.raises(ConfigError, match=word):
        FigalornConfig.from_dict(raw)


def test_what_the_attention_part_refuses():
    shared = type("Shared", (), {"position": staticmethod(lambda spec: build("position", spec))})
    names = {k: k for k in ("q", "k", "v", "o", "g", "sink", "lq1", "lk1", "lq2", "lk2", "q_norm", "k_norm", "q_bias", "k_bias", "v_bias")}
    base = {"hidden_size": 32, "num_heads": 4, "num_kv_heads": 2, "head_dim": 8, "eps": 1e-5, "position": PartSpec("none"), "qk_norm": False,
            "names": names}
    halves = PartSpec("rope_halves", {"theta": 100.0, "rotary_dims": 8})
    for bad in ({"difference": 0.5, "sink": True}, {"difference": 0.5, "keys_are_values": True}, {"keys_are_values": True, "value_dim": 16},
                {"difference": 0.5, "conv": 3}, {"keys_are_values": True, "qk_norm": "whole"}, {"position": halves, "conv": 2},
                {"bias": "q"}, {"difference": 0.5, "window": 9, "keep_first": 2}):
        with pytest.raises(ValueError):
            build("mixer", PartSpec("attention", {**base, **bad}), shared=shared)
    part = build("mixer", PartSpec("attention", {**base, "difference": 0.5, "value_dim": 24}), shared=shared)
    assert part.q_dim == 8 * 24 and part.cache_need().head_dim == 24 and part.prepared and not part.filtered


def test_where_a_projections_row_has_its_heads():
    two = HeadsLayout(8, 2, 2, 12, 40, 64)
    assert (two.k_off, two.v_off, two.channels, two.map_stride) == (96, 144, 224, 32)
    odd = HeadsLayout(2, 1, 2, 12, 25, 25)
    assert odd.map_stride == 12 and not odd.adds_slices
    same = HeadsLayout(6, 3, 1, 20, 20, 32, True)
    assert (same.k_off, same.v_off, same.channels) == (120, 120, 180) and same.adds_slices
