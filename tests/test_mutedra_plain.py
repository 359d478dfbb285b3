"""The plain formulas of the Mutedra decoder checked against independent ones on the CPU, the configuration, the model
as data, and the cache's pages of a window that keeps the first keys."""
import json
import math

import numpy as np
import pytest
import torch

import herbert_rs_amd as hb
from herbert_rs_amd.cache import Cache, KVNeed
from herbert_rs_amd.config import MutedraConfig
from herbert_rs_amd.config.registry import resolve_architecture
from herbert_rs_amd.engine.model import Model
from herbert_rs_amd.errors import CacheError, ConfigError, ModelLoadError
from herbert_rs_amd.parts.position import bias_by_distance, distance_bucket

from .mutedra_tiny import CONFIGS, make_folder, random_tokens
from .plain import mutedra as plain


def rand(*shape, seed=0, scale=1.0):
    return torch.randn(*shape, generator=torch.Generator().manual_seed(seed), dtype=torch.float64) * scale


def test_the_norm_bends_and_has_no_mean():
    x = rand(5, 12, seed=1)
    y = plain.dynamic_tanh(x, torch.tensor(0.7), torch.ones(12), torch.zeros(12))
    assert torch.allclose(y, (torch.exp(1.4 * x) - 1) / (torch.exp(1.4 * x) + 1))
    # an entry's value does not depend on its row's other entries
    other = x.clone()
    other[:, 1:] *= 100.0
    z = plain.dynamic_tanh(other, torch.tensor(0.7), torch.ones(12), torch.zeros(12))
    assert torch.equal(z[:, 0], y[:, 0])
    b = rand(12, seed=2)
    assert torch.allclose(plain.dynamic_tanh(torch.zeros(3, 12, dtype=torch.float64), torch.tensor(0.7), rand(12, seed=3), b), b.expand(3, 12))


@pytest.mark.parametrize("rows,bias_max", [(32, 128), (32, 200), (8, 40), (2, 7), (64, 4096), (12, 7)])
def test_distance_buckets(rows, bias_max):
    got = [plain.bucket(n, rows, bias_max) for n in range(2 * bias_max + 5)]
    half = rows // 2
    assert got[:half] == list(range(half))                        # a row a distance at first
    assert all(b - a in (0, 1) or a >= half for a, b in zip(got, got[1:])) and got == sorted(got)
    assert got[half] == half and all(g == rows - 1 for g in got[bias_max:])
    for n in range(half, bias_max):                               # the logarithm's stretch, from the border's side
        if got[n] < rows - 1:
            at = (got[n] + 1 - half) / (rows - half)
            assert n < half * (bias_max / half) ** at + 1e-6
    # the library's own, and its table by distance: the last value holds beyond the table's end
    assert [distance_bucket(n, rows, bias_max) for n in range(2 * bias_max + 5)] == got
    table = rand(rows, 3, seed=4).float()
    by_distance = bias_by_distance(table, bias_max)
    for n in range(2 * bias_max + 5):
        assert torch.equal(by_distance[min(n, by_distance.shape[0] - 1)], table[got[n]])


def test_a_bias_table_that_cannot_be():
    with pytest.raises(ValueError):
        bias_by_distance(torch.zeros(1, 2), 10)
    with pytest.raises(ValueError):
        bias_by_distance(torch.zeros(32, 2), 16)


def test_windows_and_first_keys():
    see = plain.visible(torch.arange(30), 5, 3)
    for i in range(30):
        for j in range(30):
            assert bool(see[i, j]) == (j <= i and (i - 5 < j or j in (0, 1, 2)))
    assert torch.equal(plain.visible(torch.arange(9)), torch.ones(9, 9).tril().bool())
    assert torch.equal(plain.visible(torch.arange(9), 1, 0), torch.eye(9).bool())


def test_sinks_take_their_share():
    s, see = rand(4, 4, seed=5), torch.ones(4, 4).tril().bool()
    p = plain.softmax_with_sink(s, see, 0.0)
    for i in range(4):
        e = [math.exp(float(s[i, j])) for j in range(i + 1)]
        assert torch.allclose(p[i, :i + 1], torch.tensor([v / (1 + sum(e)) for v in e], dtype=torch.float64))
    assert torch.allclose(plain.softmax_with_sink(s, see, None), torch.softmax(s.masked_fill(~see, -math.inf), -1))
    q = plain.softmax_with_sink(s, see, 2.5)
    assert torch.allclose(1 - q.sum(-1), math.exp(2.5) * q[:, 0] / torch.exp(s[:, 0]))
    assert float(plain.softmax_with_sink(s * 300, see, 0.0).isnan().sum()) == 0


def test_latent_attention_is_attention_over_built_keys():
    """Without a rotated part: plain multi-head attention whose keys and values are two matrices times the latent; with
    one: the same with the shared part joined to every head's key."""
    T, W, m = 9, 20, {"heads": 3, "dim": 4, "vdim": 5, "kv_rank": 6, "q_rank": 7, "scale": 0.4}
    for R in (0, 2):
        mm = dict(m) if not R else dict(m, rot_dim=R, rot={"dims": R, "base": 30.0})
        w = {"dq": rand(7, W, seed=1), "dq.norm": rand(7, seed=2), "uq": rand(3 * (4 + R), 7, seed=3), "dkv": rand(6 + R, W, seed=4),
             "dkv.norm": rand(6, seed=5), "uk": rand(12, 6, seed=6), "uv": rand(15, 6, seed=7), "o": rand(W, 15, seed=8)}
        if R:
            w.update(sink=rand(3, seed=9), g=rand(3, W, seed=10))
        h = rand(T, W, seed=11)
        got = plain.latent_mixer(h, w, mm, 1e-5, torch.arange(T))
        want = torch.zeros(T, 15, dtype=torch.float64)
        for i in range(T):
            cq = h[i] @ w["dq"].T
            cq = cq / math.sqrt(float((cq ** 2).mean()) + 1e-5) * w["dq.norm"]
            for a in range(3):
                q = w["uq"][a * (4 + R):(a + 1) * (4 + R)] @ cq
                e, vs = [], []
                for j in range(i + 1):
                    d = h[j] @ w["dkv"].T
                    c = d[:6] / math.sqrt(float((d[:6] ** 2).mean()) + 1e-5) * w["dkv.norm"]
                    s = float(q[:4] @ (w["uk"][4 * a:4 * a + 4] @ c))
                    if R:       # a rotation by the difference of the positions
                        t = float(i - j)
                        s += float(q[4] * (d[6] * math.cos(t) + d[7] * math.sin(t)) + q[5] * (d[7] * math.cos(t) - d[6] * math.sin(t)))
                    e.append(math.exp(s * 0.4))
                    vs.append(w["uv"][5 * a:5 * a + 5] @ c)
                total = sum(e) + (math.exp(float(w["sink"][a])) if R else 0.0)
                out = sum(p / total * v for p, v in zip(e, vs))
                if R:
                    out = out / (1 + math.exp(-float(w["g"][a] @ h[i])))
                want[i, 5 * a:5 * a + 5] = out
        assert torch.allclose(got, want @ w["o"].T)


def test_the_order_of_runs_and_what_joins_each_pass():
    cfg = {"layers": [0] * 5, "loop": {"start": 1, "stop": 3, "times": 3}}
    assert plain.runs(cfg) == [(0, None), (1, 0), (2, None), (1, 1), (2, None), (1, 2), (2, None), (3, None), (4, None)]
    raw = CONFIGS["P"][0]
    arch = resolve_architecture(raw)
    spec = arch.build_spec(MutedraConfig.from_dict(raw))
    assert [(e.layer, e.starts_pass) for e in spec.schedule] == plain.runs(raw)
    model = Model(spec)
    assert len(model.cache_needs()) == len(spec.schedule)          # every run has a cache of its own
    assert {n.keep_first for n in model.cache_needs().values()} == {0, 3}
    assert model.graph_safe


def test_portions_do_not_change_the_plain_model(tmp_path):
    """The first rows of a longer sequence are those of the shorter one."""
    cfg, w = plain.load_folder(make_folder(tmp_path, "P"))
    tokens = random_tokens(cfg["vocab"], 80, 1)
    assert torch.allclose(plain.forward(cfg, w, tokens)[:33], plain.forward(cfg, w, tokens[:33]), atol=1e-5)


@pytest.mark.parametrize("name", sorted(CONFIGS))
def test_configuration_round_trip_and_tensors(name, tmp_path):
    raw = CONFIGS[name][0]
    cfg = MutedraConfig.from_dict(raw)
    assert MutedraConfig.from_dict(json.loads(json.dumps(cfg.to_dict()))) == cfg
    folder = make_folder(tmp_path, name)
    needs = Model(resolve_architecture(raw).build_spec(cfg)).tensor_needs()
    got = hb.weights.read_tensors(folder, needs, strict=True)
    assert set(got) == set(needs) and ("loop.step" in needs) == ("loop" in raw)
    for i, layer in enumerate(raw["layers"]):
        assert (f"l{i}.norm2" in needs) == (layer["mlp"] is not None)
        assert got[f"l{i}.norm1.alpha"].shape == () and got[f"l{i}.norm1b.b"].shape == (raw["width"],)
        assert (f"l{i}.mix.sink" in needs) == (layer["type"] == "latent_attention_2")


@pytest.mark.parametrize("change,word", [
    (lambda r: r["layers"][0].update(type="mamba2"), "unknown layer type"),
    (lambda r: r["layers"][0].update(mlp={"kind": "moe"}), "unknown feed-forward"),
    (lambda r: r["layers"][1]["mixer"].update(kv_heads=4), "multiple of kv_heads"),
    (lambda r: r["layers"][1]["mixer"].pop("bias_max"), "bias_max"),
    (lambda r: r["layers"][1]["mixer"]["mask"].update(size=0), "mask.size"),
    (lambda r: r["layers"][1]["mixer"]["mask"].update(keep_first=-1), "keep_first"),
    (lambda r: r["layers"][0]["mixer"]["rot"].update(dims=6), "rot_dim"),
    (lambda r: r["layers"][2]["mixer"].pop("q_rank"), "q_rank"),
    (lambda r: r.update(loop={"start": 2, "stop": 2, "times": 2}), "loop"),
    (lambda r: r.update(loop={"start": 0, "stop": 9, "times": 2}), "loop"),
    (lambda r: r.update(logit_softcap=-1.0), "logit_softcap"),
    (lambda r: r.pop("norm"), "norm"),
])
def test_what_a_configuration_may_not_say(change, word):
    raw = json.loads(json.dumps(CONFIGS["P"][0]))
    change(raw)
    with pytest.raises(ConfigError, match=word):
        MutedraConfig.from_dict(raw)


def test_a_bias_table_of_another_number_of_heads_is_refused(tmp_path):
    from safetensors.torch import load_file, save_file
    folder = make_folder(tmp_path, "P")
    path = f"{folder}/model.safetensors"
    tensors = load_file(path)
    tensors["l1.mix.rel"] = torch.zeros(10, 7)
    save_file(tensors, path)
    raw = CONFIGS["P"][0]
    needs = Model(resolve_architecture(raw).build_spec(MutedraConfig.from_dict(raw))).tensor_needs()
    with pytest.raises(ModelLoadError, match="l1.mix.rel"):
        hb.weights.read_tensors(folder, needs)


@pytest.mark.parametrize("window,keep", [(50, 3), (64, 64), (1, 130), (100, 70), (200, 1)])
def test_pages_of_the_first_keys_stay(window, keep):
    """A slot that grows gives back the pages between the kept first keys and the window, and no other; every key that a
    later query sees lies on a page that is held; everything goes back with the slot."""
    cache = Cache({0: KVNeed(2, 8, window, keep_first=keep), 1: KVNeed(1, 4, None)}, 64 * 64, 4096, torch.float32, "cpu", max_slots=3)
    group = cache.kv_groups[KVNeed(2, 8, window, keep_first=keep)]
    whole = cache.kv_groups[KVNeed(1, 4, None)]
    rng = np.random.default_rng(window)
    for _ in range(2):
        slots = [cache.alloc_slot(), cache.alloc_slot()]
        for _ in range(40):
            for s in slots:
                n = int(rng.integers(1, 60))
                if cache.length(s) + n > 1500:
                    continue
                cache.reserve_all([(s, n)])
                first = cache.length(s)
                for p in range(first, first + n):                 # what the step's queries see is held
                    for j in {0, keep - 1, max(0, p - window + 1), p}:
                        if 0 <= j <= p:
                            assert group.table_host[s][j // 64] >= 0
                cache.commit(s, n)
                held = [p for p in range(group.pages_per_slot) if group.table_host[s][p] >= 0]
                length = cache.length(s)
                oldest = max(0, length + 1 - window) // 64
                assert held == sorted(set(range(min(-(-keep // 64), -(-length // 64)))) | set(range(oldest, -(-length // 64))))
                cache.check()
        assert whole.pages.held_count > group.pages.held_count
        with pytest.raises(CacheError):
            cache.truncate(slots[0], 10)
        for s in slots:
            cache.free_slot(s)
        cache.check()
        assert group.pages.held_count == 0


def test_a_roll_back_into_kept_pages():
    cache = Cache({0: KVNeed(1, 8, 500, keep_first=100)}, 64 * 32, 4096, torch.float32, "cpu", max_slots=1)
    group = next(iter(cache.kv_groups.values()))
    s = cache.alloc_slot()
    for n in (300, 150):
        cache.reserve_all([(s, n)])
        cache.commit(s, n)
    cache.truncate(s, 70)                       # nothing has been given up yet: the pages behind go back
    assert cache.length(s) == 70 and group.pages.held_count == 2
    cache.check()
    cache.reserve_all([(s, 700)])
    cache.commit(s, 700)
    cache.check()
    assert group.table_host[s][0] >= 0 and group.table_host[s][1] >= 0 and group.table_host[s][2] < 0


def test_a_step_that_does_not_fit_leaves_the_kept_pages_alone():
    cache = Cache({0: KVNeed(1, 8, 64, keep_first=10)}, 64 * 4, 4096, torch.float32, "cpu", max_slots=2)
    s = cache.alloc_slot()
    for _ in range(5):
        cache.reserve_all([(s, 60)])
        cache.commit(s, 60)
    before = next(iter(cache.kv_groups.values())).table_host[s].copy()
    with pytest.raises(CacheError):
        cache.reserve_all([(s, 300)])
    assert (next(iter(cache.kv_groups.values())).table_host[s] == before).all()
    cache.reserve_all([(s, 3)])
    cache.unreserve(s)
    cache.check()
