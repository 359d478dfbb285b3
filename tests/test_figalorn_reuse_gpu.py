"""The Figalorn family's mechanisms in models of another arrangement: passes that make the stream anew before pre-norm,
sandwich, post-norm and parallel blocks, the difference of two maps over a window with a norm a map, halves that turn and an
output bias, values that are the keys over chunks with a gate and stored sinks, two matrices with gelu in every kind of
block, prepared heads beside kept first keys and a bias by distance."""
import numpy as np
import pytest
import torch

from herbert_rs_amd.engine import Engine, StepEntry
from herbert_rs_amd.engine.model import Model
from herbert_rs_amd.parts import LayerSpec, ModelSpec, PartSpec, ScheduleEntry
from herbert_rs_amd.weights import random_tensors

from .bounds import rel_rms_error
from .plain import figalorn as plain
from .plain.mutedra import distance_bias, dynamic_tanh, softmax_with_sink, visible

pytestmark = pytest.mark.gpu

W, V, HEADS, KV, D, FF, SIZE, SCALE, EPS, DIFF = 96, 120, 4, 2, 24, 64, 40, 0.3, 1e-5, 0.45
HALVES = {"dims": 16, "base": 200.0, "scaling": {"factor": 3.0, "original": 100, "fast": 8.0, "slow": 1.0}}
# (layer, number of the pass that starts there): at the first block and behind blocks of every kind
SCHEDULE = [(0, 0), (1, 1), (2, 2), (3, 3), (0, 4), (1, None), (1, 5), (2, None), (3, None), (3, 6)]


def attention(p, **more):
    names = {k: p + k for k in ("q", "k", "v", "o", "g", "sink", "rel", "lq1", "lk1", "lq2", "lk2", "q_norm", "k_norm", "q_bias", "k_bias",
                                "v_bias", "o_bias")}
    halves = PartSpec("rope_halves", {"theta": HALVES["base"], "rotary_dims": HALVES["dims"],
                                      "scaling": tuple(HALVES["scaling"][k] for k in ("factor", "original", "fast", "slow"))})
    return PartSpec("attention", {"hidden_size": W, "num_heads": HEADS, "num_kv_heads": KV, "head_dim": D, "eps": EPS, "position": halves,
                                  "names": names, "qk_norm": False, "scale": SCALE, **more})


def spec():
    rms = lambda name: PartSpec("rmsnorm", {"size": W, "eps": EPS, "weight": name})
    tanh = lambda name: PartSpec("dynamic_tanh", {"size": W, "weight": name})
    gelu = lambda p: PartSpec("up_down", {"hidden_size": W, "intermediate_size": FF, "names": {"up": p + "up", "down": p + "down"}})
    layers = [LayerSpec(PartSpec("prenorm"), attention("a.", difference=DIFF, value_dim=40, window=SIZE, qk_norm=True, bias=True), gelu("a."),
                        {"input": rms("a.n1"), "post_mixer": rms("a.n2")}),
              LayerSpec(PartSpec("sandwich"), attention("b.", keys_are_values=True, chunk=SIZE, gate=True, sink=True), gelu("b."),
                        {r: tanh("b." + r) for r in ("before_mixer", "after_mixer", "before_ff", "after_ff")}),
              LayerSpec(PartSpec("postnorm", {"alpha": 1.5}), attention("c.", window=SIZE, keep_first=3, distance_bias=(60,), softcap=None),
                        gelu("c."), {"post_mixer": rms("c.n1"), "post_ff": rms("c.n2")}),
              LayerSpec(PartSpec("parallel", {"mult": 0.7}), attention("d.", difference=DIFF, gate=True, softcap=8.0), gelu("d."),
                        {"input": PartSpec("layernorm", {"size": W, "eps": EPS, "weight": "d.n"})})]
    return ModelSpec(hidden_size=W, vocab_size=V, max_positions=512,
                     embedding=PartSpec("table", {"vocab_size": V, "hidden_size": W, "weight": "emb", "scale": 1.3}),
                     layers=layers, schedule=[ScheduleEntry(i, starts_pass=t) for i, t in SCHEDULE], final_norm=rms("fn"),
                     head=PartSpec("linear", {"vocab_size": V, "hidden_size": W, "weight": "head", "tied_to_embedding": False}),
                     pass_input=PartSpec("joined_projection", {"hidden_size": W, "weight": "join"}))


def plain_attention(h, w, p):
    T, positions = h.shape[0], torch.arange(h.shape[0])
    bias = (lambda n: w[p + n + "_bias"]) if p == "a." else (lambda n: None)
    q = plain.linear(h, w[p + "q"], bias("q")).view(T, -1, D)
    k = plain.linear(h, w[p + "k"], bias("k")).view(T, -1, D)
    v = k if p == "b." else plain.linear(h, w[p + "v"], bias("v")).view(T, KV, -1)
    if p == "a.":
        q, k = plain.over_rms(q, EPS) * w["a.q_norm"], plain.over_rms(k, EPS) * w["a.k_norm"]
    q, k = plain.rotate_halves(q, positions, HALVES), plain.rotate_halves(k, positions, HALVES)
    see = {"a.": plain.visible_window(positions, SIZE), "b.": plain.visible_chunk(positions, SIZE), "c.": visible(positions, SIZE, 3),
           "d.": plain.visible_chunk(positions, None)}[p]
    maps = 2 if p in ("a.", "d.") else 1
    out = []
    for a in range(HEADS):
        g, sums = a // (HEADS // KV), []
        for m in range(maps):
            s = (q[:, a * maps + m] @ k[:, g * maps + m].T) * SCALE
            if p == "c.":
                s = s + distance_bias(w["c.rel"], positions, 60)[:, :, a]
            if p == "d.":
                s = 8.0 * torch.tanh(s / 8.0)
            sums.append(softmax_with_sink(s, see, w["b.sink"][a] if p == "b." else None) @ v[:, g])
        o = sums[0]
        if maps == 2:
            names = {n: w[p + n] for n in ("lq1", "lk1", "lq2", "lk2")}
            o = plain.over_rms(sums[0] - plain.difference_factor(names, DIFF) * sums[1], EPS) * (1 - DIFF)
        out.append(o)
    out = torch.cat(out, 1)
    if p in ("b.", "d."):
        out = out * plain.sigmoid(plain.linear(h, w[p + "g"]))
    return plain.linear(out, w[p + "o"], bias("o"))


def plain_forward(w, tokens):
    rms = lambda x, n: plain.over_rms(x, EPS) * w[n]
    tanh = lambda x, r: dynamic_tanh(x, w["b." + r + ".alpha"], w["b." + r], w["b." + r + ".b"])
    unit = lambda h, p: plain.feed_forward(h, {"up": w[p + "up"], "down": w[p + "down"]})
    x0 = w["emb"][torch.tensor(tokens)] * 1.3
    x = x0
    for layer, t in SCHEDULE:
        if t is not None:
            x = plain.loop_input(x, x0, w["join"])
        if layer == 0:
            x = x + plain_attention(rms(x, "a.n1"), w, "a.")
            x = x + unit(rms(x, "a.n2"), "a.")
        elif layer == 1:
            x = x + tanh(plain_attention(tanh(x, "before_mixer"), w, "b."), "after_mixer")
            x = x + tanh(unit(tanh(x, "before_ff"), "b."), "after_ff")
        elif layer == 2:
            x = rms(1.5 * x + plain_attention(x, w, "c."), "c.n1")
            x = rms(1.5 * x + unit(x, "c."), "c.n2")
        else:
            c = x - x.mean(-1, keepdim=True)
            h = plain.over_rms(c, EPS) * w["d.n"]
            x = x + 0.7 * (plain_attention(h, w, "d.") + unit(h, "d."))
    return plain.linear(rms(x, "fn"), w["head"]).numpy()


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_blocks_of_several_kinds_and_passes_that_make_the_stream_anew(dtype):
    s = spec()
    w = random_tensors(Model(s).tensor_needs(), 5, "float32", std=0.1, norm_std=0.1)
    w = {k: v.bfloat16().float() for k, v in w.items()}
    gen = torch.Generator().manual_seed(8)
    seqs = [torch.randint(0, V, (n,), generator=gen).tolist() for n in (150, 3, 71)]
    engine = Engine(None, s, w, dtype=dtype, max_tokens=1024)
    refs = [plain_forward(w, t) for t in seqs]

    def check(row, ref, label):
        err, rel, l2 = rel_rms_error(np.asarray(row), ref)
        assert (err <= 1e-4) if dtype == "float32" else (rel <= 0.1 and l2 <= 0.03), f"{label}: {err} {rel} {l2}"
    for again in range(2):
        slots = [engine.alloc_slot() for _ in seqs]
        at = [0, 0, 0]
        for sizes in [(2, 1, 60), (99, 1, 1)] + [(1, 0, 1)] * 9 + [(40, 1, 1)]:
            live = [i for i in range(3) if sizes[i]]
            out = engine.step([StepEntry(slots[i], seqs[i][at[i]:at[i] + sizes[i]], list(range(sizes[i]))) for i in live]).cpu().numpy()
            row = 0
            for i in live:
                for j in range(sizes[i]):
                    check(out[row], refs[i][at[i] + j], f"sequence {i}, position {at[i] + j}")
                    row += 1
                at[i] += sizes[i]
        for slot in slots:
            engine.free_slot(slot)
    engine.cache.check()
