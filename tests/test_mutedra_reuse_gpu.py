"""The Mutedra family's mechanisms in models of another arrangement: passes that start at blocks which know nothing of them
(pre-norm, post-norm) and between blocks of different kinds, a sandwich block around parts that only add, the bias by
distance and the kept first keys in the attention's other form (with a gate, a stored sink and a rotation)."""
import numpy as np
import pytest
import torch

from herbert_rs_amd.engine import Engine, StepEntry
from herbert_rs_amd.engine.model import Model
from herbert_rs_amd.errors import ConfigError
from herbert_rs_amd.parts import LayerSpec, ModelSpec, PartSpec, ScheduleEntry
from herbert_rs_amd.weights import random_tensors

from .bounds import rel_rms_error
from .plain import mutedra as plain

pytestmark = pytest.mark.gpu

W, V, HEADS, KV, D, FF, SIZE, KEEP, BIAS_MAX, SCALE, EPS = 96, 120, 4, 2, 32, 64, 40, 3, 60, 0.3, 1e-5
ROT = {"dims": 16, "base": 200.0}
# (layer, number of the pass that starts there): at a pre-norm block, at a post-norm block behind a sandwich, at a sandwich
# behind a sandwich, at a sandwich behind a pre-norm block
SCHEDULE = [(0, 0), (1, None), (1, 1), (2, 2), (0, None), (1, 3), (2, None)]


def attention(p, other_form):
    names = {k: p + k for k in ("q", "k", "v", "o", "rel") + (("g", "sink") if other_form else ())}
    position = PartSpec("rope_pairs", {"theta": ROT["base"], "rotary_dims": ROT["dims"]}) if other_form else PartSpec("none")
    return PartSpec("attention", {"hidden_size": W, "num_heads": HEADS, "num_kv_heads": KV, "head_dim": D, "eps": EPS,
                                  "position": position, "names": names, "qk_norm": False, "scale": SCALE, "window": SIZE,
                                  "keep_first": KEEP, "distance_bias": (BIAS_MAX,), "gate": other_form,
                                  "sink": True if other_form else "unit"})


def spec():
    rms = lambda name: PartSpec("rmsnorm", {"size": W, "eps": EPS, "weight": name})
    tanh = lambda name: PartSpec("dynamic_tanh", {"size": W, "weight": name})
    relu = lambda p: PartSpec("swiglu", {"hidden_size": W, "intermediate_size": FF, "activation": "relu",
                                         "names": {k: p + k for k in ("gate", "up", "down")}})
    squared = PartSpec("squared_relu", {"hidden_size": W, "intermediate_size": FF, "names": {"up": "b.up", "down": "b.down"}})
    layers = [LayerSpec(PartSpec("prenorm"), attention("a.", True), relu("a."), {"input": rms("a.n1"), "post_mixer": rms("a.n2")}),
              LayerSpec(PartSpec("sandwich"), attention("b.", True), squared,
                        {r: tanh("b." + r) for r in ("before_mixer", "after_mixer", "before_ff", "after_ff")}),
              LayerSpec(PartSpec("postnorm", {"alpha": 1.5}), attention("c.", False), relu("c."),
                        {"post_mixer": rms("c.n1"), "post_ff": rms("c.n2")})]
    return ModelSpec(hidden_size=W, vocab_size=V, max_positions=512,
                     embedding=PartSpec("table", {"vocab_size": V, "hidden_size": W, "weight": "emb", "scale": 1.3}),
                     layers=layers, schedule=[ScheduleEntry(i, starts_pass=t) for i, t in SCHEDULE], final_norm=rms("fn"),
                     head=PartSpec("linear", {"vocab_size": V, "hidden_size": W, "weight": "head", "tied_to_embedding": False,
                                              "softcap": 7.0}),
                     pass_input=PartSpec("step_and_embedding", {"hidden_size": W, "passes": 4, "weight": "steps"}))


def plain_attention(h, w, p, other_form):
    T, positions = h.shape[0], torch.arange(h.shape[0])
    q, k, v = (plain.linear(h, w[p + n]).view(T, -1, D) for n in "qkv")
    if other_form:
        q, k = plain.rotate_pairs(q, positions, ROT), plain.rotate_pairs(k, positions, ROT)
    see, bias = plain.visible(positions, SIZE, KEEP), plain.distance_bias(w[p + "rel"], positions, BIAS_MAX)
    out = torch.zeros(T, HEADS, D)
    for a in range(HEADS):
        g = a // (HEADS // KV)
        s = (q[:, a] @ k[:, g].T) * SCALE + bias[:, :, a]
        out[:, a] = plain.softmax_with_sink(s, see, w[p + "sink"][a] if other_form else 0.0) @ v[:, g]
    out = out.reshape(T, -1)
    if other_form:
        out = out * plain.sigmoid(plain.linear(h, w[p + "g"]))
    return plain.linear(out, w[p + "o"])


def plain_forward(w, tokens):
    rms = lambda x, n: plain.rms_norm(x, w[n], EPS)
    tanh = lambda x, r: plain.dynamic_tanh(x, w["b." + r + ".alpha"], w["b." + r], w["b." + r + ".b"])
    unit = lambda h, p: plain.relu_unit(h, w[p + "gate"], w[p + "up"], w[p + "down"])
    embedded = w["emb"][torch.tensor(tokens)] * 1.3
    x = embedded
    for layer, t in SCHEDULE:
        if t is not None:
            x = x + (embedded if t else 0) + w["steps"][t]
        if layer == 0:
            x = x + plain_attention(rms(x, "a.n1"), w, "a.", True)
            x = x + unit(rms(x, "a.n2"), "a.")
        elif layer == 1:
            x = x + tanh(plain_attention(tanh(x, "before_mixer"), w, "b.", True), "after_mixer")
            h = torch.clamp(plain.linear(tanh(x, "before_ff"), w["b.up"]), min=0.0) ** 2
            x = x + tanh(plain.linear(h, w["b.down"]), "after_ff")
        else:
            x = rms(1.5 * x + plain_attention(x, w, "c.", False), "c.n1")
            x = rms(1.5 * x + unit(x, "c."), "c.n2")
    return plain.capped(plain.linear(rms(x, "fn"), w["head"]), 7.0).numpy()


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_blocks_of_several_kinds_and_passes_between_them(dtype):
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


def test_a_schedule_that_names_passes_without_saying_what_joins():
    import dataclasses
    with pytest.raises(ConfigError, match="passes"):
        Model(dataclasses.replace(spec(), pass_input=None))
