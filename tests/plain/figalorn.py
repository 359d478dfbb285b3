"""Plain, slow, whole-sequence formulas of the Figalorn decoder: one function a mechanism.

A model of this design is a stack of pre-norm layers

    x <- x + mixer(n1(x));  x <- x + ff(n2(x))

with n(x) = x / sqrt(mean(x^2) + eps) (1 + w). A stretch of the layers may run several times over with the same
weights; every pass, the first one included, starts with x <- W_in [x | x0], x0 the embedding's output. A mixer is
the difference of two softmax attentions over the keys of the query's own chunk of positions, which share their
values, with biases, a rotation of neighbouring pairs and a gate an entry ("attention"), or a softmax attention over a
window whose values are the keys before their norm and rotation, with a norm a head, a rotation of halves and
capped scores ("attention_2"). The feed-forward is two matrices with the exact gelu between them. Nothing here has
a cache, a batch or code in common with the engine; everything runs on the CPU in the dtype of its inputs (float32,
or float64 to judge rounding).
"""
import json
import math
import os

import torch
from safetensors import safe_open


# ---------------------------------------------------------------- small pieces
def over_rms(x, eps):
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def norm_around_one(x, w, eps):
    return over_rms(x, eps) * (1.0 + w)


def linear(x, weight, bias=None):
    y = x @ weight.T
    return y if bias is None else y + bias


def sigmoid(x):
    return 1.0 / (1.0 + torch.exp(-x))


def gelu_erf(z):
    """z times the share of a standard normal variable that lies below z."""
    return 0.5 * z * (1.0 + torch.erf(z / math.sqrt(2.0)))


def feed_forward(h, w):
    return linear(gelu_erf(linear(h, w["up"])), w["down"])


def loop_input(x, x0, w_in):
    return linear(torch.cat([x, x0], -1), w_in)


# ---------------------------------------------------------------- rates of rotation
def base_rates(rot):
    dims = rot["dims"]
    return torch.tensor([rot["base"] ** (-2.0 * i / dims) for i in range(dims // 2)], dtype=torch.float64)


def rates_by_wavelength(rot):
    """Short wavelengths keep their rate, long ones are slowed by the factor, those between are a blend."""
    f = base_rates(rot)
    sc = rot.get("scaling")
    if sc is None:
        return f
    out = []
    for rate in f.tolist():
        wave = 2.0 * math.pi / rate
        if wave < sc["original"] / sc["high"]:
            out.append(rate)
        elif wave > sc["original"] / sc["low"]:
            out.append(rate / sc["factor"])
        else:
            s = (sc["original"] / wave - sc["low"]) / (sc["high"] - sc["low"])
            out.append((1.0 - s) * rate / sc["factor"] + s * rate)
    return torch.tensor(out, dtype=torch.float64)


def rates_by_ramp(rot):
    """(rates, factor of cosine and sine): pairs up to `lo` keep their rate, from `hi` on they are slowed by the factor,
    a straight line between; lo and hi are the pairs that turn `fast` and `slow` times in the original length."""
    f = base_rates(rot)
    sc = rot.get("scaling")
    if sc is None:
        return f, 1.0
    dims = rot["dims"]

    def pair_that_turns(times):
        return dims * math.log(sc["original"] / (2.0 * math.pi * times)) / (2.0 * math.log(rot["base"]))

    lo = max(math.floor(pair_that_turns(sc["fast"])), 0)
    hi = min(math.ceil(pair_that_turns(sc["slow"])), dims - 1)
    i = torch.arange(dims // 2, dtype=torch.float64)
    ramp = torch.clamp((i - lo) / max(hi - lo, 0.001), 0.0, 1.0)
    return f / sc["factor"] * ramp + f * (1.0 - ramp), 0.1 * math.log(sc["factor"]) + 1.0


def _angles(positions, rates, like):
    ang = positions.to(torch.float64)[:, None] * rates[None, :]
    return torch.cos(ang).to(like.dtype)[:, None, :], torch.sin(ang).to(like.dtype)[:, None, :]


def rotate_pairs(x, positions, rot):
    """x [T, heads, D]: entries 2i and 2i + 1 of the first rot.dims turn together."""
    if rot is None:
        return x
    dims = rot["dims"]
    cos, sin = _angles(positions, rates_by_wavelength(rot), x)
    out = x.clone()
    u, v = x[..., 0:dims:2], x[..., 1:dims:2]
    out[..., 0:dims:2] = u * cos - v * sin
    out[..., 1:dims:2] = v * cos + u * sin
    return out


def rotate_halves(x, positions, rot):
    """x [T, heads, D]: entries i and i + dims / 2 of the first rot.dims turn together."""
    if rot is None:
        return x
    half = rot["dims"] // 2
    rates, grow = rates_by_ramp(rot)
    cos, sin = _angles(positions, rates, x)
    cos, sin = cos * grow, sin * grow
    out = x.clone()
    u, v = x[..., :half], x[..., half:2 * half]
    out[..., :half] = u * cos - v * sin
    out[..., half:2 * half] = v * cos + u * sin
    return out


# ---------------------------------------------------------------- which keys
def visible_chunk(positions, size):
    i, j = positions[:, None], positions[None, :]
    see = j <= i
    if size is not None:
        see = see & (i // size == j // size)
    return see


def visible_window(positions, size):
    i, j = positions[:, None], positions[None, :]
    see = j <= i
    if size is not None:
        see = see & (i - j < size)
    return see


# ---------------------------------------------------------------- mixers
def difference_factor(w, diff):
    return torch.exp((w["lq1"] * w["lk1"]).sum()) - torch.exp((w["lq2"] * w["lk2"]).sum()) + diff


def difference_mixer(h, w, m, eps, positions):
    T = h.shape[0]
    H, G, D, Dv = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q = linear(h, w["q"], w["q.b"]).view(T, H * 2, D)
    k = linear(h, w["k"], w["k.b"]).view(T, G * 2, D)
    v = linear(h, w["v"], w["v.b"]).view(T, G, Dv)
    q = rotate_pairs(q, positions, m.get("rot")).view(T, H, 2, D)
    k = rotate_pairs(k, positions, m.get("rot")).view(T, G, 2, D)
    see = visible_chunk(positions, (m.get("mask") or {}).get("size"))
    lam = difference_factor(w, m["diff"])
    out = torch.zeros(T, H, Dv, dtype=h.dtype)
    for a in range(H):
        g = a // (H // G)
        maps = []
        for j in range(2):
            s = (q[:, a, j] @ k[:, g, j].T) * m["scale"]
            maps.append(torch.softmax(s.masked_fill(~see, float("-inf")), -1) @ v[:, g])
        out[:, a] = over_rms(maps[0] - lam * maps[1], eps) * (1.0 - m["diff"])
    joined = out.reshape(T, H * Dv) * sigmoid(linear(h, w["g"]))
    return linear(joined, w["o"])


def key_value_mixer(h, w, m, eps, positions):
    T = h.shape[0]
    H, G, D = m["heads"], m["kv_heads"], m["dim"]
    q = linear(h, w["q"]).view(T, H, D)
    v = linear(h, w["k"]).view(T, G, D)
    q = rotate_halves(over_rms(q, eps) * w["q.norm"], positions, m.get("rot"))
    k = rotate_halves(over_rms(v, eps) * w["k.norm"], positions, m.get("rot"))
    see = visible_window(positions, (m.get("mask") or {}).get("size"))
    out = torch.zeros(T, H, D, dtype=h.dtype)
    for a in range(H):
        g = a // (H // G)
        s = (q[:, a] @ k[:, g].T) * m["scale"]
        if m.get("softcap"):
            s = m["softcap"] * torch.tanh(s / m["softcap"])
        out[:, a] = torch.softmax(s.masked_fill(~see, float("-inf")), -1) @ v[:, g]
    return linear(out.reshape(T, H * D), w["o"])


MIXERS = {"attention": difference_mixer, "attention_2": key_value_mixer}


# ---------------------------------------------------------------- the model
def sub(tensors, prefix):
    return {k[len(prefix):]: v for k, v in tensors.items() if k.startswith(prefix)}


def runs(cfg):
    """[(layer, True where a pass starts before it)] in the order in which the layers run."""
    n, loop = len(cfg["layers"]), cfg.get("loop")
    if not loop:
        return [(i, False) for i in range(n)]
    order = [(i, False) for i in range(loop["start"])]
    for _ in range(loop["times"]):
        order += [(i, i == loop["start"]) for i in range(loop["start"], loop["stop"])]
    return order + [(i, False) for i in range(loop["stop"], n)]


def forward(cfg, tensors, tokens, dtype=torch.float32, layers_out=None, rows=None):
    """Logits [T, vocab] (or at `rows`) of one sequence from its first token on."""
    w = {k: (v.to(dtype) if v.is_floating_point() else v) for k, v in tensors.items()}
    eps = cfg["norm"]["eps"]
    tokens = torch.as_tensor(tokens, dtype=torch.long)
    positions = torch.arange(tokens.shape[0])
    x0 = w["embed"][tokens]
    x = x0
    for i, starts_pass in runs(cfg):
        if starts_pass:
            x = loop_input(x, x0, w["loop.in"])
        layer, p = cfg["layers"][i], f"l{i}."
        x = x + MIXERS[layer["type"]](norm_around_one(x, w[p + "norm1"], eps), sub(w, p + "mix."), layer["mixer"], eps,
                                      positions)
        if layer.get("mlp") is not None:
            x = x + feed_forward(norm_around_one(x, w[p + "norm2"], eps), sub(w, p + "mlp."))
        if layers_out is not None:
            layers_out.append(x.clone())
    x = norm_around_one(x, w["final.norm"], eps)
    if rows is not None:
        x = x[torch.as_tensor(rows, dtype=torch.long)]
    return linear(x, w["head"])


def greedy(cfg, tensors, prompt, n):
    """The n tokens that follow `prompt` when the most likely one (the lower of equals) is taken each time."""
    tokens, out = list(prompt), []
    for _ in range(n):
        out.append(int(torch.argmax(forward(cfg, tensors, tokens, rows=[len(tokens) - 1])[0])))
        tokens.append(out[-1])
    return out


def load_folder(folder):
    with open(os.path.join(folder, "config.json")) as f:
        cfg = json.load(f)
    tensors = {}
    with safe_open(os.path.join(folder, "model.safetensors"), "pt") as f:
        for k in f.keys():
            tensors[k] = f.get_tensor(k)
    return cfg, tensors
