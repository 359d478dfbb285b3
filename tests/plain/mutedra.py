"""Plain, slow, whole-sequence formulas of the Mutedra decoder: one function a mechanism.

Every layer norms before and after each of its two steps,

    x <- x + n1b(mixer(n1(x)));  x <- x + n2b(ff(n2(x)))

with n(x) = tanh(alpha x) w + b, which has no mean and no variance. A stretch of the layers may run several
times over with the same weights; at the start of each of its passes a vector of that pass is added to x,
and from the second pass on, before that, the embedding output once more. A mixer is a softmax attention over a
window of the last keys and the first few of the sequence, with a learned bias by distance and a one in the
softmax's denominator ("attention"), or an attention whose keys and values come from one low-rank latent a
token, its queries from a latent of their own: without any position ("latent_attention"), or with a rotated
part, a sink a head and a gate a head ("latent_attention_2"). Nothing here has a cache, a batch or code in
common with the engine; everything runs on the CPU in the dtype of its inputs (float32, or float64 to judge
rounding).
"""
import json
import math
import os

import torch
from safetensors import safe_open


# ---------------------------------------------------------------- small pieces
def dynamic_tanh(x, alpha, w, b):
    return torch.tanh(alpha * x) * w + b


def rms_norm(x, w, eps):
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps) * w


def linear(x, weight):
    return x @ weight.T


def sigmoid(x):
    return 1.0 / (1.0 + torch.exp(-x))


def relu_unit(h, gate, up, down):
    return linear(torch.clamp(linear(h, gate), min=0.0) * linear(h, up), down)


def capped(z, cap):
    return z if cap is None else cap * torch.tanh(z / cap)


# ---------------------------------------------------------------- positions
def bucket(n, rows, bias_max):
    """The table row of distance n: one a distance for the first half of the rows, then by the logarithm up to
    bias_max, the last row from there on."""
    half = rows // 2
    if n < half:
        return n
    return min(rows - 1, half + math.floor(math.log(n / half) / math.log(bias_max / half) * (rows - half)))


def distance_bias(table, positions, bias_max):
    """table [rows, heads] -> [T, T, heads], the bias of key j for query i (zero where j > i)."""
    T = positions.shape[0]
    row = [bucket(n, table.shape[0], bias_max) for n in range(int(positions.max()) + 1)]
    index = torch.tensor([[row[max(0, int(positions[i] - positions[j]))] for j in range(T)] for i in range(T)])
    return table[index]


def rotate_pairs(x, positions, rot):
    """x [T, heads, D]: entries 2i and 2i + 1 of the first rot.dims turn by position x base^(-2i / dims)."""
    dims = rot["dims"]
    rates = torch.tensor([rot["base"] ** (-2.0 * i / dims) for i in range(dims // 2)], dtype=torch.float64)
    ang = positions.to(torch.float64)[:, None] * rates[None, :]
    cos, sin = torch.cos(ang).to(x.dtype)[:, None, :], torch.sin(ang).to(x.dtype)[:, None, :]
    out = x.clone()
    u, v = x[..., 0:dims:2], x[..., 1:dims:2]
    out[..., 0:dims:2] = u * cos - v * sin
    out[..., 1:dims:2] = v * cos + u * sin
    return out


# ---------------------------------------------------------------- which keys, and their weights
def visible(positions, size=None, keep_first=0):
    """[T, T] True where query i sees key j: j <= i, and with a window only the last `size` positions and the
    sequence's first `keep_first`."""
    i, j = positions[:, None], positions[None, :]
    see = j <= i
    if size is not None:
        see = see & ((i - j < size) | (j < keep_first))
    return see


def softmax_with_sink(scores, see, sink):
    """Weights over the visible keys; the denominator also holds exp(sink) (None: nothing)."""
    s = scores.masked_fill(~see, float("-inf"))
    top = s.max(dim=-1, keepdim=True).values
    if sink is not None:
        top = torch.maximum(top, torch.full_like(top, float(sink)))
    e = torch.exp(s - top)
    total = e.sum(-1, keepdim=True)
    if sink is not None:
        total = total + torch.exp(float(sink) - top)
    return e / total


# ---------------------------------------------------------------- mixers
def attention_mixer(h, w, m, eps, positions):
    T = h.shape[0]
    H, G, D, Dv = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q = linear(h, w["q"]).view(T, H, D)
    k = linear(h, w["k"]).view(T, G, D)
    v = linear(h, w["v"]).view(T, G, Dv)
    mask = m.get("mask") or {}
    see = visible(positions, mask.get("size"), mask.get("keep_first", 0))
    bias = distance_bias(w["rel"], positions, m["bias_max"])
    out = torch.zeros(T, H, Dv, dtype=h.dtype)
    for a in range(H):
        g = a // (H // G)
        s = (q[:, a] @ k[:, g].T) * m["scale"] + bias[:, :, a]
        out[:, a] = softmax_with_sink(s, see, 0.0) @ v[:, g]
    return linear(out.reshape(T, H * Dv), w["o"])


def latent_mixer(h, w, m, eps, positions):
    """Both latent kinds: with a rotated part, sinks and gates where the layer has their sizes and tensors."""
    T = h.shape[0]
    H, D, Dv, rank, R = m["heads"], m["dim"], m["vdim"], m["kv_rank"], m.get("rot_dim", 0)
    q = linear(rms_norm(linear(h, w["dq"]), w["dq.norm"], eps), w["uq"]).view(T, H, D + R)
    down = linear(h, w["dkv"])
    c = rms_norm(down[:, :rank], w["dkv.norm"], eps)
    k = linear(c, w["uk"]).view(T, H, D)
    v = linear(c, w["uv"]).view(T, H, Dv)
    if R:
        k_rot = rotate_pairs(down[:, rank:].view(T, 1, R), positions, m["rot"])[:, 0]
        q = torch.cat([q[..., :D], rotate_pairs(q[..., D:], positions, m["rot"])], -1)
    see = visible(positions)
    out = torch.zeros(T, H, Dv, dtype=h.dtype)
    for a in range(H):
        s = q[:, a, :D] @ k[:, a].T
        if R:
            s = s + q[:, a, D:] @ k_rot.T
        out[:, a] = softmax_with_sink(s * m["scale"], see, w["sink"][a] if "sink" in w else None) @ v[:, a]
    if "g" in w:
        out = out * sigmoid(linear(h, w["g"]))[:, :, None]
    return linear(out.reshape(T, H * Dv), w["o"])


MIXERS = {"attention": attention_mixer, "latent_attention": latent_mixer, "latent_attention_2": latent_mixer}


# ---------------------------------------------------------------- the model
def sub(tensors, prefix):
    return {k[len(prefix):]: v for k, v in tensors.items() if k.startswith(prefix)}


def runs(cfg):
    """[(layer, number of the pass that starts before it or None)] in the order in which the layers run."""
    n = len(cfg["layers"])
    loop = cfg.get("loop")
    if not loop:
        return [(i, None) for i in range(n)]
    order = [(i, None) for i in range(loop["start"])]
    for t in range(loop["times"]):
        order += [(i, t if i == loop["start"] else None) for i in range(loop["start"], loop["stop"])]
    return order + [(i, None) for i in range(loop["stop"], n)]


def forward(cfg, tensors, tokens, dtype=torch.float32, layers_out=None, rows=None):
    """Logits [T, vocab] (or at `rows`) of one sequence from its first token on."""
    w = {k: (v.to(dtype) if v.is_floating_point() else v) for k, v in tensors.items()}
    eps = cfg["norm"]["eps"]
    tokens = torch.as_tensor(tokens, dtype=torch.long)
    positions = torch.arange(tokens.shape[0])
    norm = lambda name, v: dynamic_tanh(v, w[name + ".alpha"], w[name], w[name + ".b"])
    embedded = w["embed"][tokens] * cfg["embedding"]["scale"]
    x = embedded
    for i, pass_number in runs(cfg):
        if pass_number is not None:
            if pass_number > 0:
                x = x + embedded
            x = x + w["loop.step"][pass_number]
        layer, p = cfg["layers"][i], f"l{i}."
        y = MIXERS[layer["type"]](norm(p + "norm1", x), sub(w, p + "mix."), layer["mixer"], eps, positions)
        x = x + norm(p + "norm1b", y)
        if layer.get("mlp") is not None:
            f = sub(w, p + "mlp.")
            x = x + norm(p + "norm2b", relu_unit(norm(p + "norm2", x), f["gate"], f["up"], f["down"]))
        if layers_out is not None:
            layers_out.append(x.clone())
    x = norm("final.norm", x)
    if rows is not None:
        x = x[torch.as_tensor(rows, dtype=torch.long)]
    return capped(linear(x, w["head"]), cfg.get("logit_softcap"))


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
