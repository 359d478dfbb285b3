"""Small Mutedra configurations for the tests, their model folders, and the plain logits.

The configurations differ from each other in every size and option: which mixer comes first and last, keys and
values of different sizes, heads that share keys or not, one head, windows shorter than a page, a page long, longer
and none at all, none, one, a few and more than a page of kept first keys, bias tables of 2 to 64 rows that end inside and
beyond the window, latents and rotated parts that the matrix cores take and that they do not, latents of the queries
wider and narrower than those of the keys, loops over the first layers, the last, one layer or the whole model,
once to three times or none, layers without a feed-forward, capped logits or not, constants that are neither 1 nor
equal to each other.
"""
import os

import numpy as np
import torch
from safetensors import safe_open
from safetensors.torch import save_file

import herbert_rs_amd as hb

from .plain import mutedra as plain


def dense(ff):
    return {"kind": "dense", "ff": ff}


def attention(heads, kv_heads, dim, vdim, scale, bias_max, size=None, keep_first=0, mlp=None):
    m = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale, "bias_max": bias_max}
    if size is not None:
        m["mask"] = {"size": size, "keep_first": keep_first}
    return {"type": "attention", "mixer": m, "mlp": mlp}


def latent(heads, dim, vdim, kv_rank, q_rank, scale, mlp=None):
    m = {"heads": heads, "dim": dim, "vdim": vdim, "kv_rank": kv_rank, "q_rank": q_rank, "scale": scale}
    return {"type": "latent_attention", "mixer": m, "mlp": mlp}


def rotated(heads, dim, rot_dim, vdim, kv_rank, q_rank, scale, base, mlp=None):
    entry = latent(heads, dim, vdim, kv_rank, q_rank, scale, mlp)
    entry["type"] = "latent_attention_2"
    entry["mixer"].update(rot_dim=rot_dim, rot={"dims": rot_dim, "base": base})
    return entry


def model(vocab, width, layers, eps, scale=1.0, loop=None, cap=None):
    d = {"architecture": "Mutedra", "vocab": vocab, "width": width, "layers": layers, "norm": {"eps": eps},
         "embedding": {"scale": scale}}
    if loop is not None:
        d["loop"] = {"start": loop[0], "stop": loop[1], "times": loop[2]}
    if cap is not None:
        d["logit_softcap"] = cap
    return d


def _p():
    # P: sizes that no kernel's block divides, keys and values of different sizes, a window shorter than a page that
    #    ends inside the bias table, a loop over the first two of four layers, three times
    layers = [rotated(3, 20, 12, 24, 40, 56, 0.2, 300.0, mlp=dense(72)),
              attention(6, 2, 24, 40, 0.25, 90, size=50, keep_first=3, mlp=dense(100)),
              latent(5, 16, 24, 48, 24, 0.3, mlp=dense(64)),
              attention(4, 4, 32, 16, 0.2, 40, mlp=None)]
    return model(210, 96, layers, eps=1e-5, scale=1.5, loop=(0, 2, 3), cap=9.0)


def _q():
    # Q: sizes that the matrix cores take throughout; more than a page of kept first keys beside a window of two
    #    pages, and a window of one page with one kept key; a loop over two layers in the middle
    layers = [attention(4, 2, 64, 64, 0.15, 300, size=128, keep_first=70, mlp=dense(256)),
              rotated(4, 32, 32, 64, 96, 64, 0.15, 10000.0, mlp=dense(128)),
              attention(4, 1, 128, 128, 0.1, 64, size=64, keep_first=1, mlp=dense(192)),
              latent(8, 32, 32, 64, 128, 0.2, mlp=dense(256))]
    return model(384, 128, layers, eps=1e-6, scale=0.7, loop=(1, 3, 2), cap=20.0)


def _r():
    # R: one head each; values wider than a wave, keys of 48; no kept keys with a window, no window with a table of
    #    two rows; layers without a feed-forward; the whole model twice; logits as they are
    layers = [latent(1, 16, 80, 24, 8, 0.3, mlp=None),
              attention(1, 1, 48, 80, 0.15, 20, size=33, mlp=dense(24)),
              rotated(1, 8, 4, 80, 32, 48, 0.3, 50.0, mlp=None),
              attention(1, 1, 48, 80, 0.15, 7, mlp=dense(40))]
    return model(96, 64, layers, eps=1e-5, loop=(0, 4, 2))


def _s():
    # S: heads beyond 128 (the plain attention kernel in either mode); a window of 7 with 2 kept keys, a window of one
    #    key; a latent of 72 (no step of 32); one pass over the last layer, and a layer without a feed-forward before
    layers = [attention(2, 1, 160, 144, 0.08, 11, size=7, keep_first=2, mlp=dense(96)),
              latent(2, 40, 24, 72, 32, 0.2, mlp=None),
              attention(3, 1, 64, 64, 0.2, 50, size=1, keep_first=9, mlp=dense(64)),
              rotated(2, 40, 8, 24, 72, 40, 0.1, 1000.0, mlp=dense(96))]
    return model(320, 192, layers, eps=2e-5, scale=3.0, loop=(3, 4, 1), cap=30.0)


def _w():
    # W: the widths of a larger model's layers at a small depth: heads of 128, a latent of 256 + 64
    layers = [rotated(8, 64, 64, 64, 256, 192, 0.1, 10000.0, mlp=dense(1024)),
              attention(8, 2, 128, 128, 0.09, 500, size=192, keep_first=5, mlp=dense(1024)),
              latent(8, 64, 64, 256, 128, 0.12, mlp=dense(512))]
    return model(1024, 512, layers, eps=1e-6, scale=2.0, loop=(0, 2, 2), cap=25.0)


def _f():
    # F: for keys far back: scores several times as sharp as a random model's usual ones, an attention without a
    #    window whose bias table ends at 200, and one with a window of 64
    layers = [attention(4, 2, 64, 64, 1.2, 200, mlp=dense(128)),
              rotated(4, 32, 32, 32, 64, 64, 0.9, 1000.0, mlp=dense(128)),
              attention(4, 2, 64, 64, 1.2, 100, size=64, keep_first=4, mlp=dense(128)),
              latent(4, 32, 32, 64, 64, 0.9, mlp=dense(128))]
    return model(384, 128, layers, eps=1e-6, scale=1.0, cap=40.0)


# name -> (config, seed, std of the matrices, rows of the layers' bias tables in turn)
CONFIGS = {"F": (_f(), 56, 0.09, (32, 16)), "P": (_p(), 51, 0.12, (10, 8)), "Q": (_q(), 52, 0.09, (32, 64)), "R": (_r(), 53, 0.15, (12, 2)),
           "S": (_s(), 54, 0.08, (6, 24)), "W": (_w(), 55, 0.05, (48,))}


def write_folder(folder, raw, seed, std, rows=(32,), dtype="float32", scale=None):
    """A random model; the bias tables have `rows` rows in turn. `scale` {tensor name suffix: factor} multiplies tensors
    afterwards, to make a far key or a window's edge show where random weights would hide it."""
    hb.write_random_model(folder, raw, seed=seed, dtype=dtype, std=std, norm_std=0.1)
    path = os.path.join(folder, "model.safetensors")
    with safe_open(path, framework="pt") as f:
        tensors = {k: f.get_tensor(k) for k in f.keys()}
    n = 0
    for k in sorted(tensors):
        if k.endswith(".mix.rel"):
            table = torch.randn(rows[n % len(rows)], tensors[k].shape[1], generator=torch.Generator().manual_seed(seed + n))
            tensors[k] = table.to(tensors[k].dtype)
            n += 1
        for suffix, factor in (scale or {}).items():
            if k.endswith(suffix):
                tensors[k] = (tensors[k].float() * factor).to(tensors[k].dtype)
    save_file(tensors, path)
    return folder


def make_folder(root, name, dtype="float32", tag="", scale=None):
    """Write the random model `name` into root/mut_<name>_<dtype><tag> once."""
    raw, seed, std, rows = CONFIGS[name]
    folder = os.path.join(str(root), f"mut_{name}_{dtype}{tag}")
    if not os.path.exists(os.path.join(folder, "model.safetensors")):
        write_folder(folder, raw, seed, std, rows, dtype, scale)
    return folder


_folders, _logits = {}, {}


def plain_folder(folder):
    if folder not in _folders:
        _folders[folder] = plain.load_folder(folder)
    return _folders[folder]


def plain_logits(folder, tokens):
    """float32 [len(tokens), vocab] of the plain whole-sequence implementation, computed once."""
    key = (folder, tuple(tokens))
    if key not in _logits:
        cfg, w = plain_folder(folder)
        _logits[key] = plain.forward(cfg, w, list(tokens)).numpy().astype(np.float32)
    return _logits[key]


def random_tokens(vocab, n, seed):
    g = torch.Generator().manual_seed(seed)
    return torch.randint(0, vocab, (n,), generator=g).tolist()
