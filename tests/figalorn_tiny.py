"""Small Figalorn configurations for the tests, their model folders, and the plain logits.

The configurations differ from each other in every size and option: which mixer comes first and last, keys and values of
different sizes, heads that share keys or not, one head, windows and chunks shorter than a page, a page long, longer and
none at all, rotations of a whole head, of part of it and none, scaled or not, capped scores or not, loops over the first
layers, the last, one layer or the whole model, once to three times or none, layers without a feed-forward, constants
that are neither 1 nor equal to each other.
"""
import os

import numpy as np
import torch
from safetensors import safe_open
from safetensors.torch import save_file

import herbert_rs_amd as hb

from .plain import figalorn as plain


def dense(ff):
    return {"kind": "dense", "ff": ff}


def rotation(dims, base, **scaling):
    return {"dims": dims, "base": base, **({"scaling": scaling} if scaling else {})}


def difference(heads, kv_heads, dim, vdim, scale, diff, size=None, rot=None, mlp=None):
    m = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale, "diff": diff}
    if size is not None:
        m["mask"] = {"size": size}
    if rot is not None:
        m["rot"] = rot
    return {"type": "attention", "mixer": m, "mlp": mlp}


def key_value(heads, kv_heads, dim, scale, size=None, rot=None, softcap=None, mlp=None):
    m = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": dim, "scale": scale}
    if size is not None:
        m["mask"] = {"size": size}
    if rot is not None:
        m["rot"] = rot
    if softcap is not None:
        m["softcap"] = softcap
    return {"type": "attention_2", "mixer": m, "mlp": mlp}


def model(vocab, width, layers, eps, loop=None):
    d = {"architecture": "Figalorn", "vocab": vocab, "width": width, "layers": layers, "norm": {"eps": eps}}
    if loop is not None:
        d["loop"] = {"start": loop[0], "stop": loop[1], "times": loop[2]}
    return d


def _p():
    # P: sizes that no kernel's block divides, values wider and narrower than both maps' keys together, a chunk and a
    #    window shorter than a page, a loop over the first two of four layers, three times
    layers = [difference(6, 2, 12, 40, 0.3, 0.35, size=37, rot=rotation(6, 300.0, factor=4.0, low=1.0, high=4.0, original=64), mlp=dense(72)),
              key_value(6, 3, 20, 0.25, size=50, rot=rotation(12, 100.0, factor=3.0, original=80, fast=8.0, slow=1.0), softcap=6.0,
                        mlp=dense(100)),
              difference(3, 3, 20, 24, 0.2, 0.7, rot=rotation(20, 50.0)),
              key_value(5, 1, 36, 0.15, size=9, mlp=dense(40))]
    return model(210, 96, layers, eps=1e-5, loop=(0, 2, 3))


def _q():
    # Q: sizes that the matrix cores take throughout; a chunk of two pages, a window of one page, both kinds of scaled
    #    rotation over whole heads, a loop over two layers in the middle
    layers = [key_value(8, 2, 64, 0.12, size=64, rot=rotation(64, 1000.0, factor=8.0, original=256, fast=16.0, slow=2.0), softcap=20.0,
                        mlp=dense(192)),
              difference(4, 2, 64, 128, 0.125, 0.5, size=128, rot=rotation(64, 10000.0, factor=8.0, low=2.0, high=8.0, original=512),
                         mlp=dense(320)),
              key_value(4, 4, 32, 0.2, size=200, rot=rotation(16, 500.0), mlp=dense(128)),
              difference(8, 1, 16, 32, 0.25, 0.2, size=65, rot=rotation(8, 100.0), mlp=dense(256))]
    return model(384, 128, layers, eps=1e-6, loop=(1, 3, 2))


def _r():
    # R: one head each; no masks, no rotation; a layer without a feed-forward, the whole model twice
    layers = [difference(1, 1, 24, 80, 0.2, 0.45), key_value(1, 1, 80, 0.12, softcap=4.0, mlp=dense(24)),
              difference(1, 1, 40, 24, 0.15, 0.9, size=1000, mlp=dense(56))]
    return model(96, 64, layers, eps=3e-5, loop=(0, 3, 2))


def _s():
    # S: heads beyond 128 as they are kept (the plain attention kernel in either mode), many query heads a key head; a
    #    window of one key, a chunk of two; one pass over the last layer; a constant of zero
    layers = [difference(2, 1, 72, 144, 0.1, 0.3, size=70, rot=rotation(48, 1000.0, factor=2.0, low=1.0, high=3.0, original=128), mlp=dense(96)),
              key_value(2, 2, 160, 0.08, size=66, rot=rotation(160, 1000.0, factor=2.0, original=128, fast=4.0, slow=1.0), mlp=dense(64)),
              key_value(12, 1, 32, 0.2, size=1, mlp=None),
              difference(10, 1, 32, 48, 0.2, 0.0, size=2, rot=rotation(10, 70.0), mlp=dense(80))]
    return model(320, 192, layers, eps=2e-5, loop=(3, 4, 1))


def _w():
    # W: the widths of a larger model's layers at a small depth: heads of 128 and maps of 64
    layers = [key_value(8, 4, 128, 128 ** -0.5, size=192, rot=rotation(128, 10000.0, factor=4.0, original=1024, fast=32.0, slow=1.0),
                        softcap=50.0, mlp=dense(1536)),
              difference(8, 4, 64, 128, 0.125, 0.5, size=160, rot=rotation(16, 10000.0, factor=8.0, low=1.0, high=4.0, original=1024),
                         mlp=dense(1024))]
    return model(1024, 512, layers, eps=1e-6, loop=(0, 2, 2))


def _f():
    # F: for keys far back: scores a few times as sharp as a random model's usual ones, no masks but a long chunk and window
    layers = [difference(4, 2, 32, 64, 0.35, 0.3, rot=rotation(8, 10000.0), mlp=dense(128)),
              key_value(4, 2, 64, 0.4, rot=rotation(16, 10000.0), softcap=30.0, mlp=dense(128)),
              difference(4, 4, 32, 32, 0.35, 0.6, size=390, mlp=dense(128)), key_value(4, 1, 64, 0.4, size=350, mlp=dense(128))]
    return model(384, 128, layers, eps=1e-6, loop=(1, 2, 2))


# name -> (config, seed, std of the matrices)
CONFIGS = {"F": (_f(), 76, 0.09), "P": (_p(), 71, 0.12), "Q": (_q(), 72, 0.09), "R": (_r(), 73, 0.15), "S": (_s(), 74, 0.08),
           "W": (_w(), 75, 0.05)}


def write_folder(folder, raw, seed, std, dtype="float32", scale=None):
    """A random model. `scale` {tensor name suffix: factor} multiplies tensors afterwards, to make a far key or an edge show
    where random weights would hide it."""
    hb.write_random_model(folder, raw, seed=seed, dtype=dtype, std=std, norm_std=0.1)
    if scale:
        path = os.path.join(folder, "model.safetensors")
        with safe_open(path, framework="pt") as f:
            tensors = {k: f.get_tensor(k) for k in f.keys()}
        for k in tensors:
            for suffix, factor in scale.items():
                if k.endswith(suffix):
                    tensors[k] = (tensors[k].float() * factor).to(tensors[k].dtype)
        save_file(tensors, path)
    return folder


def make_folder(root, name, dtype="float32", tag="", scale=None):
    """Write the random model `name` into root/fig_<name>_<dtype><tag> once."""
    raw, seed, std = CONFIGS[name]
    folder = os.path.join(str(root), f"fig_{name}_{dtype}{tag}")
    if not os.path.exists(os.path.join(folder, "model.safetensors")):
        write_folder(folder, raw, seed, std, dtype, scale)
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
