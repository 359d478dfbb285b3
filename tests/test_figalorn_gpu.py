"""The Figalorn decoder through the engine against the plain implementation: whole prompts, decoding through the cache,
portions down to two tokens, unequal batches, slots and pages used again, sizes of several kinds, keys just inside and
just outside a chunk and a window (in prompts and in decoding, at the pages' edges), far keys, the first tokens of a
sequence, long decoding, the passes of a loop, greedy generation through the entry point, the trace program and the
command line; float32 and bfloat16."""
import numpy as np
import pytest

import herbert_rs_amd as hb
from herbert_rs_amd.engine import StepEntry

from . import replay_util as ru
from .bounds import close
from .figalorn_tiny import (CONFIGS, dense, difference, key_value, make_folder, model, plain_folder, plain_logits, random_tokens,
                            rotation, write_folder)
from .plain import figalorn as plain

pytestmark = pytest.mark.gpu

DTYPES = ["float32", "bfloat16"]


def compare(rows, folder, tokens, positions, dtype, label, bound="fig"):
    ref = plain_logits(folder, tokens)
    off = []
    for row, p in zip(rows, positions):
        assert np.isfinite(np.asarray(row)).all(), f"{label}: position {p} is not finite"
        ok, err = close(np.asarray(row), ref[p], dtype, bound, label)
        if not ok:
            off.append((p, err))
    assert not off, f"{label}: positions and errors {off[:5]}"


def feed(engine, slot, tokens, cuts):
    """The tokens of one sequence in portions that end at `cuts`; every position's logits, in order."""
    rows, at = [], 0
    for end in list(cuts) + [len(tokens)]:
        if end <= at:
            continue
        part = tokens[at:end]
        rows.append(engine.step([StepEntry(slot, part, list(range(len(part))))]).cpu().numpy())
        at = end
    return np.concatenate(rows)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", ["P", "Q", "R", "S"])
def test_whole_prompts_and_token_by_token(name, dtype, model_root):
    folder = make_folder(model_root, name, dtype)
    vocab = CONFIGS[name][0]["vocab"]
    engine = hb.load(folder, dtype=dtype, cache_tokens=1024)
    for n, seed in ((1, 1), (2, 2), (3, 6), (67, 3), (210, 4)):
        tokens = random_tokens(vocab, n, seed)
        slot = engine.alloc_slot()
        compare(feed(engine, slot, tokens, []), folder, tokens, range(n), dtype, f"{name} whole")
        engine.free_slot(slot)
    # the first tokens of a sequence one by one, then on past pages' edges, chunks' and the window's
    tokens = random_tokens(vocab, 210, 5)
    slot = engine.alloc_slot()
    compare(feed(engine, slot, tokens, range(1, 210)), folder, tokens, range(210), dtype, f"{name} one by one")
    engine.free_slot(slot)
    engine.cache.check()


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", ["P", "Q", "S"])
def test_portions_of_several_sizes_and_slots_used_again(name, dtype, model_root):
    """Portions that end beside a page's edge, a chunk's and the window's, and one long one; every pass takes the slot and
    pages that the pass before gave back."""
    folder = make_folder(model_root, name, dtype)
    vocab = CONFIGS[name][0]["vocab"]
    engine = hb.load(folder, dtype=dtype, cache_tokens=512)
    tokens = random_tokens(vocab, 260, 21)
    for cuts in ([2, 4, 7], [64, 128, 192, 256], [63, 65, 127, 129, 192, 194], [1, 3, 36, 37, 38, 49, 51, 74, 75, 100, 102, 199], [150]):
        slot = engine.alloc_slot()
        compare(feed(engine, slot, tokens, cuts), folder, tokens, range(260), dtype, f"{name} portions")
        engine.free_slot(slot)
    engine.cache.check()


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", ["P", "Q", "R", "S"])
def test_unequal_batches_against_each_alone(name, dtype, model_root):
    folder = make_folder(model_root, name, dtype)
    vocab = CONFIGS[name][0]["vocab"]
    engine = hb.load(folder, dtype=dtype, cache_tokens=1024)
    lengths = [1, 90, 33, 180, 64, 2]
    seqs = [random_tokens(vocab, n + 12, 40 + i) for i, n in enumerate(lengths)]
    for again in range(2):               # twice: the second time the slots and pages were used before
        slots = [engine.alloc_slot() for _ in seqs]
        out = engine.step([StepEntry(s, t[:n], list(range(n))) for s, t, n in zip(slots, seqs, lengths)]).cpu().numpy()
        at = 0
        for t, n in zip(seqs, lengths):
            compare(out[at:at + n], folder, t, range(n), dtype, f"{name} batch prompts")
            at += n
        live = list(range(len(seqs)))
        for step in range(12):
            if step == 5:                # a sequence ends early; its slot goes back while the others go on
                engine.free_slot(slots[live.pop(1)])
            out = engine.step([StepEntry(slots[i], [seqs[i][lengths[i] + step]], [0]) for i in live]).cpu().numpy()
            for row, i in zip(out, live):
                compare([row], folder, seqs[i], [lengths[i] + step], dtype, f"{name} batch decode")
        for i in live:
            engine.free_slot(slots[i])
        engine.cache.check()


@pytest.mark.parametrize("dtype", DTYPES)
def test_portions_of_a_batch(dtype, model_root):
    """Several sequences go on by portions of unequal sizes in the same steps, single tokens beside long portions."""
    folder = make_folder(model_root, "Q", dtype)
    vocab = CONFIGS["Q"][0]["vocab"]
    engine = hb.load(folder, dtype=dtype, cache_tokens=1024)
    seqs = [random_tokens(vocab, n, 140 + i) for i, n in enumerate([230, 71, 9])]
    slots = [engine.alloc_slot() for _ in seqs]
    at = [0, 0, 0]
    for sizes in ([2, 64, 1], [62, 1, 2], [103, 2, 3], [63, 4, 3]):
        entries, spans = [], []
        for i, n in enumerate(sizes):
            part = seqs[i][at[i]:at[i] + n]
            entries.append(StepEntry(slots[i], part, list(range(len(part)))))
            spans.append((i, at[i], len(part)))
            at[i] += len(part)
        out = engine.step(entries).cpu().numpy()
        row = 0
        for i, first, n in spans:
            compare(out[row:row + n], folder, seqs[i], range(first, first + n), dtype, "Q portions of a batch")
            row += n


@pytest.mark.parametrize("dtype", DTYPES)
def test_long_decoding(dtype, model_root):
    """500 tokens one by one: the decode steps replayed as graphs over several shapes, pages given back behind the windows."""
    folder = make_folder(model_root, "Q", dtype)
    vocab = CONFIGS["Q"][0]["vocab"]
    engine = hb.load(folder, dtype=dtype, cache_tokens=640)
    tokens = random_tokens(vocab, 530, 77)
    slot = engine.alloc_slot()
    compare(feed(engine, slot, tokens, [30] + list(range(31, 530))), folder, tokens, range(530), dtype, "Q long decode")
    engine.cache.check()
    engine.free_slot(slot)


@pytest.mark.parametrize("dtype", DTYPES)
def test_a_far_key_shows(dtype, model_root):
    """The logits depend on tokens hundreds back, in the prompt and in decoding, across the pages' edges: checked on the
    plain implementation, then the engine against it."""
    folder = make_folder(model_root, "F", dtype, tag="_sharp", scale={".mix.q": 2.0})
    vocab = CONFIGS["F"][0]["vocab"]
    tokens = random_tokens(vocab, 380, 91)
    cfg, w = plain_folder(folder)
    a = plain_logits(folder, tokens)[300:]
    for changed in (2, 70):
        other = list(tokens)
        other[changed] = (other[changed] + 1) % vocab
        b = plain.forward(cfg, w, other, rows=list(range(300, 380))).numpy()
        rms = np.sqrt(((a - b) ** 2).mean(1)) / np.sqrt((a ** 2).mean())
        assert np.median(rms) > 0.03, f"token {changed} does not show in the plain logits: {np.median(rms)}"
    engine = hb.load(folder, dtype=dtype, cache_tokens=1024)
    for cuts in ([], [128, 256], [340] + list(range(341, 380))):
        slot = engine.alloc_slot()
        compare(feed(engine, slot, tokens, cuts), folder, tokens, range(380), dtype, "F far", "figfar")
        engine.free_slot(slot)


MARK = 63           # the token whose key stands out


def edge_folder(root, kind, size, dtype):
    """One attention layer in which the key of one token stands out: every query has a large entry that does not turn (a
    channel that every embedding holds), every key a zero there but the marked token's, whose score is then far above
    the others. A query that sees a marked key gives it nearly all its weight."""
    from safetensors.torch import load_file, save_file
    rot, D = rotation(8, 100.0), 32
    if kind == "chunk":
        layer = difference(2, 1, D, 40, 0.25, 0.3, size=size, rot=rot, mlp=dense(64))
    else:
        layer = key_value(2, 1, D, 0.5, size=size, rot=rot, softcap=25.0, mlp=dense(64))
    raw = model(64, 64, [layer], eps=1e-5)
    folder = write_folder(str(root / f"edge_{kind}_{size}_{dtype}"), raw, 7, 0.2, dtype)
    path = folder + "/model.safetensors"
    t = load_file(path)
    t["embed"][:, 0] = 2.0                    # channel 0: a constant
    t["embed"][:, 1] = 0.0                    # channel 1: the mark
    t["embed"][MARK, 1] = 4.0
    t["l0.norm1"][:2] = 0.0
    q, k = t["l0.mix.q"], t["l0.mix.k"]
    q[D - 1::D] = 0.0
    q[D - 1::D, 0] = 2.0
    k[D - 1::D] = 0.0
    k[D - 1, 1] = 3.0                         # (of two maps the first alone)
    if kind == "chunk":
        t["l0.mix.q.b"][D - 1::D] = 0.0
        t["l0.mix.k.b"][D - 1::D] = 0.0
    save_file({n: v.contiguous() for n, v in t.items()}, path)
    return folder


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("kind,size", [("chunk", 7), ("chunk", 64), ("chunk", 100), ("window", 7), ("window", 64), ("window", 100)])
def test_keys_just_inside_and_just_outside_a_chunk_and_a_window(kind, size, dtype, tmp_path):
    """A marked key as a chunk's last and as its first, and in a window's middle: every position's logits whole, with
    portions that end on, before and after the edge, and one token at a time. That the key shows where it is seen, and
    only there, is checked on the plain implementation."""
    folder = edge_folder(tmp_path, kind, size, dtype)
    n = 2 * size + 80
    cfg, w = plain_folder(folder)
    engine = hb.load(folder, dtype=dtype, cache_tokens=1024)
    base = random_tokens(63, n, 12)
    for at in (size - 1, size) if kind == "chunk" else (30,):
        tokens = list(base)
        tokens[at] = MARK
        edge = at + size if kind == "window" else size
        mixer = {**cfg["layers"][0]["mixer"], "mask": {"size": size + 1}}
        other = {**cfg, "layers": [{**cfg["layers"][0], "mixer": mixer}]}
        ref, moved = plain_logits(folder, tokens), plain.forward(other, w, tokens).numpy()
        shows = np.sqrt(((moved - ref) ** 2).mean(1)) > 0.2 * np.sqrt((ref ** 2).mean())
        assert shows[edge if at < size or kind == "window" else edge + 1]
        # (in a window of few keys one key more shows by itself)
        if kind == "chunk" or size > 20:
            assert not shows[:edge].any() and (kind == "chunk" or not shows[edge + 1:].any())
        for cuts in ([], [edge], [edge - 1, edge + 1, n - 2], [at, at + 1, edge + 2], list(range(max(2, edge - 3), n))):
            slot = engine.alloc_slot()
            compare(feed(engine, slot, tokens, cuts), folder, tokens, range(n), dtype, "edge")
            engine.free_slot(slot)
    engine.cache.check()


@pytest.mark.parametrize("dtype", DTYPES)
def test_what_a_pass_starts_from_shows(dtype, tmp_path):
    """Without either half of the projection before a pass, or without it before the first pass, the plain logits move by
    more than the bounds; the engine agrees with the right ones, from one pass to four."""
    for times, loop in ((1, (0, 1)), (2, (1, 2)), (4, (0, 2))):
        raw = model(128, 64, [difference(2, 2, 16, 24, 0.25, 0.5, size=20, mlp=dense(48)), key_value(2, 1, 16, 0.25, size=30, mlp=dense(64))],
                    eps=1e-5, loop=(*loop, times))
        folder = write_folder(str(tmp_path / f"loop{times}_{dtype}"), raw, 9, 0.12, dtype)
        tokens = random_tokens(128, 50, 3)
        ref = plain_logits(folder, tokens)
        cfg, w = plain_folder(folder)
        for half in (slice(0, 64), slice(64, 128)):
            w_in = w["loop.in"].clone()
            w_in[:, half] = 0
            assert np.abs(plain.forward(cfg, {**w, "loop.in": w_in}, tokens).numpy() - ref).max() > 0.1 * np.abs(ref).max()
        engine = hb.load(folder, dtype=dtype, cache_tokens=512)
        slot = engine.alloc_slot()
        compare(feed(engine, slot, tokens, [20, 22] + list(range(23, 50))), folder, tokens, range(50), dtype, "passes")
        engine.free_slot(slot)


@pytest.mark.parametrize("dtype", DTYPES)
def test_wider_layers(dtype, model_root):
    """Heads of 128, maps of 64, feed-forwards of 1,024 and more: the sizes of a larger model's layers."""
    folder = make_folder(model_root, "W", dtype)
    vocab = CONFIGS["W"][0]["vocab"]
    engine = hb.load(folder, dtype=dtype, cache_tokens=4096, max_slots=40)
    tokens = random_tokens(vocab, 300, 5)
    rows = [0, 1, 2, 3, 63, 64, 100, 126, 127, 128, 159, 160, 161, 191, 192, 193, 255, 256, 279]
    slot = engine.alloc_slot()
    out = engine.step([StepEntry(slot, tokens[:280], rows)]).cpu().numpy()
    compare(out, folder, tokens, rows, dtype, "W prompt")
    for p in range(280, 300):
        out = engine.step([StepEntry(slot, [tokens[p]], [0])]).cpu().numpy()
        compare(out, folder, tokens, [p], dtype, "W decode")
    engine.free_slot(slot)
    for n in (20, 40):                       # products of more rows than the few-row kernel's
        seqs = [random_tokens(vocab, 9, 600 + i) for i in range(n)]
        slots = [engine.alloc_slot() for _ in range(n)]
        engine.step([StepEntry(s, t[:8], []) for s, t in zip(slots, seqs)])
        out = engine.step([StepEntry(s, [t[8]], [0]) for s, t in zip(slots, seqs)]).cpu().numpy()
        for row, t in zip(out, seqs):
            compare([row], folder, t, [8], dtype, "W many")
        for s in slots:
            engine.free_slot(s)


def drawn_configuration(seed):
    """A configuration whose sizes, options and order of layers are drawn: widths and vocabularies that are no powers of
    two, keys of 12 to 160 and values of 16 to 144, 1 to 16 heads, windows and chunks of 1 to 200 keys or none, rotations
    of part of a head or all of it, scaled or not, feed-forwards or none, a loop over any stretch of the layers once to
    three times or none, capped scores or not."""
    import random
    r = random.Random(seed)
    width = r.choice([64, 96, 136, 160, 200, 256, 320])
    layers = []
    for _ in range(r.randint(1, 4)):
        mlp = dense(r.choice([48, 100, 192, 320])) if r.random() < 0.8 else None
        kv = r.choice([1, 2, 4])
        H, size = kv * r.choice([1, 2, 3, 4]), r.choice([None, 1, 2, 5, 32, 50, 64, 129, 200])
        if r.random() < 0.5:
            dim, vdim = r.choice([12, 24, 32, 48, 60, 64, 80]), r.choice([16, 40, 64, 80, 96, 128, 144])
            rot = None
            if r.random() < 0.8:
                rot = rotation(2 * r.randint(1, dim // 2), r.choice([100.0, 10000.0]),
                               **({} if r.random() < 0.3 else dict(factor=r.choice([2.0, 8.0]), low=1.0, high=r.choice([2.0, 4.0]), original=r.choice([64, 500]))))
            layers.append(difference(H, kv, dim, vdim, r.choice([0.5, 1.0, 2.0]) * dim ** -0.5, r.choice([0.1, 0.35, 0.8]), size, rot, mlp))
        else:
            dim = r.choice([16, 24, 32, 40, 64, 80, 96, 128, 160])
            rot = None
            if r.random() < 0.8:
                rot = rotation(2 * r.randint(1, dim // 2), r.choice([100.0, 10000.0]),
                               **({} if r.random() < 0.3 else dict(factor=r.choice([2.0, 8.0]), original=r.choice([64, 500]), fast=r.choice([8.0, 32.0]), slow=1.0)))
            layers.append(key_value(H, kv, dim, r.choice([0.5, 1.0, 1.5]) * dim ** -0.5, size, rot, r.choice([None, 5.0, 30.0]), mlp))
    loop = None
    if r.random() < 0.75:
        start = r.randrange(len(layers))
        loop = (start, r.randint(start + 1, len(layers)), r.randint(1, 3))
    return model(r.choice([100, 257, 448, 600]), width, layers, eps=r.choice([1e-6, 1e-5, 3e-5]), loop=loop)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("seed", range(16))
def test_drawn_configurations(seed, dtype, tmp_path):
    """Sixteen drawn configurations: a prompt whole, decoded on, and beside a second request in portions and single
    tokens."""
    raw = drawn_configuration(seed)
    folder = write_folder(str(tmp_path / "drawn"), raw, 100 + seed, 0.1, dtype)
    vocab = raw["vocab"]
    a, b = random_tokens(vocab, 250, 300 + seed), random_tokens(vocab, 40, 400 + seed)
    engine = hb.load(folder, dtype=dtype, cache_tokens=1024)
    slot = engine.alloc_slot()
    compare(feed(engine, slot, a, [231] + list(range(232, 250))), folder, a, range(250), dtype, "drawn")
    engine.free_slot(slot)
    sa, sb = engine.alloc_slot(), engine.alloc_slot()
    out = engine.step([StepEntry(sa, a[:170], list(range(170))), StepEntry(sb, b[:3], [0, 1, 2])]).cpu().numpy()
    compare(out[:170], folder, a, range(170), dtype, "drawn")
    compare(out[170:], folder, b, range(3), dtype, "drawn")
    for i in range(8):
        out = engine.step([StepEntry(sa, [a[170 + i]], [0]), StepEntry(sb, [b[3 + i]], [0])]).cpu().numpy()
        compare([out[0]], folder, a, [170 + i], dtype, "drawn")
        compare([out[1]], folder, b, [3 + i], dtype, "drawn")
    engine.cache.check()


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", ["P", "Q"])
def test_greedy_generation_through_the_entry_point(name, dtype, model_root):
    folder = make_folder(model_root, name, dtype)
    vocab = CONFIGS[name][0]["vocab"]
    cfg, w = plain_folder(folder)
    prompts = [random_tokens(vocab, n, 60 + n) for n in (9, 1, 70)]
    got = hb.generate(folder, prompts, temperature=0.0, max_tokens=10, ignore_eos=True, no_repeat_check=True, dtype=dtype)
    for p, g in zip(prompts, got):
        assert len(g) == 10
        if dtype == "float32":
            assert g == plain.greedy(cfg, w, p, 10)
            continue
        seq = list(p)                    # bfloat16 may flip a near-tie: the token must then be close to the best
        for tok in g:
            logits = plain.forward(cfg, w, seq, rows=[len(seq) - 1])[0]
            assert float(logits.max() - logits[tok]) <= 0.05 * float(logits.std()) + 1e-6
            seq.append(tok)


@pytest.mark.parametrize("dtype", DTYPES)
def test_the_trace_program(dtype, model_root, tmp_path):
    folder = make_folder(model_root, "P", dtype)
    vocab = CONFIGS["P"][0]["vocab"]
    reqs = {f"r{i}": random_tokens(vocab, n, 200 + i) for i, n in enumerate([5, 130, 1, 66, 40])}
    for label, steps in (("whole", ru.trace_whole(reqs)), ("tail", ru.trace_tail(reqs, 20)),
                         ("batches", ru.trace_batches(reqs, 3, 0.6))):
        held = max(sum(len(t) for t in reqs.values()), 1)
        out = ru.run_trace(folder, dtype, steps, str(tmp_path / label), held, vocab)
        got = ru.collect(steps, out)
        assert len(got) == sum(len(t) for t in reqs.values())
        by_request = {}
        for (rid, pos), row in got.items():
            by_request.setdefault(rid, []).append((pos, row))
        for rid, rows in by_request.items():
            rows.sort(key=lambda pr: pr[0])
            compare([r for _, r in rows], folder, reqs[rid], [p for p, _ in rows], dtype, f"P trace {label}")


def test_the_command_line_generates_token_ids(model_root):
    """The command line serves the family as it serves any other: token ids in, token ids out (--max-tokens 6 gives
    seven tokens: it counts the decode steps after the prompt's own token), with sampling parameters too."""
    import os
    import subprocess
    import sys
    folder = make_folder(model_root, "P", "float32")
    cfg, w = plain_folder(folder)
    cli = os.path.join(ru.ROOT, "bin", "herbert-cli")
    args = [sys.executable, cli, "--model", folder, "--prompt", "5,17,3,190", "--max-tokens", "6", "--dtype", "float32",
            "--ignore-eos", "--no-repeat-check"]
    out = subprocess.run(args + ["--temperature", "0", "--verbose"], capture_output=True, text=True, timeout=240)
    assert out.returncode == 0, out.stderr
    assert [int(t) for t in out.stdout.strip().split(",")] == plain.greedy(cfg, w, [5, 17, 3, 190], 7)
    drawn = [subprocess.run(args + ["--temperature", "0.8", "--top-k", "20", "--top-p", "0.9", "--seed", "3"], capture_output=True,
                            text=True, timeout=240) for _ in range(2)]
    assert all(d.returncode == 0 for d in drawn), drawn[0].stderr
    assert drawn[0].stdout == drawn[1].stdout and len(drawn[0].stdout.strip().split(",")) == 7
