"""Each mechanism of the Mutedra decoder alone on the GPU against its plain formula: the norm without mean and variance
with the sums that join the stream beside it, the capped logits, the relu unit, the scaled embedding, the attention with
a bias by distance, kept first keys and a one in the denominator (prompts in tiles of both heights, portions, single
tokens by the fused and the unfused kernel, ranges dealt out over unequal sequences, single keys made to stand out on
either side of every edge), and the latent attention with queries from a latent of their own, sinks and no rotated
part."""
import math

import pytest
import torch

from herbert_rs_amd.cache import Cache, KVNeed
from herbert_rs_amd.kernels import latent, mfma, ops
from herbert_rs_amd.parts import PartSpec, Runtime, StepContext, build
from herbert_rs_amd.parts.linear import Linear
from herbert_rs_amd.parts.position import bias_by_distance

from .plain import mutedra as plain
from .test_vipalorn_kernels_gpu import step_meta

pytestmark = pytest.mark.gpu
DEV = "cuda"
DTYPES = [torch.float32, torch.bfloat16]


def rand(*shape, seed=0, scale=1.0):
    return torch.randn(*shape, generator=torch.Generator().manual_seed(seed)) * scale


def g(t):
    return None if t is None else t.to(DEV).contiguous()


# ---------------------------------------------------------------- norm, sums, caps
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("T,H", [(1, 24), (7, 101), (5, 2048), (300, 64)])
def test_tanh_norm_and_the_sums_beside_it(T, H, dtype):
    x, part, extra, step = rand(T, H, seed=1), 3 * rand(T, H, seed=2), rand(T, H, seed=3), rand(H, seed=4)
    wa, ba, wb, bb = 1 + 0.2 * rand(H, seed=5), 0.3 * rand(H, seed=6), 1 + 0.2 * rand(H, seed=7), 0.3 * rand(H, seed=8)
    after, before = (0.8, g(wa), g(ba)), (1.7, g(wb), g(bb))
    tol = 3e-6 if dtype == torch.float32 else 2 ** -8
    for use in range(8):
        p, e, s = (part if use & 1 else None), (extra if use & 2 else None), (step if use & 4 else None)
        want = x.clone()
        if p is not None:
            want = want + plain.dynamic_tanh(p, 0.8, wa, ba)
        if e is not None:
            want = want + e
        if s is not None:
            want = want + s
        norm = plain.dynamic_tanh(want, 1.7, wb, bb)
        for in_place in (True, False):
            xg, y = g(x.clone()), torch.full((T, H), 9.0, dtype=dtype, device=DEV)
            out = xg if in_place else torch.full((T, H), 9.0, device=DEV)
            ops.tanh_join(xg, g(p), after if p is not None else None, g(e), g(s), out, before, y)
            assert torch.allclose(out.cpu(), want, atol=3e-6, rtol=1e-6)
            assert torch.allclose(y.float().cpu(), norm, atol=tol, rtol=tol)
            assert in_place or torch.equal(xg.cpu(), x)
        only = g(x.clone())                                       # the sum alone
        ops.tanh_join(only, g(p), after if p is not None else None, g(e), g(s), only)
        assert torch.allclose(only.cpu(), want, atol=3e-6, rtol=1e-6)
    rows = torch.tensor([T - 1, 0, T // 2], dtype=torch.int32, device=DEV)
    y = torch.empty(3, H, dtype=dtype, device=DEV)
    ops.tanh_join(g(x), before=before, y=y, rows=rows)
    assert torch.allclose(y.float().cpu(), plain.dynamic_tanh(x[[T - 1, 0, T // 2]], 1.7, wb, bb), atol=tol, rtol=tol)


@pytest.mark.parametrize("H", [64, 72, 101])
@pytest.mark.parametrize("slices", [2, 4, 8])
def test_tanh_norm_of_a_product_in_slices(slices, H):
    T = 6
    x, parts = rand(T, H, seed=1), rand(slices, T, H, seed=2)
    wa, ba, wb, bb = 1 + 0.2 * rand(H, seed=5), 0.3 * rand(H, seed=6), 1 + 0.2 * rand(H, seed=7), 0.3 * rand(H, seed=8)
    want = x + plain.dynamic_tanh(parts.sum(0), 0.8, wa, ba)
    xg, y, held = g(x.clone()), torch.empty(T, H, device=DEV), g(parts)
    ops.tanh_join(xg, torch.full((T, H), float("nan"), device=DEV), (0.8, g(wa), g(ba)), x_out=xg, before=(1.7, g(wb), g(bb)), y=y,
                  part_slices=(slices, held.data_ptr(), T * H))
    assert torch.allclose(xg.cpu(), want, atol=5e-6)
    assert torch.allclose(y.cpu(), plain.dynamic_tanh(want, 1.7, wb, bb), atol=1e-5)


@pytest.mark.parametrize("M,N,K", [(1, 64, 32), (8, 256, 128), (16, 48, 320), (5, 2048, 2048), (3, 1024, 4096), (16, 16, 64), (17, 256, 512), (64, 512, 1024),
                                   (300, 128, 64)])
def test_a_product_that_joins_the_stream(M, N, K):
    """Through Linear, as the parts do it: few rows in the product's epilogue, more by way of rows or slices of K."""
    a, w = rand(M, K, seed=1).bfloat16(), rand(N, K, seed=2, scale=K ** -0.5).bfloat16()
    x, extra, step = rand(M, N, seed=3), rand(M, N, seed=4), rand(N, seed=5)
    wa, ba, wb, bb = 1 + 0.2 * rand(N, seed=6), 0.3 * rand(N, seed=7), 1 + 0.2 * rand(N, seed=8), 0.3 * rand(N, seed=9)
    p = (a.double() @ w.double().T).float()
    linear = Linear(g(w))
    from herbert_rs_amd.parts.base import TanhJoin
    for use in range(4):
        e, s = (extra if use & 1 else None), (step if use & 2 else None)
        want = x + plain.dynamic_tanh(p, 0.9, wa, ba) + (e if e is not None else 0) + (s if s is not None else 0)
        for with_y in (True, False):
            calls = [lambda xg, y, rows: linear.forward_join(g(a), rows, TanhJoin(xg, rows, (0.9, g(wa), g(ba)), g(e), g(s),
                                                                                 (1.3, g(wb), g(bb)) if with_y else None, y))]
            if M <= 16:                                          # and by name, whatever the estimate prefers
                calls.append(lambda xg, y, rows: mfma.gemm_join(g(a), linear.weight, xg, (0.9, g(wa), g(ba)), g(e), g(s),
                                                                (1.3, g(wb), g(bb)) if with_y else None, y, packed=linear.packed))
            for call in calls:
                xg, rows = g(x.clone()), torch.empty(M, N, device=DEV)
                y = torch.full((M, N), 9.0, dtype=torch.bfloat16, device=DEV) if with_y else None
                call(xg, y, rows)
                assert torch.allclose(xg.cpu(), want, atol=2e-5), f"use {use}"
                if with_y:
                    assert torch.allclose(y.float().cpu(), plain.dynamic_tanh(want, 1.3, wb, bb), atol=2 ** -7, rtol=2 ** -8)


def test_tanh_norm_far_outside_its_bend():
    x = torch.tensor([[-1e30, -50.0, 0.0, 50.0, 1e30, 1e-20, -0.0, 3.0]])
    y = torch.empty(1, 8, device=DEV)
    ops.tanh_join(g(x), before=(2.0, torch.ones(8, device=DEV), torch.zeros(8, device=DEV)), y=y)
    assert torch.allclose(y.cpu(), torch.tanh(2.0 * x), atol=1e-7)


def test_what_the_sums_refuse():
    from herbert_rs_amd.errors import BackendError
    x = torch.zeros(2, 8, device=DEV)
    w = torch.ones(8, device=DEV)
    with pytest.raises(BackendError):
        ops.tanh_join(x, part=x.clone(), x_out=x)                  # a part without its norm
    with pytest.raises(BackendError):
        ops.tanh_join(x, before=(1.0, w, w), y=x)                  # the normed rows over the stream
    with pytest.raises(BackendError):
        ops.tanh_join(x)
    with pytest.raises(BackendError):
        ops.softcap(x, 0.0)


def test_capped_logits_and_the_scaled_embedding():
    z = rand(5, 333, seed=1, scale=40.0)
    got = g(z.clone())
    ops.softcap(got, 17.0)
    assert torch.allclose(got.cpu(), plain.capped(z, 17.0), atol=2e-5)
    for H in (20, 64):
        for dtype in DTYPES:
            table = rand(50, H, seed=2).to(dtype)
            ids = torch.tensor([49, 0, 7, 7], dtype=torch.int32, device=DEV)
            out = torch.empty(4, H, device=DEV)
            ops.embed(ids, g(table), out, scale=2.75)
            assert torch.equal(out.cpu(), table.float()[[49, 0, 7, 7]] * 2.75)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("T,W,I", [(1, 64, 96), (5, 128, 64), (20, 64, 320), (70, 96, 32), (300, 256, 512), (9, 40, 24), (600, 128, 1024)])
def test_relu_unit(T, W, I, dtype):
    """Few rows to many, sizes with the activation in the product's epilogue and without it."""
    rt = Runtime(dtype, DEV)
    part = build("feed_forward", PartSpec("swiglu", {"hidden_size": W, "intermediate_size": I, "activation": "relu",
                                                     "names": {"gate": "g", "up": "u", "down": "d"}}), shared=None)
    tensors = {"g": rand(I, W, seed=1, scale=W ** -0.5).to(dtype), "u": rand(I, W, seed=2, scale=W ** -0.5).to(dtype),
               "d": rand(W, I, seed=3, scale=I ** -0.5).to(dtype)}
    part.load(tensors, rt)
    h, x = rand(T, W, seed=4).to(dtype), rand(T, W, seed=5)
    want = plain.relu_unit(h.float(), *(tensors[k].float() for k in "gud"))
    ctx = StepContext(rt=rt, meta=None, cache=None)
    got = g(x.clone())
    part.forward(ctx, g(h), got)
    tol = 2e-5 if dtype == torch.float32 else 0.02
    assert torch.allclose(got.cpu(), x + want, atol=tol * float(want.abs().max()) + 1e-6)
    fresh = torch.full((T, W), 7.0, device=DEV)
    ctx.fresh_rows = fresh                                         # rows that hold nothing yet are stored to
    part.forward(ctx, g(h), fresh)
    assert torch.allclose(fresh.cpu(), want, atol=tol * float(want.abs().max()) + 1e-6)


# ---------------------------------------------------------------- attention
def head_size(dtype, dim):
    return dim if dtype == torch.float32 else next((t for t in mfma.ATTENTION_HEAD_DIMS if dim <= t), dim)


def attend(q, k, v, table, bias_max, size, keep, scale):
    """The heads' outputs [T, H, D] by the plain formulas."""
    T, H, D = q.shape
    positions = torch.arange(T)
    see = plain.visible(positions, size, keep)
    bias = plain.distance_bias(table, positions, bias_max)
    out = torch.zeros(T, H, v.shape[2])
    for a in range(H):
        kv = a // (H // k.shape[1])
        out[:, a] = plain.softmax_with_sink((q[:, a] @ k[:, kv].T) * scale + bias[:, :, a], see, 0.0) @ v[:, kv]
    return out


class Sequence:
    """Keys and values of one slot, fed in portions, and the outputs so far."""

    def __init__(self, n, nq, nkv, dim, hd, dtype, seed, marks=()):
        r = lambda *s, i: rand(*s, seed=10 * seed + i).to(dtype).float()
        self.q, self.k, self.v = r(n, nq, dim, i=1), r(n, nkv, dim, i=2), r(n, nkv, dim, i=3)
        self.q[:, :, 0] = 4.0                                      # what a marked key answers to
        self.k[:, :, 0] = 0.0
        for p in marks:
            if 0 <= p < n:
                self.k[p, :, 0] = 24.0
        self.n, self.at, self.got = n, 0, []
        pad = lambda t: torch.nn.functional.pad(t, (0, hd - dim)).reshape(n, -1)
        self.rows = torch.cat([pad(self.q), pad(self.k), pad(self.v)], 1)


ATTENTION_CASES = [
    # nq, nkv, dim, bias rows, bias_max, window, kept
    (4, 2, 64, 32, 200, 100, 5),
    (8, 2, 128, 16, 90, 64, 70),
    (3, 3, 32, 8, 40, 7, 2),
    (6, 2, 96, 32, 250, None, 0),
    (2, 1, 160, 12, 60, 50, 3),
    (40, 2, 32, 2, 9, 129, 1),
    (4, 4, 48, 64, 2000, 64, 64),
    (5, 1, 128, 32, 150, 1, 0),
]


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("nq,nkv,dim,rows,bias_max,size,keep", ATTENTION_CASES)
def test_attention_with_distances_and_kept_keys(nq, nkv, dim, rows, bias_max, size, keep, dtype):
    """A sequence of 330 tokens beside a short one, in portions and single tokens, three passes over slots that were used
    before: tiles of 64 and of 32 tokens by name, single tokens by the kernel that writes its own key and by the
    one that finds it written. Keys at the last kept position, at the first that is not kept, at the window's edge and
    far back are marked: they hold the weight wherever they are seen. That they do is checked on the plain formulas."""
    n, n_short, hd, scale = 330, 9, head_size(dtype, dim), 0.9 * dim ** -0.5
    table = 1.5 * rand(rows, nq, seed=9)
    edge = size if size else 70
    # (one marked key a sequence: two of them at once would hide each other)
    for mark in sorted({keep - 1, keep, keep + 40, edge}):
        if mark < 0:
            continue
        seq, short = Sequence(n, nq, nkv, dim, hd, dtype, 1, (mark,)), Sequence(n_short, nq, nkv, dim, hd, dtype, 2, (1,))
        want, want_short = (attend(s.q, s.k, s.v, table, bias_max, size, keep, scale) for s in (seq, short))
        if size and mark + size < n and mark <= keep + 40:
            wrong = {keep - 1: (size, keep - 1), keep: (size, keep + 1)}.get(mark, (size + 1, keep))
            other = attend(seq.q, seq.k, seq.v, table, bias_max, *wrong, scale)
            if mark in (keep - 1, keep, keep + 40):
                assert float((other - want)[mark + size].abs().max()) > 0.5 * float(want.abs().max())
        by_distance = bias_by_distance(table, bias_max).to(DEV)
        bias, raw = ops.DistanceBias(by_distance), ops.DistanceBias(by_distance / scale)
        zeros = torch.zeros(nq, device=DEV)
        cache = Cache({0: KVNeed(nkv, hd, size, keep_first=keep if size else 0)}, 64 * 12, 4096, dtype, DEV, max_slots=3)
        kv = cache.kv_view(0)
        for height, fused in ((None, True), (64, False), (32, True)):
            a, b = cache.alloc_slot(), cache.alloc_slot()
            seq.at = short.at = 0
            seq.got, short.got = [], []
            for n_a, n_b in [(2, 2), (61, 3), (2, 1), (135, 3)] + [(1, 0)] * 20 + [(70, 0)] + [(1, 0)] * 40:
                slots, parts = ([a, b], [(seq, n_a), (short, n_b)]) if n_b else ([a], [(seq, n_a)])
                meta = step_meta(cache, slots, [m for _, m in parts])
                proj = g(torch.cat([s.rows[s.at:s.at + m] for s, m in parts]))
                T = proj.shape[0]
                out = torch.full((T, nq * hd), 9.0, dtype=dtype, device=DEV)
                q = torch.empty(T, nq * hd, dtype=dtype, device=DEV)
                cores = dtype == torch.bfloat16 and mfma.attention_supported(q, kv, nq, nkv, hd)
                if cores and fused and meta.max_new == 1:
                    mfma.attention_decode_fused(proj, None, None, None, None, meta, kv, out, nq, nkv, hd, 0.0, scale, size,
                                                sinks=zeros, bias=raw, keep_first=keep if size else 0)
                else:
                    ops.qk_norm_rope_write(proj, None, None, None, None, 0, meta, kv, q, nq, nkv, hd, 0.0)
                    if cores:
                        mfma.attention(q, meta, kv, out, nq, nkv, hd, scale, size, tile_height=height if meta.max_new > 1 else None,
                                       sinks=zeros, bias=raw, keep_first=keep if size else 0)
                    else:
                        ops.attention_plain(q, meta, kv, out, nq, nkv, hd, scale, size, sinks=zeros, bias=bias,
                                            keep_first=keep if size else 0)
                rows_out, row = out.float().cpu().view(T, nq, hd)[..., :dim], 0
                for s, m in parts:
                    s.got.append(rows_out[row:row + m])
                    s.at += m
                    row += m
            tol = 3e-5 if dtype == torch.float32 else 0.02
            for s, ref in ((seq, want), (short, want_short)):
                err = (torch.cat(s.got) - ref).abs().amax((1, 2))
                assert float(err.max()) <= tol * float(ref.abs().max()), \
                    f"mark {mark}, height {height}: position {int(err.argmax())}, error {float(err.max())}"
            cache.free_slot(a)
            cache.free_slot(b)
            cache.check()


@pytest.mark.parametrize("nq,nkv,hd,size", [(8, 4, 128, None), (4, 2, 64, None), (8, 2, 128, 600)])
def test_single_tokens_of_unequal_sequences(nq, nkv, hd, size):
    """Sequences of 2,000 to 20 tokens in one step of single tokens: the grid dealt out by a list (without a window), or
    cut into equal ranges, with the sum's one and the biases in the merge."""
    dtype, scale, keep = torch.bfloat16, hd ** -0.5, 66 if size else 0
    table, bias_max = rand(32, nq, seed=3), 900
    lengths = [2000, 130, 20, 300]
    cache = Cache({0: KVNeed(nkv, hd, size, keep_first=keep)}, 64 * 50, 4096, dtype, DEV, max_slots=4)
    kv = cache.kv_view(0)
    seqs = [Sequence(n, nq, nkv, hd, hd, dtype, 20 + i, (n // 2, 3)) for i, n in enumerate(lengths)]
    slots = [cache.alloc_slot() for _ in seqs]
    raw = ops.DistanceBias(bias_by_distance(table, bias_max).to(DEV) / scale)
    zeros = torch.zeros(nq, device=DEV)
    meta = step_meta(cache, slots, [n - 1 for n in lengths])
    proj = g(torch.cat([s.rows[:-1] for s in seqs]))
    q = torch.empty(proj.shape[0], nq * hd, dtype=dtype, device=DEV)
    ops.qk_norm_rope_write(proj, None, None, None, None, 0, meta, kv, q, nq, nkv, hd, 0.0)
    meta = step_meta(cache, slots, [1] * 4)
    assert size or mfma._decode_ranges(meta, nkv, 0) is not None
    out = torch.empty(4, nq * hd, dtype=dtype, device=DEV)
    mfma.attention_decode_fused(g(torch.cat([s.rows[-1:] for s in seqs])), None, None, None, None, meta, kv, out, nq, nkv, hd, 0.0,
                                scale, size, sinks=zeros, bias=raw, keep_first=keep)
    for s, row in zip(seqs, out.float().cpu().view(4, nq, hd)):
        n = s.n
        see = plain.visible(torch.arange(n), size, keep)[n - 1:]
        index = torch.tensor([plain.bucket(n - 1 - j, 32, bias_max) for j in range(n)])
        for a in range(nq):
            kvh = a // (nq // nkv)
            scores = (s.k[:, kvh] @ s.q[-1, a]) * scale + table[index, a]
            want = (plain.softmax_with_sink(scores[None], see, 0.0) @ s.v[:, kvh])[0]
            assert float((row[a] - want).abs().max()) <= 0.02 * float(want.abs().max()) + 2e-3


def test_what_the_attention_refuses():
    from herbert_rs_amd.errors import BackendError
    shared = type("Shared", (), {"position": staticmethod(lambda spec: build("position", spec))})
    base = {"hidden_size": 32, "num_heads": 2, "num_kv_heads": 1, "head_dim": 16, "eps": 1e-5, "position": PartSpec("none"),
            "qk_norm": False, "names": {k: k for k in ("q", "k", "v", "o", "rel")}}
    for bad in ({"keep_first": 3}, {"keep_first": -1, "window": 4}, {"distance_bias": (20,), "softcap": 3.0},
                {"keep_first": 2, "window": 5, "chunk": 4}, {"sink": "two"}):
        with pytest.raises(ValueError):
            build("mixer", PartSpec("attention", {**base, **bad}), shared=shared)
    cache = Cache({0: KVNeed(1, 32)}, 128, 256, torch.bfloat16, DEV, max_slots=1)
    meta = step_meta(cache, [cache.alloc_slot()], [5])
    q = torch.zeros(5, 64, dtype=torch.bfloat16, device=DEV)
    bias = ops.DistanceBias(torch.zeros(9, 2, device=DEV))
    with pytest.raises(BackendError):
        mfma.attention(q, meta, cache.kv_view(0), torch.empty_like(q), 2, 1, 32, 1.0, 0, bias=bias, softcap=2.0)
    with pytest.raises(BackendError):
        mfma.attention(q, meta, cache.kv_view(0), torch.empty_like(q), 2, 1, 32, 1.0, 0, keep_first=4)
    with pytest.raises(BackendError):
        mfma.attention(q, meta, cache.kv_view(0), torch.empty_like(q), 2, 1, 32, 1.0, 0, bias=ops.DistanceBias(torch.zeros(9, 3, device=DEV)))


# ---------------------------------------------------------------- latent attention
LATENT_CASES = [
    # heads, dim, rot_dim, vdim, kv_rank, q_rank
    (4, 32, 32, 64, 96, 64),
    (3, 20, 12, 24, 40, 56),
    (8, 64, 0, 32, 128, 96),
    (1, 16, 0, 80, 24, 8),
    (20, 32, 64, 32, 256, 160),
    (5, 40, 0, 24, 72, 40),
]


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("H,D,R,Dv,rank,q_rank", LATENT_CASES)
def test_latent_attention_part(H, D, R, Dv, rank, q_rank, dtype):
    """The part by itself over two slots used twice: a prompt whole, in portions, and single tokens whose keys are cut into
    ranges; sinks that take most of a row's weight, some of it, and none."""
    W, n, n_short, eps = 96, 300, 11, 1e-5
    m = {"heads": H, "dim": D, "vdim": Dv, "kv_rank": rank, "q_rank": q_rank, "scale": 2.0 * (D + R) ** -0.5}
    names = {"dq": "dq", "dq_norm": "dq.norm", "uq": "uq", "dkv": "dkv", "dkv_norm": "dkv.norm", "uk": "uk", "uv": "uv", "o": "o"}
    sizes = {"dq": (q_rank, W), "uq": (H * (D + R), q_rank), "dkv": (rank + R, W), "uk": (H * D, rank), "uv": (H * Dv, rank), "o": (W, H * Dv)}
    if R:
        m.update(rot_dim=R, rot={"dims": R, "base": 500.0})
        names.update(sink="sink", g="g")
        sizes["g"] = (H, W)
    w = {k: rand(*s, seed=30 + i, scale=s[1] ** -0.5).to(dtype) for i, (k, s) in enumerate(sizes.items())}
    w["dq.norm"], w["dkv.norm"] = (1 + 0.2 * rand(q_rank, seed=1)).to(dtype), (1 + 0.2 * rand(rank, seed=2)).to(dtype)
    if R:
        w["sink"] = torch.linspace(-40.0, 6.0, H).to(dtype) if H > 1 else torch.tensor([1.5]).to(dtype)
    shared = type("Shared", (), {"position": staticmethod(lambda spec: build("position", spec))})
    position = PartSpec("rope", {"theta": 500.0, "rotary_dims": R, "max_positions": 4096, "tables": False}) if R else PartSpec("none")
    part = build("mixer", PartSpec("latent_attention", {
        "hidden_size": W, "heads": H, "dim": D, "rot_dim": R, "vdim": Dv, "kv_rank": rank, "q_rank": q_rank, "scale": m["scale"],
        "eps": eps, "position": position, "names": names, "gate": "head", "pairs": True, "sink": bool(R)}), shared=shared)
    assert set(part.tensor_needs()) == set(w)
    rt = Runtime(dtype, DEV)
    part.position.load({}, rt)
    part.load(w, rt)
    h, hs = rand(n, W, seed=3).to(dtype), rand(n_short, W, seed=4).to(dtype)
    wf = {k: v.float() for k, v in w.items()}
    want, want_short = (plain.latent_mixer(v.float(), wf, m, eps, torch.arange(v.shape[0])) for v in (h, hs))
    cache = Cache({0: part.cache_need()}, 64 * 12, 4096, dtype, DEV, max_slots=3)
    for steps in ([(n, n_short)], [(2, 2), (61, 3), (2, 1), (135, 5)] + [(1, 0)] * 100):
        a, b = cache.alloc_slot(), cache.alloc_slot()
        at, got = [0, 0], [[], []]
        for counts in steps:
            live = [i for i in (0, 1) if counts[i]]
            meta = step_meta(cache, [(a, b)[i] for i in live], [counts[i] for i in live])
            y = g(torch.cat([(h, hs)[i][at[i]:at[i] + counts[i]] for i in live]))
            x = torch.full((y.shape[0], W), 5.0, device=DEV)
            ctx = StepContext(rt=rt, meta=meta, cache=cache)
            ctx.fresh_rows = x
            part.forward(ctx, y, x)
            row = 0
            for i in live:
                got[i].append(x[row:row + counts[i]].cpu())
                at[i] += counts[i]
                row += counts[i]
        tol = 3e-5 if dtype == torch.float32 else 0.03
        for rows, ref in ((got[0], want), (got[1], want_short)):
            err = (torch.cat(rows) - ref).abs().amax(1)
            assert float(err.max()) <= tol * float(ref.abs().max()), f"position {int(err.argmax())}: {float(err.max())}"
        cache.free_slot(a)
        cache.free_slot(b)
    cache.check()


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("rank,rot", [(128, 0), (40, 8)])
def test_a_sink_far_above_and_far_below_the_scores(rank, rot, dtype):
    """Sinks of -1000, 0 and 1000: nothing, a share of one, everything."""
    H, n = 3, 90
    cache = Cache({0: KVNeed(1, rank + rot, None, values=False)}, 64 * 4, 256, dtype, DEV, max_slots=1)
    slot = cache.alloc_slot()
    kv = cache.kv_view(0)
    rows = rand(n, rank + rot, seed=1, scale=0.3).to(dtype)
    page = cache.kv_view(0).page_table
    sinks = torch.tensor([-1000.0, 0.0, 1000.0], device=DEV)
    for counts in ([n], [n - 1, 1]):
        for c in counts:
            meta = step_meta(cache, [slot], [c])
            for p in range(n):
                kv.k[int(page[slot, p // 64]), 0, p % 64] = g(rows[p]) if p < cache.length(slot) else 0
            q = rand(c, H * (rank + rot), seed=2)
            out = torch.empty(c, H * rank, dtype=dtype, device=DEV)
            if latent.mfma_takes(kv, rank, rot):
                latent.latent_attention_mfma(g(q), meta, kv, out, None, 0, H, rank, rot, 0.2, Runtime(dtype, DEV).buffer, sinks=sinks)
            else:
                latent.latent_attention_plain(g(q), meta, kv, out, None, 0, H, rank, rot, 0.2, sinks=sinks)
            got = out.float().cpu().view(c, H, rank)
            first = cache.length(slot) - c
            for t in range(c):
                keys = rows[:first + t + 1].float()
                for a in range(H):
                    s = keys @ q[t].view(H, -1)[a] * 0.2
                    want = plain.softmax_with_sink(s[None], torch.ones(1, len(s)).bool(), float(sinks[a]))[0] @ keys[:, :rank]
                    assert torch.allclose(got[t, a], want, atol=2e-5 if dtype == torch.float32 else 6e-3)
        cache.truncate(slot, 0)
