"""Each mechanism of the Figalorn decoder alone on the GPU against its plain formula: a step's angles, the preparation of
heads (biases, a norm a head, both rotations, two maps side by side, values that are the keys), the difference of two
maps, both attentions from the projection's rows to the heads' outputs (prompts in tiles of both heights, portions, single
tokens inside the decode attention and beside it, in one range and in many, from K slices, dealt out over unequal
sequences, with single keys that stand out on either side of every edge), the exact gelu in a product's epilogue and
beside it, and what a pass over the layers starts from."""
import pytest
import torch

from herbert_rs_amd.cache import Cache, KVNeed
from herbert_rs_amd.errors import BackendError
from herbert_rs_amd.kernels import heads, mfma, ops
from herbert_rs_amd.kernels.heads import HeadsLayout
from herbert_rs_amd.parts import PartSpec, Runtime, StepContext, build
from herbert_rs_amd.parts.linear import Linear
from herbert_rs_amd.parts.position import RotaryHalves, RotaryPairs

from .plain import figalorn as plain
from .plain.modasun import relu_squared
from .test_vipalorn_kernels_gpu import step_meta

pytestmark = pytest.mark.gpu
DEV = "cuda"
DTYPES = [torch.float32, torch.bfloat16]
F64 = torch.float64


def rand(*shape, seed=0, scale=1.0):
    return torch.randn(*shape, generator=torch.Generator().manual_seed(seed)) * scale


def g(t):
    return None if t is None else t.to(DEV).contiguous()


# ---------------------------------------------------------------- angles
def test_a_steps_angles():
    positions = torch.tensor([0, 1, 2, 63, 1000, 99999, 1 << 20], dtype=torch.int32)
    for part, rot in ((RotaryPairs(10000.0, 48, (8.0, 1.0, 4.0, 512)), {"dims": 48, "base": 10000.0}),
                      (RotaryHalves(500.0, 20, (4.0, 256, 16.0, 2.0)), {"dims": 20, "base": 500.0})):
        rates = torch.tensor(part.pair_rates_host(), dtype=F64)
        table = torch.empty(7, part.rotary_dims // 2, 2, device=DEV)
        heads.step_angles(g(positions), g(rates), part.amplitude, table)
        ang = positions.double()[:, None] * rates[None]
        want = torch.stack([torch.cos(ang), torch.sin(ang)], -1) * part.amplitude
        assert float((table.cpu().double() - want).abs().max()) < 3e-7


# ---------------------------------------------------------------- from the projection's rows to the heads' outputs
class Case:
    """One attention: the layout of its rows, its constants, and the plain formulas from rows to outputs."""

    def __init__(self, H, G, dim, vdim, maps, same, rot, halves, norm, bias, gate, size, windowed, softcap=None, diff=0.4, seed=0,
                 factor=1.0):
        self.H, self.G, self.dim, self.vdim, self.maps, self.same = H, G, dim, vdim, maps, same
        self.rot, self.halves, self.size, self.windowed, self.softcap, self.diff = rot, halves, size, windowed, softcap, diff
        self.scale = factor * dim ** -0.5
        self.eps, self.lam, self.gate = 1e-5, 0.55, gate
        probe = self.layout(torch.float32)
        self.q_w = 1 + 0.3 * rand(dim, seed=seed + 1) if norm else None
        self.k_w = 1 + 0.3 * rand(dim, seed=seed + 2) if norm else None
        self.bias = 0.5 * rand(probe.channels, seed=seed + 3) if bias else None
        self.ld = probe.channels + (H * vdim if gate else 0)
        if rot is None:
            self.rates, self.amplitude, self.rot_dims = None, 1.0, 0
        else:
            self.rates, self.amplitude = plain.rates_by_ramp(rot) if halves else (plain.rates_by_wavelength(rot), 1.0)
            self.rot_dims = rot["dims"]

    def layout(self, dtype):
        hd = max(self.maps * self.dim, self.vdim)
        if dtype == torch.bfloat16:
            hd = next((t for t in mfma.ATTENTION_HEAD_DIMS if hd <= t), hd)
        return HeadsLayout(self.H * self.maps, self.G, self.maps, self.dim, self.vdim, hd, self.same)

    def angles(self, meta):
        if self.rates is None:
            return None
        table = torch.empty(meta.num_tokens, self.rot_dims // 2, 2, device=DEV)
        heads.step_angles(meta.positions, g(self.rates), self.amplitude, table)
        return table

    def split(self, rows, positions):
        """q [T, H maps, dim], k [T, G maps, dim], v [T, G, vdim], ready for the scores."""
        L, T = self.layout(torch.float32), rows.shape[0]
        x = rows[:, :L.channels] + (0 if self.bias is None else self.bias)
        q = x[:, :L.k_off].reshape(T, -1, self.dim)
        k = x[:, L.k_off:L.k_off + self.G * self.maps * self.dim].reshape(T, -1, self.dim)
        v = x[:, L.v_off:L.v_off + self.G * self.vdim].reshape(T, self.G, self.vdim)
        if self.q_w is not None:
            q, k = plain.over_rms(q, self.eps) * self.q_w, plain.over_rms(k, self.eps) * self.k_w
        turn = plain.rotate_halves if self.halves else plain.rotate_pairs
        return turn(q, positions, self.rot), turn(k, positions, self.rot), v

    def outputs(self, rows, size=None, last=None):
        """[T, H vdim] (the last so many rows) by the plain formulas, `size` in place of the case's own."""
        T = rows.shape[0]
        first = 0 if last is None else T - last
        positions = torch.arange(T)
        q, k, v = self.split(rows, positions)
        see = (plain.visible_window if self.windowed else plain.visible_chunk)(positions, size or self.size)[first:]
        out = torch.zeros(T - first, self.H, self.vdim)
        for a in range(self.H):
            kv = a // (self.H // self.G)
            sums = []
            for m in range(self.maps):
                s = (q[first:, a * self.maps + m] @ k[:, kv * self.maps + m].T) * self.scale
                if self.softcap:
                    s = self.softcap * torch.tanh(s / self.softcap)
                sums.append(torch.softmax(s.masked_fill(~see, float("-inf")), -1) @ v[:, kv])
            o = sums[0]
            if self.maps == 2:
                o = plain.over_rms(sums[0] - self.lam * sums[1], self.eps) * (1 - self.diff)
            out[:, a] = o
        out = out.reshape(T - first, -1)
        if self.gate:
            out = out * plain.sigmoid(rows[first:, -self.H * self.vdim:])
        return out

    def run(self, rows, meta, kv, dtype, inside, height=None, slices=1):
        """The product's way through the kernels: `inside` the attention (single tokens: everything; prompts: what follows it)
        where that can be, else beside it."""
        L, T = self.layout(dtype), rows.shape[0]
        proj, cut = g(rows), None
        if slices > 1:
            parts = rand(slices, *rows.shape, seed=99)
            parts[-1] = rows - parts[:-1].sum(0)
            held = g(parts)
            cut, proj = (slices, held.data_ptr(), rows.numel()), torch.full_like(proj, float("nan"))
        own = torch.full((T, self.H * self.vdim), 9.0, dtype=dtype, device=DEV)
        gate_off = L.channels if self.gate else None
        mixing = {"lam": self.lam, "factor": 1 - self.diff} if self.maps == 2 else {}
        masks = {"window": self.size} if self.windowed else {"chunk": self.size}
        prep = (g(self.bias), g(self.q_w), g(self.k_w), self.angles(meta), self.rot_dims, self.halves, self.eps)
        if inside and mfma.decode_heads_fusable(meta, kv, L, dtype):
            mfma.attention_decode_heads(proj, L, *prep, meta, kv, own, self.scale, softcap=self.softcap, gate_off=gate_off,
                                        slices=cut, **masks, **mixing)
            return own.float().cpu()
        q = torch.full((T, L.nq * L.hd), 9.0, dtype=dtype, device=DEV)
        heads.prepare(proj, L, *prep, meta, kv, q, cut)
        if meta.max_new > 1 and inside and mfma.heads_supported(kv, L, dtype):
            mfma.attention_heads(q, L, meta, kv, own, self.scale, softcap=self.softcap, proj=proj, gate_off=gate_off, eps=self.eps,
                                 slices=cut, tile_height=height, **masks, **mixing)
            return own.float().cpu()
        cores = dtype == torch.bfloat16 and mfma.attention_supported(q, kv, L.nq, L.nkv, L.hd)
        attn = torch.full(q.shape, 9.0, dtype=dtype if cores or self.maps == 1 else torch.float32, device=DEV)
        chunk = None if self.windowed else self.size
        window = self.size if self.windowed else None
        if cores:
            mfma.attention(q, meta, kv, attn, L.nq, L.nkv, L.hd, self.scale, window, tile_height=height if meta.max_new > 1 else None,
                           chunk=chunk, softcap=self.softcap)
        else:
            ops.attention_plain(q, meta, kv, attn, L.nq, L.nkv, L.hd, self.scale, window, chunk=chunk, softcap=self.softcap)
        if self.maps == 2:
            heads.difference(attn, proj, gate_off, own, self.H, L.hd, self.vdim, eps=self.eps, slices=cut, **mixing)
        else:
            ops.gate_heads(attn, proj if self.gate else None, L.channels, own, self.H, L.hd, self.vdim)
        return own.float().cpu()

    def cache(self, dtype, pages, slots):
        L = self.layout(dtype)
        return Cache({0: KVNeed(L.nkv, L.hd, self.size if self.windowed else None)}, 64 * pages, 1 << 20, dtype, DEV, max_slots=slots)


SCALED_PAIRS = dict(factor=4.0, low=1.0, high=4.0, original=200)
SCALED_HALVES = dict(factor=3.0, original=300, fast=16.0, slow=1.0)
CASES = {
    # H, G, dim, vdim, maps, same, rot, halves, norm, bias, gate, size, windowed
    "two maps": Case(6, 2, 32, 64, 2, False, {"dims": 8, "base": 900.0, "scaling": SCALED_PAIRS}, False, False, True, True, 100, False),
    "two maps of 64": Case(4, 2, 64, 128, 2, False, {"dims": 64, "base": 10000.0}, False, False, True, True, 64, False),
    "two normed maps": Case(2, 2, 24, 40, 2, False, {"dims": 16, "base": 100.0}, True, True, False, False, 50, True, softcap=9.0),
    "two maps, narrow values": Case(3, 3, 20, 16, 2, False, None, False, False, True, True, 7, False),
    "two maps, wide": Case(2, 1, 72, 150, 2, False, {"dims": 10, "base": 50.0}, False, False, True, True, 130, False),
    "many heads a key": Case(32, 2, 16, 32, 2, False, {"dims": 16, "base": 50.0}, False, False, True, True, None, False),
    "keys are values": Case(8, 4, 64, 64, 1, True, {"dims": 64, "base": 800.0, "scaling": SCALED_HALVES}, True, True, False, False, 65, True, 12.0),
    "keys are values, 128": Case(4, 1, 128, 128, 1, True, {"dims": 128, "base": 10000.0, "scaling": SCALED_HALVES}, True, True, False, False, 64, True, 20.0),
    "keys are values, kept larger": Case(6, 3, 48, 48, 1, True, {"dims": 20, "base": 70.0}, True, True, False, False, 7, True, 5.0),
    "keys are values, odd": Case(3, 1, 27, 27, 1, True, {"dims": 14, "base": 70.0}, True, True, True, False, 100, True, None),
    "keys are values, wide": Case(2, 2, 160, 160, 1, True, {"dims": 96, "base": 300.0}, True, True, False, True, None, True, 15.0),
    "plain heads with a gate": Case(4, 2, 32, 24, 1, False, {"dims": 12, "base": 60.0}, False, False, False, True, 33, False, 8.0),
    "one key": Case(5, 5, 32, 32, 1, True, {"dims": 32, "base": 60.0}, True, True, False, False, 1, True, 4.0),
}


def close_rows(got, want, dtype, label):
    # (bfloat16: the prompt kernels hand the two maps' sums on in bfloat16, and their difference is normed)
    tol = 5e-5 if dtype == torch.float32 else 0.025
    err = (got - want).abs().amax(1)
    assert float(err.max()) <= tol * float(want.abs().max()), f"{label}: row {int(err.argmax())}, error {float(err.max())}"


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", sorted(CASES))
def test_prepared_heads(name, dtype):
    """Queries, keys and values as they are kept, entry by entry; every entry that is no head's own is zero. Steps of few
    tokens and many, from whole sums and from K slices."""
    case = CASES[name]
    L = case.layout(dtype)
    for counts, slices in (((3, 1), 1), ((70, 33), 1), ((150, 2), 2), ((130, 70), 8)):
        if slices > 1 and (dtype == torch.float32 or not L.adds_slices or case.ld % 4):
            continue
        cache = case.cache(dtype, 12, 2)
        kv = cache.kv_view(0)
        slots = [cache.alloc_slot(), cache.alloc_slot()]
        meta = step_meta(cache, slots, list(counts))
        rows = rand(sum(counts), case.ld, seed=5)
        proj, cut = g(rows), None
        if slices > 1:
            parts = rand(slices, *rows.shape, seed=6)
            parts[-1] = rows - parts[:-1].sum(0)
            held = g(parts)
            cut, proj = (slices, held.data_ptr(), rows.numel()), torch.full_like(proj, float("nan"))
        q = torch.full((rows.shape[0], L.nq * L.hd), 9.0, dtype=dtype, device=DEV)
        heads.prepare(proj, L, g(case.bias), g(case.q_w), g(case.k_w), case.angles(meta), case.rot_dims, case.halves, case.eps, meta,
                      kv, q, cut)
        q, kp, vp = q.float().cpu().view(-1, L.nq, L.hd), kv.k.float().cpu(), kv.v.float().cpu()
        table, at = kv.page_table.cpu(), 0
        tol = 2e-5 if dtype == torch.float32 else 2 ** -7
        for slot, n in zip(slots, counts):
            wq, wk, wv = case.split(rows[at:at + n], torch.arange(n))
            want_q, want_k, want_v = torch.zeros(n, L.nq, L.hd), torch.zeros(n, L.nkv, L.hd), torch.zeros(n, L.nkv, L.hd)
            want_v[..., :case.vdim] = wv
            for m in range(case.maps):
                span = slice(m * L.map_stride, m * L.map_stride + case.dim)
                want_q[:, m::case.maps, span] = wq[:, m::case.maps]
                want_k[:, :, span] = wk[:, m::case.maps]
            assert torch.allclose(q[at:at + n], want_q, atol=tol, rtol=tol)
            for p in range(n):
                page = int(table[slot, p // 64])
                if page < 0:                                # behind a window: given back
                    continue
                assert torch.allclose(kp[page, :, p % 64], want_k[p], atol=tol, rtol=tol)
                assert torch.allclose(vp[page, :, :, p % 64], want_v[p], atol=tol, rtol=tol)
            at += n


class Fed:
    def __init__(self, rows):
        self.rows, self.at, self.got = rows, 0, []


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", sorted(CASES))
def test_attention_from_rows_to_outputs(name, dtype):
    """A sequence of 330 tokens beside a short one, in portions and single tokens, over slots that were used before: tiles of
    both heights by name, single tokens inside the decode attention and beside it."""
    case, n = CASES[name], 330
    rows, short = rand(n, case.ld, seed=11), rand(9, case.ld, seed=12)
    want, want_short = case.outputs(rows), case.outputs(short)
    cache = case.cache(dtype, 14, 3)
    kv = cache.kv_view(0)
    for inside, height in ((True, None), (False, 64), (True, 64), (False, 32), (True, 32)):
        a, b = cache.alloc_slot(), cache.alloc_slot()
        fa, fb = Fed(rows), Fed(short)
        for n_a, n_b in [(2, 2), (61, 3), (2, 1), (135, 3)] + [(1, 0)] * 20 + [(70, 0)] + [(1, 0)] * 40:
            both = [(a, fa, n_a)] + ([(b, fb, n_b)] if n_b else [])
            meta = step_meta(cache, [s for s, _, _ in both], [m for _, _, m in both])
            out = case.run(torch.cat([f.rows[f.at:f.at + m] for _, f, m in both]), meta, kv, dtype, inside, height)
            at = 0
            for _, f, m in both:
                f.got.append(out[at:at + m])
                f.at += m
                at += m
        assert fa.at == n
        close_rows(torch.cat(fa.got), want, dtype, f"{name}, inside {inside}, height {height}")
        close_rows(torch.cat(fb.got), want_short, dtype, f"{name}, short")
        cache.free_slot(a)
        cache.free_slot(b)
        cache.check()


@pytest.mark.parametrize("name", ["two maps of 64", "keys are values, 128", "two maps", "keys are values", "keys are values, kept larger",
                                  "many heads a key", "two normed maps", "plain heads with a gate"])
@pytest.mark.parametrize("ranges", [1, 2, None])
def test_single_tokens_in_one_range_and_in_many(name, ranges, monkeypatch):
    """The decode attention that writes the heads' outputs itself (one range a sequence) and the one that leaves that to the
    merge; the projection whole and in 2, 4 and 8 K slices (heads kept at 128)."""
    case, dtype = CASES[name], torch.bfloat16
    if ranges is not None:
        def cut(meta, nkv, window, chunk=0, keep_first=0):
            span = (meta.context_bucket + 63) // 64
            if window or chunk:
                span = min(span, ((window or chunk) + 63) // 64 + 1)
            per = -(-span // ranges)
            return -(-span // per), per
        monkeypatch.setattr(mfma, "_decode_split", cut)
        monkeypatch.setattr(mfma, "_decode_ranges", lambda *a, **k: None)
    lengths = [260, 1, 64, 65, 130]
    rows = [rand(n, case.ld, seed=30 + i) for i, n in enumerate(lengths)]
    want = [case.outputs(r, last=1) for r in rows]
    for slices in (1, 2, 4, 8) if case.layout(dtype).hd == 128 else (1,):
        cache = case.cache(dtype, 20, 5)
        kv = cache.kv_view(0)
        slots = [cache.alloc_slot() for _ in lengths]
        long = [i for i, n in enumerate(lengths) if n > 1]
        meta = step_meta(cache, [slots[i] for i in long], [lengths[i] - 1 for i in long])
        case.run(torch.cat([rows[i][:-1] for i in long]), meta, kv, dtype, False)
        meta = step_meta(cache, slots, [1] * 5)
        out = case.run(torch.cat([r[-1:] for r in rows]), meta, kv, dtype, True, slices=slices)
        for i in range(5):
            close_rows(out[i:i + 1], want[i], dtype, f"{name}, ranges {ranges}, slices {slices}, sequence {i}")


@pytest.mark.parametrize("maps", [1, 2])
def test_single_tokens_of_unequal_sequences(maps):
    """Sequences of 2,000 to 20 tokens in one step of single tokens: the grid dealt out by a list, the difference, gate and own
    size in the merge."""
    if maps == 2:
        case = Case(8, 4, 64, 128, 2, False, {"dims": 16, "base": 1000.0}, False, False, True, True, None, False)
    else:
        case = Case(8, 4, 48, 48, 1, True, {"dims": 48, "base": 1000.0, "scaling": SCALED_HALVES}, True, True, False, False, None, True, 10.0)
    dtype, lengths = torch.bfloat16, [2000, 130, 20, 300]
    rows = [rand(n, case.ld, seed=40 + i) for i, n in enumerate(lengths)]
    cache = case.cache(dtype, 50, 4)
    kv = cache.kv_view(0)
    slots = [cache.alloc_slot() for _ in lengths]
    case.run(torch.cat([r[:-1] for r in rows]), step_meta(cache, slots, [n - 1 for n in lengths]), kv, dtype, False)
    meta = step_meta(cache, slots, [1] * 4)
    assert mfma._decode_ranges(meta, 4, 0) is not None
    out = case.run(torch.cat([r[-1:] for r in rows]), meta, kv, dtype, True)
    for i in range(4):
        close_rows(out[i:i + 1], case.outputs(rows[i], last=1), dtype, f"sequence {i}")


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("maps,size", [(2, 7), (2, 64), (2, 100), (1, 7), (1, 64), (1, 100), (1, 129)])
def test_keys_on_either_side_of_an_edge(maps, size, dtype):
    """A key that every query answers to (an entry of its own, not rotated) with nearly all its weight: as a chunk's last and
    first key, and where a window just reaches and just does not. That it shows where it is seen, and only there, is
    checked on the plain formulas; whole prompts, portions around the edge, and single tokens."""
    n = 2 * size + 70
    if maps == 2:
        case = Case(4, 2, 32, 64, 2, False, {"dims": 8, "base": 90.0}, False, False, True, True, size, False, factor=1.5)
        marks = (size - 1, size)
    else:
        case = Case(4, 2, 64, 64, 1, True, {"dims": 16, "base": 90.0}, True, True, False, False, size, True, 30.0, factor=2.0)
        marks = (20,)
    L = case.layout(torch.float32)
    for mark in marks:
        rows = rand(n, case.ld, seed=50)
        last = case.dim - 1
        q = rows[:, :L.k_off].view(n, -1, case.dim)
        k = rows[:, L.k_off:L.k_off + case.G * maps * case.dim].view(n, -1, case.dim)
        if case.bias is not None:
            case.bias[last:L.k_off:case.dim] = 0.0
            case.bias[L.k_off + last:L.k_off + case.G * maps * case.dim:case.dim] = 0.0
        q[..., last] = 6.0
        k[..., last] = 0.0
        k[mark, ::maps, last] = 12.0 if maps == 2 else 40.0          # (the first map alone, where there are two)
        want = case.outputs(rows)
        wrong = case.outputs(rows, size=size + 1)
        moved = (wrong - want).abs().amax(1) > 0.25 * float(want.abs().max())
        assert moved[(size if mark < size else size + 1) if maps == 2 else mark + size]
        cache = case.cache(dtype, 12, 2)
        kv = cache.kv_view(0)
        edge = mark + size if maps == 1 else size
        for inside, height, cuts in ((True, None, []), (True, 64, [edge]), (False, 32, [edge - 1, edge + 1, n - 2]),
                                     (True, None, list(range(max(2, edge - 3), min(n, edge + 6)))), (False, None, list(range(edge - 2, edge + 3)))):
            slot, at, got = cache.alloc_slot(), 0, []
            for end in cuts + [n]:
                meta = step_meta(cache, [slot], [end - at])
                got.append(case.run(rows[at:end], meta, kv, dtype, inside, height))
                at = end
            close_rows(torch.cat(got), want, dtype, f"mark {mark}, cuts {cuts[:3]}")
            cache.free_slot(slot)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("T,H,hd,vdim", [(1, 3, 64, 40), (5, 8, 128, 128), (70, 2, 128, 96), (9, 2, 320, 300), (4, 5, 33, 33), (3, 4, 32, 6)])
def test_difference_of_two_maps(T, H, hd, vdim, dtype):
    for attn_dtype in {dtype, torch.float32}:
        one_difference(T, H, hd, vdim, attn_dtype, dtype)


def one_difference(T, H, hd, vdim, attn_dtype, dtype):
    attn = rand(T, 2 * H, hd, seed=1).to(attn_dtype)
    rows = rand(T, 8 + H * vdim, seed=2)
    a = attn.float()[..., :vdim]
    want = plain.over_rms(a[:, ::2] - 0.7 * a[:, 1::2], 1e-3).reshape(T, -1) * 0.35
    tol = 3e-6 if dtype == torch.float32 else 2 ** -8
    for gate in (None, 8):
        for slices in (1, 3):
            cut = None
            if slices > 1:
                parts = rand(slices, *rows.shape, seed=3)
                parts[-1] = rows - parts[:-1].sum(0)
                held = g(parts)
                cut = (slices, held.data_ptr(), rows.numel())
            out = torch.full((T, H * vdim), 9.0, dtype=dtype, device=DEV)
            heads.difference(g(attn.view(T, -1)), g(rows), gate, out, H, hd, vdim, 0.7, 0.35, 1e-3, cut)
            ref = want if gate is None else want * plain.sigmoid(rows[:, 8:])
            assert torch.allclose(out.float().cpu(), ref, atol=tol, rtol=tol)


def test_what_the_preparation_refuses():
    case = CASES["two maps"]
    L = case.layout(torch.bfloat16)
    cache = case.cache(torch.bfloat16, 4, 1)
    kv, meta = cache.kv_view(0), step_meta(cache, [cache.alloc_slot()], [3])
    rows, q = g(rand(3, case.ld)), torch.empty(3, L.nq * L.hd, dtype=torch.bfloat16, device=DEV)
    args = (None, None, None, None, 0, False, 1e-5, meta, kv, q)
    heads.prepare(rows, L, *args)
    with pytest.raises(BackendError):
        heads.prepare(rows[:, :L.channels - 4].contiguous(), L, *args)                       # rows too short
    with pytest.raises(BackendError):
        heads.prepare(rows, L, None, None, None, None, 8, False, 1e-5, meta, kv, q)          # a rotation without angles
    with pytest.raises(BackendError):
        heads.prepare(rows, L, None, torch.ones(L.dim, device=DEV), None, None, 0, False, 1e-5, meta, kv, q)
    with pytest.raises(BackendError):
        heads.prepare(rows, HeadsLayout(L.nq, L.nkv, 2, L.dim, L.vdim, 128), *args)          # not the cache's heads
    with pytest.raises(BackendError):
        mfma.attention_decode_heads(rows, L, None, None, None, None, 0, False, 1e-5, meta, kv, q, 1.0)      # three tokens a sequence


# ---------------------------------------------------------------- the exact gelu, the squared relu
TILES = (0, 112, 122, 123, 124, 142, 184, 186, 188, 2112, 4122, 2188)
FORMULAS = {"gelu": plain.gelu_erf, "relu_squared": relu_squared}


@pytest.mark.parametrize("activation", sorted(FORMULAS))
@pytest.mark.parametrize("M,N,K", [(1, 64, 32), (5, 48, 320), (16, 20000, 64), (16, 96, 512), (17, 256, 512), (64, 512, 1024), (300, 128, 96),
                                   (520, 640, 512), (129, 72, 1024), (700, 1000, 512)])
def test_a_product_with_its_activation(M, N, K, activation):
    a, w = rand(M, K, seed=1).bfloat16(), (rand(N, K, seed=2) * 2 * K ** -0.5).bfloat16()
    want = FORMULAS[activation](a.double() @ w.double().T).float()
    linear = Linear(g(w))
    for tile in TILES:
        rows = {112: 32, 124: 1 << 20, 184: 1 << 20}.get(tile % 1000, 1 << 20)
        if tile and (K % 64 and tile != 123 or M > rows or tile >= 1000 and (K // 64) // (tile // 1000) < 4):
            continue
        out = torch.full((M, N), 9.0, dtype=torch.bfloat16, device=DEV)
        mfma.gemm_activated(g(a), linear.weight, out, activation, packed=linear.packed, tile=tile)
        assert torch.allclose(out.float().cpu(), want, atol=2e-3, rtol=2 ** -7), f"tile {tile}"
    if M <= 16:                                          # rows that are half normed
        scale = 0.5 + torch.rand(M, generator=torch.Generator().manual_seed(3))
        squares = torch.zeros((K + 15) // 16, mfma.padded_rows(M))
        squares[0, :M] = K * (1 / scale ** 2 - 1e-5)
        out = torch.full((M, N), 9.0, dtype=torch.bfloat16, device=DEV)
        mfma.gemm_activated(g(a), linear.weight, out, activation, packed=linear.packed, row_scale=(g(squares), 1e-5))
        want = FORMULAS[activation]((a.double() @ w.double().T) * scale.double()[:, None]).float()
        assert torch.allclose(out.float().cpu(), want, atol=2e-3, rtol=2 ** -7)


def test_the_products_gelu_over_its_whole_range():
    """The identity as the matrix: what the epilogue makes of a number, against the exact gelu, rounding to bfloat16 apart."""
    z = torch.cat([torch.linspace(-14, 14, 4000), torch.tensor([0.0, -0.0, 1e-30, -1e-30, 300.0, -300.0])]).bfloat16()
    a = torch.zeros(z.shape[0], 64)
    a[:, 0] = z.float()
    w = torch.zeros(64, 64)
    w[:, 0] = 1.0
    out = torch.empty(z.shape[0], 64, dtype=torch.bfloat16, device=DEV)
    mfma.gemm_activated(g(a.bfloat16()), g(w.bfloat16()), out, "gelu")
    want = plain.gelu_erf(z.double())
    got = out.double().cpu()
    assert torch.equal(got, got[:, :1].expand_as(got))
    assert bool(((got[:, 0] - want).abs() <= want.abs() * 2 ** -8 + 3e-7).all())
    for dtype, tol in ((torch.float32, 2e-7), (torch.bfloat16, 2 ** -8)):
        out = torch.empty(z.shape[0], dtype=dtype, device=DEV)
        ops.activate(g(z.float()), out, "gelu")
        assert bool(((out.double().cpu() - want).abs() <= want.abs() * tol + 1e-6).all())


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("T,W,I", [(1, 64, 96), (5, 128, 64), (20, 64, 320), (70, 96, 32), (300, 256, 512), (9, 40, 24), (600, 128, 1024)])
def test_two_matrices_with_an_activation(T, W, I, dtype):
    """Few rows to many, sizes with the activation in the product's epilogue and without it."""
    for activation, formula in FORMULAS.items():
        rt = Runtime(dtype, DEV)
        part = build("feed_forward", PartSpec("up_down", {"hidden_size": W, "intermediate_size": I, "activation": activation,
                                                          "names": {"up": "u", "down": "d"}}), shared=None)
        up, down = rand(I, W, seed=1, scale=W ** -0.5).to(dtype), rand(W, I, seed=2, scale=I ** -0.5).to(dtype)
        part.load({"u": up, "d": down}, rt)
        h, x = rand(T, W, seed=4).to(dtype), rand(T, W, seed=5)
        want = plain.linear(formula(plain.linear(h.float(), up.float())), down.float())
        ctx, got = StepContext(rt=rt, meta=None, cache=None), g(x.clone())
        part.forward(ctx, g(h), got)
        tol = 2e-5 if dtype == torch.float32 else 0.02
        assert torch.allclose(got.cpu(), x + want, atol=tol * float(want.abs().max()) + 1e-6)


# ---------------------------------------------------------------- what a pass starts from
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("T,W", [(1, 64), (7, 96), (20, 128), (150, 256), (5, 72), (3, 33)])
def test_a_pass_starts_from_the_stream_and_the_embedding(T, W, dtype):
    rt = Runtime(dtype, DEV)
    part = build("pass_input", PartSpec("joined_projection", {"hidden_size": W, "weight": "w"}))
    w = rand(W, 2 * W, seed=1, scale=W ** -0.5).to(dtype)
    part.load({"w": w}, rt)
    x0, x = rand(T, W, seed=2), rand(T, W, seed=3)
    ctx, stream = StepContext(rt=rt, meta=None, cache=None), g(x0.clone())
    kept = part.begin(ctx, stream)
    assert torch.equal(stream.cpu(), x0)
    tol = 1e-5 if dtype == torch.float32 else 0.02
    want = plain.loop_input(x0, x0, w.float())
    part.forward(ctx, stream, kept)
    assert torch.allclose(stream.cpu(), want, atol=tol * float(want.abs().max()))
    stream.copy_(x)                                      # a later pass: another stream beside the same embedding
    want = plain.loop_input(x, x0, w.float())
    part.forward(ctx, stream, kept)
    assert torch.allclose(stream.cpu(), want, atol=tol * float(want.abs().max()))
