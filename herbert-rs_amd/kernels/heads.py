"""Host side of the kernels between an attention's projection and its scores, and between its weighted sums and its
output projection, for heads that are not kept as they are projected (csrc/heads.hip; the same for one token a
sequence inside the decode attention, mfma.attention_decode_heads). Not in xigh/herbert-rs.
"""
from dataclasses import dataclass

import torch

from ..errors import BackendError
from . import lib
from .ops import _check, _check_paged, _ptr, _stream, dtype_code

MAX_WIDTH = 1024          # columns of one head (all maps) that the preparing kernel holds


@dataclass(frozen=True)
class HeadsLayout:
    """Where a projection's row [nq x dim queries | nkv x maps x dim keys | nkv x vdim values | ...] has its heads and how
    they are kept. nq counts maps: a head of the model with two maps is two neighbouring query heads here. maps: keys
    of so many maps lie side by side in a kept head of hd entries, map m's at m x map_stride. Values that are the keys as
    projected (keys_are_values): v_off is k_off."""
    nq: int
    nkv: int
    maps: int
    dim: int
    vdim: int
    hd: int
    keys_are_values: bool = False

    @property
    def map_stride(self):
        return self.hd // 2 if self.maps == 2 and self.hd % 2 == 0 else self.dim

    @property
    def adds_slices(self):
        """True if `prepare` adds up the K slices of such a projection (of a row width that four divides) itself."""
        return self.dim % 4 == 0 and self.vdim % 4 == 0

    @property
    def k_off(self):
        return self.nq * self.dim

    @property
    def v_off(self):
        return self.k_off if self.keys_are_values else self.k_off + self.nkv * self.maps * self.dim

    @property
    def channels(self):
        return self.v_off + self.nkv * (self.maps * self.dim if self.keys_are_values else self.vdim)


def step_angles(positions, rates, amplitude, table):
    """table f32 [T, half, 2] = amplitude x (cosine, sine) of positions int32 [T] x rates f64 [half]."""
    T, half = positions.shape[0], rates.shape[0]
    _check(positions, "positions", torch.int32, (T,))
    _check(rates, "rates", torch.float64, (half,))
    _check(table, "angles", torch.float32, (T, half, 2))
    lib.call("heads", "hb_step_angles", positions.data_ptr(), rates.data_ptr(), half, float(amplitude), table.data_ptr(), T,
             _stream())


def check_operands(layout, proj, angles, rot_dims, bias, q_norm_w, k_norm_w):
    T, ld = proj.shape
    _check(proj, "proj", torch.float32, (T, ld))
    if ld < layout.channels:
        raise BackendError(f"heads: rows of {ld} do not hold {layout.channels} columns")
    if angles is not None:
        _check(angles, "angles", torch.float32, (T, rot_dims // 2, 2))
    elif rot_dims:
        raise BackendError("heads: a rotation needs the step's angles")
    if bias is not None:
        _check(bias, "bias", torch.float32, (layout.channels,))
    if (q_norm_w is None) != (k_norm_w is None):
        raise BackendError("heads: queries and keys are normed together")
    for w, name in ((q_norm_w, "q_norm"), (k_norm_w, "k_norm")):
        if w is not None:
            _check(w, name, torch.float32, (layout.dim,))


def slice_args(slices, proj):
    """(number, pointer, floats between two) of a projection whose K slices are still apart (None: it is whole)."""
    return slices if slices is not None else (1, proj.data_ptr(), 0)


def prepare(proj, layout, bias, q_norm_w, k_norm_w, angles, rot_dims, halves, eps, meta, cache, q_out, slices=None):
    """Biases [channels], a norm a head or map (weights [dim]), the rotation of rot_dims entries by the step's angles (pairs
    of neighbours, or of halves), q to q_out [T, nq x hd], keys and values to the tokens' pages. slices: as
    mfma.gemm(..., defer_slices=True) gives them (proj itself is then not read)."""
    T, ld = proj.shape
    L = layout
    check_operands(L, proj, angles, rot_dims, bias, q_norm_w, k_norm_w)
    _check_paged(meta, cache, T)
    _check(q_out, "q_out", cache.k.dtype, (T, L.nq * L.hd))
    if tuple(cache.k.shape[1:]) != (L.nkv, cache.page_size, L.hd):
        raise BackendError(f"cache pages {list(cache.k.shape)} do not fit {L.nkv} kv heads of {L.hd}")
    n, src, stride = slice_args(slices, proj)
    lib.call("heads", "hb_heads_prepare", src, ld, n, stride, _ptr(bias), _ptr(q_norm_w), _ptr(k_norm_w), _ptr(angles),
             meta.positions.data_ptr(), meta.seq_of.data_ptr(), meta.slots.data_ptr(), cache.page_table.data_ptr(),
             cache.page_table.shape[1], cache.page_size, q_out.data_ptr(), cache.k.data_ptr(), cache.v.data_ptr(),
             dtype_code(q_out), T, L.nq, L.nkv, L.maps, L.dim, L.vdim, L.hd, L.map_stride, L.k_off, L.v_off, int(rot_dims),
             1 if halves else 0, float(eps), _stream())


def difference(attn, proj, gate_off, out, heads, hd, vdim, lam, factor, eps, slices=None):
    """out[t, h vdim + d] = o factor / sqrt(mean(o^2) + eps) x sigmoid(gate), o = a1 - lam a2 with a1, a2 the kept heads 2h and
    2h + 1 of attn [T, 2 heads x hd] and the gate in proj's columns from gate_off on (None: no gate). attn may be
    float32 beside outputs of another type: the maps' sums are then not rounded before they are taken from each other."""
    T = attn.shape[0]
    _check(attn, "attn", torch.float32 if attn.dtype == torch.float32 else out.dtype, (T, 2 * heads * hd))
    _check(out, "out", None, (T, heads * vdim))
    gate, ld, n, stride = None, 0, 1, 0
    if gate_off is not None:
        _check(proj, "gate", torch.float32, (T, None))
        ld = proj.shape[1]
        if gate_off < 0 or gate_off + heads * vdim > ld:
            raise BackendError("difference: the gate's columns lie outside the rows")
        n, src, stride = slice_args(slices, proj)
        gate = src + 4 * gate_off
    lib.call("heads", "hb_heads_difference", attn.data_ptr(), dtype_code(attn), dtype_code(out), gate, ld, n, stride, out.data_ptr(), T, heads, hd,
             vdim, float(lam), float(factor), float(eps), _stream())
