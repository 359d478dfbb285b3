"""Position encodings. A mixer takes one as a parameter; "none" is a valid choice.

"rope": half-split rotation with a table built as the reference builds it
(crates/backends/backend_common/src/loader_common.rs:179-202):
inv_freq_i = 1 / theta^(2i / R), angle = float32(pos) * inv_freq_i in float32,
cos and sin of it for every position below max_positions.
Scaled frequencies, all in float32 as there: "linear" divides every inv_freq by the factor
(:205-228); "yarn" keeps those whose wavelength 2 pi / inv_freq is below original_max / beta_fast,
divides by the factor those above original_max / beta_slow, and blends in between with
smooth = (original_max / wavelength - beta_slow) / (beta_fast - beta_slow) (:239-287).

"rope_pairs" and "rope_halves" (not in the reference): rates in float64, a table of the step's own angles instead of one
for all positions (TurnsByAngles).
"""
import math

import torch

from ..kernels import heads
from .base import Part
from .registry import register


def distance_bucket(n, rows, bias_max):
    """The row of a table of `rows` learned biases that the distance n takes: a row a distance for the first half of
    them, then rows that grow with the distance's logarithm up to bias_max, the last row from there on."""
    half = rows // 2
    if n < half:
        return n
    return min(rows - 1, half + math.floor(math.log(n / half) / math.log(bias_max / half) * (rows - half)))


def bias_by_distance(table, bias_max):
    """table f32 [rows, heads] -> f32 [length, heads]: the biases of the distances 0 .. length - 1, the last of which
    holds for every distance beyond it."""
    rows = table.shape[0]
    if rows < 2 or not bias_max > rows // 2:
        raise ValueError(f"a table of {rows} biases needs two rows and a largest distance beyond half of them, not {bias_max}")
    length = max(rows // 2, math.ceil(bias_max)) + 1
    index = torch.tensor([distance_bucket(n, rows, bias_max) for n in range(length)], dtype=torch.long)
    return table[index.to(table.device)].contiguous()


@register("position", "none")
class NoPosition(Part):
    graph_safe = True

    def __init__(self, **_):
        pass

    def rotation(self):
        return None

    def rotation_rates(self):
        return None


@register("position", "rope")
class RotaryHalfSplit(Part):
    graph_safe = True

    def __init__(self, theta, rotary_dims, max_positions, scaling=None, tables=True):
        """tables False: no cos / sin tables are built (`rotation()` is then None); a mixer whose kernels
        take the angles from `rotation_rates()` needs none, and its positions have no bound but the cache's."""
        self.tables = bool(tables)
        if rotary_dims % 2:
            raise ValueError("rotary_dims must be even")
        self.theta = float(theta)
        self.rotary_dims = int(rotary_dims)
        self.max_positions = int(max_positions)
        # (type, factor, original_max_position_embeddings, beta_fast, beta_slow)
        self.scaling = tuple(scaling) if scaling else ("default", 1.0, None, 32.0, 1.0)
        if self.scaling[0] not in ("default", "linear", "yarn"):
            raise ValueError(f"unknown rope scaling {self.scaling[0]!r}")
        self.cos = self.sin = None

    def inv_freq(self):
        half = self.rotary_dims // 2
        theta = torch.tensor(self.theta, dtype=torch.float32)
        exponent = (2.0 * torch.arange(half, dtype=torch.float32)) / float(self.rotary_dims)
        inv_freq = 1.0 / torch.pow(theta, exponent)
        kind, factor, original, beta_fast, beta_slow = self.scaling
        f32 = lambda v: torch.tensor(v, dtype=torch.float32)
        if kind == "linear":
            inv_freq = 1.0 / (torch.pow(theta, exponent) * f32(factor))
        elif kind == "yarn":
            original = f32(float(original if original is not None else self.max_positions))
            low, high = original / f32(beta_fast), original / f32(beta_slow)
            wavelen = f32(2.0) * f32(math.pi) / inv_freq
            smooth = (original / wavelen - f32(beta_slow)) / (f32(beta_fast) - f32(beta_slow))
            scaled = inv_freq / f32(factor)
            blend = (1.0 - smooth) * scaled + smooth * inv_freq
            inv_freq = torch.where(wavelen < low, inv_freq, torch.where(wavelen > high, scaled, blend))
        return inv_freq

    def load(self, tensors, rt):
        inv_freq = self.inv_freq()
        self.rates = inv_freq.contiguous().to(rt.device)
        if not self.tables:
            return
        pos = torch.arange(self.max_positions, dtype=torch.float32)
        ang = pos[:, None] * inv_freq[None, :]
        self.cos = torch.cos(ang).contiguous().to(rt.device)
        self.sin = torch.sin(ang).contiguous().to(rt.device)

    def rotation(self):
        if not self.tables:
            return None
        return self.cos, self.sin, self.rotary_dims

    def rotation_rates(self):
        """(inv_freq float32 [rotary_dims / 2] on the GPU, rotary_dims): entry i turns by position * inv_freq[i]."""
        return self.rates, self.rotary_dims


class TurnsByAngles(Part):
    """Rotations without tables for all positions: rates [rotary_dims / 2] in float64, from which a step's angles are worked
    out once for all layers that turn alike, so no table bounds the positions. A subclass has theta, rotary_dims, halves
    (True: entry i turns with entry i + rotary_dims / 2; False: 2i with 2i + 1), amplitude (cosine and sine are
    multiplied by it) and pair_rates_host()."""
    graph_safe = True
    halves = False
    amplitude = 1.0

    def pair_rates_host(self):
        raise NotImplementedError

    def load(self, tensors, rt):
        self.rates = torch.tensor(self.pair_rates_host(), dtype=torch.float64).to(rt.device)

    def rotation(self):
        return None

    def rotation_rates(self):
        return None

    def step_angles(self, ctx):
        """(angles f32 [T, rotary_dims / 2, 2]: cosine and sine for the step's tokens, rotary_dims, halves)."""
        table = ctx.angles.get(id(self))
        if table is None:
            table = ctx.rt.buffer(f"step angles {id(self)}", (ctx.meta.num_tokens, self.rotary_dims // 2, 2), torch.float32)
            heads.step_angles(ctx.meta.positions, self.rates, self.amplitude, table)
            ctx.angles[id(self)] = table
        return table, self.rotary_dims, self.halves


@register("position", "rope_halves")
class RotaryHalves(TurnsByAngles):
    """Rotation of halves: entries i and i + rotary_dims / 2 of a head turn by position x theta^(-2i / rotary_dims).
    scaling = (factor, original, fast, slow): pair i keeps its rate up to i = lo, has it divided by factor from i = hi on, and
    goes over in a straight line between; lo and hi are the (rounded outwards) pairs that turn `fast` and `slow` times in
    `original` positions. Cosine and sine are then multiplied by 0.1 ln(factor) + 1."""
    halves = True

    def __init__(self, theta, rotary_dims, scaling=None):
        if rotary_dims % 2 or rotary_dims <= 0:
            raise ValueError("rotary_dims must be even and positive")
        self.theta, self.rotary_dims = float(theta), int(rotary_dims)
        self.scaling = None if scaling is None else tuple(float(v) for v in scaling)
        if self.scaling is not None:
            self.amplitude = 0.1 * math.log(self.scaling[0]) + 1.0
        self.rates = None

    def pair_rates_host(self):
        dims = self.rotary_dims
        rates = [self.theta ** (-2.0 * i / dims) for i in range(dims // 2)]
        if self.scaling is None:
            return rates
        factor, original, fast, slow = self.scaling
        turning = lambda times: dims * math.log(original / (2.0 * math.pi * times)) / (2.0 * math.log(self.theta))
        lo, hi = max(math.floor(turning(fast)), 0), min(math.ceil(turning(slow)), dims - 1)
        out = []
        for i, rate in enumerate(rates):
            ramp = min(max((i - lo) / max(hi - lo, 0.001), 0.0), 1.0)
            out.append(rate / factor * ramp + rate * (1.0 - ramp))
        return out


@register("position", "rope_pairs")
class RotaryPairs(TurnsByAngles):
    """Rotation of neighbouring pairs: entries 2i and 2i + 1 of a head's first `rotary_dims` turn by
    position x theta^(-2i / rotary_dims). No tables: a mixer's kernel takes the rates (float64) and computes
    a position's angle, its sine and its cosine itself, so no table bounds the positions.
    scaling = (factor, low, high, original): a rate whose wavelength 2 pi / rate lies beyond original / low is
    divided by factor, one under original / high stays, and between the two, with
    s = (original / wavelength - low) / (high - low), the rate is (1 - s) rate / factor + s rate.
    scaling = ("linear", factor): every rate is divided by factor."""
    def __init__(self, theta, rotary_dims, scaling=None):
        if rotary_dims % 2 or rotary_dims <= 0:
            raise ValueError("rotary_dims must be even and positive")
        self.theta, self.rotary_dims = float(theta), int(rotary_dims)
        self.linear = None
        if scaling is not None and scaling[0] == "linear":
            self.linear, scaling = float(scaling[1]), None
            if self.linear <= 0:
                raise ValueError("the rates' divisor must be positive")
        self.scaling = None if scaling is None else tuple(float(v) for v in scaling)
        self.rates = None

    def pair_rates_host(self):
        rates = []
        for i in range(self.rotary_dims // 2):
            rate = self.theta ** (-2.0 * i / self.rotary_dims)
            if self.linear is not None:
                rate = rate / self.linear
            if self.scaling is not None:
                factor, low, high, original = self.scaling
                wavelength = 2.0 * math.pi / rate
                if wavelength > original / low:
                    rate = rate / factor
                elif wavelength >= original / high:
                    s = (original / wavelength - low) / (high - low)
                    rate = (1.0 - s) * rate / factor + s * rate
            rates.append(rate)
        return rates

    def pair_rates(self):
        """(rates float64 [rotary_dims / 2] on the GPU, rotary_dims)."""
        return self.rates, self.rotary_dims
