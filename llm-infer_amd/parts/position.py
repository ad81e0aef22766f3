from __future__ import annotations

import torch

from ..kernels import ops
from ..registry import register_position
from .base import Part


@register_position("rope")
class RotaryPosition(Part):
    """Rotation of q and k by position: angle = pos * theta^(-i / rotary_dim) for the pair
    that starts at dimension i (include/kernels_cpu.hpp:82-100).  ``pairing`` "adjacent"
    rotates (i, i+1) as the reference does; "half" rotates (i/2, i/2 + rotary_dim/2), the order of
    a checkpoint whose q and k rows were never permuted for the reference (docs/gguf.md:487-493).
    ``scaling_factor`` divides every frequency (linear scaling of positions).  ``wavelength_scaling`` {"factor", "low",
    "high", "original"} stretches by wavelength instead: with l = 2 pi / f, a frequency whose l is shorter than
    original / high stays, one whose l is longer than original / low becomes f / factor, and between the two
    s = (original / l - low) / (high - low) blends them, (1 - s) f / factor + s f; the frequencies are then made in
    float64 and rounded once.  ``yarn`` {"factor", "original", "fast", "slow"} stretches by dimension: with D(t) = rotary_dim
    ln(original / (2 pi t)) / (2 ln theta), the pairs up to max(floor(D(fast)), 0) keep their frequency, those from
    min(ceil(D(slow)), rotary_dim - 1) on are divided by factor, a linear ramp between the two blends, and sine and cosine
    are multiplied by ``magnitude`` = 0.1 ln(factor) + 1 (1 without ``yarn``); only mixers whose own kernels turn their
    dimensions take a magnitude.

    The kernels rotate adjacent pairs only.  A half-paired model runs on them unchanged because a
    score is a sum over the dimensions of a head and does not care about their order: the mixer asks
    ``head_row_order`` once, when it binds its weights, and puts the rows of every q and k head into
    that order (row 2j <- row j, row 2j+1 <- row j + rotary_dim/2), after which pair j sits in
    (2j, 2j+1) with the same frequency as before.  Values and the output projection are untouched.

    A position encoding is a part like the others: it may own tensors (``params`` under its
    ``prefix``, handed over by ``bind``); this one owns none.  It keeps a table of one frequency per
    rotated pair; another encoding of this family (scaled, interpolated, with learned factors) only
    fills the table differently.  Layers whose position specs are equal share one instance.  Its
    duties towards a mixer: ``head_row_order`` (the order it wants the rows of a q or k head in, or
    None) and ``project_rotate_store`` / ``rotate_store``: rotate q and k of the step's tokens, write
    k and v into the layer's pages, and return q.
    """

    def __init__(self, *, theta: float, rotary_dim: int, head_dim: int, pairing: str = "adjacent",
                 scaling_factor: float = 1.0, wavelength_scaling: dict | None = None, yarn: dict | None = None,
                 prefix: str = "", dtype, device):
        if yarn is not None and wavelength_scaling is not None:
            raise ValueError("rotation: one way of stretching the frequencies")
        self.rotary_dim, self.head_dim, self.pairing, self.theta = rotary_dim, head_dim, pairing, float(theta)
        self.scaling_factor = float(scaling_factor)
        self.prefix = prefix
        i = torch.arange(0, rotary_dim, 2, dtype=torch.float32)
        # 1 / powf(theta, i / rotary_dim) in float32, as kernels_cpu.hpp:87
        inv = 1.0 / torch.pow(torch.tensor(float(theta), dtype=torch.float32), i / float(rotary_dim))
        if wavelength_scaling is not None:
            inv = scaled_by_wavelength(float(theta), rotary_dim, wavelength_scaling)
        self.magnitude = 1.0
        if yarn is not None:
            inv, self.magnitude = scaled_by_ramp(float(theta), rotary_dim, yarn)
        if self.scaling_factor != 1.0:
            # linear scaling: every frequency divided by the factor, i.e. positions counted in its units
            inv = inv / self.scaling_factor
        self.inv_freq = inv.to(device) if device is not None else inv
        self.dtype = dtype

    def head_row_order(self, head_dim: int):
        """The order in which a mixer must keep the rows of each q and k head (new row i holds the
        checkpoint's row ``order[i]``), or None for the checkpoint's own order."""
        if self.pairing != "half" or self.rotary_dim == 0:
            return None
        half = self.rotary_dim // 2
        order = list(range(head_dim))
        for j in range(half):
            order[2 * j], order[2 * j + 1] = j, j + half
        return order

    def _plain_turn(self):
        if self.magnitude != 1.0:
            raise ValueError("rotation with a magnitude: not built for mixers that turn q and k in their product")

    def rotate_store(self, qkv, ctx, kv_view, n_heads, n_kv_heads, head_dim):
        self._plain_turn()
        k = v = table = stride = None
        if n_kv_heads > 0:
            k, v, table, stride = kv_view.k, kv_view.v, kv_view.page_table, kv_view.page_stride
        return ops.rope_store(qkv, self.inv_freq, self.rotary_dim, False, ctx.pos, ctx.tok_slot,
                              table, stride, k, v, n_heads, n_kv_heads, head_dim, self.dtype,
                              kv_round=getattr(kv_view, "round_to", None))

    def project_rotate_store(self, h, w, ctx, kv_view, n_heads, n_kv_heads, head_dim):
        """q, k, v = h W^T, rotated and stored (the rows of W's q and k heads in ``head_row_order``); with
        16-bit storage the rotation and the cache write happen in the product's epilogue."""
        self._plain_turn()
        return _project(self, h, w, ctx, kv_view, n_heads, n_kv_heads, head_dim, self.inv_freq, self.rotary_dim,
                        True, self._table(ctx))

    def step_table(self):
        """(key, frequencies) of the table of angles that this part will ask a step for, or None.  Whoever
        builds a step and knows its positions early (the recorded decode step's bookkeeping kernel) may fill
        the table itself and leave it in the step under that key."""
        if self.rotary_dim == 0 or self.dtype == torch.float32:
            return None
        # keyed by the frequencies themselves: two encodings that fill them differently never share a table
        return ("rope_table", self.inv_freq.data_ptr(), self.rotary_dim), self.inv_freq

    def _table(self, ctx):
        """cos and sin of every token's angles, computed once per step and shared by all layers that
        rotate with the same frequencies."""
        wanted = self.step_table()
        if wanted is None:
            return None
        return ctx.shared(wanted[0], lambda: ops.rope_table(self.inv_freq, ctx.pos, ctx.n_tokens))


def scaled_by_wavelength(theta: float, rotary_dim: int, scaling: dict) -> torch.Tensor:
    """theta^(-2i / rotary_dim) for every pair i, stretched by wavelength (see ``RotaryPosition``); float64 throughout,
    rounded to float32 at the end."""
    import math
    factor, low, high, original = (float(scaling[k]) for k in ("factor", "low", "high", "original"))
    if not (factor > 0 and high > low >= 0 and original > 0):
        raise ValueError("wavelength scaling: factor and original positive, high above low")
    out = []
    for i in range(rotary_dim // 2):
        f = theta ** (-2.0 * i / rotary_dim)
        wavelength = 2.0 * math.pi / f
        if wavelength > original / low if low > 0 else False:
            f = f / factor
        elif wavelength >= original / high:
            s = (original / wavelength - low) / (high - low)
            f = (1.0 - s) * f / factor + s * f
        out.append(f)
    return torch.tensor(out, dtype=torch.float64).to(torch.float32)


def scaled_by_ramp(theta: float, rotary_dim: int, scaling: dict) -> tuple:
    """(theta^(-2i / rotary_dim) for every pair i, stretched along a ramp of the pairs, and the factor of sine and cosine;
    see ``RotaryPosition``); float64 throughout, the frequencies rounded to float32 at the end."""
    import math
    factor, original, fast, slow = (float(scaling[k]) for k in ("factor", "original", "fast", "slow"))
    if not (factor > 0 and original > 0 and fast > 0 and slow > 0 and theta > 0 and theta != 1.0):
        raise ValueError("yarn: factor, original, fast and slow positive, a base other than 1")

    def pair_that_turns(times):                  # ``times`` times over the original positions, as a fraction of a pair
        return rotary_dim * math.log(original / (2.0 * math.pi * times)) / (2.0 * math.log(theta))
    begin = max(math.floor(pair_that_turns(fast)), 0)
    end = min(math.ceil(pair_that_turns(slow)), rotary_dim - 1)
    out = []
    for i in range(rotary_dim // 2):
        f = theta ** (-2.0 * i / rotary_dim)
        ramp = min(max((i - begin) / max(end - begin, 0.001), 0.0), 1.0)
        out.append(f / factor * ramp + f * (1.0 - ramp))
    return torch.tensor(out, dtype=torch.float64).to(torch.float32), 0.1 * math.log(factor) + 1.0


def _project(part, h, w, ctx, kv_view, n_heads, n_kv_heads, head_dim, inv_freq, rotary_dim, fusable, table=None):
    if fusable and part.dtype != torch.float32 and h.dtype == part.dtype:
        k = v = ptab = stride = None
        if n_kv_heads > 0:
            k, v, ptab, stride = kv_view.k, kv_view.v, kv_view.page_table, kv_view.page_stride
        return ops.linear_rope_store(h, w, inv_freq, rotary_dim, ctx.pos, ctx.tok_slot, ptab, stride, k, v,
                                     n_heads, n_kv_heads, head_dim, part.dtype, cos_sin=table)
    qkv = ops.linear(h, w, out_dtype=torch.float32)
    return part.rotate_store(qkv, ctx, kv_view, n_heads, n_kv_heads, head_dim)


@register_position("rope_half")
class HalfRotaryPosition(RotaryPosition):
    """The same frequencies for mixers whose own kernel turns dimension i together with i + rotary_dim / 2
    (``ops.rot_store``): nothing is asked of the mixer's rows, and no table of angles of the step."""

    def __init__(self, **kw):
        kw.pop("pairing", None)
        super().__init__(pairing="half", **kw)

    def head_row_order(self, head_dim: int):
        return None

    def step_table(self):
        return None


@register_position("none")
class NoPosition(Part):
    """No position encoding: q passes unrotated, k and v are written as they are."""

    def __init__(self, *, prefix: str = "", dtype, device, **_):
        self.dtype, self.prefix = dtype, prefix

    def rotate_store(self, qkv, ctx, kv_view, n_heads, n_kv_heads, head_dim):
        k = v = table = stride = None
        if n_kv_heads > 0:
            k, v, table, stride = kv_view.k, kv_view.v, kv_view.page_table, kv_view.page_stride
        return ops.rope_store(qkv, None, 0, False, ctx.pos, ctx.tok_slot, table, stride, k, v, n_heads, n_kv_heads,
                              head_dim, self.dtype, kv_round=getattr(kv_view, "round_to", None))

    def project_rotate_store(self, h, w, ctx, kv_view, n_heads, n_kv_heads, head_dim):
        return _project(self, h, w, ctx, kv_view, n_heads, n_kv_heads, head_dim, None, 0, True)
