"""Rotary position tables: the frequency of every pair of columns, from a mixer's constants."""

import math

import torch


def rotary_table(dims, base, scaling=None, device=None):
    """``(inv_freq float32 [dims / 2], factor for cos and sin)``: ``f_i = base^(-2i / dims)``.

    With ``scaling = {factor, original, fast, slow}`` (the interpolation by wavelength known as
    YaRN): pairs that turn more than ``fast`` times within ``original`` positions keep ``f_i``,
    pairs that turn fewer than ``slow`` times get ``f_i / factor``, a linear ramp over the pair
    index between the two; cos and sin are multiplied by ``0.1 ln(factor) + 1``.

    With ``scaling = {factor, original, low, high}`` (the interpolation by wavelength of Llama 3.1): pairs
    with a wavelength ``2 pi / f_i`` below ``original / high`` keep ``f_i``, above ``original / low`` they get
    ``f_i / factor``, between the two ``((1 - s) / factor + s) f_i`` with ``s`` linear in the inverse
    wavelength; cos and sin as they are.  Computed in float64 on the host, once, when the weights are loaded."""
    dims, base = int(dims), float(base)
    if dims % 2 or dims < 0:
        raise ValueError(f"{dims} turning columns: an even number is needed")
    f = [base ** (-2.0 * i / dims) for i in range(dims // 2)]
    mult = 1.0
    if scaling and "high" in scaling:
        factor, original, low, high = (float(scaling[k]) for k in ("factor", "original", "low", "high"))
        for i, fi in enumerate(f):
            turns = original * fi / (2.0 * math.pi)  # within ``original`` positions
            if turns < low:
                f[i] = fi / factor
            elif turns <= high:
                s = (turns - low) / (high - low) if high > low else 1.0
                f[i] = (1.0 - s) * fi / factor + s * fi
    elif scaling:
        factor, original = float(scaling["factor"]), float(scaling["original"])

        def pair_of(turns):
            return dims * math.log(original / (2.0 * math.pi * turns)) / (2.0 * math.log(base))

        lo = max(math.floor(pair_of(float(scaling["fast"]))), 0)
        hi = min(math.ceil(pair_of(float(scaling["slow"]))), dims - 1)
        for i, fi in enumerate(f):
            ramp = min(max((i - lo) / max(hi - lo, 0.001), 0.0), 1.0)
            f[i] = fi / factor * ramp + fi * (1.0 - ramp)
        mult = 0.1 * math.log(factor) + 1.0
    return torch.tensor(f, dtype=torch.float64).float().to(device), mult
