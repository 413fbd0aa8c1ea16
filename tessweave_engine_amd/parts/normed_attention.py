"""Grouped-query attention without a rotation, whose heads' queries and keys are normed: a branch of a `ParallelMixer`.

    q = W_q h, k = W_k h, v = W_v h (no biases);  q_h <- t(p) * q_h / rms(q_h),  k_g <- k_g / rms(k_g)      (no weights)
    t(p) = 1 + coef * ln(floor((p + 1) / every) + 1)                     positions enter as the queries' temperature
    score = cap * tanh(scale * q . k / cap), softmax over the keys up to the query, W_o on the heads' sums

Query head a reads key head a // (heads / kv_heads); values have a size of their own. The packed product leaves float32
rows; norms and temperature are float32, one kernel forms them, rounds queries, keys and values once and writes the pages.
The attention itself is the engine's (`paged_attention`): keys and values are laid out with the larger of their sizes,
rounded up to 16, tails of zeros.
"""
from __future__ import annotations

from ..cache.spec import CacheNeed, PagedKV
from ..kernels import ops
from .attention import paged_attention
from .parallel import MixerBranch


def _round_up(v, m):
    return (int(v) + m - 1) // m * m


class NormedAttention(MixerBranch):
    def __init__(self, prefix, q_heads, kv_heads, dim, value_dim, scale, eps, softcap=None, temperature=None,
                 names=("q", "k", "v", "o")):
        """eps: of the heads' norms; softcap: the scores' cap, or None; temperature: (coef, every), or None."""
        if q_heads % kv_heads:
            raise ValueError("q_heads must be a multiple of kv_heads")
        if not (1 <= int(dim) <= 256 and 1 <= int(value_dim) <= 256):
            raise ValueError("the attention kernels take key and value sizes up to 256")
        if temperature is not None and int(temperature[1]) <= 0:
            raise ValueError("the temperature's step must be positive")
        self.names = [prefix + n for n in names]
        self.q_heads, self.kv_heads, self.dim, self.value_dim = int(q_heads), int(kv_heads), int(dim), int(value_dim)
        self.head_dev = _round_up(max(self.dim, self.value_dim), 16)
        self.scale, self.eps = float(scale), float(eps)
        self.softcap = float(softcap) if softcap else 0.0
        self.temperature = (float(temperature[0]), int(temperature[1])) if temperature is not None else None
        H, G = self.q_heads, self.kv_heads
        self.rows = [H * self.dim, G * self.dim, G * self.value_dim]
        self.columns, at = [], 0
        for rows in self.rows:                                   # (every matrix's columns begin 16-byte aligned)
            self.columns.append(at)
            at += _round_up(rows, 4)

    def in_matrices(self):
        return [(name, rows, False, (rows, _round_up(rows, 4))) for name, rows in zip(self.names, self.rows)]

    def out_matrix(self):
        return (self.names[3], self.q_heads * self.value_dim, (self.value_dim, self.head_dev))

    def cache_need(self):
        return CacheNeed(paged=PagedKV(self.kv_heads, self.head_dev))

    def forward(self, ctx, run, proj, out, scale):
        if scale != 1.0:
            raise ValueError("this branch's result is not scaled: give the mixer result norms")
        H, G, Dp = self.q_heads, self.kv_heads, self.head_dev
        keys, values, g = ctx.cache.keys_values(run.cache_slot)
        group = ctx.groups[g]
        q = ctx.scratch("normed.q", (ctx.n_tokens, H * Dp))
        ops.head_finish(proj, *self.columns, ctx.positions[0], q, keys, values, group.slot_mapping, H, G, self.dim,
                        self.value_dim, self.eps, temperature=self.temperature)
        paged_attention(ctx, q, keys, values, group, out, H, G, Dp, self.scale, softcap=self.softcap)
