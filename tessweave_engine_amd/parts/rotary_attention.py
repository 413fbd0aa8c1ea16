"""Attention over pages with rotated queries and keys, as branches of a `ParallelMixer` (alone, or beside others).

`RotaryAttention`: grouped-query attention, no biases, values of a size of their own:

    q = rotate(norm(W_q h)), k = rotate(norm(W_k h)), v = W_v h
    score = scale * q . k over the keys up to the query;  softmax, its denominator with exp(sink_h) more where there are sinks
    result = [ .. sum_j p_j v_j * sigmoid(W_g h)_h .. ]              (one gate a head, where there are gates)

norm: over each head with one weight for all heads ("head"), over the whole row at once ("row"), or none.

`DifferentialAttention` (Ye et al., "Differential Transformer"), with biases, in chunks: a query sees only keys of its own chunk of
positions (counted from the sequence's start). A head has two maps of queries and keys over the same values:

    a_m = softmax(scale * q_m . k_m) v, m = 1, 2
    o = a_1 - lambda a_2,  lambda = exp(lq1 . lk1) - exp(lq2 . lk2) + diff;   result = unit(o) * (1 - diff) * sigmoid(W_g h)_h

It may read another layer's keys and values (`reads_other`): it then has no matrices for them, and its schedule entry names
that layer's cache slot without writing it. A key lies in the page with its two maps side by side; a map's query has zeros
in the other map's place. So the engine's attention kernels run both maps as one attention of twice the heads.

The packed product leaves float32 rows (or split-K sums): biases, norms, rotation, gates and the cache write are one kernel
(`ops.rows_finish`, which also forms the angles), float32 with one rounding. Keys and values are laid out with the larger of their sizes, rounded up to
16, tails of zeros. A branch's weight in its mixer's sum multiplies the values before they are rounded into the pages
(attention is linear in them), or the combined maps.
"""
from __future__ import annotations

import torch

from ..cache.spec import CacheNeed, PagedKV
from ..kernels import ops
from ..weights.spec import NORMAL, ONE_PLUS_NORMAL, VECTOR, TensorSpec
from .attention import paged_attention
from .parallel import MixerBranch


def _round_up(v, m):
    return (int(v) + m - 1) // m * m


class RotaryAttention(MixerBranch):
    takes_partials = True
    maps = 1

    def __init__(self, prefix, q_heads, kv_heads, dim, value_dim, position, scale, eps, norm=None, sink=False, gate=False, bias=False,
                 chunk=None, retain=None, reads_other=False, names=("q", "k", "v", "g", "o"), norm_suffix=".norm", sink_name="sink"):
        """position: a rotary part over at most dim elements (shared by layers); eps: of the queries' and keys' norm; chunk: size of
        the chunks a query stays in, or None; retain: the chunk sizes of every layer that reads this layer's pages."""
        if q_heads % kv_heads:
            raise ValueError("q_heads must be a multiple of kv_heads")
        if not (1 <= int(dim) * self.maps <= 256 and 1 <= int(value_dim) <= 256):
            raise ValueError("the attention kernels take key sizes (of all maps together) and value sizes up to 256")
        if position.rotary_dim > dim:
            raise ValueError("the rotary encoding must cover at most dim elements")
        self.names = [prefix + n for n in names]
        self.q_heads, self.kv_heads, self.dim, self.value_dim = int(q_heads), int(kv_heads), int(dim), int(value_dim)
        self.position, self.scale, self.eps, self.norm = position, float(scale), float(eps), norm
        self.has_gate, self.has_bias, self.reads_other = bool(gate), bool(bias), bool(reads_other)
        self.chunk = int(chunk) if chunk else None
        self.retain = tuple(retain) if retain else ((self.chunk,) if self.chunk else ())
        self.head_dev = _round_up(max(self.maps * self.dim, self.value_dim), 16)
        self.norm_names = [self.names[0] + norm_suffix, self.names[1] + norm_suffix]
        self.sink_name = prefix + sink_name if sink else None
        self.q_weight = self.k_weight = self.sink = None
        H, G, M = self.q_heads, self.kv_heads, self.maps
        self.rows = {"q": H * M * self.dim}
        if not self.reads_other:
            self.rows.update(k=G * M * self.dim, v=G * self.value_dim)
        if self.has_gate:
            self.rows["g"] = H
        at, columns = 0, {}
        for key, rows in self.rows.items():                      # (every matrix's columns begin 16-byte aligned)
            columns[key] = at
            at += _round_up(rows, 4)
        self.columns = tuple(columns.get(key) for key in "qkvg")

    def parts(self):
        return [self.position]

    def in_matrices(self):
        name = dict(zip("qkvg", self.names))
        return [(name[key], rows, self.has_bias and key != "g", (rows, _round_up(rows, 4))) for key, rows in self.rows.items()]

    def out_matrix(self):
        return (self.names[4], self.q_heads * self.value_dim, (self.value_dim, self.head_dev))

    def tensor_specs(self):
        specs = []
        if self.norm:
            heads = (1, 1) if self.norm == "head" else (self.q_heads * self.maps, self.kv_heads * self.maps)
            specs += [TensorSpec(name, (k * self.dim,), VECTOR, ONE_PLUS_NORMAL)
                      for name, k in list(zip(self.norm_names, heads))[:1 if self.reads_other else 2]]
        if self.sink_name:
            specs.append(TensorSpec(self.sink_name, (self.q_heads,), VECTOR, NORMAL))
        return specs

    def bind(self, tensors, dtype, device):
        if self.norm:
            self.q_weight = tensors.pop(self.norm_names[0]).contiguous()
            self.k_weight = tensors.pop(self.norm_names[1]).contiguous() if not self.reads_other else None
        if self.sink_name:
            self.sink = tensors.pop(self.sink_name).contiguous()
        self.position.bind(tensors, dtype, device)               # shared by layers; binding again is harmless

    def weight_tensors(self):
        return [t for t in (self.q_weight, self.k_weight, self.sink) if t is not None]

    def cache_need(self):
        return CacheNeed(paged=PagedKV(self.kv_heads, self.head_dev, chunks=self.retain))

    def _finish(self, ctx, run, proj, bias, value_scale):
        """(queries, keys, values, cache group, gate): the projection's rows normed and turned, keys and values written."""
        n, H = ctx.n_tokens, self.q_heads
        if run.writes_cache == self.reads_other:
            raise ValueError("the schedule and the layer disagree about who writes the cache slot")
        keys, values, g = ctx.cache.keys_values(run.cache_slot)
        group = ctx.groups[g]
        q = ctx.scratch("rotary.q", (n, H * self.maps * self.head_dev))
        gate = ctx.scratch("rotary.gate", (n, H), torch.float32) if self.has_gate else None
        ops.rows_finish(proj, self.columns, self.norm, self.q_weight, self.k_weight, self.position.angles(ctx), q, keys, values,
                        group.slot_mapping, gate, H, self.kv_heads, self.dim, self.value_dim, self.eps, maps=self.maps,
                        adjacent=self.position.pairing == "adjacent", value_scale=value_scale, bias=bias)
        return q, keys, values, group, gate

    def forward(self, ctx, run, proj, out, scale, bias=None):
        q, keys, values, group, gate = self._finish(ctx, run, proj, bias, scale)
        paged_attention(ctx, q, keys, values, group, out, self.q_heads, self.kv_heads, self.head_dev, self.scale,
                        chunk=self.chunk or 0, sink=self.sink, gate=gate)


class DifferentialAttention(RotaryAttention):
    maps = 2

    def __init__(self, prefix, q_heads, kv_heads, dim, value_dim, position, scale, eps, diff, chunk=None, retain=None, reads_other=False,
                 names=("q", "k", "v", "g", "o"), lambda_names=("lq1", "lk1", "lq2", "lk2")):
        super().__init__(prefix, q_heads, kv_heads, dim, value_dim, position, scale, eps, gate=True, bias=True, chunk=chunk, retain=retain,
                         reads_other=reads_other, names=names)
        self.diff, self.lambda_names = float(diff), [prefix + n for n in lambda_names]
        self.value_dev = _round_up(self.value_dim, 8)            # (rows of the output product's input stay 16-byte aligned)
        self.weight = None

    def out_matrix(self):
        return (self.names[4], self.q_heads * self.value_dim, (self.value_dim, self.value_dev))

    def tensor_specs(self):
        return super().tensor_specs() + [TensorSpec(name, (self.dim,), VECTOR, NORMAL) for name in self.lambda_names]

    def bind(self, tensors, dtype, device):
        super().bind(tensors, dtype, device)
        q1, k1, q2, k2 = (tensors.pop(name).double() for name in self.lambda_names)
        # one number the layer's weights fix: formed once
        self.weight = float(torch.exp((q1 * k1).sum()) - torch.exp((q2 * k2).sum()) + self.diff)

    def forward(self, ctx, run, proj, out, scale, bias=None):
        n, H = ctx.n_tokens, self.q_heads
        q, keys, values, group, gate = self._finish(ctx, run, proj, bias, 1.0)
        maps = ctx.scratch("rotary.maps", (n, 2 * H * self.head_dev), torch.float32)
        paged_attention(ctx, q, keys, values, group, maps, 2 * H, self.kv_heads, self.head_dev, self.scale, chunk=self.chunk or 0)
        ops.map_difference(maps, out, H, self.value_dim, self.weight, (1.0 - self.diff) * scale, self.eps, gate=gate)
