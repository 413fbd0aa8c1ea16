"""Recurrences with a matrix state per head that decays from token to token (kernels: `ops.linear_state`).

`StateSpace`: the state-space recurrence of Mamba-2 (Dao and Gu, "Transformers are SSMs: Generalized Models and Efficient
Algorithms Through Structured State Space Duality") as a mixer:

    [z | x | B | C | delta] = W_in h;  x, B, C through one short causal convolution per channel (with bias) and SiLU
    delta <- softplus(delta + dt_bias);  per head  S <- exp(-exp(A_log) delta) S + delta B x^T,  y = S^T C + D x
    out = W_o ( norm_weight * unit_in_parts(y * silu(z)) )           heads // groups heads in a row share a group's B and C

`GatedLinearAttention` (Yang et al., "Gated Linear Attention Transformers with Hardware-Efficient Training"): one of the
branches of a `ParallelMixer`:

    q = W_q h * dim^-1/2, k = W_k h, v = W_v h;  log a = log sigmoid(W_up (W_low h) + b) / tau     (per head and key element)
    S <- diag(a) S + k v^T,  o = S^T q;   out = W_o [ .. norm_weight * unit(o_h) .. ] * silu(W_g h)

`LightningAttention` (Qin et al., "Lightning Attention-2: A Free Lunch for Handling Unlimited Sequence Lengths in Large Language
Models"), another branch:

    q = silu(W_q h), k = silu(W_k h), v = silu(W_v h);  S <- decay_h S + k v^T,  o = S^T q          (decays: constants)
    out = W_o ( norm_weight * unit(o over all heads) * sigmoid(W_g h) )

The state S (and the convolution's last inputs) are float32 states of the cache slot, zero when a request opens. The
packed products leave float32 rows; convolution, decays, states, norms and all products with a state are float32 in both
precisions. One-token (and few-token) sequences are walked token by token, longer portions run in chunks on the matrix
unit: the same sums in another order.
"""
from __future__ import annotations

import torch

from ..cache.spec import CacheNeed, FixedState
from ..kernels import ops
from ..weights.spec import NORMAL, ONE_PLUS_NORMAL, VECTOR, TensorSpec
from .base import Mixer
from .convolution import CausalConv
from .linear import Linear
from .parallel import MixerBranch

MAX_KEY = 256                   # key elements the kernels take


def _round_up(v, m):
    return (int(v) + m - 1) // m * m


def state_need(heads, dim, value_dim):
    """The float32 state of `ops.linear_state`: [heads, values, keys], both rounded up to 16."""
    return FixedState((heads, _round_up(value_dim, 16), _round_up(dim, 16)), "float32")


def all_walked(ctx):
    """Does every sequence of the step bring so few tokens that it is walked?"""
    return ctx.max_q_len <= ops.LINEAR_STATE_WALK_TOKENS


def run_linear_state(ctx, src, state, out, heads, dim, value_dim, **options):
    """A step's sequences through the recurrence: few tokens a sequence walked, prompt portions in chunks."""
    common = (state, ctx.q_start, ctx.state_slots)
    columns = [options.pop(k) for k in ("q_col", "k_col", "v_col")]
    portions = ctx.n_seqs - ctx.n_decode
    walked = ctx.n_seqs if all_walked(ctx) else ctx.n_decode
    if walked:
        ops.linear_state(src, *columns, *common, 0, walked, out, heads, dim, value_dim, walk=True, **options)
    if portions and walked < ctx.n_seqs:
        floats = ops.linear_state_workspace_floats(portions, ctx.max_q_len, heads, dim, value_dim)
        ws = ctx.workspace.get("linear_state.segments", (floats,), torch.float32) if floats else None
        ops.linear_state(src, *columns, *common, ctx.n_decode, portions, out, heads, dim, value_dim, walk=False,
                         max_q_len=ctx.max_q_len, workspace=ws, **options)
    return out


class StateSpace(Mixer):
    STATE, CONV_STATE = "state_space.s", "state_space.conv"

    def __init__(self, prefix, hidden, heads, value_dim, state, groups, taps, norm_parts, eps,
                 names=("in", "conv", "dt_bias", "A_log", "D", "norm", "o"), bias_suffix=".b", suffix=""):
        """value_dim: a head's size of x and y; state: the size of a group's B and C; norm_parts: into how many equal
        parts the norm cuts the row of all heads; eps: of that norm; names: the checkpoint's, behind the prefix."""
        if heads % groups or (heads * value_dim) % norm_parts:
            raise ValueError("heads must be a multiple of groups, and the row of all heads one of the norm's parts")
        if not 1 <= int(state) <= MAX_KEY:
            raise ValueError(f"the recurrence's kernels take states of up to {MAX_KEY} elements")
        self.heads, self.value_dim, self.state, self.groups = int(heads), int(value_dim), int(state), int(groups)
        self.norm_parts, self.eps = int(norm_parts), float(eps)
        n_in, conv, *extras, norm, o = (prefix + n for n in names)
        self.extras, self.norm_name = extras, norm
        self.inner = self.heads * self.value_dim
        self.channels = self.inner + 2 * self.groups * self.state
        width = self.inner + self.channels + self.heads
        self.proj = Linear([n_in], hidden, [width], pad_out=(width, _round_up(width, 4)), suffixes=(suffix, bias_suffix))
        self.width_dev = _round_up(width, 4)                     # (rows of the packed product stay 16-byte aligned)
        self.conv = CausalConv(conv, self.channels, taps, self.CONV_STATE, bias_name=conv + bias_suffix)
        self.o = Linear([o], self.inner, [hidden], suffixes=(suffix, bias_suffix))
        self.dt_bias = self.A_log = self.skip = self.norm_weight = None

    def parts(self):
        return [self.proj, self.conv, self.o]

    def tensor_specs(self):
        dt_bias, a_log, skip = self.extras
        H = (self.heads,)
        return (self.proj.tensor_specs() + self.conv.tensor_specs() + self.o.tensor_specs() +
                [TensorSpec(dt_bias, H, VECTOR, NORMAL), TensorSpec(a_log, H, VECTOR, NORMAL), TensorSpec(skip, H, VECTOR, ONE_PLUS_NORMAL),
                 TensorSpec(self.norm_name, (self.inner,), VECTOR, ONE_PLUS_NORMAL)])

    def bind(self, tensors, dtype, device):
        for p in self.parts():
            p.bind(tensors, dtype, device)
        self.dt_bias, self.A_log, self.skip = (tensors.pop(name).contiguous() for name in self.extras)
        self.norm_weight = tensors.pop(self.norm_name).contiguous()

    def weight_tensors(self):
        return [self.dt_bias, self.A_log, self.skip, self.norm_weight]

    def cache_need(self):
        return CacheNeed(states=((self.STATE, state_need(self.heads, self.state, self.value_dim)), self.conv.state_need()))

    def forward(self, ctx, run, h, x, accumulate=True):
        n, inner, N = ctx.n_tokens, self.inner, self.state
        proj = ctx.scratch("state_space.proj", (n, self.width_dev), torch.float32)
        self.proj.forward(ctx, h, proj)
        xbc = ctx.scratch("state_space.xbc", (n, self.channels), torch.float32)
        self.conv.forward(ctx, run, proj[:, inner:inner + self.channels], out32=xbc, activation="silu")
        y = ctx.scratch("state_space.y", (n, inner), torch.float32)
        run_linear_state(ctx, xbc, ctx.cache.states[run.cache_slot][self.STATE], y, self.heads, N, self.value_dim, v_col=0,
                         k_col=inner, q_col=inner + self.groups * N, groups=self.groups, raw=proj, raw_col=inner + self.channels,
                         dt_bias=self.dt_bias, A_log=self.A_log, skip=self.skip)
        act = ctx.scratch("state_space.act", (n, inner))
        ops.gate_group_norm(y, proj[:, :inner], self.norm_weight, act, self.norm_parts, self.eps)
        if ctx.defer_sums and self.o.deferrable(n):
            return self.o.forward_partials(ctx, act, "o")          # whoever runs next adds them up
        self.o.forward(ctx, act, x, residual=x if accumulate else None)
        return None


class GatedLinearAttention(MixerBranch):
    STATE = "linear_attention.s"

    def __init__(self, prefix, heads, dim, value_dim, rank, tau, eps, names=("q", "k", "v", "g", "a1", "a2", "norm", "o"),
                 bias_suffix=".b"):
        """rank: of the decay's low-rank product; tau: the root taken of the decay; eps: of the heads' norm."""
        if not 1 <= int(dim) <= MAX_KEY:
            raise ValueError(f"the recurrence's kernels take keys of up to {MAX_KEY} elements")
        if not float(tau) > 0 or int(rank) <= 0:
            raise ValueError("tau and the rank must be positive")
        self.heads, self.dim, self.value_dim, self.rank = int(heads), int(dim), int(value_dim), int(rank)
        self.tau, self.eps = float(tau), float(eps)
        self.names = [prefix + n for n in names]
        self.up_name, self.norm_name, self.o_name = self.names[5:]
        self.bias_name = self.up_name + bias_suffix
        self.up = self.bias = self.norm_weight = None
        H, D, E = self.heads, self.dim, self.value_dim
        self.rows = [H * D, H * D, H * E, H * E, self.rank]
        self.columns, at = [], 0
        for rows in self.rows:                                   # (every matrix's columns begin 16-byte aligned)
            self.columns.append(at)
            at += _round_up(rows, 4)

    def in_matrices(self):
        return [(name, rows, False, (rows, _round_up(rows, 4))) for name, rows in zip(self.names, self.rows)]

    def out_matrix(self):
        return (self.o_name, self.heads * self.value_dim, None)

    def tensor_specs(self):
        HD = self.heads * self.dim
        return [TensorSpec(self.up_name, (HD, self.rank), VECTOR, NORMAL), TensorSpec(self.bias_name, (HD,), VECTOR, NORMAL),
                TensorSpec(self.norm_name, (self.value_dim,), VECTOR, ONE_PLUS_NORMAL)]

    def bind(self, tensors, dtype, device):
        self.up = tensors.pop(self.up_name).t().contiguous()     # float32 [rank, heads * dim]
        self.bias = tensors.pop(self.bias_name).contiguous()
        self.norm_weight = tensors.pop(self.norm_name).contiguous()

    def weight_tensors(self):
        return [self.up, self.bias, self.norm_weight]

    def cache_need(self):
        return CacheNeed(states=((self.STATE, state_need(self.heads, self.dim, self.value_dim)),))

    def forward(self, ctx, run, proj, out, scale):
        if scale != 1.0:
            raise ValueError("this branch's result is not scaled: give the mixer result norms")
        n, H, D, E = ctx.n_tokens, self.heads, self.dim, self.value_dim
        q, k, v, g, low = self.columns
        if all_walked(ctx):                                      # the walking kernel forms the decays itself
            decays = dict(low_rank=(proj[:, low:low + self.rank], self.up, self.bias, self.tau))
        else:
            decays = dict(logs=ctx.scratch("linear_attention.logs", (n, H * D), torch.float32))
            ops.decay_logs(proj[:, low:low + self.rank], self.up, self.bias, self.tau, decays["logs"])
        o = ctx.scratch("linear_attention.o", (n, H * E), torch.float32)
        run_linear_state(ctx, proj, ctx.cache.states[run.cache_slot][self.STATE], o, H, D, E, q_col=q, k_col=k, v_col=v,
                         q_scale=D ** -0.5, **decays)
        ops.head_norm_gate(o, proj[:, g:g + H * E], self.norm_weight, out, H, E, self.eps)


class LightningAttention(MixerBranch):
    STATE = "lightning_attention.s"

    def __init__(self, prefix, heads, dim, value_dim, decay, eps, names=("q", "k", "v", "g", "norm", "o")):
        """decay: one constant per head, in (0, 1]; eps: of the norm over all heads."""
        if not 1 <= int(dim) <= MAX_KEY:
            raise ValueError(f"the recurrence's kernels take keys of up to {MAX_KEY} elements")
        self.decays = [float(d) for d in decay]
        if len(self.decays) != int(heads) or not all(0.0 < d <= 1.0 for d in self.decays):
            raise ValueError("one decay in (0, 1] per head is needed")
        self.heads, self.dim, self.value_dim, self.eps = int(heads), int(dim), int(value_dim), float(eps)
        self.names = [prefix + n for n in names]
        self.norm_name, self.o_name = self.names[4:]
        self.decay = self.norm_weight = None
        H, D, E = self.heads, self.dim, self.value_dim
        self.rows = [H * D, H * D, H * E, H * E]
        self.columns, at = [], 0
        for rows in self.rows:                                   # (every matrix's columns begin 16-byte aligned)
            self.columns.append(at)
            at += _round_up(rows, 4)
        self.inner, self.inner_dev = H * E, _round_up(H * E, 8)  # (rows of the output product's input stay 16-byte aligned)

    def in_matrices(self):
        return [(name, rows, False, (rows, _round_up(rows, 4))) for name, rows in zip(self.names, self.rows)]

    def out_matrix(self):
        return (self.o_name, self.inner, (self.inner, self.inner_dev))

    def tensor_specs(self):
        return [TensorSpec(self.norm_name, (self.inner,), VECTOR, ONE_PLUS_NORMAL)]

    def bind(self, tensors, dtype, device):
        self.norm_weight = tensors.pop(self.norm_name).contiguous()
        self.decay = torch.tensor(self.decays, dtype=torch.float32, device=device)        # constants of the configuration

    def weight_tensors(self):
        return [self.norm_weight]

    def cache_need(self):
        return CacheNeed(states=((self.STATE, state_need(self.heads, self.dim, self.value_dim)),))

    def forward(self, ctx, run, proj, out, scale):
        n, H, D, E = ctx.n_tokens, self.heads, self.dim, self.value_dim
        q, k, v, g = self.columns
        o = ctx.scratch("lightning_attention.o", (n, H * E), torch.float32)
        run_linear_state(ctx, proj, ctx.cache.states[run.cache_slot][self.STATE], o, H, D, E, q_col=q, k_col=k, v_col=v,
                         decay=self.decay, activation="silu")
        if self.inner_dev != self.inner:
            out[:, self.inner:].zero_()                          # (meets zero columns, but must not hold NaN)
        ops.gate_group_norm(o, proj[:, g:g + self.inner], self.norm_weight, out[:, :self.inner], 1, self.eps, after=True, scale=scale)
