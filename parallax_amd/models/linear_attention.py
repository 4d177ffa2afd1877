"""Recurrent sequence mixers whose state lives in the engine's per-request
slots: gated linear attention (below), minGRU (class MinGRU), the matrix LSTM
(class MLSTM), linear attention with a fixed decay per head (class
DecayLinearAttention: retention, lightning attention) and the gated delta rule
(class GatedDeltaRule).

Gated linear attention (GLA): a matrix-valued recurrent state per head with
a data-dependent decay per key channel,

    S_t = diag(alpha_t) S_(t-1) + k_t v_t^T,     o_t = S_t^T (q_t / sqrt(dk)),
    alpha_t = sigmoid(W_a2 W_a1 h_t + b)^(1/tau),

followed by a per-head RMS norm of o (weight shared by heads), a silu output
gate and the output projection. The state lives in the engine's
LinearStateCache slots in fp32; prompt portions and decode steps both run
ops.gla_recurrence (one HIP kernel, token-serial inside, column-parallel
across the state), so a prompt gives the same state however it is cut.
Decay, gate of the recurrence and the norm are fp32; projections run in the
activation dtype.
"""

from __future__ import annotations

from typing import Sequence

import torch
import torch.nn as nn

from .. import ops
from ..parallel.layers import MergedColumnParallelLinear, RowParallelLinear
from .forward_meta import ForwardMeta


class GatedLinearAttention(nn.Module):
    def __init__(self, hidden_size: int, heads: int, key_dim: int,
                 value_dim: int, tau: float, norm_eps: float,
                 state_layer_idx: int, decay_rank: int = 32):
        super().__init__()
        self.heads, self.dk, self.dv = heads, key_dim, value_dim
        self.tau = float(tau)
        self.eps = norm_eps
        self.state_layer_idx = state_layer_idx
        # one GEMM for q | k | v | output gate
        self.in_proj = MergedColumnParallelLinear(
            hidden_size,
            [heads * key_dim, heads * key_dim, heads * value_dim, heads * value_dim],
        )
        # low-rank decay projection; the rank follows the checkpoint's tensors
        self.decay_down = nn.Parameter(torch.empty(decay_rank, hidden_size),
                                       requires_grad=False)
        self.decay_up = nn.Parameter(torch.empty(heads * key_dim, decay_rank),
                                     requires_grad=False)
        self.decay_bias = nn.Parameter(torch.empty(heads * key_dim),
                                       requires_grad=False)
        self.norm_weight = nn.Parameter(torch.empty(value_dim), requires_grad=False)
        self.o_proj = RowParallelLinear(heads * value_dim, hidden_size)

    def load_decay(self, which: str, t: torch.Tensor) -> None:
        """a1 / a2 carry the decay rank in their shape."""
        name = "decay_down" if which == "a1" else "decay_up"
        setattr(self, name, nn.Parameter(t.clone(), requires_grad=False))

    def forward(self, x: torch.Tensor, meta: ForwardMeta) -> torch.Tensor:
        q, k, v, g = self.in_proj.split_output(self.in_proj(x))
        z = ops.linear(ops.linear(x, self.decay_down), self.decay_up)
        state = meta.linear_cache.recurrent_states[self.state_layer_idx]
        o = ops.gla_recurrence(
            q, k, v, z, self.decay_bias, state, meta.linear_slots,
            meta.query_bounds(), meta.positions, 1.0 / self.tau, self.dk ** -0.5,
        )
        return self.o_proj(ops.gated_rmsnorm(o, g, self.norm_weight, self.eps,
                                             x.dtype))


class MinGRU(nn.Module):
    """minGRU: a gated recurrence over a vector state whose gates read only
    the current token, so the whole portion's gate pre-activations come from
    one GEMM and the recurrence itself is elementwise,

        f_t = sigma(W_z h_t + b_z)            (update gate),
        p_t = W_x h_t + b_x,   c_t = p_t + 1/2 where p_t >= 0, sigma(p_t) below,
        S_t = S_(t-1) + f_t (c_t - S_(t-1)),   o_t = S_t * silu(W_g h_t),

    followed by the output projection. The state [width] lives in the
    engine's LinearStateCache slots in fp32; gates, candidate and state are
    fp32 whatever the activation dtype. Prompt portions and decode steps run
    the same kernel (ops.mingru_scan), token-serial per channel.

    own_proj False: the module has no input projection of its own; a caller
    that merges it with other projections of the same input hands the
    pre-activations [z | u | g] (`proj_sizes` wide) to mix()."""

    def __init__(self, hidden_size: int, width: int, state_layer_idx: int,
                 own_proj: bool = True):
        super().__init__()
        self.width = int(width)
        self.state_layer_idx = state_layer_idx
        self.proj_sizes = [self.width] * 3       # z | u | g
        self.in_proj = MergedColumnParallelLinear(hidden_size, self.proj_sizes) \
            if own_proj else None
        self.z_bias = nn.Parameter(torch.empty(self.width), requires_grad=False)
        self.x_bias = nn.Parameter(torch.empty(self.width), requires_grad=False)
        self.o_proj = RowParallelLinear(self.width, hidden_size)
        self._b32 = None

    def invalidate_constants(self) -> None:
        self._b32 = None

    def mix(self, zug: torch.Tensor, meta: ForwardMeta) -> torch.Tensor:
        """zug [T, 3 * width] (a strided view is fine) -> S_t * silu(g_t)."""
        if self._b32 is None or self._b32[0].device != zug.device:
            self._b32 = (self.z_bias.detach().float().contiguous(),
                         self.x_bias.detach().float().contiguous())
        state = meta.linear_cache.recurrent_states[self.state_layer_idx]
        return ops.mingru_scan(zug, self._b32[0], self._b32[1], state,
                               meta.linear_slots, meta.query_bounds(),
                               meta.positions, self.o_proj.weight.dtype)

    def forward(self, x: torch.Tensor, meta: ForwardMeta) -> torch.Tensor:
        return self.o_proj(self.mix(self.in_proj(x), meta))


class MLSTM(nn.Module):
    """Matrix LSTM (the mLSTM cell of xLSTM): per head a matrix memory S
    [dim, vdim], a normaliser n [dim] and a running maximum m with scalar
    exponential gates,

        i = cap tanh((W_i h + b_i) / cap),
        f = logsigmoid(cap tanh((W_f h + b_f) / cap)),
        m' = max(f + m, i),
        S <- exp(f + m - m') S + exp(i - m') k v^T,   n likewise with k alone,
        o = S^T q / (max(|n . q|, exp(-m')) + 1e-6),   q = W_q h / sqrt(dim),

    all three starting at zero; each head's o is divided by its RMS, the heads
    together are multiplied by a weight and by sigmoid(W_g h) before the
    output projection. State, gates, normalisation and output gate are fp32
    (ops.mlstm); so are the gates' pre-activations (ops.linear_f32), which end
    in exponentials. The state lives in LinearStateCache slots, one row
    [S | n | m] per head. A layer that runs several times per token names the
    state of the pass when it is called."""

    def __init__(self, hidden_size: int, heads: int, dim: int, vdim: int,
                 gate_cap: float, norm_eps: float, state_layer_idx: int = 0):
        super().__init__()
        self.heads, self.dim, self.vdim = heads, dim, vdim
        self.cap, self.eps = float(gate_cap), float(norm_eps)
        self.state_layer_idx = state_layer_idx
        # one GEMM for q | k | v | output gate
        self.in_proj = MergedColumnParallelLinear(
            hidden_size, [heads * dim, heads * dim, heads * vdim, heads * vdim])
        # input gates, then forget gates
        self.gate_weight = nn.Parameter(torch.empty(2 * heads, hidden_size),
                                        requires_grad=False)
        self.gate_bias = nn.Parameter(torch.empty(2 * heads), requires_grad=False)
        self.norm_weight = nn.Parameter(torch.empty(heads * vdim),
                                        requires_grad=False)
        self.o_proj = RowParallelLinear(heads * vdim, hidden_size)
        self._b32 = None

    def load_gate(self, which: int, w=None, b=None) -> None:
        """which: 0 = input gate, 1 = forget gate."""
        rows = slice(which * self.heads, (which + 1) * self.heads)
        if w is not None:
            self.gate_weight.data[rows].copy_(w)
        if b is not None:
            self.gate_bias.data[rows].copy_(b)

    def invalidate_constants(self) -> None:
        self._b32 = None

    def forward(self, x: torch.Tensor, meta: ForwardMeta,
                state_layer_idx=None) -> torch.Tensor:
        if self._b32 is None or self._b32.device != x.device:
            self._b32 = self.gate_bias.detach().float().contiguous()
        q, k, v, g = self.in_proj.split_output(self.in_proj(x))
        idx = self.state_layer_idx if state_layer_idx is None else state_layer_idx
        o = ops.mlstm(q, k, v, g, ops.linear_f32(x, self.gate_weight),
                      self._b32, self.norm_weight, self.cap, self.eps,
                      meta.linear_cache.recurrent_states[idx],
                      meta.linear_slots, meta.query_bounds(), meta.positions,
                      x.dtype)
        return self.o_proj(o)


class DecayLinearAttention(nn.Module):
    """Linear attention with one fixed decay per head, no softmax and no
    denominator,

        S_t = decay_h S_(t-1) + k_t v_t^T,     o_t = S_t^T q_t,

    S [dim, vdim] from zero, then a norm, an output gate and the output
    projection. Switches make it retention (q and k rotated by position on
    their first rot_dims dimensions, pairs i, i + rot_dims / 2; k times
    k_scale; each head's o divided by its RMS; silu gate) or lightning
    attention (silu on q, k and v; the heads normed together with a weight,
    `norm_all`; sigmoid gate). Angles, decays, state, norm and gate are fp32
    (ops.decay_attention, ops.gated_rmsnorm); the state lives in
    LinearStateCache slots.

    own_proj False: a caller merges the input projections [q | k | v | g]
    (`proj_sizes`) with others of the same input and hands their columns to
    mix()."""

    def __init__(self, hidden_size: int, heads: int, dim: int, vdim: int,
                 decay: Sequence[float], norm_eps: float, state_layer_idx: int, *,
                 silu: bool = False, rot_dims: int = 0, rot_base: float = 10000.0,
                 k_scale: float = 1.0, norm_all: bool = False,
                 gate_act: str = "silu", own_proj: bool = True):
        super().__init__()
        if len(decay) != heads:
            raise ValueError(f"{len(decay)} decays for {heads} heads")
        if rot_dims % 2 or rot_dims > dim:
            raise ValueError(f"cannot rotate {rot_dims} of {dim} dimensions")
        self.heads, self.dim, self.vdim = heads, dim, vdim
        self.eps = norm_eps
        self.state_layer_idx = state_layer_idx
        self.silu, self.k_scale = bool(silu), float(k_scale)
        self.norm_all, self.gate_act = bool(norm_all), gate_act
        self._powers = ops.decay_powers(decay)
        self._rot_key = (int(rot_dims), float(rot_base))
        self._freq = None
        if rot_dims:
            i = torch.arange(0, rot_dims, 2, dtype=torch.float64)
            self._freq = (float(rot_base) ** (-i / rot_dims)).float()
        self.proj_sizes = [heads * dim, heads * dim, heads * vdim, heads * vdim]
        self.in_proj = MergedColumnParallelLinear(hidden_size, self.proj_sizes) \
            if own_proj else None
        self.norm_weight = nn.Parameter(torch.empty(heads * vdim),
                                        requires_grad=False) if norm_all else None
        self.o_proj = RowParallelLinear(heads * vdim, hidden_size)

    def invalidate_constants(self) -> None:
        pass

    def mix(self, qkvg: torch.Tensor, meta: ForwardMeta) -> torch.Tensor:
        """qkvg: the projections' columns (a strided view is fine) -> [T, heads
        * vdim]."""
        T, H = qkvg.shape[0], self.heads
        q, k, v, g = torch.split(qkvg, self.proj_sizes, dim=-1)
        dev = qkvg.device
        if self._powers.device != dev:
            self._powers = self._powers.to(dev)
            self._freq = self._freq.to(dev) if self._freq is not None else None
        cs = meta.rope_table(self._rot_key, self._freq) \
            if self._freq is not None else None
        o = ops.decay_attention(
            q.view(T, H, self.dim), k.view(T, H, self.dim), v.view(T, H, self.vdim),
            self._powers, self.k_scale, self.silu, cs,
            meta.linear_cache.recurrent_states[self.state_layer_idx],
            meta.linear_slots, meta.query_bounds(), meta.positions)
        return ops.gated_rmsnorm(o, g, self.norm_weight, self.eps,
                                 self.o_proj.weight.dtype, whole=self.norm_all,
                                 act=self.gate_act)

    def forward(self, x: torch.Tensor, meta: ForwardMeta) -> torch.Tensor:
        return self.o_proj(self.mix(self.in_proj(x), meta))


class GatedDeltaRule(nn.Module):
    """Gated delta rule: `kv_heads` query/key heads of width dim, `heads` value
    heads of width vdim (head h reads q/k head h // (heads / kv_heads)). q, k
    and v pass a causal depthwise convolution over time and silu; q and k
    become unit vectors, q times dim^-1/2; beta = sigmoid(W_b h), g =
    exp(-exp(A_log) softplus(W_a h + dt_bias)), one each per head:

        S <- g S,   u = beta (v - S^T k),   S <- S + k u^T,   o = S^T q;

    each head's o is divided by its RMS, times a weight shared by the heads,
    times silu(W_g h), then the output projection. Unit norms, gates, decays,
    state and the head norm are fp32; so are the gates' pre-activations
    (ops.linear_f32), which end in exponentials. The state and the
    convolution's last inputs live in LinearStateCache slots."""

    def __init__(self, hidden_size: int, heads: int, kv_heads: int, dim: int,
                 vdim: int, taps: int, norm_eps: float, state_layer_idx: int):
        super().__init__()
        if heads % kv_heads:
            raise ValueError(f"{heads} heads do not divide into {kv_heads} "
                             "query/key heads")
        if taps < 1:
            raise ValueError("a convolution has at least one tap")
        self.heads, self.kv_heads, self.dim, self.vdim = heads, kv_heads, dim, vdim
        self.eps = norm_eps
        self.state_layer_idx = state_layer_idx
        self.conv_sizes = [kv_heads * dim, kv_heads * dim, heads * vdim]
        self.conv_width = sum(self.conv_sizes)
        # one GEMM for q | k | v | output gate
        self.in_proj = MergedColumnParallelLinear(
            hidden_size, self.conv_sizes + [heads * vdim])
        self.conv_weight = nn.Parameter(torch.empty(self.conv_width, taps),
                                        requires_grad=False)
        # step sizes, then decays
        self.gate_weight = nn.Parameter(torch.empty(2 * heads, hidden_size),
                                        requires_grad=False)
        self.a_log = nn.Parameter(torch.empty(heads), requires_grad=False)
        self.dt_bias = nn.Parameter(torch.empty(heads), requires_grad=False)
        self.norm_weight = nn.Parameter(torch.empty(vdim), requires_grad=False)
        self.o_proj = RowParallelLinear(heads * vdim, hidden_size)
        self._f32 = None

    def load_conv(self, which: int, t: torch.Tensor) -> None:
        """which: 0 = q, 1 = k, 2 = v; t [channels, taps]."""
        off = sum(self.conv_sizes[:which])
        self.conv_weight.data[off : off + self.conv_sizes[which]].copy_(t)

    def load_gate(self, which: int, t: torch.Tensor) -> None:
        """which: 0 = step size, 1 = decay."""
        self.gate_weight.data[which * self.heads : (which + 1) * self.heads].copy_(t)

    def invalidate_constants(self) -> None:
        self._f32 = None

    def forward(self, x: torch.Tensor, meta: ForwardMeta) -> torch.Tensor:
        if self._f32 is None or self._f32[0].device != x.device:
            self._f32 = tuple(p.detach().float().contiguous().to(x.device)
                              for p in (self.a_log, self.dt_bias))
        T, cache, idx = x.shape[0], meta.linear_cache, self.state_layer_idx
        y = self.in_proj(x)
        cu = meta.query_bounds()
        mixed = ops.short_conv(y[:, : self.conv_width], self.conv_weight,
                               cache.conv_states[idx], meta.linear_slots, cu,
                               meta.positions, x.dtype)
        q, k, v = torch.split(mixed, self.conv_sizes, dim=-1)
        o = ops.gated_delta_rule(
            q.view(T, self.kv_heads, self.dim), k.view(T, self.kv_heads, self.dim),
            v.view(T, self.heads, self.vdim), ops.linear_f32(x, self.gate_weight),
            *self._f32, cache.recurrent_states[idx], meta.linear_slots, cu,
            meta.positions)
        return self.o_proj(ops.gated_rmsnorm(o, y[:, self.conv_width :],
                                             self.norm_weight, self.eps, x.dtype))
