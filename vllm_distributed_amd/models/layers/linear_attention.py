"""Linear attention with a recurrent state per request: a decay per head or per key channel, the gated delta rule, a state-space
recurrence whose decay depends on the token (per head, or per channel and state), or a gated linear unit per channel.

Per head ``S_t = decay[h] * S_(t-1) + k_t v_t^T`` and ``o_t = S_t^T q_t``: no softmax, no cache that grows with the
sequence.  What a request carries from token to token is the ``dim x vdim`` matrix ``S`` of every head, in fp32, one
slot per row of the worker's persistent batch (``AttentionMetadata.state_slots``; the model runner allocates the
tensor next to the KV cache and adds a spare slot for the padding rows of captured decode batches).  Nothing is cleared
when a slot changes owner: rows that start at position 0 take the state as zero whatever the slot holds.
"""
from __future__ import annotations

from typing import Optional, Sequence, Tuple

import torch
import torch.nn as nn

from ... import ops
from .attention import get_forward_context
from .linear import ColumnParallelLinear, ReplicatedLinear
from .short_conv import ShortConv, SlotState, conv_rows


class DecayLinearAttention(nn.Module):
    """Reads ``[q | k | v]`` from the leading columns of a fused projection (``activation``: through SiLU first),
    returns the fp32 heads ``[T, H * vdim]`` side by side."""
    state_dtype = torch.float32

    def __init__(self, num_heads: int, dim: int, vdim: int, decay: Sequence[float], layer_idx: int,
                 activation: bool = True):
        super().__init__()
        if len(decay) != num_heads:
            raise ValueError(f"layer {layer_idx}: {len(decay)} decays for {num_heads} heads")
        self.num_heads, self.dim, self.vdim = num_heads, dim, vdim
        self.layer_idx, self.activation = layer_idx, activation
        # fp32 from the configuration's doubles (the recurrence multiplies by exactly this number every token)
        self.register_buffer("decay", torch.tensor([float(d) for d in decay], dtype=torch.float32), persistent=False)
        self.state: Optional[torch.Tensor] = None

    # ---- per-request state, owned by the model runner
    def state_shape(self, num_slots: int) -> Tuple[int, int, int, int]:
        return (num_slots, self.num_heads, self.dim, self.vdim)

    def state_values_per_slot(self) -> int:
        return self.num_heads * self.dim * self.vdim

    def bind_state(self, state: Optional[torch.Tensor]) -> None:
        self.state = state

    def forward(self, x: torch.Tensor) -> torch.Tensor:
        md = get_forward_context().attn_metadata
        if md is None:                    # memory-profiling pass: no state bound
            return x.new_zeros((x.shape[0], self.num_heads * self.vdim), dtype=torch.float32)
        return ops.decay_linear_attention(x, self.num_heads, self.dim, self.vdim, self.decay, self.state,
                                          md.state_slots, md.query_start_loc, md.seq_lens, self.activation,
                                          md.max_query_len)


class GatedLinearHeads(nn.Module):
    """Gated linear attention between its input projection and its output projection: per head ``S <- diag(alpha) S + k v^T``
    and ``o = dim^-0.5 S^T q`` with a decay per head and key channel that comes from the token through a narrow middle,
    ``alpha = sigmoid(a2 a + bias)^(1 / tau)``; then each head's RMS norm (``norm[vdim]``, shared) times ``silu(gate)``.
    ``sizes``: the sub-matrices ``[q | k | v | gate | a]`` whose products ``forward`` reads side by side (the caller may
    fuse them with those of other consumers of the same input).  The state tensor is a ``layers.short_conv.SlotState``."""

    def __init__(self, width: int, heads: int, dim: int, vdim: int, rank: int, tau: float, eps: float, layer_idx: int,
                 dtype: torch.dtype):
        super().__init__()
        self.heads, self.dim, self.vdim, self.rank, self.tau = heads, dim, vdim, rank, float(tau)
        self.eps, self.dtype, self.layer_idx = eps, dtype, layer_idx
        self.sizes, self.out_cols = [heads * dim, heads * dim, heads * vdim, heads * vdim, rank], heads * vdim
        self.a2 = ReplicatedLinear(rank, heads * dim, False, dtype)
        self.a2_bias = nn.Parameter(torch.zeros(heads * dim, dtype=torch.float32), requires_grad=False)
        self.norm = nn.Parameter(torch.zeros(vdim, dtype=torch.float32), requires_grad=False)
        self.slot_state = SlotState((heads, dim, vdim), torch.float32)

    def forward(self, x: torch.Tensor) -> torch.Tensor:
        """``x[T, sum(sizes)]`` (rows may be strided) -> the gated heads ``[T, heads * vdim]``."""
        md = get_forward_context().attn_metadata
        vs = self.heads * self.vdim
        if md is None:                    # memory-profiling pass: no state bound
            return x.new_zeros((x.shape[0], vs))
        lo = 2 * self.heads * self.dim + vs
        alpha = ops.low_rank_decay(x[:, lo + vs:lo + vs + self.rank], self.a2.weight, self.a2_bias, self.tau)
        o = ops.decay_linear_attention(x, self.heads, self.dim, self.vdim, alpha, self.slot_state.state, md.state_slots,
                                       md.query_start_loc, md.seq_lens, False, md.max_query_len, self.dim ** -0.5)
        return ops.gated_rms_norm(o, self.norm, x[:, lo:lo + vs], self.eps, self.dtype, group=self.vdim, silu=True)


class GatedDeltaRule(nn.Module):
    """The gated delta rule: per value head a ``dim x vdim`` fp32 state with
    ``S <- g * S`` (one decay per key channel, by rows; ``head_decay``: one per head), ``u = b (v - S^T k)``, ``S <- S + k u^T``, ``o = S^T q``, on
    unit-length q and k (q times ``dim^-0.5``), ``b = sigmoid(beta)`` and ``g = exp(-exp(a_log[h]) * softplus(dt +
    dt_bias))``.  ``heads`` value heads share ``qk_heads`` query / key heads in runs of neighbours.  The state tensors
    are ``layers.short_conv.SlotState`` objects the caller owns (one per run of the layer); ``forward`` reads
    ``[q | k | v]`` from the leading columns of ``x`` and returns the fp32 heads ``[T, heads * vdim]`` side by side."""

    def __init__(self, heads: int, qk_heads: int, dim: int, vdim: int, layer_idx: int, norm_eps: float = 1e-6,
                 head_decay: bool = False):
        super().__init__()
        if heads % qk_heads:
            raise ValueError(f"layer {layer_idx}: {heads} value heads do not divide over {qk_heads} query / key heads")
        self.heads, self.qk_heads, self.dim, self.vdim = heads, qk_heads, dim, vdim
        self.layer_idx, self.norm_eps = layer_idx, float(norm_eps)
        self.a_log = nn.Parameter(torch.zeros(heads, dtype=torch.float32), requires_grad=False)
        self.dt_bias = nn.Parameter(torch.zeros(heads if head_decay else heads * dim, dtype=torch.float32),
                                    requires_grad=False)

    def per_slot_shape(self) -> Tuple[int, int, int]:
        return (self.heads, self.dim, self.vdim)

    def forward(self, x: torch.Tensor, beta: torch.Tensor, dt: torch.Tensor, state: Optional[torch.Tensor]) -> torch.Tensor:
        md = get_forward_context().attn_metadata
        if md is None or state is None:   # memory-profiling pass: no state bound
            return x.new_zeros((x.shape[0], self.heads * self.vdim), dtype=torch.float32)
        return ops.gated_delta_rule(x, self.heads, self.qk_heads, self.dim, self.vdim, beta, dt, self.dt_bias,
                                    self.a_log, state, md.state_slots, md.query_start_loc, md.seq_lens, self.norm_eps,
                                    md.max_query_len)


class SelectiveStateSpace(nn.Module):
    """A state-space recurrence in its dual (attention-like) form: per head an ``n_state x vdim`` fp32 state with
    ``S <- exp(-exp(a_log[h]) * d) * S + d * B u^T`` and ``y = S^T C + d_skip[h] * u``, where the step size
    ``d = softplus(dt + dt_bias[h])`` comes from the token (unbounded above); ``heads`` heads share ``groups`` B / C vectors
    in runs of neighbours.  The state tensors are ``layers.short_conv.SlotState`` objects the caller owns;
    ``forward`` reads ``[u | B | C]`` from the leading columns of ``x`` and returns the fp32 heads
    ``[T, heads * vdim]`` side by side.  ``skip`` False: no ``d_skip`` term."""

    def __init__(self, heads: int, groups: int, vdim: int, n_state: int, layer_idx: int, skip: bool = True):
        super().__init__()
        if groups < 1 or heads % groups:
            raise ValueError(f"layer {layer_idx}: {heads} heads do not divide over {groups} B / C groups")
        self.heads, self.groups, self.vdim, self.n_state = heads, groups, vdim, n_state
        self.layer_idx = layer_idx
        f32 = torch.float32
        self.a_log = nn.Parameter(torch.zeros(heads, dtype=f32), requires_grad=False)
        self.dt_bias = nn.Parameter(torch.zeros(heads, dtype=f32), requires_grad=False)
        self.d_skip = nn.Parameter(torch.zeros(heads, dtype=f32), requires_grad=False) if skip else None

    @property
    def channels(self) -> int:
        """Columns ``forward`` reads: ``[u | B | C]``."""
        return self.heads * self.vdim + 2 * self.groups * self.n_state

    def per_slot_shape(self) -> Tuple[int, int, int]:
        return (self.heads, self.n_state, self.vdim)

    def forward(self, x: torch.Tensor, dt: torch.Tensor, state: Optional[torch.Tensor]) -> torch.Tensor:
        md = get_forward_context().attn_metadata
        if md is None or state is None:   # memory-profiling pass: no state bound
            return x.new_zeros((x.shape[0], self.heads * self.vdim), dtype=torch.float32)
        return ops.selective_scan(x, dt, self.heads, self.groups, self.vdim, self.n_state, self.a_log, self.dt_bias,
                                  self.d_skip, state, md.state_slots, md.query_start_loc, md.seq_lens,
                                  md.max_query_len)


class ChannelStateSpace(nn.Module):
    """A selective scan in its per-channel form: every one of ``channels`` channels has a state vector of ``n_state``
    fp32 values with decays of its own, ``S[c, n] <- exp(-exp(a_log[c, n]) d_c) S[c, n] + d_c u_c B_n`` and
    ``y_c = sum_n S[c, n] C_n + d_skip[c] u_c``, with the step size ``d = softplus(dt + dt_bias)`` per channel and token
    and ``B``, ``C`` shared by the channels; the output is multiplied by ``silu(gate)`` on its way out.  The state tensors
    are ``layers.short_conv.SlotState`` objects the caller owns."""

    def __init__(self, channels: int, n_state: int, layer_idx: int):
        super().__init__()
        self.channels, self.n_state, self.layer_idx = channels, n_state, layer_idx
        f32 = torch.float32
        self.a_log = nn.Parameter(torch.zeros(channels, n_state, dtype=f32), requires_grad=False)
        self.dt_bias = nn.Parameter(torch.zeros(channels, dtype=f32), requires_grad=False)
        self.d_skip = nn.Parameter(torch.zeros(channels, dtype=f32), requires_grad=False)

    def per_slot_shape(self) -> Tuple[int, int]:
        return (self.channels, self.n_state)

    def forward(self, u: torch.Tensor, dt: torch.Tensor, bc: torch.Tensor, gate: torch.Tensor,
                state: Optional[torch.Tensor]) -> torch.Tensor:
        md = get_forward_context().attn_metadata
        if md is None or state is None:   # memory-profiling pass: no state bound
            return torch.zeros_like(u)
        return ops.channel_scan(u, dt, bc, self.n_state, self.a_log, self.dt_bias, self.d_skip, gate, state,
                                md.state_slots, md.query_start_loc, md.seq_lens, md.max_query_len)


class GatedUnitRecurrence(nn.Module):
    """A real-gated linear recurrence, one fp32 number of state per channel: ``S <- a S + sqrt(1 - a^2) i u`` with
    ``log a = -strength * r * softplus(lam)``; the gates ``r`` and ``i`` are sigmoids of block-diagonal projections of
    the input ``u`` itself (``blocks`` equal runs of channels, square matrices ``ra[b]`` and ``ri[b]`` stored out by in).
    The first token takes no special path.  The output is ``S * gelu_tanh(gate + gate_bias)``: the other branch of the
    block, still in front of its bias and activation, joins in the same launch.  The state tensors are
    ``layers.short_conv.SlotState`` objects the caller owns."""

    def __init__(self, width: int, blocks: int, layer_idx: int, dtype: torch.dtype, strength: float = 8.0):
        super().__init__()
        if blocks < 1 or width % blocks:
            raise ValueError(f"layer {layer_idx}: {width} channels do not split into {blocks} equal blocks")
        self.width, self.blocks, self.layer_idx, self.strength = width, blocks, layer_idx, float(strength)
        n, f32 = width // blocks, torch.float32
        self.ra = nn.Parameter(torch.empty(blocks, n, n, dtype=dtype), requires_grad=False)
        self.ri = nn.Parameter(torch.empty(blocks, n, n, dtype=dtype), requires_grad=False)
        self.ra_bias = nn.Parameter(torch.zeros(width, dtype=f32), requires_grad=False)
        self.ri_bias = nn.Parameter(torch.zeros(width, dtype=f32), requires_grad=False)
        self.lam = nn.Parameter(torch.zeros(width, dtype=f32), requires_grad=False)
        self.gate_bias = nn.Parameter(torch.zeros(width, dtype=f32), requires_grad=False)
        self.register_buffer("rate", None)        # strength * softplus(lam), made once the checkpoint is in

    def finalize_weights(self) -> None:
        lam = self.lam.data.double()
        self.rate = (self.strength * torch.where(lam > 30, lam, torch.log1p(torch.exp(lam.clamp(max=30.0))))).float()

    def per_slot_shape(self) -> Tuple[int]:
        return (self.width,)

    def forward(self, u: torch.Tensor, gate: torch.Tensor, state: Optional[torch.Tensor]) -> torch.Tensor:
        md = get_forward_context().attn_metadata
        if md is None or state is None:   # memory-profiling pass: no state bound
            return torch.zeros_like(u)
        return ops.gated_unit_step(u, self.ra, self.ra_bias, self.ri, self.ri_bias, self.rate, gate, self.gate_bias,
                                   state, md.state_slots, md.query_start_loc, md.seq_lens, md.max_query_len)


class DeltaRuleMixer(nn.Module):
    """Everything of a gated-delta-rule mixer between its input and its output projection: one fused projection
    ``[q | k | v | beta | decay rank | gate rank]``, the two low-rank up-projections, convolution + SiLU over
    ``[q | k | v]``, the recurrence, and the per-head RMS norm times the sigmoid gate.  ``direct``: the decay (one per
    head) and the gate are projections of the input themselves, ``[q | k | v | gate | beta | decay]``, without a low
    rank in between.  ``silu_gate``: the gate passes SiLU instead of a sigmoid.  ``passes``: how many times the
    layer runs in a forward pass over these weights (each run with convolution tails and a state of its own);
    ``forward`` writes ``scale * normed, gated heads`` into the columns it is given, so a caller may fuse several
    mixers' output projections."""

    def __init__(self, width: int, m: dict, eps: float, layer_idx: int, dtype: torch.dtype, passes: int, scale: float,
                 direct: bool = False, silu_gate: bool = False):
        super().__init__()
        self.heads, self.qk_heads = int(m["heads"]), int(m.get("kv_heads") or m["heads"])
        self.dim, self.vdim = int(m["dim"]), int(m.get("vdim") or m["dim"])
        self.direct, self.silu_gate = bool(direct), bool(silu_gate)
        self.eps, self.dtype, self.out_scale = eps, dtype, float(scale)
        qs, vs = self.qk_heads * self.dim, self.heads * self.vdim
        self.channels, self.out_cols = 2 * qs + vs, vs
        if self.direct:
            self.proj = ColumnParallelLinear(width, [qs, qs, vs, vs, self.heads, self.heads], False, dtype)
        else:
            self.decay_rank, self.gate_rank = int(m["decay_rank"]), int(m["gate_rank"])
            self.proj = ColumnParallelLinear(width, [qs, qs, vs, self.heads, self.decay_rank, self.gate_rank], False, dtype)
            self.a2 = ReplicatedLinear(self.decay_rank, self.heads * self.dim, False, dtype)
            self.g2 = ReplicatedLinear(self.gate_rank, vs, False, dtype)
        self.conv = ShortConv([qs, qs, vs], int(m.get("conv") or 1), dtype)
        self.rule = GatedDeltaRule(self.heads, self.qk_heads, self.dim, self.vdim, layer_idx, head_decay=self.direct)
        self.conv_states = [SlotState((max(self.conv.taps - 1, 1), self.channels)) for _ in range(passes)]
        self.rule_states = [SlotState(self.rule.per_slot_shape(), torch.float32) for _ in range(passes)]
        self.norm = nn.Parameter(torch.zeros(self.vdim, dtype=torch.float32), requires_grad=False)

    def forward(self, h: torch.Tensor, index: int, out: torch.Tensor) -> None:
        ctx = get_forward_context()
        md = ctx.attn_metadata
        x = self.proj(h)
        c = self.channels
        if self.direct:
            gate, lo = x[:, c:c + self.out_cols], c + self.out_cols
            beta, dt = x[:, lo:lo + self.heads], x[:, lo + self.heads:lo + 2 * self.heads]
        else:
            beta = x[:, c:c + self.heads]
            dt = self.a2(x[:, c + self.heads:c + self.heads + self.decay_rank])
            gate = self.g2(x[:, c + self.heads + self.decay_rank:])
        if md is None:                    # memory-profiling pass: no state
            out.zero_()
            return
        qkv = ops.short_conv_act(x, c, self.conv.weight_t, self.conv_states[index].state, md.state_slots,
                                 md.query_start_loc, md.seq_lens, conv_rows(md, ctx.positions), ctx.positions, True,
                                 md.num_prefills > 0)
        o = self.rule(qkv, beta, dt, self.rule_states[index].state)
        ops.gated_rms_norm(o, self.norm, gate, self.eps, self.dtype, group=self.vdim, scale=self.out_scale, out=out,
                           silu=self.silu_gate)
