"""Recurrent mixers whose state is a matrix per head, moved by a decay and a weight per head or by the
delta rule (``csrc/matrix_state.hip``)."""

import torch

from ..ops import kernels
from ..weights.loader import MATRIX, VECTOR, ParamSpec
from .base import CoreMixer, SlotStateSpec
from .registry import register_mixer


def _slot_floats(*pieces):
    """Floats of a slot that holds the pieces one behind the other, rounded up to 16 bytes."""
    return -(-sum(pieces) // 4) * 4


# tokens beyond one per item from which a bfloat16 step runs a decayed recurrence in chunks
CHUNKS_FROM = 128


def _chunks(ctx, state, dtype, heads, key_dim, value_dim, ones=False):
    """What ``kernels.state_scan`` needs to run this step in chunks, or None where it walks token by token."""
    items = ctx.slots.numel()
    if dtype != torch.bfloat16 or ctx.tokens - items < CHUNKS_FROM:
        return None
    workspace, slots, size = ctx.workspace, state.shape[0], kernels.STATE_CHUNK
    # (the scratch is asked for at its largest, so that it never moves under recorded launches)
    most = workspace.max_rows // size + slots
    index = ctx.shared_calls.get("state_pieces")
    if index is None:
        # once per step, for all layers
        index = (workspace.flat("state_piece_cu", most + 1, torch.int32),
                 workspace.flat("state_item_first", slots + 1, torch.int32), ctx.tokens // size + items)
        kernels.scan_pieces(ctx.cu_tokens, items, size, index[2], index[0], index[1])
        ctx.shared_calls["state_pieces"] = index
    records, totals = kernels.state_chunk_floats(most, heads, key_dim, value_dim, ones)
    name = f"{heads}x{key_dim}x{value_dim}{'+1' if ones else ''}"
    return index + (workspace.flat("state_records_" + name, records, torch.float32),
                    workspace.flat("state_totals_" + name, totals, torch.float32))


def _check_key_dim(dim):
    if not 0 < dim <= 256:
        raise ValueError(f"key head size {dim} must lie in 1..256")


def _check_taps(taps):
    if not 1 <= taps <= 64:
        raise ValueError(f"taps {taps} must lie in 1..64")


@register_mixer("channel_delta")
class ChannelDelta(CoreMixer):
    """The gated delta rule with a decay per key channel.  With ``h`` the layer's input and ``conv`` a causal
    convolution per channel over ``taps`` inputs (no bias) followed by silu:

        q = unit(conv(W_q h)) key_dim^(-1/2),  k = unit(conv(W_k h))     (key_heads x key_dim)
        v = conv(W_v h)                                                  (heads x value_dim)
        beta = sigmoid(W_b h),  g = exp(-exp(A) softplus(W_a2 (W_a1 h) + b))     (heads;  heads x key_dim)
        S' = diag(g) S,  S = S' + k (beta (v - S'^T k))^T,  o = S^T q            (per head)
        out = W_o (rms_norm_per_head(o) * w_norm * sigmoid(W_g2 (W_g1 h)))

    ``unit(x) = x / sqrt(sum(x^2) + 1e-6)`` per head; head ``h`` reads key head ``h // (heads / key_heads)``.  The
    slot keeps S and the convolution's last ``taps - 1`` inputs, both zero at the start.  One packed product gives
    ``[q | k | v | low-rank decay | low-rank gate | beta]`` in float."""

    def __init__(self, width: int, dtype, heads: int, key_heads: int, key_dim: int, value_dim: int, taps: int,
                 decay_rank: int, gate_rank: int, norm_eps: float, ride: int = 0):
        if heads % key_heads:
            raise ValueError(f"heads ({heads}) must be a multiple of key_heads ({key_heads})")
        _check_key_dim(key_dim)
        _check_taps(taps)
        self.heads, self.key_heads = heads, key_heads
        self.key_dim, self.value_dim = key_dim, value_dim
        self.taps = taps
        self.decay_rank, self.gate_rank = decay_rank, gate_rank
        self.norm_eps = float(norm_eps)
        self.key_cols, self.value_cols = key_heads * key_dim, heads * value_dim
        self.channels = 2 * self.key_cols + self.value_cols
        self.history = heads * value_dim * key_dim
        super().__init__(width, dtype, self.channels + decay_rank + gate_rank + heads, self.value_cols, ride)

    def core_parameters(self):
        return {
            "conv.weight": ParamSpec((self.channels, self.taps), VECTOR),
            "decay.weight": ParamSpec((self.heads * self.key_dim, self.decay_rank), MATRIX),
            "decay.bias": ParamSpec((self.heads * self.key_dim,), VECTOR),
            "decay.log": ParamSpec((self.heads,), VECTOR),
            "gate.weight": ParamSpec((self.value_cols, self.gate_rank), MATRIX),
            "norm.gamma": ParamSpec((self.value_dim,), VECTOR),
        }

    def bind_core(self, tensors, device):
        self.conv_weight = tensors["conv.weight"].t().contiguous()
        self.decay_weight = tensors["decay.weight"].unsqueeze(0)
        # equal sizes: both low-rank products as one block-diagonal one
        self.low_weights = None
        if self.decay_rank == self.gate_rank and self.heads * self.key_dim == self.value_cols:
            self.low_weights = torch.stack([tensors["decay.weight"], tensors["gate.weight"]]).contiguous()
        self.decay_bias = tensors["decay.bias"]
        self.decay_log = tensors["decay.log"]
        self.gate_weight = tensors["gate.weight"].unsqueeze(0)
        self.norm_gamma = tensors["norm.gamma"]

    def cache_spec(self):
        return SlotStateSpec((_slot_floats(self.history, (self.taps - 1) * self.channels),), torch.float32)

    def core(self, proj, col, out, ctx, cache):
        tokens, workspace = ctx.tokens, ctx.workspace
        heads, dk, dv = self.heads, self.key_dim, self.value_dim
        low_col = col + self.channels
        gate_col = low_col + self.decay_rank
        decays = heads * dk
        both, raw_decay, gate = workspace.column_views("delta_low", decays + self.value_cols, torch.float32, tokens,
                                                       (decays, self.value_cols))
        if self.low_weights is not None:
            kernels.block_linear(proj[:, low_col:gate_col + self.gate_rank], self.decay_rank, self.low_weights, None,
                                 both, decays)
        else:
            kernels.block_linear(proj[:, low_col:gate_col], 0, self.decay_weight, None, raw_decay, decays)
            kernels.block_linear(proj[:, gate_col:gate_col + self.gate_rank], 0, self.gate_weight, None, gate,
                                 self.value_cols)
        mixed, q, k, v = workspace.column_views("delta_inputs", self.channels, torch.float32, tokens,
                                                (self.key_cols, self.key_cols, self.value_cols))
        decay = workspace.first_rows("delta_decay", heads * dk, torch.float32, tokens)
        take = workspace.first_rows("delta_take", heads, torch.float32, tokens)
        kernels.state_prepare(
            proj, col, self.conv_weight, None, cache.state, self.history, mixed, "delta", decay, take,
            self.decay_log, self.decay_bias, gate_col + self.gate_rank, ctx.tok_item, ctx.cu_tokens, ctx.slots,
            z=raw_decay, per_head=dk, unit_heads=2 * self.key_heads, head=dk, scale_heads=self.key_heads,
            q_scale=dk ** -0.5)
        o = workspace.first_rows("delta_out", self.value_cols, torch.float32, tokens)
        kernels.state_scan(q, k, v, decay, take, cache.state, o, ctx.cu_tokens, ctx.slots, "delta", heads,
                           self.key_heads, dk, dv, longest=1 if ctx.decode_only else 0,
                           raw=proj[:, col:col + self.channels], taps=self.taps, history=self.history)
        kernels.state_output(o, heads, dv, self.norm_gamma, self.norm_eps, heads, out, behind=gate)


@register_mixer("matrix_memory")
class MatrixMemory(CoreMixer):
    """A matrix memory with exponential gates (the mLSTM of xLSTM).  With ``h`` the layer's input:

        q = W_q h key_dim^(-1/2),  k = W_k h,  v = W_v h              (heads x key_dim / value_dim)
        i = c tanh((W_i h + b_i) / c),  f = log sigmoid(c tanh((W_f h + b_f) / c))        (per head)
        m_t = max(f + m_(t-1), i)
        S_t = e^(f + m_(t-1) - m_t) S_(t-1) + e^(i - m_t) k v^T,   n_t likewise with k alone
        o = S_t^T q / (max(|n_t . q|, e^(-m_t)) + 1e-6)
        out = W_o (rms_norm_per_head(o) * w_norm * sigmoid(W_g h))

    ``n`` is one more column of S, whose value is always one.  The slot keeps S with that column and m, all
    zero at the start.  One packed product gives ``[q | k | v | gate | i | f]`` in float."""

    def __init__(self, width: int, dtype, heads: int, key_dim: int, value_dim: int, gate_cap: float,
                 norm_eps: float, ride: int = 0):
        _check_key_dim(key_dim)
        if not gate_cap > 0:
            raise ValueError("the gates' cap must be positive")
        self.heads, self.key_dim, self.value_dim = heads, key_dim, value_dim
        self.gate_cap = float(gate_cap)
        self.norm_eps = float(norm_eps)
        self.key_cols, self.value_cols = heads * key_dim, heads * value_dim
        self.maxima = heads * (value_dim + 1) * key_dim
        super().__init__(width, dtype, 2 * self.key_cols + 2 * self.value_cols + 2 * heads, self.value_cols, ride)

    def core_parameters(self):
        return {
            "input_gate.bias": ParamSpec((self.heads,), VECTOR),
            "forget_gate.bias": ParamSpec((self.heads,), VECTOR),
            "norm.gamma": ParamSpec((self.value_cols,), VECTOR),
        }

    def bind_core(self, tensors, device):
        self.input_bias = tensors["input_gate.bias"]
        self.forget_bias = tensors["forget_gate.bias"]
        self.norm_gamma = tensors["norm.gamma"]

    def cache_spec(self):
        return SlotStateSpec((_slot_floats(self.maxima, self.heads),), torch.float32)

    def core(self, proj, col, out, ctx, cache):
        tokens, workspace = ctx.tokens, ctx.workspace
        heads, dk, dv = self.heads, self.key_dim, self.value_dim
        k_col = col + self.key_cols
        v_col = k_col + self.key_cols
        gate_col = v_col + self.value_cols
        i_col = gate_col + self.value_cols
        decay = workspace.first_rows("memory_decay", heads, torch.float32, tokens)
        take = workspace.first_rows("memory_take", heads, torch.float32, tokens)
        floor = workspace.first_rows("memory_floor", heads, torch.float32, tokens)
        kernels.memory_gates(proj, i_col, i_col + heads, self.input_bias, self.forget_bias, self.gate_cap,
                             cache.state, self.maxima, decay, take, floor, ctx.cu_tokens, ctx.slots)
        o = workspace.first_rows("memory_out", heads * (dv + 1), torch.float32, tokens)
        kernels.state_scan(proj[:, col:k_col], proj[:, k_col:v_col], proj[:, v_col:gate_col], decay, take, cache.state,
                           o, ctx.cu_tokens, ctx.slots, "decayed", heads, heads, dk, dv, ones=True,
                           q_scale=dk ** -0.5, longest=1 if ctx.decode_only else 0,
                           chunks=_chunks(ctx, cache.state, self.dtype, heads, dk, dv, ones=True))
        kernels.state_output(o, heads, dv, self.norm_gamma, self.norm_eps, heads, out, floor=floor,
                             behind=proj[:, gate_col:i_col])


@register_mixer("head_state_space")
class HeadStateSpace(CoreMixer):
    """A state-space mixer with one decay per head (Mamba-2).  With ``h`` the layer's input:

        [z | x | B | C | dt] = W_in h      (heads x value_dim twice, groups x states twice, heads)
        x, B, C pass a causal convolution per channel over ``taps`` inputs, with bias, and silu
        dt = softplus(dt + b_dt),   S_t = exp(-exp(A) dt) S_(t-1) + dt B x^T     (per head, S: states x value_dim)
        y = S_t^T C + D x
        out = W_o (rms_norm(y * silu(z)) * w_norm)       the norm over ``norm_groups`` equal runs of columns

    Head ``h`` reads group ``h // (heads / groups)`` of B and C.  The slot keeps S and the convolution's last
    ``taps - 1`` inputs, both zero at the start.  ``out_scale`` multiplies the result (folded into ``w_norm``)."""

    def __init__(self, width: int, dtype, heads: int, value_dim: int, states: int, groups: int, taps: int,
                 norm_groups: int, norm_eps: float, out_scale: float = 1.0, ride: int = 0):
        if heads % groups:
            raise ValueError(f"heads ({heads}) must be a multiple of groups ({groups})")
        if heads * value_dim % norm_groups:
            raise ValueError(f"{heads * value_dim} columns do not split into {norm_groups} equal runs")
        _check_key_dim(states)
        _check_taps(taps)
        self.heads, self.value_dim = heads, value_dim
        self.states, self.groups = states, groups
        self.taps = taps
        self.norm_groups = norm_groups
        self.norm_eps = float(norm_eps)
        self.out_scale = float(out_scale)
        self.inner = heads * value_dim
        self.channels = self.inner + 2 * groups * states
        self.history = self.inner * states
        super().__init__(width, dtype, 2 * self.inner + 2 * groups * states + heads, self.inner, ride)

    def core_parameters(self):
        return {
            "conv.weight": ParamSpec((self.channels, self.taps), VECTOR),
            "conv.bias": ParamSpec((self.channels,), VECTOR),
            "step.bias": ParamSpec((self.heads,), VECTOR),
            "decay.log": ParamSpec((self.heads,), VECTOR),
            "skip": ParamSpec((self.heads,), VECTOR),
            "norm.gamma": ParamSpec((self.inner,), VECTOR),
        }

    def bind_core(self, tensors, device):
        self.conv_weight = tensors["conv.weight"].t().contiguous()
        self.conv_bias = tensors["conv.bias"]
        self.step_bias = tensors["step.bias"]
        self.decay_log = tensors["decay.log"]
        self.skip = tensors["skip"]
        gamma = tensors["norm.gamma"]
        self.norm_gamma = gamma if self.out_scale == 1.0 else gamma * self.out_scale

    def cache_spec(self):
        return SlotStateSpec((_slot_floats(self.history, (self.taps - 1) * self.channels),), torch.float32)

    def core(self, proj, col, out, ctx, cache):
        tokens, workspace = ctx.tokens, ctx.workspace
        heads, dv, states, inner = self.heads, self.value_dim, self.states, self.inner
        x_col = col + inner
        step_col = x_col + self.channels
        mixed, x, b, c = workspace.column_views("space_inputs", self.channels, torch.float32, tokens,
                                                (inner, self.groups * states, self.groups * states))
        decay = workspace.first_rows("space_decay", heads, torch.float32, tokens)
        take = workspace.first_rows("space_take", heads, torch.float32, tokens)
        kernels.state_prepare(proj, x_col, self.conv_weight, self.conv_bias, cache.state, self.history, mixed,
                              "decayed", decay, take, self.decay_log, self.step_bias, step_col, ctx.tok_item,
                              ctx.cu_tokens, ctx.slots)
        o = workspace.first_rows("space_out", inner, torch.float32, tokens)
        kernels.state_scan(c, b, x, decay, take, cache.state, o, ctx.cu_tokens, ctx.slots, "decayed", heads,
                           self.groups, states, dv, longest=1 if ctx.decode_only else 0,
                           raw=proj[:, x_col:step_col], taps=self.taps, history=self.history,
                           chunks=_chunks(ctx, cache.state, self.dtype, heads, states, dv))
        kernels.state_output(o, heads, dv, self.norm_gamma, self.norm_eps, self.norm_groups, out, skip=self.skip,
                             u=x, before=proj[:, col:x_col])
