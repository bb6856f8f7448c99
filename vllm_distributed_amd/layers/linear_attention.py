"""Linear-attention mixers with decay and a fixed-size recurrent state per request.

    q, k = W_q x, W_k x (heads x D), v = W_v x (heads x Dv); the first ``rot_dims`` values of every q / k head rotated
           (value i paired with i + rot_dims / 2, fp32 angles); q times q_scale, k times k_scale
    decay  one number per head (``decay``: a list; retention), or per token, head and key channel
           sigmoid(W_a2 (W_a1 x) + b)^(1 / tau) (``decay_rank``, ``tau``; gated linear attention)
    S <- diag(decay) S + k v^T;  o = S^T q          (S: [D, Dv] per head, fp32)
    out = W_o ((o / rms(o) per head [* norm]) * silu(W_g x))

One GEMM produces everything that reads x.  The state lives in the runner's per-request state slots, the mechanism of
the other recurrent mixers; rotation, scaling, decays, the recurrence and the output norm are fp32
(ops/csrc/linear_attention.hip).
"""
from __future__ import annotations

import math
from typing import Optional, Sequence

import torch
import torch.nn as nn

from .. import ops
from ..forward_context import get_forward_context
from ..models.mamba import StateSpaceLayer
from ..parallel.state import get_tensor_model_parallel_world_size
from .hyper_connections import _fp32_param
from .linear import MergedColumnParallelLinear, ReplicatedLinear, RowParallelLinear, row_padding, zero_tail_rows
from .rotary import half_split_cos_sin

MIN_LOG_DECAY = -1e4              # a decay of zero, kept finite


class DecayedLinearAttention(StateSpaceLayer):
    def __init__(self, hidden_size: int, num_heads: int, head_dim: int, v_head_dim: int, eps: float, *,
                 decay: Optional[Sequence[float]] = None, decay_rank: Optional[int] = None, tau: float = 1.0,
                 out_norm: bool = False, rot_dims: int = 0, rot_base: float = 10000.0,
                 rot_scaling: Optional[dict] = None, q_scale: float = 1.0, k_scale: float = 1.0, quant_config=None,
                 prefix: str = ""):
        super().__init__()
        if get_tensor_model_parallel_world_size() > 1:
            raise NotImplementedError("linear-attention layers run with tensor_parallel_size=1")
        H, D, Dv = int(num_heads), int(head_dim), int(v_head_dim)
        if (decay is None) == (decay_rank is None):
            raise ValueError(f"{prefix}: either a decay per head or the rank of a decay projection")
        if decay is not None and (len(decay) != H or not all(0.0 <= float(d) <= 1.0 for d in decay)):
            raise ValueError(f"{prefix}: {len(decay)} decays for {H} heads, or one outside [0, 1]")
        if rot_dims % 2 or rot_dims > D:
            raise ValueError(f"{prefix}: {rot_dims} rotated dimensions do not fit an even part of {D}")
        self.num_heads, self.head_dim, self.v_head_dim = H, D, Dv
        self.eps, self.tau = float(eps), float(tau)
        self.q_scale, self.k_scale = float(q_scale), float(k_scale)
        self.rot_dims, self.rot_base, self.rot_scaling = int(rot_dims), float(rot_base), rot_scaling
        self.layer_name = prefix
        self.conv_dtype = torch.float32
        self.state_dtypes = (torch.float32, torch.float32)
        self.decay_rank = int(decay_rank) if decay_rank is not None else None
        # q | k | v | output gate (| decay low-rank), rows padded for aligned consumers
        self.sizes = [H * D, H * D, H * Dv, H * Dv] + ([self.decay_rank] if self.decay_rank is not None else [])
        pad = row_padding(sum(self.sizes))
        self.in_proj = MergedColumnParallelLinear(hidden_size, self.sizes + ([pad] if pad else []), bias=False,
                                                  quant_config=quant_config, prefix=f"{prefix}.in_proj")
        zero_tail_rows(self.in_proj, pad)
        if self.decay_rank is not None:
            self.decay_up = ReplicatedLinear(self.decay_rank, H * D, bias=False, prefix=f"{prefix}.decay_up")
            self.decay_bias = _fp32_param((H * D,), 0.0)
            self.log_decay = None
        else:
            self.register_buffer("log_decay", torch.tensor(
                [max(math.log(float(d)), MIN_LOG_DECAY) if float(d) > 0 else MIN_LOG_DECAY for d in decay],
                dtype=torch.float32), persistent=False)
        self.norm_weight = _fp32_param((Dv,)) if out_norm else None
        self.o_proj = RowParallelLinear(H * Dv, hidden_size, bias=False, quant_config=quant_config,
                                        prefix=f"{prefix}.o_proj")
        self._cos_sin: Optional[torch.Tensor] = None

    def state_shapes(self) -> tuple:
        # no convolution part: a 16-byte placeholder
        return ((1, 4), (self.num_heads, self.v_head_dim, self.head_dim))

    def _table(self, device) -> Optional[torch.Tensor]:
        if self.rot_dims == 0:
            return None
        if self._cos_sin is None or self._cos_sin.device != device:
            self._cos_sin = half_split_cos_sin(self.max_model_len + 1, self.rot_dims, self.rot_base, self.rot_scaling,
                                               device)
        return self._cos_sin

    def forward(self, x: torch.Tensor, positions: torch.Tensor) -> torch.Tensor:
        md = get_forward_context().attn_metadata
        H, D, Dv = self.num_heads, self.head_dim, self.v_head_dim
        p = self.in_proj(x)
        nk, nv = H * D, H * Dv
        gate0 = 2 * nk + nv
        z = None
        if self.decay_rank is not None:
            z = self.decay_up(p[:, gate0 + nv: gate0 + nv + self.decay_rank])
        if md is None or self.ssm_state is None:          # memory-profiling run
            o = p[:, 2 * nk: gate0] * p[:, gate0: gate0 + nv]
            return self.o_proj((o if z is None else o + z[:, :1]).contiguous())
        T, n = p.shape[0], md.num_actual_tokens
        S = md.num_decode_seqs + md.num_prefill_seqs
        out = ops.linear_attention(
            p[:n, :nk], p[:n, nk: 2 * nk], p[:n, 2 * nk: gate0], p[:n, gate0: gate0 + nv], self.norm_weight,
            self.ssm_state, md.query_start_loc[:S + 1], md.seq_lens[:S], self.slot_table(md)[:S], H, D, Dv, self.eps,
            md.max_query_len, log_decay=self.log_decay, z=z[:n] if z is not None else None,
            z_bias=self.decay_bias if z is not None else None, tau=self.tau, cos_sin=self._table(p.device),
            positions=positions[:n], rot=self.rot_dims, q_scale=self.q_scale, k_scale=self.k_scale,
            first_long_seq=first_long_sequence(md))
        if n < T:
            out = torch.cat([out, out.new_zeros((T - n, out.shape[1]))], dim=0)
        return self.o_proj(out)


def first_long_sequence(md) -> int:
    """Sequences of a step before this one bring few tokens each (the step's decode group)."""
    return md.num_decode_seqs if md.max_decode_query_len <= ops.RECURRENT_STEP_TOKENS else 0
