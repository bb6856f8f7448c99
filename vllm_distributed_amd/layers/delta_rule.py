"""Gated delta-rule mixer (a linear-attention layer with a fixed-size recurrent state per request), with one decay per
head and key channel or one per head.

    q, k, v = silu(short causal convolution over time of the projections), per channel
    q, k  <- unit vectors per head (q also times dim^-1/2);  head h reads q / k head h // (heads / kv_heads)
    beta   = sigmoid(W_b x);   decay = exp(-exp(A_log[h]) * softplus(W_a2 (W_a1 x) + dt_bias))   [heads, dim]
    S <- diag(decay) S;  u = beta (v - S^T k);  S <- S + k u^T;  o = S^T q      (S: [dim, vdim] per head, fp32)
    out = W_o (o / rms(o) * norm * sigmoid(W_g2 (W_g1 x)))

``decay_rank`` and ``gate_rank`` None: one decay per head and a full-rank SiLU gate,
    decay = exp(-exp(A_log[h]) * softplus(W_a x + dt_bias))   [heads];   out = W_o (o / rms(o) * norm * silu(W_g x))

The state (S and the convolution's last taps - 1 inputs) lives in the runner's per-request state slots, the
mechanism of the other recurrent mixers; everything the recurrence consumes besides the projections is fp32.
Kernels: ops/csrc/delta_rule.hip (the recurrence, norms, decays, gates, output norm), ops/csrc/mamba.hip (the
convolution, shared with the state-space mixers).
"""
from __future__ import annotations

from typing import Optional

import torch
import torch.nn as nn
import torch.nn.functional as F

from .. import ops
from ..forward_context import get_forward_context
from ..models.mamba import StateSpaceLayer
from ..parallel.state import get_tensor_model_parallel_world_size
from .hyper_connections import _fp32_param
from .linear import (MergedColumnParallelLinear, ReplicatedLinear, RowParallelLinear, row_padding, set_weight_attrs,
                     zero_tail_rows)
from .linear_attention import first_long_sequence


class GatedDeltaRule(StateSpaceLayer):
    def __init__(self, hidden_size: int, num_heads: int, num_kv_heads: int, head_dim: int, v_head_dim: int,
                 conv_taps: int, decay_rank: Optional[int], gate_rank: Optional[int], eps: float, quant_config=None,
                 prefix: str = ""):
        super().__init__()
        if get_tensor_model_parallel_world_size() > 1:
            raise NotImplementedError("delta-rule layers run with tensor_parallel_size=1")
        if num_heads % num_kv_heads:
            raise ValueError(f"{num_heads} heads do not divide into {num_kv_heads} query/key heads")
        H, G, D, Dv = num_heads, num_kv_heads, head_dim, v_head_dim
        self.num_heads, self.num_kv_heads, self.head_dim, self.v_head_dim = H, G, D, Dv
        self.taps, self.eps = int(conv_taps), float(eps)
        if (decay_rank is None) != (gate_rank is None):
            raise ValueError(f"{prefix}: decays per key channel come with a low-rank gate, decays per head with a full one")
        self.per_head = decay_rank is None
        if not self.per_head:
            self.decay_rank, self.gate_rank = int(decay_rank), int(gate_rank)
        self.layer_name = prefix
        dtype = torch.get_default_dtype()
        self.conv_dtype = dtype
        self.state_dtypes = (dtype, torch.float32)
        self.conv_dim = 2 * G * D + H * Dv
        # one GEMM for everything that reads x: q | k | v | decay low-rank | gate low-rank | beta, or, with decays per
        # head, q | k | v | gate | beta | decay (rows padded for aligned consumers)
        self.sizes = [G * D, G * D, H * Dv] + ([H * Dv, H, H] if self.per_head
                                               else [self.decay_rank, self.gate_rank, H])
        pad = row_padding(sum(self.sizes)) if self.per_head else 0
        self.in_proj = MergedColumnParallelLinear(hidden_size, self.sizes + ([pad] if pad else []), bias=False,
                                                  quant_config=quant_config, prefix=f"{prefix}.in_proj")
        zero_tail_rows(self.in_proj, pad)
        if not self.per_head:
            self.decay_up = ReplicatedLinear(self.decay_rank, H * D, bias=False, prefix=f"{prefix}.decay_up")
            self.gate_up = ReplicatedLinear(self.gate_rank, H * Dv, bias=False, prefix=f"{prefix}.gate_up")
        self.o_proj = RowParallelLinear(H * Dv, hidden_size, bias=False, quant_config=quant_config,
                                        prefix=f"{prefix}.o_proj")
        self.conv_weight = nn.Parameter(torch.zeros((self.conv_dim, self.taps), dtype=dtype), requires_grad=False)
        offs = [0, G * D, 2 * G * D]

        def load_conv(param, t, shard_id=None):
            if shard_id is None:
                param.data.copy_(t.reshape(param.shape))
            else:
                t = t.reshape(t.shape[0], -1)
                param.data[offs[shard_id]: offs[shard_id] + t.shape[0]].copy_(t)
        set_weight_attrs(self.conv_weight, {"weight_loader": load_conv})
        self.A_log = _fp32_param((H,), 0.0)
        self.dt_bias = _fp32_param((H if self.per_head else H * D,), 0.0)
        self.norm_weight = _fp32_param((Dv,))

    def state_shapes(self) -> tuple:
        return ((self.conv_dim, max(self.taps - 1, 1)), (self.num_heads, self.v_head_dim, self.head_dim))

    def forward(self, x: torch.Tensor) -> torch.Tensor:
        md = get_forward_context().attn_metadata
        H, G, D, Dv, C = self.num_heads, self.num_kv_heads, self.head_dim, self.v_head_dim, self.conv_dim
        p = self.in_proj(x)
        if self.per_head:
            gate = p[:, C: C + H * Dv]
            b_raw, a_raw = p[:, C + H * Dv: C + H * Dv + H], p[:, C + H * Dv + H: C + H * Dv + 2 * H]
        else:
            ra, rg = self.decay_rank, self.gate_rank
            a_raw = self.decay_up(p[:, C: C + ra])
            gate = self.gate_up(p[:, C + ra: C + ra + rg])
            b_raw = p[:, C + ra + rg:]
        if md is None or self.conv_state is None:          # memory-profiling run
            return self.o_proj((gate * p[:, 2 * G * D: C]).contiguous() + a_raw[:, :1])
        T, n = p.shape[0], md.num_actual_tokens
        S = md.num_decode_seqs + md.num_prefill_seqs
        tbl = self.slot_table(md)[:S]
        qsl, lens = md.query_start_loc[:S + 1], md.seq_lens[:S]
        if self.taps == 1:                                 # no earlier inputs, nothing carried
            xc = F.silu(p[:n, :C].float() * self.conv_weight.float().view(1, -1)).to(p.dtype)
        else:
            xc = ops.causal_conv1d(p[:n, :C], self.conv_weight, None, self.conv_state, qsl, lens, tbl, md.max_query_len)
        args = (xc, a_raw[:n], b_raw[:n], gate[:n], self.A_log, self.dt_bias, self.norm_weight, self.ssm_state, qsl, lens,
                tbl, H, G, D, Dv, self.eps)
        if self.per_head:
            out = ops.gated_delta_rule_head(*args, md.max_query_len, first_long_sequence(md))
        else:
            out = ops.gated_delta_rule(*args)
        if n < T:
            out = torch.cat([out, out.new_zeros((T - n, out.shape[1]))], dim=0)
        return self.o_proj(out)
