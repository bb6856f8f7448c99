"""RWKV-style time mixing: linear attention whose projections read mixes of a token's input with the one before it, with a
decay per token, head and key channel and a bonus for the own token, and a fixed-size recurrent state per request.

    mix_s = x + (x' - x) * mu_s            s = r, k, v, g, w;  x': the input of the token before (zeros before the first)
    r, k, v = W_s mix_s (heads x D),  gate = silu(W_g mix_g)
    decay  = exp(-exp(W_w2 tanh(W_w1 mix_w) + w0))                   per head and key channel
    o = (S + diag(u) k v^T)^T r,   S <- diag(decay) S + k v^T        (S: [D, D] per head, fp32)
    out = W_o (o / rms(o) per head * norm * gate)

The state (S and the last input row) lives in the runner's per-request state slots, the mechanism of the other recurrent
mixers; the mixes are formed in fp32 in one launch, decays, the recurrence and the output norm are fp32.
Kernels: ops/csrc/token_shift.hip (the mixes), ops/csrc/linear_attention.hip (the recurrence with its bonus, decays, norm
and gate; shared with the other decaying memories).
"""
from __future__ import annotations

import torch
import torch.nn as nn

from .. import ops
from ..forward_context import get_forward_context
from ..models.mamba import StateSpaceLayer
from ..parallel.state import get_tensor_model_parallel_world_size
from .hyper_connections import _fp32_param
from .linear import RowParallelLinear, row_padding, set_weight_attrs
from .linear_attention import first_long_sequence

MIXES = ("r", "k", "v", "g", "w")


def _padded(shape: tuple, dtype: torch.dtype) -> nn.Parameter:
    """A zero-filled parameter that may be larger than its checkpoint tensor (aligned rows and columns)."""
    p = nn.Parameter(torch.zeros(shape, dtype=dtype), requires_grad=False)

    def load(param, t, *_):
        param.data[: t.shape[0], : t.shape[1]].copy_(t)
    set_weight_attrs(p, {"weight_loader": load})
    return p


class WKVMixer(StateSpaceLayer):
    def __init__(self, hidden_size: int, num_heads: int, head_dim: int, decay_rank: int, eps: float, quant_config=None,
                 prefix: str = ""):
        super().__init__()
        if get_tensor_model_parallel_world_size() > 1:
            raise NotImplementedError("wkv layers run with tensor_parallel_size=1")
        H, D, W = int(num_heads), int(head_dim), int(hidden_size)
        self.num_heads, self.head_dim, self.hidden_size, self.eps = H, D, W, float(eps)
        self.layer_name = prefix
        dtype = torch.get_default_dtype()
        self.conv_dtype = dtype
        self.state_dtypes = (dtype, torch.float32)
        self.mu = nn.Parameter(torch.zeros((len(MIXES), W), dtype=torch.float32), requires_grad=False)
        # r | k | v | g, each over a mix of its own
        self.in_weight = nn.Parameter(torch.zeros((4, H * D, W), dtype=dtype), requires_grad=False)

        def load_part(param, t, shard_id):
            param.data[shard_id].copy_(t.reshape(param.shape[1:]))
        for p in (self.mu, self.in_weight):
            set_weight_attrs(p, {"weight_loader": load_part})
        rank = int(decay_rank)
        rank += row_padding(rank)
        self.decay_down, self.decay_up = _padded((rank, W), dtype), _padded((H * D, rank), dtype)
        self.decay_bias = _fp32_param((H * D,), 0.0)
        self.bonus = _fp32_param((H * D,), 0.0)
        self.norm_weight = _fp32_param((H * D,))
        self.o_proj = RowParallelLinear(H * D, W, bias=False, quant_config=quant_config, prefix=f"{prefix}.o_proj")

    def state_shapes(self) -> tuple:
        return ((1, self.hidden_size), (self.num_heads, self.head_dim, self.head_dim))

    def forward(self, x: torch.Tensor) -> torch.Tensor:
        md = get_forward_context().attn_metadata
        H, D = self.num_heads, self.head_dim
        if md is None or self.ssm_state is None:          # memory-profiling run: the projections carry the footprint
            p = ops.grouped_linear(x.unsqueeze(0).expand(4, *x.shape).contiguous(), self.in_weight)
            return self.o_proj(p[0] * p[3])
        T, n = x.shape[0], md.num_actual_tokens
        S = md.num_decode_seqs + md.num_prefill_seqs
        qsl, lens, tbl = md.query_start_loc[:S + 1], md.seq_lens[:S], self.slot_table(md)[:S]
        mix = ops.token_shift_mix(x[:n], self.mu, self.conv_state, qsl, lens, tbl, md.max_query_len)
        r, k, v, gate = ops.grouped_linear(mix[:4], self.in_weight)
        z = ops.linear(ops.activation(ops.linear(mix[4], self.decay_down), "tanh"), self.decay_up)
        out = ops.linear_attention(r, k, v, gate, self.norm_weight, self.ssm_state, qsl, lens, tbl, H, D, D, self.eps,
                                   md.max_query_len, z=z, z_bias=self.decay_bias, decay_exp=True, bonus=self.bonus,
                                   first_long_seq=first_long_sequence(md))
        if n < T:
            out = torch.cat([out, out.new_zeros((T - n, out.shape[1]))], dim=0)
        return self.o_proj(out)
