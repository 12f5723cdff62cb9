"""Matrix memory (the mLSTM cell of xLSTM): a linear-attention layer with exponential input gates, log-sigmoid forget gates, a
normaliser vector beside the state and a running maximum that keeps both in range:

    q = W_q h * D^-1/2, k = W_k h   (H heads of D),   v = W_v h   (H heads of Dv)
    i = cap tanh((W_i h + b_i) / cap),   f = logsigmoid(cap tanh((W_f h + b_f) / cap))        one number per head
    m' = max(f + m, i)  (m from 0);   S <- e^(f+m-m') S + e^(i-m') k v^T;   n <- e^(f+m-m') n + e^(i-m') k
    o = S^T q / (max(|n . q|, e^(-m')) + 1e-6)
    y = W_o [ o_h / rms(o_h) * w_h * sigmoid(W_g h)_h ]_h

Serving state per sequence (one slot of the engine's state manager): S, n and m in f32. One GEMM for q | k | v | gate | i | f, the
recurrence with its gates (mix_ops.gated_scan), the division, norm and gate (mix_ops.scaled_head_norm_gate) and the output
GEMM. A ragged step carries any number of new tokens per sequence; a sequence without context starts from zeros without the
slot being cleared.
"""
from __future__ import annotations

import torch
from torch import nn

from .. import mix_ops
from ..utils.context import get_context
from .linear import MergedColumnParallelLinear, RowParallelLinear
from .tp import tp_size


class MatrixMemory(nn.Module):
    uses_state_slots = True

    def __init__(self, width: int, heads: int, dim: int, vdim: int, gate_cap: float, norm_eps: float = 1e-6):
        super().__init__()
        assert tp_size() == 1, "the matrix memory is not sharded: run it with tensor_parallel_size 1"
        assert heads >= 1 and dim >= 1 and vdim >= 1 and gate_cap > 0
        self.H, self.D, self.Dv, self.cap, self.norm_eps = heads, dim, vdim, float(gate_cap), float(norm_eps)
        self.sizes = [heads * dim, heads * dim, heads * vdim, heads * vdim, heads, heads]      # q | k | v | gate | i | f
        self.offsets = [sum(self.sizes[:j]) for j in range(len(self.sizes) + 1)]
        f32 = dict(dtype=torch.float32)
        self.in_proj = MergedColumnParallelLinear(width, self.sizes, bias=False)
        self.o_proj = RowParallelLinear(heads * vdim, width, bias=False)
        self.i_bias = nn.Parameter(torch.zeros(heads, **f32))
        self.f_bias = nn.Parameter(torch.zeros(heads, **f32))
        self.out_norm_weight = nn.Parameter(torch.ones(heads * vdim, **f32))
        self.state = self.norm_state = self.max_state = torch.tensor([])

    # -- cache protocol of the model runner
    @property
    def _copies(self) -> int:
        return mix_ops.scan_copies(self.Dv)

    def cache_bytes(self, block_size: int, act_bytes: int) -> tuple[int, int]:
        """(bytes per cache page, bytes per state slot)."""
        return 0, self.H * (self.D * self.Dv + self.D + self._copies) * 4

    def bind_cache(self, num_blocks: int, block_size: int, num_slots: int, device, dtype) -> None:
        kw = dict(dtype=torch.float32, device=device)
        self.state = torch.zeros(num_slots, self.H, self.D, self.Dv, **kw)
        self.norm_state = torch.zeros(num_slots, self.H, self.D, **kw)
        self.max_state = torch.zeros(num_slots, self.H, self._copies, **kw)

    def forward(self, h: torch.Tensor) -> torch.Tensor:
        step = get_context().ragged
        proj = self.in_proj(h)
        q, k, v, gate, i, f = (proj[:, a:b] for a, b in zip(self.offsets, self.offsets[1:]))
        o, den = mix_ops.gated_scan(mix_ops.SCAN_LOG_GATES, q, k, v, i, self.i_bias, self.f_bias, step, self.state, self.H, self.H,
                                    self.D, self.Dv, a2=f, q_scale=self.D ** -0.5, cap=self.cap, norm_state=self.norm_state,
                                    max_state=self.max_state)
        y = mix_ops.scaled_head_norm_gate(o, gate, self.out_norm_weight, self.norm_eps, h.dtype, "sigmoid", den=den)
        return self.o_proj(y)
