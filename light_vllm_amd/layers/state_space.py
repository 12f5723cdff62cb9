"""State-space mixer of Mamba-2 (state-space duality): a scalar decay per head and token, keys and queries (B, C) shared by groups
of heads, a skip of the input and an output gated before it is normed:

    [z | x | B | C | dt] = W_in h        (inner = H * Dv | inner | G * N | G * N | H)
    x, B, C = silu(conv(x | B | C) + b)  (causal, one filter per channel)
    dt = softplus(dt + dt_bias);   S <- exp(-exp(A_log) dt) S + dt B x^T;   y = S^T C + D x          per head, B, C of its group
    out = W_o [ parts of (y * silu(z)), each divided by its own root mean square, times w ]

Serving state per sequence (one slot of the engine's state manager): S [H, N, Dv] in f32 and the last taps - 1 convolution
inputs. One GEMM in, the convolution (mix_ops.causal_conv), the recurrence (mix_ops.gated_scan), the gate and norm
(mix_ops.grouped_gate_norm), one GEMM out.
"""
from __future__ import annotations

import torch
from torch import nn

from .. import mix_ops
from ..utils.context import get_context
from .linear import ColumnParallelLinear, RowParallelLinear
from .tp import tp_size


class StateSpaceMixer(nn.Module):
    uses_state_slots = True

    def __init__(self, width: int, heads: int, vdim: int, state: int, groups: int, conv_taps: int, norm_groups: int = 1,
                 norm_eps: float = 1e-6):
        super().__init__()
        assert tp_size() == 1, "the state-space mixer is not sharded: run it with tensor_parallel_size 1"
        assert heads % groups == 0 and conv_taps >= 1 and (heads * vdim) % norm_groups == 0
        self.H, self.Dv, self.N, self.G, self.taps = heads, vdim, state, groups, conv_taps
        self.norm_groups, self.norm_eps = norm_groups, float(norm_eps)
        self.inner = heads * vdim
        self.channels = self.inner + 2 * groups * state                  # convolved: x | B | C
        f32 = dict(dtype=torch.float32)
        self.in_proj = ColumnParallelLinear(width, self.inner + self.channels + heads, bias=False)      # z | x | B | C | dt
        self.o_proj = RowParallelLinear(self.inner, width, bias=False)
        self.conv_weight = nn.Parameter(torch.zeros(self.channels, conv_taps, **f32))       # last column: current token
        self.conv_bias = nn.Parameter(torch.zeros(self.channels, **f32))
        self.dt_bias = nn.Parameter(torch.zeros(heads, **f32))
        self.A_log = nn.Parameter(torch.zeros(heads, **f32))
        self.skip = nn.Parameter(torch.zeros(heads, **f32))
        self.out_norm_weight = nn.Parameter(torch.ones(self.inner, **f32))
        self.conv_state = self.state = torch.tensor([])

    # -- cache protocol of the model runner
    def cache_bytes(self, block_size: int, act_bytes: int) -> tuple[int, int]:
        """(bytes per cache page, bytes per state slot)."""
        return 0, self.inner * self.N * 4 + max(self.taps - 1, 1) * self.channels * act_bytes

    def bind_cache(self, num_blocks: int, block_size: int, num_slots: int, device, dtype) -> None:
        self._conv_buf = torch.zeros(num_slots, max(self.taps - 1, 1), self.channels, dtype=dtype, device=device)
        self.conv_state = self._conv_buf[:, :self.taps - 1]      # taps == 1: an empty view that still has an address
        self.state = torch.zeros(num_slots, self.H, self.N, self.Dv, dtype=torch.float32, device=device)

    def forward(self, h: torch.Tensor) -> torch.Tensor:
        step = get_context().ragged
        proj = self.in_proj(h)
        z = proj[:, :self.inner]
        dt = proj[:, self.inner + self.channels:]
        u = mix_ops.causal_conv(proj[:, self.inner:self.inner + self.channels], self.conv_weight, self.conv_bias, self.conv_state,
                                step, silu=True)
        x, B, C = torch.split(u, [self.inner, self.G * self.N, self.G * self.N], dim=1)
        o = mix_ops.gated_scan(mix_ops.SCAN_STEP, C, B, x, dt, self.dt_bias, self.A_log, step, self.state, self.H, self.G, self.N,
                               self.Dv, p2=self.skip)
        y = mix_ops.grouped_gate_norm(o.view(-1, self.inner), z, self.out_norm_weight, self.norm_groups, self.norm_eps)
        return self.o_proj(y)
