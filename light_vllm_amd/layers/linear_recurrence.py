"""Recurrent block of Griffin: a real-gated linear recurrent unit (RG-LRU) behind a short convolution, beside a gelu branch
(Soham De et al., "Griffin: Mixing Gated Linear Recurrences with Local Attention for Efficient Language Models", 2024):

    y = gelu(W_y h + b_y)                       u = conv(W_x h + b_x) + b_conv      (causal, one filter per channel)
    r, i = sigmoid(A_b u_b + c_b), sigmoid(B_b u_b + d_b)                          for each of `blocks` equal parts u_b of u
    log a = -C r softplus(lam),   S <- a S + sqrt(1 - a^2) i u,   out = W_o (S y)

C = 8 is the block's constant (`decay_scale`); the state starts at zero, also for the first token. Serving state per sequence
(one slot of the engine's state manager): S [N] in f32 and the convolution's last taps - 1 inputs. One launch for the
convolution (mix_ops.causal_conv), one for gates, recurrence, gelu and product (mix_ops.gated_linear_recurrence; two when a few
long prompts have to fill the chip).

Built `fused`, a module has no projections of its own: the caller passes the columns [y | x] of a wider projection and the
place of S y in a wider row (layers.parallel_block). With `share` it runs with another module's parameters and keeps a state of
its own.
"""
from __future__ import annotations

import torch
import torch.nn.functional as F
from torch import nn

from .. import mix_ops
from ..utils.context import get_context
from .linear import MergedColumnParallelLinear, RowParallelLinear
from .tp import tp_size


class GatedLinearRecurrence(nn.Module):
    uses_state_slots = True
    bias = True               # both branches' projections have one

    def __init__(self, width: int, channels: int, blocks: int, conv_taps: int, decay_scale: float = 8.0, fused: bool = False,
                 share: "GatedLinearRecurrence | None" = None):
        super().__init__()
        assert tp_size() == 1, "the gated linear recurrence is not sharded: run it with tensor_parallel_size 1"
        assert channels % blocks == 0 and conv_taps >= 1
        self.N, self.blocks, self.taps, self.decay_scale = channels, blocks, conv_taps, float(decay_scale)
        self.sizes = [channels, channels]                                    # y | x
        self.out_size = channels
        n = channels // blocks
        if share is None:
            f32 = dict(dtype=torch.float32)
            self.in_proj = None if fused else MergedColumnParallelLinear(width, self.sizes, bias=True)
            self.o_proj = None if fused else RowParallelLinear(channels, width, bias=False)
            self.conv_weight = nn.Parameter(torch.zeros(channels, conv_taps, **f32))       # last column: current token
            self.conv_bias = nn.Parameter(torch.zeros(channels, **f32))
            self.gate_weight = nn.Parameter(torch.empty(blocks, 2, n, n))                  # recurrence gate, input gate: [out, in]
            self.gate_bias = nn.Parameter(torch.zeros(blocks, 2, n, **f32))
            self.lam = nn.Parameter(torch.zeros(channels, **f32))
        else:
            assert (share.sizes, share.blocks, share.taps) == (self.sizes, blocks, conv_taps)
            self.in_proj, self.o_proj, self.lam = share.in_proj, share.o_proj, share.lam
            self.conv_weight, self.conv_bias = share.conv_weight, share.conv_bias
            self.gate_weight, self.gate_bias = share.gate_weight, share.gate_bias
        self.conv_state = self.state = torch.tensor([])

    # -- cache protocol of the model runner
    def cache_bytes(self, block_size: int, act_bytes: int) -> tuple[int, int]:
        return 0, self.N * 4 + max(self.taps - 1, 1) * self.N * act_bytes

    def bind_cache(self, num_blocks: int, block_size: int, num_slots: int, device, dtype) -> None:
        self._conv_buf = torch.zeros(num_slots, max(self.taps - 1, 1), self.N, dtype=dtype, device=device)
        self.conv_state = self._conv_buf[:, :self.taps - 1]      # one tap: an empty view that still has an address
        self.state = torch.zeros(num_slots, self.N, dtype=torch.float32, device=device)
        self.rate = (-self.decay_scale * F.softplus(self.lam.detach().double())).float().contiguous()     # log a per unit of r

    def forward(self, h: torch.Tensor, proj: torch.Tensor | None = None, col0: int = 0, out: torch.Tensor | None = None) -> torch.Tensor:
        step = get_context().ragged
        if proj is None:
            proj, col0 = self.in_proj(h), 0
        N = self.N
        u = mix_ops.causal_conv(proj[:, col0 + N:col0 + 2 * N], self.conv_weight, self.conv_bias, self.conv_state, step)
        o = mix_ops.gated_linear_recurrence(u, proj[:, col0:col0 + N], self.gate_weight, self.gate_bias, self.rate, self.state, step,
                                            self.blocks, out)
        return o if self.o_proj is None else self.o_proj(o)
