"""Time mixing in the manner of RWKV: every input of the recurrence reads its own mix of the token's h and its predecessor's, every row of
the state decays at a rate the token chooses, and the current token is read with a bonus before it is written:

    mix_s = h + (h' - h) mu_s        for s in r, k, v, g, w; h' = the previous token's h, zeros for the first
    r, k, v = W_r mix_r, W_k mix_k, W_v mix_v (H heads of D);   gate = silu(W_g mix_g)
    w = exp(-exp(W_w2 tanh(W_w1 mix_w) + w0))                   one number per head and row of its state
    o = (S + diag(u) k v^T)^T r;   then S <- diag(w) S + k v^T
    y = W_o [ o_h / rms(o_h) * w_h * gate_h ]_h

Serving state per sequence (one slot of the engine's state manager): S [H, D, D] in f32 and the previous token's h. One
launch for the five mixes (mix_ops.token_shift), one batched GEMM for r, k, v and g (their weights lie side by side, input
dimension first), two thin ones for the decay, the recurrence (mix_ops.gated_scan), norm and gate
(mix_ops.scaled_head_norm_gate), the output GEMM.

The module projects its own mixes, so `sizes` is empty: beside another mixer it takes no columns of a shared projection.
"""
from __future__ import annotations

import torch
from torch import nn

from .. import mix_ops
from ..utils.context import get_context
from .linear import ColumnParallelLinear, RowParallelLinear
from .tp import tp_size

BATCHED = ("r", "k", "v", "g")        # order of the batched projections; the decay's mix follows them


class TimeMixing(nn.Module):
    uses_state_slots = True

    def __init__(self, width: int, heads: int, dim: int, decay_rank: int, norm_eps: float = 1e-6):
        super().__init__()
        assert tp_size() == 1, "the time mixing is not sharded: run it with tensor_parallel_size 1"
        assert heads >= 1 and dim >= 1 and decay_rank >= 1
        self.W, self.H, self.D, self.norm_eps = width, heads, dim, float(norm_eps)
        self.sizes: list = []
        n = heads * dim
        f32 = dict(dtype=torch.float32)
        self.mix_weight = nn.Parameter(torch.zeros(len(BATCHED) + 1, width, **f32))       # r, k, v, g, w
        self.proj_weight = nn.Parameter(torch.empty(len(BATCHED), width, n))              # [in, out] each
        self.decay_down = ColumnParallelLinear(width, decay_rank, bias=False)
        self.decay_up = ColumnParallelLinear(decay_rank, n, bias=False)
        self.decay_bias = nn.Parameter(torch.zeros(n, **f32))
        self.bonus = nn.Parameter(torch.zeros(heads, dim, **f32))
        self.out_norm_weight = nn.Parameter(torch.ones(n, **f32))
        self.o_proj = RowParallelLinear(n, width, bias=False)
        self.shift_state = self.state = torch.tensor([])

    # -- cache protocol of the model runner
    def cache_bytes(self, block_size: int, act_bytes: int) -> tuple[int, int]:
        """(bytes per cache page, bytes per state slot)."""
        return 0, self.H * self.D * self.D * 4 + self.W * act_bytes

    def bind_cache(self, num_blocks: int, block_size: int, num_slots: int, device, dtype) -> None:
        self.shift_state = torch.zeros(num_slots, self.W, dtype=dtype, device=device)
        self.state = torch.zeros(num_slots, self.H, self.D, self.D, dtype=torch.float32, device=device)

    def forward(self, h: torch.Tensor, proj: torch.Tensor | None = None, col0: int = 0) -> torch.Tensor:
        """proj, col0: not used (the mixers of a pair are called alike)."""
        step = get_context().ragged
        n = len(BATCHED)
        mixes = mix_ops.token_shift(h, self.mix_weight, self.shift_state, step)
        r, k, v, g = torch.bmm(mixes[:n], self.proj_weight)
        w = self.decay_up(mix_ops.unary_act(self.decay_down(mixes[n]), "tanh"))
        o = mix_ops.gated_scan(mix_ops.SCAN_ROW_DECAY, r, k, v, w, self.decay_bias, self.bonus, step, self.state, self.H, self.H,
                               self.D, self.D)
        y = mix_ops.scaled_head_norm_gate(o, g, self.out_norm_weight, self.norm_eps, h.dtype, "silu")
        return self.o_proj(y)
