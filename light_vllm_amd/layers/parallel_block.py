"""A sequence mixer and a gated feed-forward side by side on one normed input, as two GEMMs around their kernels:

    [mixer's inputs | gate | up] = W_in h (+ biases of the mixer's part)
    y = [W_o | W_down] [mixer's outputs ; act(gate) * up]      =  mixer(h) + ff(h)

The mixer is built `fused`: it reads its columns of the joint projection and leaves its outputs in the left columns of the row
that the output GEMM multiplies, the gated unit writes the columns behind them. The sum of the two sublayers is the
inner sum of that GEMM, in its f32 accumulators, rounded once. ff = 0: the mixer alone.

With `share` a block runs with the parameters of another one; its mixer is a module of its own (cache, state).
"""
from __future__ import annotations

import torch
from torch import nn

from .activation import GatedAct
from .linear import MergedColumnParallelLinear, RowParallelLinear


class ParallelBlock(nn.Module):

    def __init__(self, width: int, mixer: nn.Module, ff: int = 0, act: str = "relu", share: "ParallelBlock | None" = None):
        super().__init__()
        self.mix, self.ff, self.split = mixer, ff, sum(mixer.sizes)
        self.sizes = list(mixer.sizes) + ([ff, ff] if ff else [])
        self.act_fn = GatedAct(act) if ff else None
        if share is None:
            bias = bool(getattr(mixer, "bias", False))
            self.in_proj = MergedColumnParallelLinear(width, self.sizes, bias=bias)
            if bias:
                self.in_proj.bias.data.zero_()       # the feed-forward's part has no bias and stays 0
            self.out_proj = RowParallelLinear(mixer.out_size + ff, width, bias=False)
        else:
            assert share.sizes == self.sizes
            self.in_proj, self.out_proj = share.in_proj, share.out_proj

    def forward(self, h: torch.Tensor) -> torch.Tensor:
        proj = self.in_proj(h)
        n = self.mix.out_size
        z = torch.empty(h.size(0), n + self.ff, dtype=h.dtype, device=h.device)
        self.mix(h, proj, 0, out=z[:, :n])
        if self.ff:
            self.act_fn(proj[:, self.split:], out=z[:, n:])
        return self.out_proj(z)
