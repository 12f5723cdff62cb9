"""Latent attention: keys and values of all heads are up-projections of one small latent vector per
token, and only that latent (plus, optionally, one rotated positional key part shared by all heads)
is cached.

    c_q = rms_norm(W_dq h) * w_q          q_h = W_uq,h c_q            = [q_h^n (dim) | q_h^r (rot_dim)]
    [c' | k^r'] = W_dkv h                 c = rms_norm(c') * w_kv     k^r = rotate(k^r', position)
    k_h = W_uk,h c,   v_h = W_uv,h c      score_h(i, j) = (q_h^n(i) . k_h(j) + rotate(q_h^r(i)) . k^r(j)) * scale
    o_h = softmax_j<=i(score_h) v_h,      y = W_o [gate_h * o_h]_h,   gate = sigmoid(W_g h)

Served in the absorbed form: q_h^n . (W_uk,h c) = (W_uk,h^T q_h^n) . c, and sum_j p_j W_uv,h c_j =
W_uv,h sum_j p_j c_j, so every head attends to the cached rows [c | k^r] themselves (keys: the whole
row, values: its first kv_rank entries) and the per-head matrices act on queries and outputs only,
as two batched GEMMs. A decoded token therefore reads kv_rank + rot_dim numbers per cached token
instead of heads * (dim + vdim), and one attention kernel serves prompts, portions and single tokens:
the paged windowed kernel with one kv head, a window no sequence reaches, no pooled blocks and no sink.

The output gate is one number per head (`gate="head"`), one per output channel (`gate="channel"`), or absent (None).
Rotation: the first rot_dims entries of the rot_dim-wide positional part, entries i and i + rot_dims/2 (or, with `interleaved`, 2i
and 2i + 1) form a pair, angle = position * base^(-2i/rot_dims), frequencies optionally rescaled and cosines and sines multiplied by
a factor (mix_ops.rotary_inv_freq, rotary_magnitude); rot_dim = 0 gives position-free attention.

With `window` a position sees itself and the window - 1 tokens before it; with `sink` the softmax denominator of head h also holds
exp(sink_h), a learned number.

q_rank = None: queries come straight from the layer's input, q = W_q h. One launch then norms and rotates everything that is
rotated or cached (mix_ops.latent_store), and both batched GEMMs write where the next step reads. Such a module can be built
`fused`: its input and output projections belong to the caller, who passes the columns of a wider projection and the place of the
per-head outputs in a wider row (layers.parallel_block).
"""
from __future__ import annotations

import torch
from torch import nn

from .. import mix_ops
from ..utils.context import get_context
from .linear import ColumnParallelLinear, MergedColumnParallelLinear, RowParallelLinear
from .tp import tp_size

NO_WINDOW = 1 << 30       # a window no sequence reaches: plain causal attention


class LatentAttention(nn.Module):
    uses_pages = True

    def __init__(self, width: int, heads: int, dim: int, vdim: int, q_rank: int | None, kv_rank: int, scale: float,
                 rot_dim: int = 0, rot_dims: int = 0, rot_base: float = 10000.0, gate: str | None = "head",
                 norm_eps: float = 1e-6, share: "LatentAttention | None" = None, interleaved: bool = False,
                 rot_scaling: dict | None = None, window: int = NO_WINDOW, sink: bool = False, fused: bool = False):
        super().__init__()
        assert tp_size() == 1, "latent attention is not sharded: run it with tensor_parallel_size 1"
        assert gate in ("head", "channel", None) and 0 <= rot_dims <= rot_dim and rot_dims % 2 == 0 and window >= 1
        if q_rank is None:
            assert gate is None, "queries straight from the input come without an output gate"
        else:
            assert not (fused or interleaved or rot_scaling) and gate is not None
        self.H, self.Dn, self.Dr, self.Dv, self.Rq, self.R = heads, dim, rot_dim, vdim, q_rank, kv_rank
        self.rot_dims, self.rot_base, self.scale, self.norm_eps = rot_dims, float(rot_base), float(scale), norm_eps
        self.interleaved, self.rot_scaling, self.window = interleaved, rot_scaling, window
        self.gate_per_channel = gate == "channel"
        self.out_size = heads * vdim
        if q_rank is None:
            self.sizes = [heads * (dim + rot_dim), kv_rank + rot_dim]                                    # q | dkv
        else:
            self.sizes = [q_rank, kv_rank + rot_dim, heads * vdim if self.gate_per_channel else heads]   # dq | dkv | gate
        if share is None:
            f32 = dict(dtype=torch.float32)
            self.in_proj = None if fused else MergedColumnParallelLinear(width, self.sizes, bias=False)
            self.uq = ColumnParallelLinear(q_rank, heads * (dim + rot_dim), bias=False) if q_rank is not None else None
            self.uk = nn.Parameter(torch.empty(heads, dim, kv_rank))        # W_uk per head, [dim, kv_rank]
            self.uv = nn.Parameter(torch.empty(heads, kv_rank, vdim))       # W_uv per head, transposed: [kv_rank, vdim]
            self.o_proj = None if fused else RowParallelLinear(heads * vdim, width, bias=False)
            self.q_norm_weight = nn.Parameter(torch.ones(q_rank, **f32)) if q_rank is not None else None
            self.kv_norm_weight = nn.Parameter(torch.ones(kv_rank, **f32))
            self.sink = nn.Parameter(torch.zeros(heads, **f32)) if sink else None
        else:       # the same weights as another layer; cache and position in the model are this layer's own
            assert (share.sizes, share.H, share.Dn, share.Dr, share.Dv) == (self.sizes, heads, dim, rot_dim, vdim)
            self.in_proj, self.uq, self.uk, self.uv, self.o_proj = share.in_proj, share.uq, share.uk, share.uv, share.o_proj
            self.q_norm_weight, self.kv_norm_weight, self.sink = share.q_norm_weight, share.kv_norm_weight, share.sink
        self.inv_freq = None          # f32 [rot_dims/2], made with the cache
        self.cache = torch.tensor([])  # [pages, page, kv_rank + rot_dim]; bound by the runner

    # -- cache protocol of the model runner
    def cache_bytes(self, block_size: int, act_bytes: int) -> tuple[int, int]:
        return block_size * (self.R + self.Dr) * act_bytes, 0

    def bind_cache(self, num_blocks: int, block_size: int, num_slots: int, device, dtype) -> None:
        self.cache = torch.zeros(num_blocks, block_size, self.R + self.Dr, dtype=dtype, device=device)
        self.inv_freq = mix_ops.rotary_inv_freq(max(self.rot_dims, 2), self.rot_base, device, self.rot_scaling)
        self.magnitude = mix_ops.rotary_magnitude(self.rot_scaling)

    def _attend(self, q_abs: torch.Tensor, step) -> torch.Tensor:
        """Per-head weighted sums of the cached latents, [T, H * R]."""
        rows = self.cache.unsqueeze(2)                                                              # [pages, page, 1, R + Dr]
        return mix_ops.window_pool_attention(q_abs, rows, rows[..., :self.R], None, None, None, step, self.H, 1, self.R + self.Dr,
                                             self.R, self.window, 0, self.scale, has_sink=False, sinks=self.sink)

    def forward(self, h: torch.Tensor, proj: torch.Tensor | None = None, col0: int = 0, out: torch.Tensor | None = None) -> torch.Tensor:
        """proj, col0: a projection of h computed by the caller whose columns from col0 on are this mixer's. A fused module writes
        the per-head outputs [T, out_size] into `out` and returns that."""
        step = get_context().ragged
        if self.Rq is None:
            return self._forward_direct(h, step, proj, col0, out)
        T, H, R, Dn, Dr = h.size(0), self.H, self.R, self.Dn, self.Dr
        proj = self.in_proj(h)
        cq = mix_ops.latent_prep(proj, 0, self.Rq, self.q_norm_weight, self.kv_norm_weight, self.inv_freq, self.cache,
                                 step, self.Rq, R, Dr, self.rot_dims, self.norm_eps)
        q = self.uq(cq)
        q_lat = torch.bmm(q.view(T, H, Dn + Dr)[:, :, :Dn].transpose(0, 1), self.uk)              # [H, T, R]
        q_abs = mix_ops.latent_q_finish(q, q_lat, self.inv_freq, step, H, Dn, Dr, R, self.rot_dims)
        o_lat = self._attend(q_abs, step)
        o = torch.bmm(o_lat.view(T, H, R).transpose(0, 1), self.uv)                                 # [H, T, Dv]
        gate = proj[:, self.sizes[0] + self.sizes[1]:]
        return self.o_proj(mix_ops.latent_out_gate(o, gate, self.gate_per_channel))

    def _forward_direct(self, h, step, proj, col0, out):
        T, H, R, Dn, Dr = h.size(0), self.H, self.R, self.Dn, self.Dr
        if proj is None:
            proj, col0 = self.in_proj(h), 0
        q_abs = torch.empty(T, H, R + Dr, dtype=h.dtype, device=h.device)
        mix_ops.latent_store(proj, col0, col0 + self.sizes[0], self.kv_norm_weight, self.inv_freq, self.magnitude, q_abs, self.cache,
                             step, H, Dn, Dr, R, self.rot_dims, self.interleaved, self.norm_eps)
        q = proj[:, col0:col0 + self.sizes[0]].view(T, H, Dn + Dr)
        torch.bmm(q[:, :, :Dn].transpose(0, 1), self.uk, out=q_abs[:, :, :R].transpose(0, 1))
        o_lat = self._attend(q_abs.view(T, H * (R + Dr)), step)
        o = out if out is not None else torch.empty(T, H * self.Dv, dtype=h.dtype, device=h.device)
        torch.bmm(o_lat.view(T, H, R).transpose(0, 1), self.uv, out=o.view(T, H, self.Dv).transpose(0, 1))
        return o if self.o_proj is None else self.o_proj(o)
