"""Softmax attention whose positions enter as a learned bias of the distance and whose values are its keys:

    q = W_q h + b_q,  k = W_k h + b_k,  v = k                                 (H query heads, G key/value heads of D)
    q^ = q / rms(q) * w_q,  k^ = k / rms(k) * w_k                             rms over the D entries of a head, weights shared by heads
    score_h(i, j) = q^_h(i) . k^_g(j) * scale + rel[bucket(i - j), h],        0 <= i - j < window,  g = h / (H / G)
    o_h = sum_j p_h(i, j) v_g(j),   p the softmax with exp(sink_h) in its denominator as well

Buckets: one per distance for the first half of the table's rows, spaced by the logarithm from there on (mix_ops.distance_bias,
which spells the table out by distance when the cache is made: the attention kernel looks a distance up, nothing else).

Keys and values are one cached row: the key as projected. Its norm is a number per head beside it, and the weights w_k are
folded into the queries', q^ . k^ = ((q / rms(q) * w_q * w_k) . k) / rms(k). A token therefore costs the cache G * D entries and G
numbers instead of 2 * G * D, and a decoded token reads each row once for its score and its value.

Built `fused`, a module has no projections of its own: the caller passes the columns [q | k] of a wider projection and the
place of the per-head outputs in a wider row (layers.parallel_block). With `share` it runs with another module's parameters
and keeps a cache of its own.
"""
from __future__ import annotations

import torch
from torch import nn

from .. import mix_ops
from ..utils.context import get_context
from .linear import MergedColumnParallelLinear, RowParallelLinear
from .tp import tp_size

NO_WINDOW = 1 << 30       # a window no sequence reaches: plain causal attention


class DistanceBiasAttention(nn.Module):
    uses_pages = True
    bias = True               # the projection of q and k has one

    def __init__(self, width: int, heads: int, kv_heads: int, dim: int, scale: float, rel_rows: int, rel_far: int,
                 window: int = NO_WINDOW, norm_eps: float = 1e-6, fused: bool = False, share: "DistanceBiasAttention | None" = None):
        super().__init__()
        assert tp_size() == 1, "the distance-biased attention is not sharded: run it with tensor_parallel_size 1"
        assert heads % kv_heads == 0 and window >= 1
        self.H, self.G, self.D, self.scale, self.window = heads, kv_heads, dim, float(scale), window
        self.rel_far, self.norm_eps = rel_far, float(norm_eps)
        self.sizes = [heads * dim, kv_heads * dim]                           # q | k
        self.out_size = heads * dim
        if share is None:
            f32 = dict(dtype=torch.float32)
            self.in_proj = None if fused else MergedColumnParallelLinear(width, self.sizes, bias=True)
            self.o_proj = None if fused else RowParallelLinear(heads * dim, width, bias=False)
            self.q_norm_weight = nn.Parameter(torch.ones(dim, **f32))
            self.k_norm_weight = nn.Parameter(torch.ones(dim, **f32))
            self.rel = nn.Parameter(torch.zeros(rel_rows, heads, **f32))
            self.sink = nn.Parameter(torch.zeros(heads, **f32))
        else:
            assert (share.sizes, share.H, share.G, share.D) == (self.sizes, heads, kv_heads, dim)
            self.in_proj, self.o_proj, self.rel, self.sink = share.in_proj, share.o_proj, share.rel, share.sink
            self.q_norm_weight, self.k_norm_weight = share.q_norm_weight, share.k_norm_weight
        self.cache = self.key_scale = torch.tensor([])

    # -- cache protocol of the model runner
    def cache_bytes(self, block_size: int, act_bytes: int) -> tuple[int, int]:
        return block_size * self.G * (self.D * act_bytes + 4), 0

    def bind_cache(self, num_blocks: int, block_size: int, num_slots: int, device, dtype) -> None:
        self.cache = torch.zeros(num_blocks, block_size, self.G, self.D, dtype=dtype, device=device)
        self.key_scale = torch.zeros(num_blocks, block_size, self.G, dtype=torch.float32, device=device)
        self.qk_weight = (self.q_norm_weight.detach() * self.k_norm_weight.detach()).contiguous()
        self.dist_bias = mix_ops.distance_bias(self.rel.detach(), self.rel_far, self.window)

    def forward(self, h: torch.Tensor, proj: torch.Tensor | None = None, col0: int = 0, out: torch.Tensor | None = None) -> torch.Tensor:
        step = get_context().ragged
        if proj is None:
            proj, col0 = self.in_proj(h), 0
        q = mix_ops.head_norm_store(proj, col0, col0 + self.sizes[0], self.qk_weight, self.cache, self.key_scale, step, self.H, self.G,
                                    self.D, self.norm_eps)
        o = mix_ops.window_pool_attention(q, self.cache, self.cache, None, None, None, step, self.H, self.G, self.D, self.D,
                                          self.window, 0, self.scale, has_sink=False, sinks=self.sink, key_scale=self.key_scale,
                                          dist_bias=self.dist_bias, out=out)
        return o if self.o_proj is None else self.o_proj(o)
