"""Feditar: a decoder-only model on one f32 residual whose layers mix the sequence with a matrix memory, a state-space
recurrence, or attention and time mixing side by side; its embedding also reads the previous token and the position.

config.json (`architecture: "Feditar"`) lists the layers. Each names its type:
  "mlstm"     matrix memory with capped exponential gates, a normaliser and a running maximum (layers.matrix_memory)
  "mamba2"    state-space recurrence with grouped keys and queries behind a short convolution (layers.state_space)
  "parallel"  two mixers read the same normed input. Left: softmax attention with grouped key/value heads, a short
              convolution on q, k and v, a query factor that grows with the position and capped scores. Right: time mixing
              with shifted inputs and a decay per row of its state (layers.time_mixing). The layer takes half the sum of
              the two outputs, each divided by its root mean square over the width and weighted.
and its feed-forward: "dense" (W_down relu(W_up h)^2) or none. A layer is pre-normed, norm weights are held as offsets from
one. The embedding is the token's row times a constant plus a row of a table hashed from the previous token and this one plus
the position's row, normed; the output head is the token table itself.

Sizes, layer order and constants come from the config; the rank of the time mixing's thin decay factors, which the config does
not name, comes from the checkpoint's tensor shapes (or from the optional mixer key `decay_rank` when a model is built
without a checkpoint).

The model runs ragged steps only (utils.context.RaggedStep). Checkpoint tensors: embed, bigram, pos, embed.norm, final.norm,
l<i>.norm1|norm2, mlstm: l<i>.mix.q|k|v|g|o|norm|i|f (+ .b), mamba2: l<i>.mix.in|conv (+ .b) |dt_bias|A_log|D|norm|o,
parallel: l<i>.mix.left.q|k|v (+ .conv) |o|out and l<i>.mix.right.mu.*|r|k|v|g|w1|w2|w0|u|norm|o|out, dense:
l<i>.mlp.up|down; linear weights stored [out, in].
"""
from __future__ import annotations

import json
import os
from dataclasses import dataclass, field
from typing import Any, Optional

import torch
from torch import nn

from ..layers.activation import Act
from ..layers.embed_head import PairPositionEmbedding, ParallelLMHead
from ..layers.layernorm import OffsetRMSNorm
from ..layers.linear import ColumnParallelLinear, RowParallelLinear
from ..layers.matrix_memory import MatrixMemory
from ..layers.parallel_mixer import ParallelMixers
from ..layers.rotary_attention import GatedRotaryAttention
from ..layers.state_space import StateSpaceMixer
from ..layers.time_mixing import BATCHED, TimeMixing
from ..utils.loader import tensor_shapes

PAIR_SCALE = 0.5           # the parallel mixer takes half the sum of its two normed outputs
NORM_WEIGHT_OFFSET = 1.0   # norm weights are offsets from one

MIXER_KEYS = {
    "mlstm": ("heads", "dim", "vdim", "gate_cap"),
    "mamba2": ("heads", "vdim", "state", "groups", "conv", "norm_groups"),
    "parallel": ("left", "right"),
}
LEFT_KEYS = ("heads", "kv_heads", "dim", "vdim", "scale", "conv")
RIGHT_KEYS = ("heads", "dim")


@dataclass
class FeditarConfig:
    """config.json of a Feditar checkpoint. Attribute names the engine reads from any model config
    (vocab_size, hidden_size, max_position_embeddings, torch_dtype) are provided as well."""
    vocab: int
    width: int
    norm_eps: float
    max_position_embeddings: int
    embedding_scale: float = 1.0
    pair: Optional[tuple] = None                 # (buckets, mul_prev, mul_cur) of the hashed pair table
    layers: list = field(default_factory=list)
    torch_dtype: Any = torch.bfloat16
    architectures: tuple = ("Feditar",)

    @property
    def vocab_size(self) -> int:
        return self.vocab

    @property
    def hidden_size(self) -> int:
        return self.width

    @property
    def num_hidden_layers(self) -> int:
        return len(self.layers)

    @classmethod
    def from_dict(cls, d: dict, shapes: Optional[dict] = None) -> "FeditarConfig":
        for key in ("vocab", "width", "layers", "norm", "max_positions"):
            if key not in d:
                raise ValueError(f"Feditar config lacks '{key}'")

        def need(i, what, m, keys):
            missing = [k for k in keys if k not in m]
            if missing:
                raise ValueError(f"layer {i} ({what}) lacks {missing}")

        layers = []
        for i, L in enumerate(d["layers"]):
            kind, m = L["type"], dict(L["mixer"])
            if kind not in MIXER_KEYS:
                raise ValueError(f"layer {i}: unknown mixer type '{kind}'")
            need(i, kind, m, MIXER_KEYS[kind])
            if kind == "parallel":
                m["left"], m["right"] = dict(m["left"]), dict(m["right"])
                need(i, "left mixer", m["left"], LEFT_KEYS)
                need(i, "right mixer", m["right"], RIGHT_KEYS)
                temp = m["left"].get("q_temp")
                if temp and (int(temp["every"]) != temp["every"] or int(temp["every"]) < 1):
                    raise ValueError(f"layer {i}: q_temp.every must be a positive whole number")
                tensor = f"l{i}.mix.right.w1"
                if shapes is not None and tensor in shapes:
                    m["right"]["decay_rank"] = int(shapes[tensor][0])
                elif "decay_rank" not in m["right"]:
                    raise ValueError(f"layer {i}: 'decay_rank' is neither in the config nor given by a tensor '{tensor}'")
            mlp = L.get("mlp")
            if mlp is not None:
                mlp = dict(mlp)
                if mlp.get("kind") != "dense":
                    raise ValueError(f"layer {i}: unknown feed-forward kind '{mlp.get('kind')}'")
                need(i, "feed-forward", mlp, ("ff",))
            layers.append({"type": kind, "mixer": m, "mlp": mlp})
        emb = d.get("embedding") or {}
        pair = emb.get("bigram")
        if pair:
            pair = (int(pair["buckets"]), int(pair["mul_prev"]), int(pair["mul_cur"]))
        return cls(vocab=int(d["vocab"]), width=int(d["width"]), norm_eps=float(d["norm"]["eps"]),
                   max_position_embeddings=int(d["max_positions"]), embedding_scale=float(emb.get("scale", 1.0)),
                   pair=pair or None, layers=layers)

    @classmethod
    def from_pretrained(cls, path: str) -> "FeditarConfig":
        with open(os.path.join(path, "config.json")) as f:
            return cls.from_dict(json.load(f), tensor_shapes(path))


class SquaredReluMLP(nn.Module):
    """W_down relu(W_up h)^2."""

    def __init__(self, width: int, ff: int):
        super().__init__()
        self.up_proj = ColumnParallelLinear(width, ff, bias=False)
        self.act_fn = Act("relu2")
        self.down_proj = RowParallelLinear(ff, width, bias=False)

    def forward(self, x):
        return self.down_proj(self.act_fn(self.up_proj(x)))


def _make_mixer(config: FeditarConfig, spec: dict):
    W, m, eps = config.width, spec["mixer"], config.norm_eps
    if spec["type"] == "mlstm":
        return MatrixMemory(W, int(m["heads"]), int(m["dim"]), int(m["vdim"]), float(m["gate_cap"]), norm_eps=eps)
    if spec["type"] == "mamba2":
        return StateSpaceMixer(W, int(m["heads"]), int(m["vdim"]), int(m["state"]), int(m["groups"]), int(m["conv"]),
                               norm_groups=int(m["norm_groups"]), norm_eps=eps)
    a, b = m["left"], m["right"]
    temp = a.get("q_temp")
    left = GatedRotaryAttention(W, int(a["heads"]), int(a["kv_heads"]), int(a["dim"]), int(a["vdim"]), float(a["scale"]),
                                rot_dims=0, bias=False, head_temp=False, gate=None, fused_input=True, conv_taps=int(a["conv"]),
                                q_temp=(temp["coef"], temp["every"]) if temp else None, softcap=float(a.get("softcap") or 0.0))
    right = TimeMixing(W, int(b["heads"]), int(b["dim"]), int(b["decay_rank"]), norm_eps=eps)
    return ParallelMixers(W, left, right, eps=eps, scale=PAIR_SCALE)


class FeditarLayer(nn.Module):

    def __init__(self, config: FeditarConfig, spec: dict):
        super().__init__()
        W, eps = config.width, config.norm_eps
        self.norm1 = OffsetRMSNorm(W, eps, NORM_WEIGHT_OFFSET)
        self.mix = _make_mixer(config, spec)
        self.mlp = None
        if spec["mlp"] is not None:
            self.norm2 = OffsetRMSNorm(W, eps, NORM_WEIGHT_OFFSET)
            self.mlp = SquaredReluMLP(W, int(spec["mlp"]["ff"]))


class FeditarForCausalLM(nn.Module):
    ragged_steps = True           # the runner feeds utils.context.RaggedStep batches
    config_class = FeditarConfig

    def __init__(self, config: FeditarConfig):
        super().__init__()
        self.config = config
        self.embed = PairPositionEmbedding(config.vocab, config.width, config.embedding_scale, config.pair,
                                           config.max_position_embeddings, config.norm_eps, NORM_WEIGHT_OFFSET)
        self.layers = nn.ModuleList([FeditarLayer(config, spec) for spec in config.layers])
        self.final_norm = OffsetRMSNorm(config.width, config.norm_eps, NORM_WEIGHT_OFFSET)
        self.lm_head = ParallelLMHead(config.vocab, config.width)
        self.lm_head.weight = self.embed.weight    # the head is the token table, without its factor
        self.layer_outputs: Optional[list] = None  # set to [] to record the residual after every layer

    @staticmethod
    def _sublayer(mix, out) -> dict:
        """Arguments of the residual update that takes a mixer's output."""
        if isinstance(mix, ParallelMixers):
            return dict(y1=out[0], y2=out[1], post_w1=mix.left_out, post_w2=mix.right_out, pair_scale=mix.scale, pair_eps=mix.eps)
        return dict(y1=out)

    def forward(self, input_ids: torch.Tensor, positions: torch.Tensor) -> torch.Tensor:
        norms = [layer.norm1 for layer in self.layers] + [self.final_norm]
        x, h = self.embed(input_ids, norms[0])     # the residual, f32 throughout, and its first norm
        for i, layer in enumerate(self.layers):
            update = self._sublayer(layer.mix, layer.mix(h))
            if layer.mlp is not None:
                h = layer.norm2(x, **update)
                update = dict(y1=layer.mlp(h))
            h = norms[i + 1](x, **update)          # x += this layer's last sublayer, then the next norm
            if self.layer_outputs is not None:
                self.layer_outputs.append(x.clone())
        return h

    def compute_logits(self, hidden_states):
        return self.lm_head(hidden_states)

    def greedy_tokens(self, hidden_states):
        return self.lm_head.greedy_tokens(hidden_states)

    # ------------------------------------------------------------------ checkpoint
    def weight_targets(self) -> dict:
        """checkpoint tensor name -> (parameter, where, shape): where is None (the whole parameter), the index of a part of
        a merged projection, ("rows", offset, size), ("row", index), or ("transposed", index) for one matrix of a batch that
        holds the input dimension first."""
        t = {}
        W = self.config.width

        def whole(name, param, shape=None):
            t[name] = (param, None, tuple(param.shape if shape is None else shape))

        whole("embed", self.embed.weight)
        if self.embed.pair_weight is not None:
            whole("bigram", self.embed.pair_weight)
        whole("pos", self.embed.pos_weight)
        whole("embed.norm", self.embed.norm_weight)
        whole("final.norm", self.final_norm.weight)
        for i, layer in enumerate(self.layers):
            p, mix = f"l{i}.", layer.mix
            whole(p + "norm1", layer.norm1.weight)
            if isinstance(mix, MatrixMemory):
                for j, nm in enumerate(("q", "k", "v", "g", "i", "f")):
                    t[p + "mix." + nm] = (mix.in_proj.weight, j, (mix.sizes[j], W))
                whole(p + "mix.i.b", mix.i_bias)
                whole(p + "mix.f.b", mix.f_bias)
                whole(p + "mix.norm", mix.out_norm_weight)
                whole(p + "mix.o", mix.o_proj.weight)
            elif isinstance(mix, StateSpaceMixer):
                whole(p + "mix.in", mix.in_proj.weight)
                whole(p + "mix.conv", mix.conv_weight)
                whole(p + "mix.conv.b", mix.conv_bias)
                whole(p + "mix.dt_bias", mix.dt_bias)
                whole(p + "mix.A_log", mix.A_log)
                whole(p + "mix.D", mix.skip)
                whole(p + "mix.norm", mix.out_norm_weight)
                whole(p + "mix.o", mix.o_proj.weight)
            else:
                left, right = mix.left, mix.right
                q = p + "mix.left."
                at = 0
                for j, nm in enumerate(("q", "k", "v")):
                    n = left.sizes[j]
                    t[q + nm] = (mix.in_proj.weight, j, (n, W))
                    t[q + nm + ".conv"] = (left.conv_weight, ("rows", at, n), (n, left.conv_taps))
                    at += n
                whole(q + "o", left.o_proj.weight)
                whole(q + "out", mix.left_out)
                q = p + "mix.right."
                n = right.H * right.D
                for j, nm in enumerate(BATCHED + ("w",)):
                    t[q + "mu." + nm] = (right.mix_weight, ("row", j), (W,))
                for j, nm in enumerate(BATCHED):
                    t[q + nm] = (right.proj_weight, ("transposed", j), (n, W))
                whole(q + "w1", right.decay_down.weight)
                whole(q + "w2", right.decay_up.weight)
                whole(q + "w0", right.decay_bias)
                whole(q + "u", right.bonus)
                whole(q + "norm", right.out_norm_weight)
                whole(q + "o", right.o_proj.weight)
                whole(q + "out", mix.right_out)
            if layer.mlp is not None:
                whole(p + "norm2", layer.norm2.weight)
                whole(p + "mlp.up", layer.mlp.up_proj.weight)
                whole(p + "mlp.down", layer.mlp.down_proj.weight)
        return t

    def load_weights(self, tensors) -> None:
        """tensors: iterable of (checkpoint name, tensor). Every parameter must be covered."""
        targets = self.weight_targets()
        seen = set()
        for name, tensor in tensors:
            if name not in targets:
                raise KeyError(f"checkpoint tensor '{name}' has no place in this Feditar configuration")
            param, where, shape = targets[name]
            if tuple(tensor.shape) != shape:
                raise ValueError(f"'{name}': shape {tuple(tensor.shape)} does not fit {shape}")
            if where is None:
                loader = getattr(param, "weight_loader", None)
                if loader is not None:
                    loader(param, tensor)
                else:
                    param.data.copy_(tensor)
            elif isinstance(where, tuple) and where[0] == "rows":
                param.data[where[1]:where[1] + where[2]].copy_(tensor)
            elif isinstance(where, tuple) and where[0] == "row":
                param.data[where[1]].copy_(tensor)
            elif isinstance(where, tuple):
                param.data[where[1]].copy_(tensor.t())
            else:
                param.weight_loader(param, tensor, where)
            seen.add(name)
        missing = sorted(set(targets) - seen)
        if missing:
            raise KeyError(f"checkpoint lacks {missing[:8]}{' ...' if len(missing) > 8 else ''}")

    @staticmethod
    def _random(name: str, shape):
        """(mean, standard deviation) of a random stand-in for checkpoint tensor `name`. Scales keep activations of order
        one through any depth and the recurrences remembering."""
        leaf = name.rsplit(".", 1)[-1]
        if name in ("embed.norm", "final.norm") or leaf in ("norm1", "norm2"):
            return 0.0, 0.1
        if leaf in ("norm", "out"):
            return 1.0, 0.1
        if name.endswith(".f.b"):
            return 3.0, 1.0
        if leaf == "w0":
            return -3.0, 1.0
        if leaf == "dt_bias":
            return -3.0, 1.0
        if leaf in ("A_log", "b"):
            return 0.0, 0.3
        if leaf in ("D", "u") or ".mu." in name:
            return 0.5, 0.3
        if leaf == "conv":
            return 0.0, shape[-1] ** -0.5
        return 0.0, (shape[-1] ** -0.5 if len(shape) == 2 else 0.5)

    @torch.no_grad()
    def init_random_on_device(self, seed: int = 0) -> None:
        """Fast random fill on the parameters' own device (benchmarks: values differ between devices)."""
        gens, done = {}, set()
        for name, (param, _, shape) in self.weight_targets().items():
            if id(param) in done:
                continue                    # merged tensors are filled once
            done.add(id(param))
            g = gens.get(param.device)
            if g is None:
                g = gens[param.device] = torch.Generator(device=param.device).manual_seed(seed)
            mean, std = self._random(name, shape)
            param.normal_(mean, std, generator=g)

    def random_weights(self, seed: int = 0):
        """(name, tensor) pairs of a seeded random checkpoint of this configuration, for runs without
        weights on disk."""
        from ..utils.loader import full_random_tensor
        for name, (_, _, shape) in self.weight_targets().items():
            mean, std = self._random(name, shape)
            yield name, mean + full_random_tensor(name, shape, seed, std)
