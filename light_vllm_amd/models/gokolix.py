"""Gokolix: a decoder-only model on one f32 residual whose layers run a sequence mixer and a gated feed-forward side by side, with
a stretch of layers that is applied several times over and re-reads the embeddings ahead of every pass.

config.json (`architecture: "Gokolix"`) lists the layers. Each names its mixer type:
  "latent_attention"  windowed attention over a cached latent, interleaved rotation with YaRN frequencies on a part of the
                      queries and one shared key part, learned sinks (layers.latent_attention)
  "attention"         windowed attention on normed queries and keys with a learned bias by distance and learned sinks, whose
                      values are its unnormed keys (layers.biased_attention)
  "rglru"             Griffin's recurrent block: a real-gated linear recurrent unit behind a short convolution, beside a gelu
                      branch (layers.linear_recurrence)
and its feed-forward: "dense" (W_down (relu(W_gate h) * W_up h)) or none. Both read h = norm(x) and x += mixer(h) + ff(h)
(layers.parallel_block); norm weights are held as offsets from one. The embedding is multiplied by a constant; the output head is
the table itself.

`loop` (start, stop, times) applies layers start .. stop-1 `times` times back to back with one set of weights, each pass on pages
and state of its own. Ahead of every pass x <- W_loop [x ; x_0] + step_t, x_0 being the scaled embeddings and t the number of the
pass. W_loop's half for x_0 is multiplied once per step and kept in f32; the half for x multiplies the residual as the sum of
two bf16 numbers (mix_ops.residual_split) and accumulates onto it, so that the residual is never rounded to 16 bits.

Sizes, layer order and constants come from the config; the rows of the distance-bias tables, which the config does not name, come
from the checkpoint's tensor shapes (or from the optional mixer key `rel_rows` when a model is built without a checkpoint).

The model runs ragged steps only (utils.context.RaggedStep). Checkpoint tensors: embed, loop.in, loop.step, final.norm, l<i>.norm1,
latent_attention: l<i>.mix.q|dkv|dkv.norm|uk|uv|sink|o, attention: l<i>.mix.q|k (+ .b, .norm) |rel|sink|o,
rglru: l<i>.mix.y|x|conv (+ .b) |ra|ri (+ .b) |lam|o, dense: l<i>.mlp.gate|up|down; linear weights stored [out, in].
"""
from __future__ import annotations

import json
import os
from dataclasses import dataclass, field
from typing import Any, Optional

import torch
from torch import nn

from .. import mix_ops
from ..layers.biased_attention import DistanceBiasAttention
from ..layers.embed_head import ParallelLMHead, VocabParallelEmbedding
from ..layers.latent_attention import NO_WINDOW, LatentAttention
from ..layers.layernorm import OffsetRMSNorm
from ..layers.linear_recurrence import GatedLinearRecurrence
from ..layers.parallel_block import ParallelBlock
from ..utils.loader import tensor_shapes

NORM_WEIGHT_OFFSET = 1.0   # norm weights are offsets from one
DECAY_SCALE = 8.0          # log a = -8 r softplus(lam)

MIXER_KEYS = {
    "latent_attention": ("heads", "dim", "vdim", "kv_rank", "scale"),
    "attention": ("heads", "kv_heads", "dim", "scale", "bias_max"),
    "rglru": ("width", "blocks", "conv"),
}


@dataclass
class GokolixConfig:
    """config.json of a Gokolix checkpoint. Attribute names the engine reads from any model config
    (vocab_size, hidden_size, max_position_embeddings, torch_dtype) are provided as well."""
    vocab: int
    width: int
    norm_eps: float
    embedding_scale: float = 1.0
    layers: list = field(default_factory=list)
    loop_start: int = 0
    loop_stop: int = 0
    loop_times: int = 1
    has_loop: bool = False                       # the config names a loop (its tensors exist even if the stretch is empty)
    torch_dtype: Any = torch.bfloat16
    max_position_embeddings: int = 1 << 30       # positions are rotated on the fly: any length the cache holds
    architectures: tuple = ("Gokolix",)

    @property
    def vocab_size(self) -> int:
        return self.vocab

    @property
    def hidden_size(self) -> int:
        return self.width

    @property
    def num_hidden_layers(self) -> int:
        return len(self.layers)

    def runs(self) -> list:
        """(layer index, pass number or None) in running order; a pass number marks the first layer of a pass."""
        n, a, b = len(self.layers), self.loop_start, self.loop_stop
        if not b > a:
            return [(i, None) for i in range(n)]
        order = [(i, None) for i in range(a)]
        for t in range(self.loop_times):
            order += [(i, t if i == a else None) for i in range(a, b)]
        return order + [(i, None) for i in range(b, n)]

    @classmethod
    def from_dict(cls, d: dict, shapes: Optional[dict] = None) -> "GokolixConfig":
        for key in ("vocab", "width", "layers", "norm"):
            if key not in d:
                raise ValueError(f"Gokolix config lacks '{key}'")
        layers = []
        for i, L in enumerate(d["layers"]):
            kind, m = L["type"], dict(L["mixer"])
            if kind not in MIXER_KEYS:
                raise ValueError(f"layer {i}: unknown mixer type '{kind}'")
            need = MIXER_KEYS[kind] + (("rot",) if kind == "latent_attention" and int(m.get("rot_dim") or 0) > 0 else ())
            missing = [k for k in need if k not in m]
            if missing:
                raise ValueError(f"layer {i} ({kind}): mixer lacks {missing}")
            if kind == "attention":
                if int(m.get("vdim", m["dim"])) != int(m["dim"]):
                    raise ValueError(f"layer {i}: values are the keys, vdim {m['vdim']} is not dim {m['dim']}")
                tensor = f"l{i}.mix.rel"
                if shapes is not None and tensor in shapes:
                    m["rel_rows"] = int(shapes[tensor][0])
                elif "rel_rows" not in m:
                    raise ValueError(f"layer {i}: 'rel_rows' is neither in the config nor given by a tensor '{tensor}'")
                if not (m["rel_rows"] >= 2 and m["bias_max"] > m["rel_rows"] // 2):
                    raise ValueError(f"layer {i}: bias_max {m['bias_max']} does not fit {m['rel_rows']} rows of distance biases")
            mlp = L.get("mlp")
            if mlp is not None:
                mlp = dict(mlp)
                if mlp.get("kind") != "dense":
                    raise ValueError(f"layer {i}: unknown feed-forward kind '{mlp.get('kind')}'")
                if "ff" not in mlp:
                    raise ValueError(f"layer {i}: feed-forward lacks ['ff']")
            layers.append({"type": kind, "mixer": m, "mlp": mlp})
        loop = d.get("loop") or {}
        start, stop, times = int(loop.get("start", 0)), int(loop.get("stop", 0)), int(loop.get("times", 1))
        if loop and not (0 <= start <= stop <= len(layers) and times >= 1):
            raise ValueError(f"loop {loop} does not fit {len(layers)} layers")
        return cls(vocab=int(d["vocab"]), width=int(d["width"]), norm_eps=float(d["norm"]["eps"]),
                   embedding_scale=float((d.get("embedding") or {}).get("scale", 1.0)), layers=layers, loop_start=start,
                   loop_stop=stop, loop_times=times, has_loop=bool(loop))

    @classmethod
    def from_pretrained(cls, path: str) -> "GokolixConfig":
        with open(os.path.join(path, "config.json")) as f:
            return cls.from_dict(json.load(f), tensor_shapes(path))


def _window(m: dict) -> int:
    size = (m.get("mask") or {}).get("size")
    return int(size) if size else NO_WINDOW


def _make_mixer(config: GokolixConfig, spec: dict, share=None):
    W, m, eps = config.width, spec["mixer"], config.norm_eps
    if spec["type"] == "latent_attention":
        rot_dim, rot = int(m.get("rot_dim") or 0), m.get("rot") or {}
        return LatentAttention(W, int(m["heads"]), int(m["dim"]), int(m["vdim"]), None, int(m["kv_rank"]), float(m["scale"]),
                               rot_dim=rot_dim, rot_dims=int(rot.get("dims", rot_dim)) if rot_dim else 0,
                               rot_base=float(rot.get("base", 10000.0)), rot_scaling=rot.get("scaling") or None, interleaved=True,
                               gate=None, norm_eps=eps, window=_window(m), sink=True, fused=True, share=share)
    if spec["type"] == "attention":
        return DistanceBiasAttention(W, int(m["heads"]), int(m["kv_heads"]), int(m["dim"]), float(m["scale"]), int(m["rel_rows"]),
                                     m["bias_max"], window=_window(m), norm_eps=eps, fused=True, share=share)
    return GatedLinearRecurrence(W, int(m["width"]), int(m["blocks"]), int(m["conv"]), DECAY_SCALE, fused=True, share=share)


class GokolixLayer(nn.Module):
    """One layer, or (with `source`) one more pass of a looped layer: the same parameters, cache and state of its own."""

    def __init__(self, config: GokolixConfig, spec: dict, source: "GokolixLayer | None" = None):
        super().__init__()
        mixer = _make_mixer(config, spec, source.block.mix if source is not None else None)
        self.norm1 = source.norm1 if source is not None else OffsetRMSNorm(config.width, config.norm_eps, NORM_WEIGHT_OFFSET)
        self.block = ParallelBlock(config.width, mixer, int(spec["mlp"]["ff"]) if spec["mlp"] is not None else 0, "relu",
                                   share=source.block if source is not None else None)


class GokolixForCausalLM(nn.Module):
    ragged_steps = True           # the runner feeds utils.context.RaggedStep batches
    config_class = GokolixConfig

    def __init__(self, config: GokolixConfig):
        super().__init__()
        self.config = config
        W = config.width
        self.embed = VocabParallelEmbedding(config.vocab, W)
        self.layers = nn.ModuleList([GokolixLayer(config, spec) for spec in config.layers])
        # later passes of the looped layers: modules of their own (cache, state), parameters of the first pass
        self.repeats = nn.ModuleList()
        self.order: list = []                     # (layer module, pass number or None) in running order
        seen = set()
        for i, t in config.runs():
            layer = self.layers[i]
            if i in seen:
                layer = GokolixLayer(config, config.layers[i], layer)
                self.repeats.append(layer)
            seen.add(i)
            self.order.append((layer, t))
        self.loop_x = self.loop_x0 = self.loop_step = None
        # W_loop in two halves; the one for the residual is laid out for [high | low] where activations are bf16
        self.split = self.embed.weight.dtype == torch.bfloat16
        if config.has_loop:
            self.loop_x = nn.Parameter(torch.empty(W, 2 * W if self.split else W))
            self.loop_x0 = nn.Parameter(torch.empty(W, W))
            self.loop_step = nn.Parameter(torch.zeros(config.loop_times, W, dtype=torch.float32))
        self.final_norm = OffsetRMSNorm(W, config.norm_eps, NORM_WEIGHT_OFFSET)
        self.lm_head = ParallelLMHead(config.vocab, W)
        self.lm_head.weight = self.embed.weight    # the head is the table, without the embedding's factor
        self.layer_outputs: Optional[list] = None  # set to [] to record the residual after every layer run

    def forward(self, input_ids: torch.Tensor, positions: torch.Tensor) -> torch.Tensor:
        cfg, order = self.config, self.order
        act = self.embed.weight.dtype
        looped = any(t is not None for _, t in order)
        enters = bool(order) and order[0][1] is not None
        # the residual, f32 throughout
        x, rows, split = mix_ops.scaled_embedding(input_ids, self.embed.weight, cfg.embedding_scale, want_rows=looped,
                                                  want_split=enters and self.split)
        if looped:                                 # W_loop's share of the embeddings, the same for every pass
            x0 = mix_ops.mm_f32(rows, self.loop_x0.t()).mul_(cfg.embedding_scale)

        def enter(r, y):
            """Adds the last layer's output y, does what comes ahead of run r, and returns (residual, its norm for run r)."""
            norm = order[r][0].norm1 if r < len(order) else self.final_norm
            t = order[r][1] if r < len(order) else None
            if t is None:
                return x, norm(x, y, act_dtype=act)
            if self.split:
                a = split if y is None and split is not None else mix_ops.residual_split(x, y)
            else:
                if y is not None:
                    mix_ops.residual_add_norm(x, y)
                a = x
            nx = mix_ops.mm_f32(a, self.loop_x.t(), add=x0)
            return nx, mix_ops.sandwich_add_norm(nx, None, None, None, self.loop_step[t], norm.weight, norm.offset, norm.eps, act)

        x, h = enter(0, None)
        for r, (layer, _) in enumerate(order):
            y = layer.block(h)
            if self.layer_outputs is not None:     # the residual as the layer leaves it, before the next pass begins
                self.layer_outputs.append(x + y.float())
            x, h = enter(r + 1, y)
        return h

    def compute_logits(self, hidden_states):
        return self.lm_head(hidden_states)

    def greedy_tokens(self, hidden_states):
        return self.lm_head.greedy_tokens(hidden_states)

    # ------------------------------------------------------------------ checkpoint
    def weight_targets(self) -> dict:
        """checkpoint tensor name -> (views that receive it, shape in the checkpoint). A tensor is reshaped to its view, which
        may be rows or columns of a merged weight or a transposed one."""
        t = {}
        W = self.config.width

        def put(name, view, shape=None):
            views = view if isinstance(view, list) else [view]
            t[name] = ([v.data for v in views], tuple(views[0].shape if shape is None else shape))

        put("embed", self.embed.weight)
        put("final.norm", self.final_norm.weight)
        if self.loop_step is not None:
            # [W, 2W] = [half for x | half for x0]: views of both, filled by _place
            t["loop.in"] = ([self.loop_x.data, self.loop_x0.data], (W, 2 * W))
            put("loop.step", self.loop_step)
        for i, layer in enumerate(self.layers):
            p, mix, block = f"l{i}.", layer.block.mix, layer.block
            put(p + "norm1", layer.norm1.weight)
            w, b, at = block.in_proj.weight, block.in_proj.bias, 0
            kind = self.config.layers[i]["type"]
            names = {"latent_attention": ("q", "dkv"), "attention": ("q", "k"), "rglru": ("y", "x")}[kind]
            for nm, n in zip(names, mix.sizes):
                put(p + "mix." + nm, w[at:at + n])
                if b is not None:
                    put(p + f"mix.{nm}.b", b[at:at + n])
                at += n
            put(p + "mix.o", block.out_proj.weight[:, :mix.out_size])
            if block.ff:
                put(p + "mlp.gate", w[at:at + block.ff])
                put(p + "mlp.up", w[at + block.ff:])
                put(p + "mlp.down", block.out_proj.weight[:, mix.out_size:])
            if kind == "latent_attention":
                put(p + "mix.dkv.norm", mix.kv_norm_weight)
                put(p + "mix.uk", mix.uk, (mix.H * mix.Dn, mix.R))
                put(p + "mix.uv", mix.uv.transpose(1, 2), (mix.H * mix.Dv, mix.R))
                put(p + "mix.sink", mix.sink)
            elif kind == "attention":
                put(p + "mix.q.norm", mix.q_norm_weight)
                put(p + "mix.k.norm", mix.k_norm_weight)
                put(p + "mix.rel", mix.rel)
                put(p + "mix.sink", mix.sink)
            else:
                put(p + "mix.conv", mix.conv_weight)
                put(p + "mix.conv.b", mix.conv_bias)
                for j, nm in enumerate(("ra", "ri")):
                    put(p + "mix." + nm, mix.gate_weight[:, j])
                    put(p + f"mix.{nm}.b", mix.gate_bias[:, j])
                put(p + "mix.lam", mix.lam)
        return t

    def _place(self, name: str, views: list, tensor: torch.Tensor) -> None:
        if name == "loop.in":
            W = self.config.width
            for at in range(0, views[0].size(1), W):        # [high | low] meet the same weights
                views[0][:, at:at + W].copy_(tensor[:, :W])
            views[1].copy_(tensor[:, W:])
            return
        for v in views:
            v.copy_(tensor.reshape(v.shape))

    def load_weights(self, tensors) -> None:
        """tensors: iterable of (checkpoint name, tensor). Every parameter must be covered."""
        targets = self.weight_targets()
        seen = set()
        for name, tensor in tensors:
            if name not in targets:
                raise KeyError(f"checkpoint tensor '{name}' has no place in this Gokolix configuration")
            views, shape = targets[name]
            if tuple(tensor.shape) != shape:
                raise ValueError(f"'{name}': shape {tuple(tensor.shape)} does not fit {shape}")
            self._place(name, views, tensor)
            seen.add(name)
        missing = sorted(set(targets) - seen)
        if missing:
            raise KeyError(f"checkpoint lacks {missing[:8]}{' ...' if len(missing) > 8 else ''}")

    @staticmethod
    def _random(name: str, shape):
        """(mean, standard deviation) of a random stand-in for checkpoint tensor `name`. Scales keep activations of order
        one through any depth and the recurrences remembering."""
        leaf = name.rsplit(".", 1)[-1]
        if name == "final.norm" or leaf == "norm1":
            return 0.0, 0.1
        if leaf == "norm":
            return 1.0, 0.1
        if leaf == "lam":
            return -3.0, 1.0
        if leaf in ("b", "sink", "rel", "step"):
            return 0.0, 0.3
        return 0.0, (shape[-1] ** -0.5 if len(shape) > 1 else 0.5)

    @torch.no_grad()
    def init_random_on_device(self, seed: int = 0) -> None:
        """Fast random fill on the parameters' own device (benchmarks: values differ between devices)."""
        gens = {}
        for name, (views, shape) in self.weight_targets().items():
            dev = views[0].device
            g = gens.get(dev)
            if g is None:
                g = gens[dev] = torch.Generator(device=dev).manual_seed(seed)
            mean, std = self._random(name, shape)
            self._place(name, views, torch.empty(shape, dtype=views[0].dtype, device=dev).normal_(mean, std, generator=g))

    def random_weights(self, seed: int = 0):
        """(name, tensor) pairs of a seeded random checkpoint of this configuration, for runs without
        weights on disk."""
        from ..utils.loader import full_random_tensor
        for name, (_, shape) in self.weight_targets().items():
            mean, std = self._random(name, shape)
            yield name, mean + full_random_tensor(name, shape, seed, std)
