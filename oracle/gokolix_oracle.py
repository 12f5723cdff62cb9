"""Plain, slow restatement of the Gokolix layers in float64, one function per mechanism, whole
sequences at a time (no cache, no state slots, no batching, no merged weights, no fused steps). Test
infrastructure only: it shares no code with the package and is what the engine's results are compared with.

W is a dict of float64 tensors under the checkpoint's names; cfg is the parsed config.json. `cache_round` is applied
to what attention multiplies (queries, keys, values), for comparisons against caches of a narrower format."""
from __future__ import annotations

import math

import torch

F64 = torch.float64


def unit_rms(x, eps):
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def offset_norm(x, w, eps):
    """RMS norm whose weight is held as an offset from one."""
    return unit_rms(x, eps) * (1.0 + w)


def gelu_tanh(z):
    return 0.5 * z * (1.0 + torch.tanh(math.sqrt(2.0 / math.pi) * (z + 0.044715 * z ** 3)))


def softplus(z):
    return torch.clamp(z, min=0.0) + torch.log1p(torch.exp(-z.abs()))


# ------------------------------------------------------------------------------------ rotation
def yarn(rot):
    """(frequencies [dims/2], factor on cos and sin) of a rotation with or without length scaling."""
    dims, base = int(rot["dims"]), float(rot["base"])
    f = [base ** (-2.0 * i / dims) for i in range(dims // 2)]
    s = rot.get("scaling")
    if not s:
        return f, 1.0
    factor, original = float(s["factor"]), float(s["original"])

    def index_of(turns):
        """The (fractional) pair index whose wave turns `turns` times over the original length."""
        return dims * math.log(original / (2.0 * math.pi * turns)) / (2.0 * math.log(base))

    lo = max(math.floor(index_of(float(s["fast"]))), 0)
    hi = min(math.ceil(index_of(float(s["slow"]))), dims - 1)
    out = []
    for i, fi in enumerate(f):
        ramp = min(max((i - lo) / max(hi - lo, 0.001), 0.0), 1.0)
        out.append(fi / factor * ramp + fi * (1.0 - ramp))
    return out, 0.1 * math.log(factor) + 1.0


def rotate(x, rot):
    """x [T, ..., d], row t at position t: pairs (2i, 2i + 1) of the first rot.dims entries."""
    f, mag = yarn(rot)
    y = x.clone()
    for t in range(x.shape[0]):
        for i, fi in enumerate(f):
            c, s = mag * math.cos(t * fi), mag * math.sin(t * fi)
            u, v = x[t, ..., 2 * i], x[t, ..., 2 * i + 1]
            y[t, ..., 2 * i] = u * c - v * s
            y[t, ..., 2 * i + 1] = v * c + u * s
    return y


# ----------------------------------------------------------------------------------- attention
def sees(i, j, window):
    """Whether position i sees position j (window None: every earlier one)."""
    return 0 <= i - j and (window is None or i - j < window)


def sink_softmax_head(score, v, sink, window):
    """score(i, j) -> number; v [T, Dv]; sink: a number whose exponential joins every denominator, or None."""
    T = v.shape[0]
    out = []
    for i in range(T):
        js = [j for j in range(T) if sees(i, j, window)]
        s = score(i, js)
        m = float(s.max()) if sink is None else max(float(s.max()), float(sink))
        e = torch.exp(s - m)
        den = e.sum() + (math.exp(float(sink) - m) if sink is not None else 0.0)
        out.append((e / den) @ v[js])
    return torch.stack(out)


def window_of(m):
    mask = m.get("mask") or {}
    return int(mask["size"]) if mask.get("size") else None


def latent_attention(h, W, p, m, eps, cache_round=None):
    T = h.shape[0]
    H, Dn, Dr, Dv, R = m["heads"], m["dim"], int(m.get("rot_dim", 0)), m["vdim"], m["kv_rank"]
    q = (h @ W[p + "q"].T).view(T, H, Dn + Dr)
    d = h @ W[p + "dkv"].T
    c = unit_rms(d[:, :R], eps) * W[p + "dkv.norm"]
    k_rot, q_rot = d[:, R:], q[..., Dn:]
    if Dr:
        k_rot, q_rot = rotate(k_rot, m["rot"]), rotate(q_rot, m["rot"])
    if cache_round is not None:
        c, k_rot, q_rot = cache_round(c), cache_round(k_rot), cache_round(q_rot)
    k = (c @ W[p + "uk"].T).view(T, H, Dn)
    v = (c @ W[p + "uv"].T).view(T, H, Dv)
    heads = []
    for hd in range(H):
        def score(i, js, hd=hd):
            return (k[js, hd] @ q[i, hd, :Dn] + k_rot[js] @ q_rot[i, hd]) * float(m["scale"])
        heads.append(sink_softmax_head(score, v[:, hd], W[p + "sink"][hd], window_of(m)))
    return torch.cat(heads, -1) @ W[p + "o"].T


def distance_bucket(n, rows, far):
    """Row of the bias table for distance n: one row each for the nearest rows/2 distances, the others spaced by the
    logarithm up to `far`, from which on all share the last row."""
    half = rows // 2
    if n < half:
        return n
    return min(rows - 1, half + math.floor(math.log(n / half) / math.log(far / half) * (rows - half)))


def attention(h, W, p, m, eps, cache_round=None):
    T = h.shape[0]
    H, G, D = m["heads"], m["kv_heads"], m["dim"]
    k0 = (h @ W[p + "k"].T + W[p + "k.b"]).view(T, G, D)
    q = unit_rms((h @ W[p + "q"].T + W[p + "q.b"]).view(T, H, D), eps) * W[p + "q.norm"]
    v = k0 if cache_round is None else cache_round(k0)
    k = unit_rms(k0, eps) * W[p + "k.norm"]
    if cache_round is not None:
        q, k = cache_round(q), cache_round(k)
    rel = W[p + "rel"]
    heads = []
    for hd in range(H):
        g = hd // (H // G)

        def score(i, js, hd=hd, g=g):
            bias = torch.stack([rel[distance_bucket(i - j, rel.shape[0], m["bias_max"]), hd] for j in js])
            return (k[js, g] @ q[i, hd]) * float(m["scale"]) + bias
        heads.append(sink_softmax_head(score, v[:, g], W[p + "sink"][hd], window_of(m)))
    return torch.cat(heads, -1) @ W[p + "o"].T


# -------------------------------------------------------------------------- gated linear recurrence
def causal_conv(u, w, bias):
    """u [T, C], w [C, taps]: y_t = sum_j w[:, j] u_(t - taps + 1 + j) + bias, zeros before the start."""
    T, C = u.shape
    taps = w.shape[1]
    y = torch.zeros(T, C, dtype=F64)
    for t in range(T):
        for j in range(taps):
            s = t - (taps - 1) + j
            if s >= 0:
                y[t] += w[:, j] * u[s]
        y[t] += bias
    return y


def lru_gates(u, W, p, blocks):
    """Recurrence and input gate of every channel from its part of u."""
    T, N = u.shape
    n = N // blocks
    r, i = torch.zeros(T, N, dtype=F64), torch.zeros(T, N, dtype=F64)
    for b in range(blocks):
        part = u[:, b * n:(b + 1) * n]
        r[:, b * n:(b + 1) * n] = torch.sigmoid(part @ W[p + "ra"][b].T + W[p + "ra.b"][b])
        i[:, b * n:(b + 1) * n] = torch.sigmoid(part @ W[p + "ri"][b].T + W[p + "ri.b"][b])
    return r, i


def lru_scan(u, r, i, lam):
    """S_t = a S_(t-1) + sqrt(1 - a^2) i u channel by channel, log a = -8 r softplus(lam)."""
    S = torch.zeros(u.shape[1], dtype=F64)
    out = []
    for t in range(u.shape[0]):
        log_a = -8.0 * r[t] * softplus(lam)
        S = torch.exp(log_a) * S + torch.sqrt(-torch.expm1(2.0 * log_a)) * i[t] * u[t]
        out.append(S)
    return torch.stack(out)


def rglru(h, W, p, m):
    y = gelu_tanh(h @ W[p + "y"].T + W[p + "y.b"])
    u = causal_conv(h @ W[p + "x"].T + W[p + "x.b"], W[p + "conv"], W[p + "conv.b"])
    r, i = lru_gates(u, W, p, int(m["blocks"]))
    return (lru_scan(u, r, i, W[p + "lam"]) * y) @ W[p + "o"].T


# --------------------------------------------------------------------------------------- model
def dense_ff(h, W, p):
    return (torch.clamp(h @ W[p + "gate"].T, min=0.0) * (h @ W[p + "up"].T)) @ W[p + "down"].T


def mixer(h, W, p, spec, eps, cache_round=None):
    if spec["type"] == "latent_attention":
        return latent_attention(h, W, p, spec["mixer"], eps, cache_round)
    if spec["type"] == "attention":
        return attention(h, W, p, spec["mixer"], eps, cache_round)
    if spec["type"] == "rglru":
        return rglru(h, W, p, spec["mixer"])
    raise ValueError(spec["type"])


def layer(x, W, i, spec, eps, cache_round=None):
    """Mixer and feed-forward side by side on one normed input."""
    p = f"l{i}."
    h = offset_norm(x, W[p + "norm1"], eps)
    y = mixer(h, W, p + "mix.", spec, eps, cache_round)
    if spec.get("mlp") is not None:
        y = y + dense_ff(h, W, p + "mlp.")
    return x + y


def enter_pass(x, x0, W, t):
    """What happens to the residual right before a pass of the looped stretch."""
    return torch.cat([x, x0], -1) @ W["loop.in"].T + W["loop.step"][t]


def forward(tokens, W, cfg, cache_round=None):
    """-> (logits [T, vocab], [residual after every layer run])."""
    eps = float(cfg["norm"]["eps"])
    x0 = W["embed"][[int(t) for t in tokens]] * float((cfg.get("embedding") or {}).get("scale", 1.0))
    x, trail = x0, []
    n = len(cfg["layers"])
    loop = cfg.get("loop")
    start, stop, times = (int(loop["start"]), int(loop["stop"]), int(loop["times"])) if loop else (n, n, 0)

    def run(i):
        nonlocal x
        x = layer(x, W, i, cfg["layers"][i], eps, cache_round)
        trail.append(x)

    for i in range(start):
        run(i)
    for t in range(times):
        x = enter_pass(x, x0, W, t)
        for i in range(start, stop):
            run(i)
    for i in range(stop, n):
        run(i)
    return offset_norm(x, W["final.norm"], eps) @ W["embed"].T, trail


# ------------------------------------------------------------------------------ random checkpoints
REL_ROWS = 32


def tensor_shapes(cfg) -> dict:
    """name -> shape of every tensor a checkpoint of this configuration holds. The rows of the distance-bias table are no part
    of the configuration: `rel_rows` of an attention mixer here, REL_ROWS without one."""
    W = int(cfg["width"])
    t = {"embed": (int(cfg["vocab"]), W), "final.norm": (W,)}
    if cfg.get("loop"):
        t.update({"loop.in": (W, 2 * W), "loop.step": (int(cfg["loop"]["times"]), W)})
    for i, L in enumerate(cfg["layers"]):
        p, m = f"l{i}.", L["mixer"]
        t[p + "norm1"] = (W,)
        q = p + "mix."
        if L["type"] == "latent_attention":
            H, Dn, Dr, Dv, R = m["heads"], m["dim"], int(m.get("rot_dim", 0)), m["vdim"], m["kv_rank"]
            t.update({q + "q": (H * (Dn + Dr), W), q + "dkv": (R + Dr, W), q + "dkv.norm": (R,), q + "uk": (H * Dn, R),
                      q + "uv": (H * Dv, R), q + "sink": (H,), q + "o": (W, H * Dv)})
        elif L["type"] == "attention":
            H, G, D = m["heads"], m["kv_heads"], m["dim"]
            t.update({q + "q": (H * D, W), q + "q.b": (H * D,), q + "k": (G * D, W), q + "k.b": (G * D,), q + "q.norm": (D,),
                      q + "k.norm": (D,), q + "rel": (int(m.get("rel_rows", REL_ROWS)), H), q + "sink": (H,), q + "o": (W, H * D)})
        else:
            N, B = m["width"], m["blocks"]
            t.update({q + "y": (N, W), q + "y.b": (N,), q + "x": (N, W), q + "x.b": (N,), q + "conv": (N, m["conv"]),
                      q + "conv.b": (N,), q + "ra": (B, N // B, N // B), q + "ra.b": (B, N // B), q + "ri": (B, N // B, N // B),
                      q + "ri.b": (B, N // B), q + "lam": (N,), q + "o": (W, N)})
        if L.get("mlp") is not None:
            ff = int(L["mlp"]["ff"])
            t.update({p + "mlp.gate": (ff, W), p + "mlp.up": (ff, W), p + "mlp.down": (W, ff)})
    return t


def random_weights(cfg, seed: int) -> dict:
    """A seeded checkpoint, float64 values that bfloat16 holds exactly. Scales keep activations of order one and make the
    sinks, the distance biases, the old taps and both gates matter, with states that remember for tens to hundreds of tokens."""
    g = torch.Generator().manual_seed(seed)
    scale = float((cfg.get("embedding") or {}).get("scale", 1.0))
    out = {}
    for name, shape in tensor_shapes(cfg).items():
        leaf = name.rsplit(".", 1)[-1]
        x = torch.randn(tuple(shape), generator=g)
        if name == "final.norm" or leaf == "norm1":
            x = 0.3 * x
        elif leaf == "norm":
            x = 1.0 + 0.3 * x
        elif name == "embed":
            x = x / max(scale, 1.0)
        elif leaf == "step":
            x = 0.4 * x
        elif leaf == "sink":
            x = 0.5 + 0.7 * x
        elif leaf == "rel":
            x = 1.2 * x
        elif leaf == "lam":
            x = -3.5 + 1.5 * x
        elif leaf == "b":
            x = 0.4 * x
        elif leaf == "conv":
            x = x / shape[-1] ** 0.5
        elif leaf in ("ra", "ri"):
            x = 1.5 * x / shape[-1] ** 0.5
        else:
            x = x / shape[-1] ** 0.5
        out[name] = x.to(torch.bfloat16).to(F64)
    return out
