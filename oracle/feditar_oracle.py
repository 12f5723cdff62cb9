"""Plain, slow restatement of the Feditar layers in float64, one function per mechanism, whole
sequences at a time (no cache, no state slots, no batching, no merged weights, no fused steps). Test
infrastructure only: it shares no code with the package and is what the engine's results are compared with.

W is a dict of float64 tensors under the checkpoint's names; cfg is the parsed config.json."""
from __future__ import annotations

import math

import torch

F64 = torch.float64


def unit_rms(x, eps):
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def offset_norm(x, w, eps):
    """RMS norm whose weight is held as an offset from one."""
    return unit_rms(x, eps) * (1.0 + w)


def silu(z):
    return z * torch.sigmoid(z)


def softplus(z):
    return torch.clamp(z, min=0.0) + torch.log1p(torch.exp(-z.abs()))


def log_sigmoid(z):
    return -softplus(-z)


# ----------------------------------------------------------------------------------- embedding
def embed_tokens(tokens, W, cfg):
    """Scaled token row + row of the hashed pair (previous token, token) + row of the position, then the norm."""
    e = cfg["embedding"]
    eps = float(cfg["norm"]["eps"])
    rows = []
    for p, tok in enumerate(tokens):
        x = W["embed"][tok] * float(e.get("scale", 1.0))
        b = e.get("bigram")
        if b:
            n = int(b["buckets"])
            row = n if p == 0 else (tokens[p - 1] * int(b["mul_prev"]) + tok * int(b["mul_cur"])) % n
            x = x + W["bigram"][row]
        rows.append(x + W["pos"][p])
    return offset_norm(torch.stack(rows), W["embed.norm"], eps)


# ---------------------------------------------------------------------------------- convolution
def causal_conv(u, w, bias=None):
    """u [T, C], w [C, taps]: y_t = sum_j w[:, j] u_(t - taps + 1 + j) (+ bias), zeros before the start."""
    T, C = u.shape
    taps = w.shape[1]
    y = torch.zeros(T, C, dtype=F64)
    for t in range(T):
        for j in range(taps):
            s = t - (taps - 1) + j
            if s >= 0:
                y[t] += w[:, j] * u[s]
        if bias is not None:
            y[t] += bias
    return y


# ----------------------------------------------------------------------------------- attention
def query_temperature(p, q_temp):
    """The factor on the query at position p."""
    if not q_temp:
        return 1.0
    return 1.0 + float(q_temp["coef"]) * math.log(math.floor((p + 1) / q_temp["every"]) + 1)


def capped_softmax_head(q, k, v, scale, cap):
    """One head, causal: q [T, D], k [T, D], v [T, Dv]; scores pass cap * tanh(score / cap) (cap None: unchanged)."""
    out = []
    for i in range(q.shape[0]):
        s = (k[:i + 1] @ q[i]) * scale
        if cap:
            s = cap * torch.tanh(s / cap)
        e = torch.exp(s - s.max())
        out.append((e / e.sum()) @ v[:i + 1])
    return torch.stack(out)


def conv_attention(h, W, p, m, cache_round=None):
    """Left half of the parallel mixer: short convolutions on q, k and v, a query factor that grows with the
    position, capped scores, plain causal softmax."""
    T = h.shape[0]
    H, G, D, Dv = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q = causal_conv(h @ W[p + "q"].T, W[p + "q.conv"]).view(T, H, D)
    k = causal_conv(h @ W[p + "k"].T, W[p + "k.conv"]).view(T, G, D)
    v = causal_conv(h @ W[p + "v"].T, W[p + "v.conv"]).view(T, G, Dv)
    temp = torch.tensor([query_temperature(t, m.get("q_temp")) for t in range(T)], dtype=F64)
    q = q * temp[:, None, None]
    heads = []
    for hq in range(H):
        g = hq // (H // G)
        qh, kh, vh = q[:, hq], k[:, g], v[:, g]
        if cache_round is not None:
            qh, kh, vh = cache_round(qh), cache_round(kh), cache_round(vh)
        heads.append(capped_softmax_head(qh, kh, vh, float(m["scale"]), m.get("softcap")))
    return torch.cat(heads, -1) @ W[p + "o"].T


# ---------------------------------------------------------------------------------- time mixing
def token_shift(h, mu):
    """h + (previous token's h - h) * mu, the first token's predecessor being zeros."""
    prev = torch.cat([torch.zeros(1, h.shape[1], dtype=F64), h[:-1]])
    return h + (prev - h) * mu


def bonus_recurrence(r, k, v, w, u):
    """One head. r, k, w [T, D], v [T, Dv], u [D]: the read-out adds the current token's k v^T with factor u to the old
    state; then every row of the state decays by its own w and takes k v^T."""
    S = torch.zeros(r.shape[1], v.shape[1], dtype=F64)
    out = []
    for t in range(r.shape[0]):
        kv = torch.outer(k[t], v[t])
        out.append((S + u[:, None] * kv).T @ r[t])
        S = w[t][:, None] * S + kv
    return torch.stack(out)


def time_mixing(h, W, p, m, eps):
    T = h.shape[0]
    H, D = m["heads"], m["dim"]
    mix = {c: token_shift(h, W[p + "mu." + c]) for c in "rkvgw"}
    r, k, v = ((mix[c] @ W[p + c].T).view(T, H, D) for c in "rkv")
    gate = silu(mix["g"] @ W[p + "g"].T)
    w = torch.exp(-torch.exp(torch.tanh(mix["w"] @ W[p + "w1"].T) @ W[p + "w2"].T + W[p + "w0"])).view(T, H, D)
    o = torch.stack([bonus_recurrence(r[:, hd], k[:, hd], v[:, hd], w[:, hd], W[p + "u"][hd]) for hd in range(H)], 1)
    y = unit_rms(o, eps).reshape(T, H * D) * W[p + "norm"] * gate
    return y @ W[p + "o"].T


def parallel_mixer(h, W, p, m, eps, cache_round=None):
    left = conv_attention(h, W, p + "left.", m["left"], cache_round)
    right = time_mixing(h, W, p + "right.", m["right"], eps)
    return 0.5 * (unit_rms(left, eps) * W[p + "left.out"] + unit_rms(right, eps) * W[p + "right.out"])


# ---------------------------------------------------------------------------------- matrix memory
def matrix_memory(q, k, v, i, f):
    """One head of the mLSTM cell. q, k [T, D], v [T, Dv], i, f [T] log gates; running maximum from 0."""
    D, Dv = q.shape[1], v.shape[1]
    S, n, m = torch.zeros(D, Dv, dtype=F64), torch.zeros(D, dtype=F64), 0.0
    out = []
    for t in range(q.shape[0]):
        new = max(float(f[t]) + m, float(i[t]))
        a, b = math.exp(float(f[t]) + m - new), math.exp(float(i[t]) - new)
        m = new
        S = a * S + b * torch.outer(k[t], v[t])
        n = a * n + b * k[t]
        out.append((S.T @ q[t]) / (max(abs(float(n @ q[t])), math.exp(-m)) + 1e-6))
    return torch.stack(out)


def mlstm_mixer(h, W, p, m, eps):
    T = h.shape[0]
    H, D, Dv, cap = m["heads"], m["dim"], m["vdim"], float(m["gate_cap"])
    q = (h @ W[p + "q"].T).view(T, H, D) * D ** -0.5
    k = (h @ W[p + "k"].T).view(T, H, D)
    v = (h @ W[p + "v"].T).view(T, H, Dv)
    i = cap * torch.tanh((h @ W[p + "i"].T + W[p + "i.b"]) / cap)
    f = log_sigmoid(cap * torch.tanh((h @ W[p + "f"].T + W[p + "f.b"]) / cap))
    o = torch.stack([matrix_memory(q[:, hd], k[:, hd], v[:, hd], i[:, hd], f[:, hd]) for hd in range(H)], 1)
    y = unit_rms(o, eps).reshape(T, H * Dv) * W[p + "norm"] * torch.sigmoid(h @ W[p + "g"].T)
    return y @ W[p + "o"].T


# --------------------------------------------------------------------------- state-space duality
def ssd_head(x, B, C, dt, A_log, D):
    """One head: x [T, Dv], B, C [T, N], dt [T]."""
    S = torch.zeros(B.shape[1], x.shape[1], dtype=F64)
    out = []
    for t in range(x.shape[0]):
        S = math.exp(-math.exp(float(A_log)) * float(dt[t])) * S + float(dt[t]) * torch.outer(B[t], x[t])
        out.append(S.T @ C[t] + float(D) * x[t])
    return torch.stack(out)


def mamba2_mixer(h, W, p, m, eps):
    T = h.shape[0]
    H, Dv, N, G = m["heads"], m["vdim"], m["state"], m["groups"]
    inner = H * Dv
    z, xBC, dt = torch.split(h @ W[p + "in"].T, [inner, inner + 2 * G * N, H], dim=-1)
    xBC = silu(causal_conv(xBC, W[p + "conv"], W[p + "conv.b"]))
    x, B, C = torch.split(xBC, [inner, G * N, G * N], dim=-1)
    x, B, C = x.view(T, H, Dv), B.reshape(T, G, N), C.reshape(T, G, N)
    dt = softplus(dt + W[p + "dt_bias"])
    y = torch.stack([ssd_head(x[:, hd], B[:, hd // (H // G)], C[:, hd // (H // G)], dt[:, hd], W[p + "A_log"][hd],
                              W[p + "D"][hd]) for hd in range(H)], 1).reshape(T, inner)
    ng = int(m["norm_groups"])
    y = unit_rms((y * silu(z)).view(T, ng, inner // ng), eps).reshape(T, inner) * W[p + "norm"]
    return y @ W[p + "o"].T


# --------------------------------------------------------------------------------------- model
def dense_ff(h, W, p):
    a = torch.clamp(h @ W[p + "up"].T, min=0.0)
    return (a * a) @ W[p + "down"].T


def mixer(h, W, p, spec, eps, cache_round=None):
    if spec["type"] == "parallel":
        return parallel_mixer(h, W, p, spec["mixer"], eps, cache_round)
    if spec["type"] == "mlstm":
        return mlstm_mixer(h, W, p, spec["mixer"], eps)
    if spec["type"] == "mamba2":
        return mamba2_mixer(h, W, p, spec["mixer"], eps)
    raise ValueError(spec["type"])


def layer(x, W, i, spec, eps, cache_round=None):
    p = f"l{i}."
    x = x + mixer(offset_norm(x, W[p + "norm1"], eps), W, p + "mix.", spec, eps, cache_round)
    if spec.get("mlp") is not None:
        x = x + dense_ff(offset_norm(x, W[p + "norm2"], eps), W, p + "mlp.")
    return x


def forward(tokens, W, cfg, cache_round=None):
    """-> (logits [T, vocab], [residual after every layer])."""
    eps = float(cfg["norm"]["eps"])
    x = embed_tokens([int(t) for t in tokens], W, cfg)
    trail = []
    for i, spec in enumerate(cfg["layers"]):
        x = layer(x, W, i, spec, eps, cache_round)
        trail.append(x)
    return offset_norm(x, W["final.norm"], eps) @ W["embed"].T, trail


# ------------------------------------------------------------------------------ random checkpoints
def tensor_shapes(cfg) -> dict:
    """name -> shape of every tensor a checkpoint of this configuration holds. The rank of the decay's thin factors is no part
    of the configuration: `decay_rank` of a right mixer here, 5 without one."""
    W = int(cfg["width"])
    t = {"embed": (int(cfg["vocab"]), W), "pos": (int(cfg["max_positions"]), W), "embed.norm": (W,), "final.norm": (W,)}
    b = (cfg.get("embedding") or {}).get("bigram")
    if b:
        t["bigram"] = (int(b["buckets"]) + 1, W)
    for i, L in enumerate(cfg["layers"]):
        p, m = f"l{i}.", L["mixer"]
        t[p + "norm1"] = (W,)
        q = p + "mix."
        if L["type"] == "mlstm":
            H, D, Dv = m["heads"], m["dim"], m["vdim"]
            t.update({q + "q": (H * D, W), q + "k": (H * D, W), q + "v": (H * Dv, W), q + "g": (H * Dv, W), q + "o": (W, H * Dv),
                      q + "norm": (H * Dv,), q + "i": (H, W), q + "i.b": (H,), q + "f": (H, W), q + "f.b": (H,)})
        elif L["type"] == "mamba2":
            H, inner, C = m["heads"], m["heads"] * m["vdim"], m["heads"] * m["vdim"] + 2 * m["groups"] * m["state"]
            t.update({q + "in": (inner + C + H, W), q + "conv": (C, m["conv"]), q + "conv.b": (C,), q + "dt_bias": (H,),
                      q + "A_log": (H,), q + "D": (H,), q + "norm": (inner,), q + "o": (W, inner)})
        else:
            a, r = m["left"], m["right"]
            H, G, D, Dv = a["heads"], a["kv_heads"], a["dim"], a["vdim"]
            for nm, n in (("q", H * D), ("k", G * D), ("v", G * Dv)):
                t.update({q + "left." + nm: (n, W), q + "left." + nm + ".conv": (n, a["conv"])})
            t.update({q + "left.o": (W, H * Dv), q + "left.out": (W,)})
            H, n, R = r["heads"], r["heads"] * r["dim"], int(r.get("decay_rank", 5))
            for c in "rkvgw":
                t[q + "right.mu." + c] = (W,)
            for c in "rkvg":
                t[q + "right." + c] = (n, W)
            t.update({q + "right.w1": (R, W), q + "right.w2": (n, R), q + "right.w0": (n,), q + "right.u": (H, r["dim"]),
                      q + "right.norm": (n,), q + "right.o": (W, n), q + "right.out": (W,)})
        if L.get("mlp") is not None:
            t.update({p + "norm2": (W,), p + "mlp.up": (L["mlp"]["ff"], W), p + "mlp.down": (W, L["mlp"]["ff"])})
    return t


def random_weights(cfg, seed: int) -> dict:
    """A seeded checkpoint, float64 values that bfloat16 holds exactly. Scales keep activations of order one and make the
    hashed pairs, the positions, the old taps, the shifted inputs, the gates and the skips all matter, with states that remember
    for tens to hundreds of tokens."""
    g = torch.Generator().manual_seed(seed)
    scale = float((cfg.get("embedding") or {}).get("scale", 1.0))
    out = {}
    for name, shape in tensor_shapes(cfg).items():
        leaf = name.rsplit(".", 1)[-1]
        x = torch.randn(tuple(shape), generator=g)
        if name in ("embed.norm", "final.norm") or leaf in ("norm1", "norm2"):
            x = 0.3 * x
        elif leaf in ("norm", "out"):
            x = 1.0 + 0.3 * x
        elif name == "embed":
            x = x / max(scale, 1.0)
        elif name in ("bigram", "pos"):
            x = 0.7 * x
        elif name.endswith(".f.b"):
            x = 2.5 + 1.5 * x
        elif name.endswith(".i.b"):
            x = -0.5 + x
        elif name.endswith("conv.b"):
            x = 0.3 * x
        elif leaf in ("i", "f"):
            x = 1.5 * x / shape[-1] ** 0.5
        elif leaf == "w0":
            x = -2.5 + 1.5 * x
        elif leaf == "dt_bias":
            x = -2.0 + x
        elif leaf == "A_log":
            x = 0.7 * x
        elif leaf in ("D", "u") or ".mu." in name:
            x = 0.5 + 0.4 * x
        elif leaf == "conv":
            x = x / shape[-1] ** 0.5
        elif ".left." in name and leaf in ("q", "k"):
            x = 1.7 * x / shape[-1] ** 0.5
        else:
            x = x / shape[-1] ** 0.5
        out[name] = x.to(torch.bfloat16).to(F64)
    return out
