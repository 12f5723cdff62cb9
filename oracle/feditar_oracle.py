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
