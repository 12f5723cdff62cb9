"""Cases of the Gokolix tests, written once and run by the CPU test file (host logic with the package's torch
restatement of the kernels) and the GPU test file (the HIP kernels): every mechanism alone against
oracle/gokolix_oracle.py, then the engine on whole prompts, token-by-token decoding, portions, mixed batches,
reused pages and slots, long decoding and greedy generation."""
from __future__ import annotations

import torch

from oracle import gokolix_oracle as oracle
from tests import _gokolix as K

F64 = torch.float64


def _dt(name):
    return {"float32": torch.float32, "bfloat16": torch.bfloat16}[name]


def _near(got, want, tol, what):
    got, want = got.detach().cpu().to(F64), want.to(F64)
    err = (got - want).abs().max().item()
    assert err <= tol * max(1.0, want.abs().max().item()), (what, err)


# Steps that feed two sequences through three state slots: whole, a sequence on a slot another one just used, portions down to
# one token, a portion beside single tokens. Each entry: [(id, tokens, slot)].
LENS = {"a": 75, "b": 40}
WALK = [[("a", 75, 1)], [("b", 30, 1), ("a", 3, 2)], [("a", 1, 2), ("b", 1, 1)], [("a", 36, 2)], [("b", 9, 1), ("a", 2, 2)], [("a", 33, 2)]]


def _walk(fn, check):
    """fn([(id, lo, hi, slot)]) -> rows of the step; check(rows, id, lo). Every sequence starts over when it has ended."""
    at = {i: 0 for i in LENS}
    for entries in WALK:
        parts = [(i, at[i], at[i] + n, s) for i, n, s in entries]
        rows = fn(parts)
        row = 0
        for i, lo, hi, _ in parts:
            check(rows[row:row + hi - lo], i, lo)
            row += hi - lo
            at[i] = 0 if hi == LENS[i] else hi


def _step(parts, device, tables=None):
    return K.make_step([hi - lo for _, lo, hi, _ in parts], [lo for _, lo, _, _ in parts], [s for *_, s in parts],
                       tables or [[0]] * len(parts), device)


def _cut(x, parts):
    return torch.cat([x[i][lo:hi] for i, lo, hi, _ in parts])


def _tables(g, page, longest=80):
    per = -(-longest // page)
    order = torch.randperm(2 * per, generator=g).tolist()
    return {"a": order[:per], "b": order[per:]}, 2 * per


def _slots(table, page, lo, n):
    return [table[p // page] * page + p % page for p in range(lo, lo + n)]


# ------------------------------------------------------------------------------- single mechanisms
def case_embedding_and_split(device, dtype):
    """The scaled rows as an f32 residual, the rows themselves, and the residual as two bf16 numbers whose products with a bf16
    weight, summed in f32, are those of the residual to f32-like accuracy; widths in and out of multiples of four."""
    from light_vllm_amd import mix_ops
    g = torch.Generator().manual_seed(1)
    for W, vocab, T, scale in ((48, 50, 7, 3.0), (37, 20, 5, 0.3), (1000, 30, 300, 1.0), (64, 9, 1, 0.7)):
        table = torch.randn(vocab, W, generator=g).to(_dt(dtype))
        ids = torch.randint(0, vocab, (T,), generator=g)
        x, rows, split = mix_ops.scaled_embedding(ids.to(device), table.to(device), scale, True, dtype == "bfloat16")
        want = table[ids].to(F64) * scale
        _near(x, want, 1e-6, ("residual", W))
        assert torch.equal(rows.cpu(), table[ids])
        if dtype == "bfloat16":
            assert torch.equal(split.cpu(), mix_ops.residual_split(x.clone()).cpu())
            y = torch.randn(T, W, generator=g).to(torch.bfloat16)
            big = (100 * torch.randn(T, W, generator=g)).to(device)
            base = big.cpu().to(F64)
            s = mix_ops.residual_split(big, y.to(device))
            want = base + y.to(F64)
            _near(big, want, 1e-6, ("updated", W))
            both = s[:, :W].cpu().to(F64) + s[:, W:].cpu().to(F64)
            assert ((both - want).abs() <= 2.0 ** -16 * want.abs() + 1e-30).all()
            w = torch.randn(24, W, generator=g).to(torch.bfloat16)
            add = torch.randn(T, 24, generator=g)
            got = mix_ops.mm_f32(s, torch.cat([w, w], 1).t().to(device), add.to(device))
            ref = want @ w.to(F64).T + add.to(F64)
            assert got.dtype == torch.float32
            _near(got, ref, 3e-5, ("product", W))
            assert (want.to(torch.bfloat16).to(F64) @ w.to(F64).T + add.to(F64) - ref).abs().max() > 3e-4 * ref.abs().max()   # one number would not do


def case_yarn_and_bias_tables(device):
    """Scaled frequencies and their factor for ramps inside, clipped at either end and of no width; bias tables spelled out by
    distance, cut by the window or where the last row begins."""
    from light_vllm_amd import mix_ops
    for dims, base, s in ((16, 10000.0, (4.0, 512, 32.0, 1.0)), (8, 100.0, (8.0, 64, 4.0, 0.5)), (64, 50000.0, (40.0, 4096, 32.0, 1.0)),
                          (2, 30.0, (1.0, 16, 2.0, 1.0)), (6, 10.0, (3.0, 100000, 1.5, 1.0)), (12, 500.0, (2.0, 8, 64.0, 16.0)),
                          (10, 1000.0, (2.0, 64, 1.0, 1.0))):
        rot = {"dims": dims, "base": base, "scaling": dict(zip(("factor", "original", "fast", "slow"), s))}
        f, mag = oracle.yarn(rot)
        got = mix_ops.rotary_inv_freq(dims, base, device, rot["scaling"]).cpu().to(F64)
        assert ((got - torch.tensor(f, dtype=F64)).abs() <= 1e-7 * torch.tensor(f, dtype=F64)).all(), (dims, base, s)
        assert abs(mix_ops.rotary_magnitude(rot["scaling"]) - mag) < 1e-12
    assert mix_ops.rotary_magnitude(None) == 1.0 and mix_ops.rotary_magnitude({"factor": 4.0, "low": 1.0, "high": 4.0, "original": 64}) == 1.0
    g = torch.Generator().manual_seed(2)
    for B, far, window, H in ((32, 128, 1 << 30, 3), (8, 15, 19, 2), (12, 40, 7, 1), (2, 3, 50, 4), (5, 33, 100, 2), (4, 1000, 400, 1), (16, 9, 64, 2)):
        rel = torch.randn(B, H, generator=g)
        table = mix_ops.distance_bias(rel.to(device), far, window).cpu()
        for n in range(min(window, 3 * far)):
            want = rel[oracle.distance_bucket(n, B, far)]
            assert torch.equal(table[:, min(n, table.size(1) - 1)], want), (B, far, n)


def case_head_norm_store(device, dtype):
    """Queries normed per head and weighted; keys stored as they are with 1 / rms beside them, in pages of any order; heads small
    enough for eps to count; head sizes in and out of what four entries a lane take."""
    from light_vllm_amd import mix_ops
    g = torch.Generator().manual_seed(3)
    tol = 1e-5 if dtype == "float32" else 1e-2
    for H, G, D, page, pad in ((4, 2, 12, 16, 4), (3, 3, 10, 16, 1), (5, 1, 66, 64, 0), (8, 4, 96, 32, 8), (2, 1, 256, 16, 0), (2, 2, 300, 16, 3), (1, 1, 1, 16, 2)):
        eps = 1e-3
        xs = {i: torch.randn(n, H * D + G * D + 2 * pad, generator=g).to(_dt(dtype)) for i, n in LENS.items()}
        xs["a"][3] *= 0.02
        w = 1 + 0.5 * torch.randn(D, generator=g)
        tables, pages = _tables(g, page)
        cache = torch.zeros(pages, page, G, D, dtype=_dt(dtype), device=device)
        ks = torch.zeros(pages, page, G, device=device)
        wd = w.to(device)

        def run(parts):
            return mix_ops.head_norm_store(_cut(xs, parts).to(device), pad, pad + H * D, wd, cache, ks, _step(parts, device, [tables[i] for i, *_ in parts]),
                                           H, G, D, eps)

        def check(rows, i, lo):
            n = len(rows)
            x = xs[i][lo:lo + n].to(F64)
            _near(rows, (oracle.unit_rms(x[:, pad:pad + H * D].view(n, H, D), eps) * w.to(F64)).reshape(n, H * D), tol, ("q", H, D, i, lo))
            sl = _slots(tables[i], page, lo, n)
            assert torch.equal(cache.view(-1, G * D)[sl].cpu(), xs[i][lo:lo + n, pad + H * D:pad + H * D + G * D])
            k = x[:, pad + H * D:pad + H * D + G * D].view(n, G, D)
            _near(ks.view(-1, G)[sl], 1 / torch.sqrt((k * k).mean(-1) + eps), 2e-6, ("key factor", H, D, i, lo))

        _walk(run, check)


def case_latent_store(device, dtype):
    """The normed latent and the rotated positional key part in the cache row, the rotated query parts behind the place of the
    absorbed queries (which stay untouched): both pairings, part of the entries rotated, none, a factor on cosines and sines."""
    from light_vllm_amd import mix_ops
    g = torch.Generator().manual_seed(4)
    tol = 1e-5 if dtype == "float32" else 1e-2
    for H, Dn, Dr, R, dims, page, pad, inter, mag in ((3, 12, 8, 24, 8, 16, 4, True, 1.2), (2, 5, 6, 9, 6, 16, 1, True, 0.8), (1, 4, 0, 12, 0, 32, 0, True, 1.0),
                                                      (4, 16, 16, 64, 8, 64, 8, True, 1.1), (2, 8, 8, 20, 8, 16, 0, False, 1.3), (5, 64, 32, 1100, 32, 16, 8, True, 1.25)):
        eps = 1e-4
        nq = H * (Dn + Dr)
        rot = {"dims": max(dims, 2), "base": 200.0}
        xs = {i: torch.randn(n, pad + nq + R + Dr, generator=g).to(_dt(dtype)) for i, n in LENS.items()}
        w = 1 + 0.3 * torch.randn(R, generator=g)
        freq = mix_ops.rotary_inv_freq(rot["dims"], rot["base"], device)
        tables, pages = _tables(g, page)
        cache = torch.zeros(pages, page, R + Dr, dtype=_dt(dtype), device=device)
        wd = w.to(device)

        def turn(x):
            """All positions from 0; a pair (i, i + dims/2) is brought to the interleaved places and back."""
            if not dims:
                return x
            y = x.clone()
            if inter:
                y[..., :dims] = oracle.rotate(x[..., :dims], rot) * mag
            else:
                half = dims // 2
                z = torch.stack([x[..., :half], x[..., half:dims]], -1).flatten(-2)
                z = oracle.rotate(z, rot) * mag
                y[..., :half], y[..., half:dims] = z[..., 0::2], z[..., 1::2]
            return y

        want_q = {i: turn(x.to(F64)[:, pad:pad + nq].view(-1, H, Dn + Dr)[..., Dn:]) for i, x in xs.items()}
        want_k = {i: torch.cat([oracle.unit_rms(x.to(F64)[:, pad + nq:pad + nq + R], eps) * w.to(F64), turn(x.to(F64)[:, pad + nq + R:])], -1)
                  for i, x in xs.items()}

        def run(parts):
            x = _cut(xs, parts).to(device)
            q = torch.full((len(x), H, R + Dr), 7.0, dtype=_dt(dtype), device=device)
            mix_ops.latent_store(x, pad, pad + nq, wd, freq, mag, q, cache, _step(parts, device, [tables[i] for i, *_ in parts]), H, Dn, Dr, R, dims, inter, eps)
            return q

        def check(rows, i, lo):
            n = len(rows)
            assert (rows[..., :R] == 7.0).all()
            _near(rows[..., R:], want_q[i][lo:lo + n], tol, ("query part", H, Dr, i, lo)) if Dr else None
            _near(cache.view(-1, R + Dr)[_slots(tables[i], page, lo, n)], want_k[i][lo:lo + n], tol, ("row", H, R, Dr, i, lo))

        _walk(run, check)


def _attend(q, k, v, factor, bias, sink, scale, window, keep=0, chunk=0):
    """Plain softmax over what each position sees. q [L, H, D], k [L, G, D], v [L, G, Dv], factor [L, G], bias(n, h), sink [H]."""
    L, H, _ = q.shape
    G = k.shape[1]
    out = torch.zeros(L, H, v.shape[2], dtype=F64)
    n = torch.arange(L)[:, None] - torch.arange(L)[None, :]
    seen = ((torch.arange(L)[:, None] // chunk == torch.arange(L)[None, :] // chunk) if chunk else n < window) | (torch.arange(L)[None, :] < keep)
    seen &= n >= 0
    for h in range(H):
        g = h // (H // G)
        s = (q[:, h] @ k[:, g].T) * scale * factor[None, :, g] + bias(n.clamp(min=0), h)
        s = s.masked_fill(~seen, float("-inf"))
        top = s.max(-1, keepdim=True).values.clamp(min=float(sink[h]))
        e = torch.exp(s - top)
        out[:, h] = (e / (e.sum(-1, keepdim=True) + torch.exp(sink[h] - top))) @ v[:, g]
    return out.reshape(L, -1)


def case_extended_attention(device, dtype):
    """Unnormed keys with a factor each, a bias by distance and head, learned sinks, windows. Beacon keys (the first token, either
    side of page and tile borders, far back) stand out among hundreds, and single distances carry a large bias; a window one token
    off, a missing factor, a bias one distance off or a missing sink moves the answer by far more than the tolerance. Keys as
    values and values of their own, outputs in wider rows, prompt-, decode- and portion-shaped launches."""
    from light_vllm_amd import mix_ops
    g = torch.Generator().manual_seed(5)
    for H, G, D, Dv, page, L, window, nb, tied, keep, chunk in (
            (4, 2, 12, 12, 16, 75, 19, 8, True, 0, 0), (5, 1, 32, 32, 16, 300, 130, 90, True, 0, 0), (2, 2, 96, 96, 64, 210, 65, 65, True, 0, 0),
            (3, 3, 16, 48, 16, 140, 64, 300, False, 0, 0), (9, 1, 16, 32, 32, 150, 33, 5, False, 3, 0), (4, 1, 64, 64, 64, 200, 1 << 30, 40, True, 0, 50),
            (2, 1, 144, 144, 64, 170, 100, 64, True, 0, 0), (1, 1, 40, 40, 16, 90, 1, 1, True, 0, 0), (2, 1, 16, 16, 64, 1250, 1200, 1150, True, 0, 0),
            (6, 2, 128, 128, 64, 130, 128, 100, True, 0, 0)):
        k = 0.3 * torch.randn(L, G, D, generator=g)
        k[:, :, 0] += 2.0 * torch.randn(L, G, generator=g)                                 # what the factors act on
        beacons = sorted({0, page - 1, page, L // 2, min(63, L - 1), min(64, L - 1)})
        for j in beacons:
            k[j, :, D - 1] += 4.0
        v = k if tied else torch.randn(L, G, Dv, generator=g)
        q = 0.3 * torch.randn(L, H, D, generator=g)
        q[:, :, D - 1] += 2.5
        q[:, :, 0] += 1.0
        factor = 0.2 + 1.5 * torch.rand(L, G, generator=g)
        factor[beacons] = 1.8
        table = 0.5 * torch.randn(H, nb, generator=g)
        edge = min(window, L) - 1
        if edge < nb:
            table[:, edge] += 4.0                                                          # the oldest key of a window
        table[:, min(16, nb - 1)] += 3.0
        sink = 4.0 + 0.5 * torch.randn(H, generator=g)
        sink[0] = 7.0
        scale = 0.4
        k, v, q = (t.to(_dt(dtype)).float() for t in (k, v, q))
        k6, v6, q6, f6, t6, s6 = (t.to(F64) for t in (k, v, q, factor, table, sink))
        args = dict(factor=f6, bias=lambda n, h: t6[h][n.clamp(max=nb - 1)], sink=s6, scale=scale, window=window, keep=keep, chunk=chunk)
        want = _attend(q6, k6, v6, **args)
        tol = 2e-4 if dtype == "float32" else 3e-2
        far = want.abs().max().item()
        wrong = [dict(factor=torch.ones_like(f6)), dict(sink=torch.full_like(s6, -1e4))]
        if window < L and not chunk:
            wrong += [dict(window=window + 1)] + ([dict(window=window - 1)] if window > 1 else [])
        if nb > 1:
            wrong.append(dict(bias=lambda n, h: t6[h][(n + 1).clamp(max=nb - 1)]))
        for other in wrong:
            assert (_attend(q6, k6, v6, **{**args, **other}) - want).abs().max().item() > 3 * tol * far, (H, D, list(other))
        per = -(-L // page)
        tb = torch.randperm(per + 2, generator=g)[:per].tolist()
        kc = torch.zeros(per + 2, page, G, D, dtype=_dt(dtype))
        vc = torch.zeros(per + 2, page, G, Dv, dtype=_dt(dtype))
        ks = torch.zeros(per + 2, page, G)
        for p in range(L):
            at = tb[p // page], p % page
            kc[at], vc[at], ks[at] = k[p].to(kc.dtype), v[p].to(vc.dtype), factor[p]
        kc, ks, td, sd = kc.to(device), ks.to(device), table.to(device), sink.to(device)
        vc = kc if tied else vc.to(device)
        qd = q.reshape(L, H * D).to(_dt(dtype)).to(device)

        def run(step, rows, what):
            wide = torch.full((len(rows), H * Dv + 24), 7.0, dtype=_dt(dtype), device=device)
            got = mix_ops.window_pool_attention(qd[rows].contiguous(), kc, vc, None, None, None, step, H, G, D, Dv, window, 0, scale, has_sink=False,
                                                sinks=sd, keep_first=keep, chunk=chunk, key_scale=ks, dist_bias=td, out=wide[:, 8:8 + H * Dv])
            _near(got, want[rows], tol, (what, H, G, D, Dv, page, window))
            assert (wide[:, :8] == 7.0).all() and (wide[:, 8 + H * Dv:] == 7.0).all()

        run(K.make_step([L], [0], [0], [tb], device), list(range(L)), "prompt")
        idx = sorted({i for j in beacons for i in (j - 1, j, j + 1, j + edge, j + edge + 1) if 0 <= i < L} | set(range(L - 5, L)))
        run(K.make_step([1] * len(idx), idx, [0] * len(idx), [tb] * len(idx), device), idx, "decode")
        run(K.make_step([1], [L - 1], [0], [tb], device), [L - 1], "one sequence")
        rows = list(range(page - 1, L - 20)) + list(range(5)) + list(range(L - 19, L))
        run(K.make_step([L - 20 - page + 1, 5, 19], [page - 1, 0, L - 19], [0, 1, 2], [tb] * 3, device), rows, "portions")
        run(K.make_step([2, 1], [L - 2, L // 2], [0, 1], [tb] * 2, device), [L - 2, L - 1, L // 2], "two tokens beside one")


def case_windowed_latent_attention(device, dtype):
    """The latent mixer alone on its paged cache: queries straight from the input, YaRN rotation, window and sinks, outputs written
    into columns of a wider row; whole, in portions, token by token, on pages another sequence used."""
    from light_vllm_amd.layers.latent_attention import LatentAttention
    from light_vllm_amd.utils.context import reset_context, set_context
    g = torch.Generator().manual_seed(6)
    for m, page in ((K.LAT_A, 16), (K.LAT_B, 16), (K.CFG_WIDE["layers"][2]["mixer"], 64)):
        W, eps = 32, 1e-5
        H, Dn, Dr, Dv, R = (m[k] for k in ("heads", "dim", "rot_dim", "vdim", "kv_rank"))
        Wt = {"q": 1.5 * torch.randn(H * (Dn + Dr), W, generator=g) / W ** 0.5, "dkv": torch.randn(R + Dr, W, generator=g) / W ** 0.5,
              "dkv.norm": 1 + 0.3 * torch.randn(R, generator=g), "uk": torch.randn(H * Dn, R, generator=g) / R ** 0.5,
              "uv": torch.randn(H * Dv, R, generator=g) / R ** 0.5, "sink": torch.randn(H, generator=g)}
        Wt = {n: t.to(torch.bfloat16) for n, t in Wt.items()}
        hs = {i: torch.randn(n, W, generator=g).to(_dt(dtype)) for i, n in LENS.items()}
        eye = {"mix." + n: t.to(F64) for n, t in Wt.items()} | {"mix.o": torch.eye(H * Dv, dtype=F64)}
        want = {i: oracle.latent_attention(h.to(F64), eye, "mix.", m, eps) for i, h in hs.items()}
        old = torch.get_default_dtype()
        torch.set_default_dtype(_dt(dtype))
        try:
            mix = LatentAttention(W, H, Dn, Dv, None, R, m["scale"], rot_dim=Dr, rot_dims=Dr, rot_base=m["rot"]["base"], gate=None, norm_eps=eps,
                                  interleaved=True, rot_scaling=m["rot"]["scaling"], window=m["mask"]["size"], sink=True, fused=True).to(device)
        finally:
            torch.set_default_dtype(old)
        with torch.no_grad():
            mix.uk.copy_(Wt["uk"].view(mix.uk.shape))
            mix.uv.copy_(Wt["uv"].view(H, Dv, R).transpose(1, 2))
            mix.kv_norm_weight.copy_(Wt["dkv.norm"])
            mix.sink.copy_(Wt["sink"])
        tables, pages = _tables(g, page)
        mix.bind_cache(pages, page, 3, device, _dt(dtype))
        w_in = torch.cat([Wt["q"], Wt["dkv"]]).to(_dt(dtype)).to(device)

        @torch.no_grad()
        def run(parts):
            h = _cut(hs, parts).to(device)
            proj = torch.cat([h[:, :8], h @ w_in.t()], 1)
            wide = torch.zeros(len(h), H * Dv + 8, dtype=_dt(dtype), device=device)
            set_context(True, ragged=_step(parts, device, [tables[i] for i, *_ in parts]))
            try:
                return mix(h, proj, 8, out=wide[:, :H * Dv])
            finally:
                reset_context()

        tol = 1e-4 if dtype == "float32" else 6e-2
        _walk(run, lambda rows, i, lo: _near(rows, want[i][lo:lo + len(rows)], tol, ("latent", H, R, i, lo)))


def case_recurrence(device, dtype):
    """Gates from block-diagonal matrices, decays from almost 1 to almost 0, the state from nothing and from what a portion left,
    the gelu branch: blocks the matrix cores take and others, one block and many, inputs and outputs as columns of wider rows of
    any alignment."""
    from light_vllm_amd import mix_ops
    g = torch.Generator().manual_seed(7)
    tol = 2e-5 if dtype == "float32" else 2e-2
    for N, blocks, pad in ((64, 2, 8), (96, 1, 8), (256, 2, 3), (160, 5, 0), (30, 3, 1), (40, 1, 0), (6, 6, 2), (600, 2, 8), (320, 1, 8)):
        n = N // blocks
        gw = (1.5 * torch.randn(blocks, 2, n, n, generator=g) / n ** 0.5).to(torch.bfloat16)
        gb = torch.randn(blocks, 2, n, generator=g)
        lam = -3.0 + 2.0 * torch.randn(N, generator=g)
        lam[0], lam[-1] = -14.0, 3.0                      # holds on for ever, forgets at once
        gb[0, 0, 0] = 4.0
        us = {i: torch.randn(t, N, generator=g).to(_dt(dtype)) for i, t in LENS.items()}
        ys = {i: (1.5 * torch.randn(t, N + 2 * pad, generator=g)).to(_dt(dtype)) for i, t in LENS.items()}
        Wt = {"ra": gw[:, 0].to(F64), "ri": gw[:, 1].to(F64), "ra.b": gb[:, 0].to(F64), "ri.b": gb[:, 1].to(F64)}
        want = {}
        for i, u in us.items():
            r, x = oracle.lru_gates(u.to(F64), Wt, "", blocks)
            want[i] = oracle.lru_scan(u.to(F64), r, x, lam.to(F64)) * oracle.gelu_tanh(ys[i].to(F64)[:, pad:pad + N])
        state = torch.full((3, N), 9.0, device=device)
        rate = (-8.0 * oracle.softplus(lam.to(F64))).float().to(device)
        gwd, gbd = gw.to(_dt(dtype)).to(device), gb.to(device)

        def run(parts):
            y = _cut(ys, parts).to(device)
            wide = torch.full((len(y), N + 2 * pad + 1), 7.0, dtype=_dt(dtype), device=device)
            got = mix_ops.gated_linear_recurrence(_cut(us, parts).to(device), y[:, pad:pad + N], gwd, gbd, rate, state, _step(parts, device), blocks,
                                                  out=wide[:, pad:pad + N])
            assert (wide[:, :pad] == 7.0).all() and (wide[:, pad + N:] == 7.0).all()
            return got

        _walk(run, lambda rows, i, lo: _near(rows, want[i][lo:lo + len(rows)], tol, ("recurrence", N, blocks, i, lo)))


def case_recurrence_long_and_many(device, dtype):
    """Sequences of many tiles beside short ones (cut into parts where a launch has few workgroups; some parts of a short sequence
    are empty), whole and continued; and single tokens of more sequences than a tile of the step kernel holds, slots in any order,
    new sequences among them."""
    from light_vllm_amd import mix_ops
    g = torch.Generator().manual_seed(8)
    tol = 2e-5 if dtype == "float32" else 2e-2
    for N, blocks in ((64, 2), (192, 1), (20, 2)):
        n = N // blocks
        gw = (torch.randn(blocks, 2, n, n, generator=g) / n ** 0.5).to(torch.bfloat16)
        gb = torch.randn(blocks, 2, n, generator=g)
        lam = -6.0 + 2.0 * torch.randn(N, generator=g)    # remembers hundreds of tokens: the parts must hand their sums on
        Wt = {"ra": gw[:, 0].to(F64), "ri": gw[:, 1].to(F64), "ra.b": gb[:, 0].to(F64), "ri.b": gb[:, 1].to(F64)}
        rate = (-8.0 * oracle.softplus(lam.to(F64))).float().to(device)
        gwd, gbd = gw.to(_dt(dtype)).to(device), gb.to(device)
        lens = [700, 130, 3, 64, 321]
        us = [torch.randn(t, N, generator=g).to(_dt(dtype)) for t in lens]
        ys = [torch.randn(t, N, generator=g).to(_dt(dtype)) for t in lens]
        want = []
        for u, y in zip(us, ys):
            r, x = oracle.lru_gates(u.to(F64), Wt, "", blocks)
            want.append(oracle.lru_scan(u.to(F64), r, x, lam.to(F64)) * oracle.gelu_tanh(y.to(F64)))
        for cuts in ([lens], [[433, 2, 1, 60, 257], [267, 128, 2, 4, 64]]):
            state = torch.full((8, N), 9.0, device=device)
            slots, at = [5, 0, 7, 2, 3], [0] * len(lens)
            for take in cuts:
                u = torch.cat([x[a:a + t] for x, a, t in zip(us, at, take)]).to(device)
                y = torch.cat([x[a:a + t] for x, a, t in zip(ys, at, take)]).to(device)
                got = mix_ops.gated_linear_recurrence(u, y, gwd, gbd, rate, state, K.make_step(take, at, slots, [[0]] * 5, device), blocks)
                row = 0
                for b, t in enumerate(take):
                    _near(got[row:row + t], want[b][at[b]:at[b] + t], tol, ("parts", N, blocks, b, at[b]))
                    row += t
                    at[b] += t
        B = 37
        slots = torch.randperm(B + 3, generator=g)[:B].tolist()
        ctx = [0 if b % 5 == 0 else 4 for b in range(B)]
        before = torch.randn(B + 3, N, generator=g)
        u, y = (torch.randn(B, N, generator=g).to(_dt(dtype)) for _ in range(2))
        state = before.clone().to(device)
        got = mix_ops.gated_linear_recurrence(u.to(device), y.to(device), gwd, gbd, rate, state, K.make_step([1] * B, ctx, slots, [[0]] * B, device), blocks)
        r, x = oracle.lru_gates(u.to(F64), Wt, "", blocks)
        log_a = rate.cpu().to(F64) * r
        old = torch.stack([before[s].to(F64) * (1.0 if c else 0.0) for s, c in zip(slots, ctx)])
        S = torch.exp(log_a) * old + torch.sqrt(-torch.expm1(2 * log_a)) * x * u.to(F64)
        _near(got, S * oracle.gelu_tanh(y.to(F64)), tol, ("single tokens", N, blocks))
        _near(state[slots], S, 1e-5, ("states", N, blocks))
        rest = [s for s in range(B + 3) if s not in slots]
        assert torch.equal(state[rest].cpu(), before[rest])


def case_gated_relu(device, dtype):
    """relu(gate) * up into columns of a wider row."""
    from light_vllm_amd import mix_ops
    g = torch.Generator().manual_seed(9)
    for T, ff, pad in ((5, 40, 8), (3, 17, 3), (2, 1024, 0), (1, 1, 1)):
        x = torch.randn(T, 2 * ff + pad, generator=g).to(_dt(dtype))
        wide = torch.full((T, ff + 2 * pad), 7.0, dtype=_dt(dtype), device=device)
        mix_ops.glu_act(x.to(device)[:, pad:], "relu", out=wide[:, pad:pad + ff])
        want = torch.clamp(x[:, pad:pad + ff].to(F64), min=0) * x[:, pad + ff:].to(F64)
        _near(wide[:, pad:pad + ff], want, 1e-6 if dtype == "float32" else 1e-2, ("glu", T, ff))
        assert (wide[:, :pad] == 7.0).all() and (wide[:, pad + ff:] == 7.0).all()


# ----------------------------------------------------------------------------------------- engine
def _model(tmp_path, cfg, seed):
    weights = oracle.random_weights(cfg, seed)
    return K.write_model(tmp_path / f"m{seed}", cfg, weights), weights


def _oracle_runs(cfg, weights, prompts):
    return {i: oracle.forward(t, weights, cfg)[0] for i, t in prompts.items()}


def case_checkpoint_placement(tmp_path):
    """Every tensor of a checkpoint lands where the oracle reads it: mixer and feed-forward side by side in the merged weights,
    both gate matrices, transposed value projections, the two halves of the loop's weight, the head on the token table, later
    passes on the first one's parameters; sizes that only the tensors give; what is missing, unknown or of another shape is refused."""
    import copy
    from light_vllm_amd.models.gokolix import GokolixConfig, GokolixForCausalLM
    from light_vllm_amd.models.registry import load_config, model_class
    cfg = copy.deepcopy(K.CFG_MAIN)
    weights = oracle.random_weights(cfg, 3)
    del cfg["layers"][3]["mixer"]["rel_rows"]
    model_dir = K.write_model(tmp_path / "m", cfg, weights)
    config = load_config(model_dir)
    assert isinstance(config, GokolixConfig) and model_class(config) is GokolixForCausalLM
    assert config.layers[3]["mixer"]["rel_rows"] == 8 and config.layers[0]["mixer"]["rel_rows"] == 12
    assert [i for i, _ in config.runs()] == [0, 1, 2, 3, 1, 2, 3, 1, 2, 3, 4, 5]
    assert [t for _, t in config.runs()] == [None, 0, None, None, 1, None, None, 2, None, None, None, None]
    old = torch.get_default_dtype()
    for dt in (torch.float32, torch.bfloat16):
        torch.set_default_dtype(dt)
        try:
            model = GokolixForCausalLM(config)
        finally:
            torch.set_default_dtype(old)
        model.load_weights(weights.items())
        assert sorted(model.weight_targets()) == sorted(weights)
        assert model.lm_head.weight is model.embed.weight
        W = 48
        w_in = weights["loop.in"]
        assert torch.equal(model.loop_x.double(), torch.cat([w_in[:, :W]] * 2, 1) if dt == torch.bfloat16 else w_in[:, :W])
        assert torch.equal(model.loop_x0.double(), w_in[:, W:])
        b1, b3, b2 = (model.layers[i].block for i in (1, 3, 2))
        assert torch.equal(b1.in_proj.weight.double(), torch.cat([weights["l1." + n] for n in ("mix.q", "mix.dkv", "mlp.gate", "mlp.up")]))
        assert torch.equal(b1.out_proj.weight.double(), torch.cat([weights["l1.mix.o"], weights["l1.mlp.down"]], 1))
        assert torch.equal(b1.mix.uv.transpose(1, 2).reshape(30, 24).double(), weights["l1.mix.uv"])
        assert torch.equal(b3.in_proj.bias.double(), torch.cat([weights["l3.mix.q.b"], weights["l3.mix.k.b"], torch.zeros(80, dtype=F64)]))
        assert torch.equal(b2.mix.gate_weight[:, 1].double(), weights["l2.mix.ri"])
        for r, (layer, _) in enumerate(model.order):
            first = model.layers[config.runs()[r][0]]
            assert layer.block.in_proj is first.block.in_proj and layer.norm1 is first.norm1
        assert model.order[4][0].block.mix is not model.order[1][0].block.mix
    short = dict(weights)
    del short["l2.mix.lam"]
    for broken, error in ((short, KeyError), ({**weights, "l0.mix.extra": torch.zeros(1)}, KeyError),
                          ({**weights, "loop.in": torch.zeros(48, 48)}, ValueError)):
        try:
            model.load_weights(broken.items())
            raise AssertionError("a wrong checkpoint went unnoticed")
        except error:
            pass
    for change in (lambda c: c["layers"][0].update(type="recurrent"), lambda c: c["layers"][2]["mixer"].pop("blocks"),
                   lambda c: c["layers"][0]["mlp"].update(kind="moe"), lambda c: c.pop("width"), lambda c: c["layers"][0]["mixer"].update(vdim=5),
                   lambda c: c["loop"].update(stop=7), lambda c: c["layers"][0]["mixer"].update(bias_max=6), lambda c: c["layers"][1]["mixer"].pop("rot")):
        bad = copy.deepcopy(K.CFG_MAIN)
        change(bad)
        try:
            GokolixConfig.from_dict(bad)
            raise AssertionError("a wrong configuration went unnoticed")
        except ValueError:
            pass


def case_layer_by_layer(device, tmp_path, cfg=None):
    """The f32 residual after every layer run of a whole prompt, against the oracle: names the first layer that differs."""
    from light_vllm_amd.engine.trace_replay import TraceReplayer
    cfg = cfg or K.CFG_MAIN
    model_dir, weights = _model(tmp_path, cfg, 4)
    tokens = K.tokens_for(cfg, 27, 5)
    want = oracle.forward(tokens, weights, cfg)[1]
    rp = TraceReplayer(model_dir, "float32", 64, device=device, slots=2, page=16)
    try:
        model = rp.engine.model_runner.model
        model.layer_outputs = []
        rp.step([{"id": "a", "tokens": tokens, "want": []}], ["a"])
        got = [x.cpu() for x in model.layer_outputs]
    finally:
        rp.close()
    assert len(got) == len(want)
    for i, (a, b) in enumerate(zip(got, want)):
        assert (a.to(F64) - b).abs().max().item() <= 3e-4 * b.abs().max().item(), f"layer run {i}"


def case_engine_schedules(device, dtype, tmp_path, cfg=None, seed=5):
    """Whole prompts, token-by-token decoding, portions down to two tokens and mixed batches of unequal requests give the logits
    of the whole-sequence oracle at every position: the first tokens, every page border (pages of 16 tokens), both sides of every
    window, portions shorter than a filter and cuts inside it."""
    cfg = cfg or K.CFG_MAIN
    model_dir, weights = _model(tmp_path, cfg, seed)
    prompts = {"a": K.tokens_for(cfg, 53, 1), "b": K.tokens_for(cfg, 21, 2), "c": K.tokens_for(cfg, 38, 3)}
    want = _oracle_runs(cfg, weights, prompts)
    schedules = {
        "whole": [[("a", 53)], [("b", 21)], [("c", 38)]],
        "decode": [[("a", 9)]] + [[("a", 1)]] * 44 + [[("b", 1)]] * 21,
        "portions": [[("a", n)] for n in (2, 3, 11, 2, 16, 1, 17, 1)] + [[("c", n)] for n in (16, 16, 2, 2, 2)],
        "mixed": [[("a", 5), ("b", 2)], [("a", 1), ("b", 7), ("c", 30)], [("c", 1), ("a", 20)], [("b", 12), ("a", 1)],
                  [("a", 26), ("c", 2)], [("c", 5)]],
    }
    for name, schedule in schedules.items():
        got = K.replay(model_dir, dtype, device, prompts, schedule, max_tokens=128, page=16, slots=3)
        for i, logits in got.items():
            if len(logits):
                err = K.rel_err(logits, want[i][:len(logits)])
                assert err <= K.TOL[dtype], (name, i, err)


def case_engine_random_config(device, dtype, tmp_path, seed):
    """A drawn configuration, prompts of a few hundred tokens on pages of 64: whole, and cut into unequal portions beside single
    tokens of another request, against the oracle at every position."""
    cfg = K.random_config(seed)
    model_dir, weights = _model(tmp_path, cfg, seed)
    prompts = {"a": K.tokens_for(cfg, 210, seed), "b": K.tokens_for(cfg, 75, seed + 1)}
    want = _oracle_runs(cfg, weights, prompts)
    schedules = {
        "whole": [[("a", 210)], [("b", 75)]],
        "mixed": [[("a", 63)], [("a", 2), ("b", 70)], [("a", 100), ("b", 1)], [("a", 1), ("b", 1)], [("a", 44), ("b", 1)], [("b", 2)]],
    }
    for name, schedule in schedules.items():
        got = K.replay(model_dir, dtype, device, prompts, schedule, max_tokens=384, page=64, slots=2)
        for i, logits in got.items():
            err = K.rel_err(logits, want[i])
            assert err <= K.TOL[dtype], (seed, name, i, err, cfg)


def case_engine_long(device, dtype, tmp_path):
    """Windows longer than pages and key tiles, states over hundreds of tokens: a prompt of 330 tokens whole, cut at odd
    places beside the single tokens of another request, and decoded token by token."""
    cfg = K.CFG_LONG
    model_dir, weights = _model(tmp_path, cfg, 11)
    prompts = {"a": K.tokens_for(cfg, 330, 41), "b": K.tokens_for(cfg, 100, 42)}
    want = _oracle_runs(cfg, weights, prompts)
    schedules = {
        "whole": [[("a", 330)], [("b", 100)]],
        "mixed": [[("a", 67)], [("a", 2), ("b", 60)], [("a", 111), ("b", 1)], [("a", 1), ("b", 1)], [("a", 89), ("b", 1)]]
                 + [[("a", 1), ("b", 1)]] * 37 + [[("a", 23)]],
    }
    for name, schedule in schedules.items():
        got = K.replay(model_dir, dtype, device, prompts, schedule, max_tokens=512, page=64, slots=2)
        for i, logits in got.items():
            err = K.rel_err(logits, want[i])
            assert err <= K.TOL[dtype], (name, i, err)


def case_engine_far_token(device, tmp_path):
    """One token changed at the start of a prompt changes the logits far beyond every window by what the oracle says, through the
    states and the chain of windows and passes; a model that forgot it would give the unchanged prompt's logits."""
    import copy
    cfg = copy.deepcopy(K.CFG_LONG)
    for L, size in zip([x for x in cfg["layers"] if "mask" in x["mixer"]], (9, 21, 17)):
        L["mixer"]["mask"]["size"] = size
    weights = oracle.random_weights(cfg, 12)
    weights["l1.mix.lam"] = weights["l1.mix.lam"] - 4.0
    model_dir = K.write_model(tmp_path / "m", cfg, weights)
    weights = {n: w.to(torch.bfloat16).to(F64) for n, w in weights.items()}
    a = K.tokens_for(cfg, 190, 51)
    b = [(a[0] + 1) % cfg["vocab"]] + a[1:]
    wa, wb = (oracle.forward(t, weights, cfg)[0][-1] for t in (a, b))
    moved = (wb - wa).abs().max().item() / wa.std().item()
    assert moved > 3e-3, "the test's weights forget: pick another seed"
    for schedule in ([[("a", 190)], [("b", 190)]], [[("a", 150), ("b", 20)], [("b", 130)]] + [[("a", 1), ("b", 1)]] * 40):
        got = K.replay(model_dir, "float32", device, {"a": a, "b": b}, schedule, max_tokens=512, page=64, slots=2)
        diff = (got["b"][-1] - got["a"][-1]).double()
        assert (diff - (wb - wa)).abs().max().item() <= 0.05 * (wb - wa).abs().max().item()


def case_engine_reuse(device, dtype, tmp_path):
    """More requests than state slots and more tokens than pages: both are given back and used again, in another order, and a
    sequence that starts on used pages and a used slot starts from nothing."""
    cfg = K.CFG_MAIN
    model_dir, weights = _model(tmp_path, cfg, 6)
    prompts = {f"r{n}": K.tokens_for(cfg, length, 10 + n) for n, length in enumerate((30, 17, 33, 9, 26, 31))}
    want = _oracle_runs(cfg, weights, prompts)
    schedule = [[("r0", 30), ("r1", 10)], [("r1", 7), ("r2", 20)], [("r3", 9), ("r2", 13)], [("r4", 13)],
                [("r5", 15), ("r4", 13)], [("r5", 16)]]
    got = K.replay(model_dir, dtype, device, prompts, schedule, max_tokens=64, page=16, slots=2)   # 4 pages, 2 slots
    for i, logits in got.items():
        K.assert_close(logits, want[i], dtype, i)


def case_engine_long_decode(device, dtype, tmp_path):
    """Hundreds of single-token steps through the caches and states."""
    cfg = K.CFG_MAIN
    model_dir, weights = _model(tmp_path, cfg, 7)
    prompts = {"a": K.tokens_for(cfg, 140, 21)}
    want = _oracle_runs(cfg, weights, prompts)
    got = K.replay(model_dir, dtype, device, prompts, [[("a", 3)]] + [[("a", 1)]] * 137, max_tokens=192, page=16, slots=1)
    K.assert_close(got["a"], want["a"], dtype, "long decode")


def case_generate(device, tmp_path, enforce_eager=True):
    """Greedy generation through LLM.generate: the scheduler admits, cuts prompts into portions under a small token budget, mixes
    them with decoding sequences, and every completion is the oracle's greedy continuation."""
    from light_vllm_amd.llm import LLM
    from light_vllm_amd.sampling_params import SamplingParams
    cfg = K.CFG_MAIN
    model_dir, weights = _model(tmp_path, cfg, 8)
    prompts = [K.tokens_for(cfg, n, 30 + n) for n in (19, 5, 33, 12, 8)]
    steps = 6
    llm = LLM(model_dir, dtype="float32", device=device, kvcache_block_size=16, max_num_seqs=3, max_cache_tokens=160,
              max_num_batched_tokens=24, long_prefill_token_threshold=10, max_model_len=64, enforce_eager=enforce_eager)
    assert llm.model_runner.enforce_eager == enforce_eager
    outs = llm.generate([list(p) for p in prompts], SamplingParams(temperature=0.0, max_tokens=steps, ignore_eos=True))
    llm.exit()
    for p, out in zip(prompts, outs):
        seq = list(p)
        for _ in range(steps):
            logits = oracle.forward(seq, weights, cfg)[0][-1]
            top2 = logits.topk(2).values
            assert (top2[0] - top2[1]).item() > 2e-4 * logits.abs().max().item(), "oracle tie: pick another seed"
            seq.append(int(logits.argmax()))
        assert out["token_ids"] == seq[len(p):]


def case_generate_bf16_graphs_like_eager(device, tmp_path):
    """bf16, sizes that take the matrix-core attention: single-token steps replayed from hipGraphs (launch geometry fixed at its
    bound, padded rows) continue every prompt like eager steps do, wherever the oracle's choice of the next token is no close
    call."""
    from light_vllm_amd.llm import LLM
    from light_vllm_amd.sampling_params import SamplingParams
    cfg = K.CFG_WIDE
    model_dir, weights = _model(tmp_path, cfg, 12)
    prompts = [K.tokens_for(cfg, n, 70 + n) for n in (40, 9, 23)]
    steps = 8
    outs = {}
    for eager in (True, False):
        llm = LLM(model_dir, dtype="bfloat16", device=device, kvcache_block_size=16, max_num_seqs=4, max_cache_tokens=256,
                  max_num_batched_tokens=64, max_model_len=64, enforce_eager=eager)
        outs[eager] = [o["token_ids"] for o in llm.generate([list(p) for p in prompts],
                                                           SamplingParams(temperature=0.0, max_tokens=steps, ignore_eos=True))]
        llm.exit()
    compared = 0
    for p, a, b in zip(prompts, outs[True], outs[False]):
        seq = list(p)
        for x, y in zip(a, b):
            logits = oracle.forward(seq, weights, cfg)[0][-1]
            top2 = logits.topk(2).values
            if (top2[0] - top2[1]).item() < 0.05 * logits.std().item() or x != int(logits.argmax()):
                break                       # a close call (or bf16 already chose otherwise): the continuations part ways
            assert x == y, (seq[len(p):], a, b)
            compared += 1
            seq.append(x)
    assert compared >= steps, "too few decided tokens: pick another seed"


def case_generate_preemption(device, tmp_path):
    """A page pool too small for the sequences that run: the scheduler preempts from the tail, frees pages and state slot, and
    recomputes the preempted sequence from its first token later; completions do not change."""
    from light_vllm_amd.llm import LLM
    from light_vllm_amd.sampling_params import SamplingParams
    cfg = K.CFG_MAIN
    model_dir, weights = _model(tmp_path, cfg, 8)
    prompts = [K.tokens_for(cfg, n, 50 + n) for n in (27, 29, 14)]
    steps = 9
    llm = LLM(model_dir, dtype="float32", device=device, kvcache_block_size=16, max_num_seqs=3, max_cache_tokens=64,
              max_num_batched_tokens=32, max_model_len=64)
    preempted = []
    original = llm.scheduler.preempt
    llm.scheduler.preempt = lambda seq: (preempted.append(seq.seq_id), original(seq))[1]
    outs = llm.generate([list(p) for p in prompts], SamplingParams(temperature=0.0, max_tokens=steps, ignore_eos=True))
    assert preempted, "the case is meant to run out of pages"
    assert llm.scheduler.block_manager.num_free_blocks == 4 and llm.scheduler.state_slots.num_free == 3
    llm.exit()
    for p, out in zip(prompts, outs):
        seq = list(p)
        for _ in range(steps):
            seq.append(int(oracle.forward(seq, weights, cfg)[0][-1].argmax()))
        assert out["token_ids"] == seq[len(p):]
