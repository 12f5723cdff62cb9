"""Cases of the Feditar tests, written once and run by the CPU test file (host logic with the package's torch
restatement of the kernels) and the GPU test file (the HIP kernels): every mechanism alone against
oracle/feditar_oracle.py, then the engine on whole prompts, token-by-token decoding, portions, mixed batches,
reused pages and slots, long decoding and greedy generation."""
from __future__ import annotations

import torch

from oracle import feditar_oracle as oracle
from tests import _feditar as K

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


def _walk(fn, check, lens=None):
    """fn([(id, lo, hi, slot)], step) -> rows of the step; check(rows, id, lo). Every sequence starts over when it has ended."""
    lens = lens or LENS
    at = {i: 0 for i in lens}
    for entries in WALK:
        parts = [(i, at[i], at[i] + n, s) for i, n, s in entries]
        rows = fn(parts)
        row = 0
        for i, lo, hi, _ in parts:
            check(rows[row:row + hi - lo], i, lo)
            row += hi - lo
            at[i] = 0 if hi == lens[i] else hi


def _step(parts, device, tables=None):
    return K.make_step([hi - lo for _, lo, hi, _ in parts], [lo for _, lo, _, _ in parts], [s for *_, s in parts],
                       tables or [[0]] * len(parts), device)


def _cut(x, parts):
    return torch.cat([x[i][lo:hi] for i, lo, hi, _ in parts])


# ------------------------------------------------------------------------------- single mechanisms
def case_embed(device, dtype):
    """Scaled token row, hashed pair row (its last row for a first token, the carried token for a portion's first one; factors
    whose products leave 32 bits), position row, two norms; each table present or not; widths in and out of multiples of four."""
    from light_vllm_amd import mix_ops
    g = torch.Generator().manual_seed(1)
    tol = 1e-5 if dtype == "float32" else 1e-2
    for W, vocab, pair, npos, scale in ((48, 50, (31, 7, 3), 80, 5.0), (37, 50, (1, 1, 1), 75, 1.0), (1000, 60, (97, 1 << 40, 5), 75, 0.5),
                                        (64, 50, None, 90, 2.0), (64, 50, (13, 2, 9), 0, 2.0)):
        eps = 1e-5
        cfg = {"norm": {"eps": eps}, "embedding": {"scale": scale}}
        Wt = {"embed": torch.randn(vocab, W, generator=g), "pos": torch.zeros(80, W), "embed.norm": 0.3 * torch.randn(W, generator=g)}
        if pair:
            cfg["embedding"]["bigram"] = dict(zip(("buckets", "mul_prev", "mul_cur"), pair))
            Wt["bigram"] = torch.randn(pair[0] + 1, W, generator=g)
        if npos:
            Wt["pos"] = torch.randn(npos, W, generator=g)
        Wt = {n: t.to(torch.bfloat16).to(F64) for n, t in Wt.items()}
        wn = 0.3 * torch.randn(W, generator=g)
        ids = {i: torch.randint(0, vocab, (n,), generator=g) for i, n in LENS.items()}
        want = {i: oracle.embed_tokens(t.tolist(), Wt, cfg) for i, t in ids.items()}
        normed = {i: oracle.offset_norm(x, wn.to(F64), eps) for i, x in want.items()}
        dev = {n: t.to(_dt(dtype)).to(device) for n, t in Wt.items() if n in ("embed", "bigram", "pos")}
        prev = torch.full((3,), 17, dtype=torch.int32, device=device)
        we = Wt["embed.norm"].float().to(device)
        hs = []

        def run(parts):
            x, h = mix_ops.embed_norm(_cut(ids, parts).to(device), dev["embed"], scale, dev.get("bigram"), *(pair or (0, 0, 0)), prev,
                                      dev["pos"] if npos else None, we, wn.to(device), 1.0, eps, _step(parts, device))
            hs.append(h)
            return torch.cat([x, h.float()], 1)

        def check(rows, i, lo):
            n = len(rows)
            _near(rows[:, :W], want[i][lo:lo + n], 2e-6, ("residual", W, i, lo))
            _near(rows[:, W:], normed[i][lo:lo + n], tol, ("first norm", W, i, lo))

        _walk(run, check)


def case_causal_conv(device, dtype):
    """Filters of 1 to 11 taps over strided columns, with and without bias and silu, channel counts in and out of multiples of
    four: whole, in portions shorter and longer than the filter and than a tile of tokens, on slots that held something else."""
    from light_vllm_amd import mix_ops
    g = torch.Generator().manual_seed(2)
    tol = 1e-5 if dtype == "float32" else 2e-2
    for C, taps, bias, silu, pad in ((24, 4, True, True, 8), (30, 3, True, True, 1), (512, 2, False, False, 4), (7, 1, True, False, 0),
                                     (16, 1, False, True, 0), (20, 6, True, True, 4), (9, 8, False, False, 3), (12, 11, True, True, 4), (640, 3, True, False, 0)):
        w = torch.randn(C, taps, generator=g) / taps ** 0.5
        b = torch.randn(C, generator=g) if bias else None
        xs = {i: torch.randn(n, C + pad, generator=g).to(_dt(dtype)) for i, n in LENS.items()}
        want = {}
        for i, x in xs.items():
            y = oracle.causal_conv(x[:, pad:].to(F64), w.to(F64), b.to(F64) if bias else None)
            want[i] = oracle.silu(y) if silu else y
        buf = torch.full((3, max(taps - 1, 1), C), 5.0, dtype=_dt(dtype), device=device)
        state = buf[:, :taps - 1]
        wd, bd = w.to(device), b.to(device) if bias else None

        def run(parts):
            x = _cut(xs, parts).to(device)
            return mix_ops.causal_conv(x[:, pad:], wd, bd, state, _step(parts, device), silu=silu)

        _walk(run, lambda rows, i, lo: _near(rows, want[i][lo:lo + len(rows)], tol, ("conv", C, taps, i, lo)))


def case_conv_qkv_store(device, dtype):
    """Convolved queries, keys and values of an attention layer: the factor of the position on the queries just before, at and
    after the positions where it changes, far along as well, keys and values in the rows of pages in any order."""
    from light_vllm_amd import mix_ops
    g = torch.Generator().manual_seed(3)
    tol = 1e-5 if dtype == "float32" else 2e-2
    for H, G, D, Dv, taps, coef, every, page in ((4, 2, 12, 8, 3, 0.4, 7, 16), (3, 3, 5, 6, 4, -0.2, 1, 16), (5, 1, 16, 70, 1, 0.3, 16, 64),
                                                 (2, 1, 8, 8, 9, 0.0, 1, 16), (2, 2, 64, 32, 2, 0.5, 33, 32)):
        C = H * D + G * (D + Dv)
        w = torch.randn(C, taps, generator=g)
        xs = {i: torch.randn(n, C, generator=g).to(_dt(dtype)) for i, n in LENS.items()}
        want = {i: oracle.causal_conv(x.to(F64), w.to(F64)) for i, x in xs.items()}
        for y in want.values():
            for p in range(len(y)):
                y[p, :H * D] *= oracle.query_temperature(p, {"coef": coef, "every": every} if coef else None)
        per = -(-80 // page)
        order = torch.randperm(2 * per, generator=g).tolist()
        tables = {"a": order[:per], "b": order[per:]}
        kc = torch.zeros(2 * per, page, G, D, dtype=_dt(dtype), device=device)
        vc = torch.zeros(2 * per, page, G, Dv, dtype=_dt(dtype), device=device)
        state = torch.full((3, max(taps - 1, 1), C), 5.0, dtype=_dt(dtype), device=device)[:, :taps - 1]
        wd = w.to(device)

        def run(parts):
            q = mix_ops.conv_qkv_store(_cut(xs, parts).to(device), wd, state, kc, vc, _step(parts, device, [tables[i] for i, *_ in parts]),
                                       H, G, D, Dv, coef, every)
            return q

        def check(rows, i, lo):
            n = len(rows)
            _near(rows, want[i][lo:lo + n, :H * D], tol, ("q", H, D, taps, i, lo))
            slots = [tables[i][p // page] * page + p % page for p in range(lo, lo + n)]
            _near(kc.view(-1, G * D)[slots], want[i][lo:lo + n, H * D:H * D + G * D], tol, ("k", H, D, taps, i, lo))
            _near(vc.view(-1, G * Dv)[slots], want[i][lo:lo + n, H * D + G * D:], tol, ("v", H, D, taps, i, lo))

        _walk(run, check)
    # far along: positions around multiples of `every`
    for p in (127, 128, 1023, 1024, 70000):
        H, D = 2, 8
        x = torch.ones(1, 4 * D).to(_dt(dtype)).to(device)
        kc, vc = torch.zeros(1, 80000, 1, D, dtype=_dt(dtype), device=device), torch.zeros(1, 80000, 1, D, dtype=_dt(dtype), device=device)
        st = torch.zeros(1, 1, 4 * D, dtype=_dt(dtype), device=device)[:, :0]
        q = mix_ops.conv_qkv_store(x, torch.ones(4 * D, 1, device=device), st, kc, vc, K.make_step([1], [p - 1], [0], [[0]], device), H, 1, D, D,
                                   0.3, 64)
        _near(q, torch.full((1, H * D), oracle.query_temperature(p - 1, {"coef": 0.3, "every": 64}), dtype=F64), tol, ("factor", p))


def case_token_shift(device, dtype):
    """h + (h' - h) mu for several mu at once; portions, reused slots; a step of thousands of tokens of several sequences
    (which takes tiles of tokens), starts of sequences anywhere in a tile."""
    from light_vllm_amd import mix_ops
    g = torch.Generator().manual_seed(4)
    tol = 1e-6 if dtype == "float32" else 1e-2
    for W, M in ((48, 5), (37, 5), (1028, 3), (64, 7)):
        mu = 0.5 + 0.5 * torch.randn(M, W, generator=g)
        hs = {i: torch.randn(n, W, generator=g).to(_dt(dtype)) for i, n in LENS.items()}
        want = {i: torch.stack([oracle.token_shift(h.to(F64), m.to(F64)) for m in mu], 1) for i, h in hs.items()}
        state = torch.full((3, W), 9.0, dtype=_dt(dtype), device=device)
        mud = mu.to(device)
        _walk(lambda parts: mix_ops.token_shift(_cut(hs, parts).to(device), mud, state, _step(parts, device)).transpose(0, 1),
              lambda rows, i, lo: _near(rows, want[i][lo:lo + len(rows)], tol, ("shift", W, M, i, lo)))
    W, M, lens = 20, 5, (700, 1, 39, 1400, 2, 33)
    mu = torch.rand(M, W, generator=g)
    h = torch.randn(sum(lens), W, generator=g).to(_dt(dtype))
    before = torch.randn(len(lens), W, generator=g).to(_dt(dtype))
    ctx = [0, 4, 9, 0, 1, 0]
    state = before.clone().to(device)
    got = mix_ops.token_shift(h.to(device), mu.to(device), state, K.make_step(lens, ctx, list(range(6)), [[0]] * 6, device))
    at = 0
    for b, n in enumerate(lens):
        rows = h[at:at + n].to(F64)
        if ctx[b]:
            rows = torch.cat([before[b:b + 1].to(F64), rows])
        ref = torch.stack([oracle.token_shift(rows, m.to(F64)) for m in mu])[:, -n:]
        _near(got[:, at:at + n], ref, tol, ("tiles", b))
        assert torch.equal(state[b].cpu(), h[at + n - 1])
        at += n


SCAN_SIZES = ((3, 3, 8, 12), (1, 1, 40, 70), (2, 2, 6, 5), (4, 2, 16, 16), (2, 1, 128, 64), (1, 1, 130, 8), (4, 4, 16, 160), (1, 1, 100, 128))
MANY = (96, 96, 40, 704)       # above a thousand workgroups: the state's rows then go over four waves instead of eight


def _scan_inputs(g, H, G, D, Dv, dtype, lens):
    q = {i: torch.randn(n, G * D, generator=g).to(_dt(dtype)) for i, n in lens.items()}
    k = {i: torch.randn(n, G * D, generator=g).to(_dt(dtype)) for i, n in lens.items()}
    v = {i: torch.randn(n, H * Dv, generator=g).to(_dt(dtype)) for i, n in lens.items()}
    return q, k, v


def _heads64(x, n):
    return {i: t.to(F64).view(len(t), n, -1) for i, t in x.items()}


def case_scan_step(device, dtype):
    """The recurrence of the state-space layers: step sizes from the softplus (large arguments too), rates, shared keys and
    queries, the skip."""
    from light_vllm_amd import mix_ops
    g = torch.Generator().manual_seed(5)
    tol = 2e-5 if dtype == "float32" else 2e-2
    for H, G, D, Dv in SCAN_SIZES + (MANY,):
        check_heads = range(H) if H < 8 else (0, 37, H - 1)
        q, k, v = _scan_inputs(g, H, G, D, Dv, dtype, LENS)
        a = {i: (3 * torch.randn(n, H, generator=g)).to(_dt(dtype)) for i, n in LENS.items()}
        a["a"][5, 0] = 30.0
        bias, rate, skip = -2 + torch.randn(H, generator=g), torch.randn(H, generator=g), torch.randn(H, generator=g)
        q6, k6, v6 = _heads64(q, G), _heads64(k, G), _heads64(v, H)
        want = {i: {h: oracle.ssd_head(v6[i][:, h], k6[i][:, h // (H // G)], q6[i][:, h // (H // G)],
                                       oracle.softplus(a[i][:, h].to(F64) + bias[h].to(F64)), rate[h].to(F64), skip[h].to(F64))
                    for h in check_heads} for i in LENS}
        state = torch.full((3, H, D, Dv), 7.0, device=device)
        bd, rd, sd = bias.to(device), rate.to(device), skip.to(device)
        spread = max(w.abs().max().item() for per in want.values() for w in per.values())

        def run(parts):
            return mix_ops.gated_scan(mix_ops.SCAN_STEP, *(_cut(x, parts).to(device) for x in (q, k, v, a)), bd, rd, _step(parts, device), state,
                                      H, G, D, Dv, p2=sd)

        def check(rows, i, lo):
            for h in check_heads:
                err = (rows[:, h].cpu().to(F64) - want[i][h][lo:lo + len(rows)]).abs().max().item()
                assert err <= tol * max(1.0, spread) * 1.0, ("step", H, G, D, Dv, i, lo, h, err)

        _walk(run, check)


def case_scan_log_gates(device, dtype):
    """The matrix memory: gates far into their caps on both sides, a running maximum that starts at 0 and stays there (small
    input gates: the floor e^-m of the normaliser rules) or climbs, scores n . q of either sign, the division and norm behind it."""
    from light_vllm_amd import mix_ops
    g = torch.Generator().manual_seed(6)
    tol = 5e-5 if dtype == "float32" else 3e-2
    sizes = [(h, d, dv, cap, ib, fb) for (h, _, d, dv), cap, ib, fb in
             zip(SCAN_SIZES, (6.0, 15.0, 1.0, 15.0, 4.0, 15.0, 8.0, 15.0), (0.0, -6.0, 1.0, 3.0, -2.0, 0.0, 2.0, -1.0), (2.0, 3.0, 0.0, 4.0, 1.0, 5.0, -2.0, 6.0))]
    for H, D, Dv, cap, ib, fb in sizes + [(96, 40, 704, 15.0, 0.5, 3.0)]:
        check_heads = range(H) if H < 8 else (0, 41, H - 1)
        q, k, v = _scan_inputs(g, H, H, D, Dv, dtype, LENS)
        ai = {i: (4 * torch.randn(n, H, generator=g)).to(_dt(dtype)) for i, n in LENS.items()}
        af = {i: (4 * torch.randn(n, H, generator=g)).to(_dt(dtype)) for i, n in LENS.items()}
        bi, bf = ib + 0.3 * torch.randn(H, generator=g), fb + 0.3 * torch.randn(H, generator=g)
        gate = {i: torch.randn(n, H * Dv, generator=g).to(_dt(dtype)) for i, n in LENS.items()}
        nw = 1 + 0.3 * torch.randn(H * Dv, generator=g)
        q6, k6, v6 = _heads64(q, H), _heads64(k, H), _heads64(v, H)
        raw, want = {}, {}
        for i in LENS:
            for h in check_heads:
                li = cap * torch.tanh((ai[i][:, h].to(F64) + bi[h].to(F64)) / cap)
                lf = oracle.log_sigmoid(cap * torch.tanh((af[i][:, h].to(F64) + bf[h].to(F64)) / cap))
                o = oracle.matrix_memory(q6[i][:, h] * D ** -0.5, k6[i][:, h], v6[i][:, h], li, lf)
                raw[i, h] = o
                want[i, h] = oracle.unit_rms(o, 1e-5) * nw[h * Dv:(h + 1) * Dv].to(F64) * torch.sigmoid(gate[i][:, h * Dv:(h + 1) * Dv].to(F64))
        state = torch.full((3, H, D, Dv), 7.0, device=device)
        ns = torch.full((3, H, D), 3.0, device=device)
        ms = torch.full((3, H, mix_ops.scan_copies(Dv)), 11.0, device=device)
        bid, bfd, nwd = bi.to(device), bf.to(device), nw.to(device)

        def run(parts):
            o, den = mix_ops.gated_scan(mix_ops.SCAN_LOG_GATES, *(_cut(x, parts).to(device) for x in (q, k, v, ai)), bid, bfd,
                                        _step(parts, device), state, H, H, D, Dv, a2=_cut(af, parts).to(device), q_scale=D ** -0.5, cap=cap,
                                        norm_state=ns, max_state=ms)
            y = mix_ops.scaled_head_norm_gate(o, _cut(gate, parts).to(device), nwd, 1e-5, _dt(dtype), "sigmoid", den=den)
            return torch.cat([(o / den[:, :, None]), y.view(-1, H, Dv).float()], -1)

        def check(rows, i, lo):
            n = len(rows)
            for h in check_heads:
                ref = raw[i, h][lo:lo + n]
                scale = raw[i, h].abs().max(-1, keepdim=True).values[lo:lo + n] + 1e-3       # read-outs differ by orders of magnitude
                err = ((rows[:, h, :Dv].cpu().to(F64) - ref).abs() / scale).max().item()
                assert err <= 2e-3, ("memory", H, D, Dv, i, lo, h, err)
                med = ((rows[:, h, :Dv].cpu().to(F64) - ref).abs() / scale).median().item()
                assert med <= 2e-5, ("memory, median", H, D, Dv, i, lo, h, med)
                e2 = (rows[:, h, Dv:].cpu().to(F64) - want[i, h][lo:lo + n]).abs()
                assert e2.max().item() <= max(tol, 5e-3) * 4 and e2.median().item() <= tol, ("normed", H, D, Dv, i, lo, h, e2.max().item())

        _walk(run, check)


def case_scan_row_decay(device, dtype):
    """Time mixing's recurrence: a decay for every row (some hold for ever, some forget at once), the bonus for the current
    token only, the read-out before the write."""
    from light_vllm_amd import mix_ops
    g = torch.Generator().manual_seed(7)
    tol = 2e-5 if dtype == "float32" else 2e-2
    for H, _, D, Dv in SCAN_SIZES + (MANY,):
        check_heads = range(H) if H < 8 else (0, 53, H - 1)
        q, k, v = _scan_inputs(g, H, H, D, Dv, dtype, LENS)
        a = {i: torch.randn(n, H * D, generator=g).to(_dt(dtype)) for i, n in LENS.items()}
        w0 = -2.5 + 1.5 * torch.randn(H * D, generator=g)
        w0[0], w0[-1] = -30.0, 6.0
        u = torch.randn(H, D, generator=g)
        q6, k6, v6 = _heads64(q, H), _heads64(k, H), _heads64(v, H)
        want = {i: {} for i in LENS}
        for i in LENS:
            w = torch.exp(-torch.exp(a[i].to(F64) + w0.to(F64))).view(-1, H, D)
            for h in check_heads:
                want[i][h] = oracle.bonus_recurrence(q6[i][:, h], k6[i][:, h], v6[i][:, h], w[:, h], u[h].to(F64))
        state = torch.full((3, H, D, Dv), 7.0, device=device)
        w0d, ud = w0.to(device), u.to(device)

        def run(parts):
            return mix_ops.gated_scan(mix_ops.SCAN_ROW_DECAY, *(_cut(x, parts).to(device) for x in (q, k, v, a)), w0d, ud, _step(parts, device), state,
                                      H, H, D, Dv)

        def check(rows, i, lo):
            for h in check_heads:
                err = (rows[:, h].cpu().to(F64) - want[i][h][lo:lo + len(rows)]).abs().max().item()
                assert err <= tol * want[i][h].abs().max().item(), ("row decay", H, D, Dv, i, lo, h, err)

        _walk(run, check)


def case_norms_and_acts(device, dtype):
    """The norm per head with weights per head, with and without a divisor (short heads, several to a wave, long ones, odd ones);
    the gate before the norm in parts of the row; the residual that receives two normed outputs; the activations."""
    from light_vllm_amd import mix_ops
    g = torch.Generator().manual_seed(8)
    tol = 1e-5 if dtype == "float32" else 2e-2
    for T, H, Dv in ((5, 3, 12), (3, 2, 10), (2, 1, 256), (9, 5, 64), (3, 2, 300), (2, 3, 640), (1, 1, 1)):
        o = 2 * torch.randn(T, H, Dv, generator=g)
        den = 0.2 + 3 * torch.rand(T, H, generator=g)
        o[0, 0] *= 1e-3                         # a head small enough for eps to count
        gate = torch.randn(T, H * Dv + 4, generator=g).to(_dt(dtype))
        nw = torch.randn(H * Dv, generator=g)
        for act, f in (("silu", oracle.silu), ("sigmoid", torch.sigmoid)):
            for d in (None, den):
                y = o.to(F64) / d.to(F64)[:, :, None] if d is not None else o.to(F64)
                want = oracle.unit_rms(y, 1e-5).reshape(T, -1) * nw.to(F64) * f(gate[:, 4:].to(F64))
                got = mix_ops.scaled_head_norm_gate(o.to(device), gate.to(device)[:, 4:], nw.to(device), 1e-5, _dt(dtype), act,
                                                    den=d.to(device) if d is not None else None)
                _near(got, want, tol, ("head norm", T, H, Dv, act, d is not None))
    for T, N, groups in ((5, 48, 2), (3, 30, 3), (2, 2048, 1), (3, 4096, 4), (2, 4608, 3), (7, 9, 9), (3, 1000, 5)):
        o, w = torch.randn(T, N, generator=g), 1 + 0.3 * torch.randn(N, generator=g)
        o[:, :N // groups] *= 30                # parts of unequal size
        z = torch.randn(T, N + 4, generator=g).to(_dt(dtype))
        y = o.to(F64) * oracle.silu(z[:, 4:].to(F64))
        want = oracle.unit_rms(y.view(T, groups, -1), 1e-5).reshape(T, N) * w.to(F64)
        _near(mix_ops.grouped_gate_norm(o.to(device), z.to(device)[:, 4:], w.to(device), groups, 1e-5), want, tol, ("parts", T, N, groups))
    for T, W in ((7, 48), (3, 37), (5, 1000)):
        x = 2 * torch.randn(T, W, generator=g)
        y1, y2 = (s * torch.randn(T, W, generator=g).to(_dt(dtype)) for s in (3, 0.1))
        p1, p2, w = (1 + 0.4 * torch.randn(W, generator=g) for _ in range(3))
        want = x.to(F64) + 0.5 * (oracle.unit_rms(y1.to(F64), 1e-4) * p1.to(F64) + oracle.unit_rms(y2.to(F64), 1e-4) * p2.to(F64))
        xd = x.clone().to(device)
        h = mix_ops.residual_pair_norm(xd, y1.to(device), y2.to(device), p1.to(device), p2.to(device), 0.5, 1e-4, w.to(device), 1.0, 1e-5)
        _near(xd, want, 2e-6, ("residual", W))
        _near(h, oracle.offset_norm(want, w.to(F64), 1e-5), tol, ("norm behind it", W))
        x2 = x.clone().to(device)
        assert mix_ops.residual_pair_norm(x2, y1.to(device), y2.to(device), p1.to(device), p2.to(device), 0.5, 1e-4) is None
        _near(x2, want, 2e-6, ("residual alone", W))
    for shape in ((5, 40), (3, 37), (2, 1024)):
        z = (2 * torch.randn(*shape, generator=g)).to(_dt(dtype))
        for act, f in (("relu2", lambda a: a.clamp(min=0) ** 2), ("tanh", torch.tanh)):
            _near(mix_ops.unary_act(z.to(device), act), f(z.to(F64)), tol, (act, shape))


def case_capped_attention(device, dtype):
    """Beacon keys (far away, the first token, either side of page and tile borders) whose scores stand out and run into the cap:
    a query among hundreds of keys takes its answer from them. Without the cap, with another cap, or with the cap before the
    scale the answer differs by far more than the tolerance. Prompt-, decode- and portion-shaped launches."""
    from light_vllm_amd import mix_ops
    g = torch.Generator().manual_seed(9)
    for H, G, D, Dv, page, L, cap, scale in ((4, 2, 12, 10, 16, 75, 3.0, 0.7), (5, 1, 32, 48, 16, 300, 6.0, 0.4), (2, 2, 64, 128, 64, 210, 5.0, 0.5),
                                             (3, 3, 16, 16, 16, 140, 40.0, 0.5), (1, 1, 80, 144, 64, 100, 4.0, 0.3), (9, 1, 16, 32, 32, 150, 2.0, 0.5)):
        e = torch.zeros(D)
        e[D - 1] = 1.0
        k, v = 0.3 * torch.randn(L, G, D, generator=g), torch.randn(L, G, Dv, generator=g)
        beacons = sorted({0, page - 1, page, L // 2, min(63, L - 1), min(64, L - 1)})
        for n, j in enumerate(beacons):
            k[j] += (5.0 + n) * e              # unequal scores that a cap brings together
        q = 0.3 * torch.randn(L, H, D, generator=g) + 3.0 * e
        k, v, q = (t.to(_dt(dtype)).float() for t in (k, v, q))

        def attend(c):
            return torch.cat([oracle.capped_softmax_head(q[:, h].to(F64), k[:, h // (H // G)].to(F64), v[:, h // (H // G)].to(F64), scale, c)
                              for h in range(H)], -1)

        want = attend(cap)
        tol = 2e-4 if dtype == "float32" else 3e-2
        if cap < 10:                           # the plain softmax and a doubled cap give something else
            for other in (None, 2 * cap):
                assert (attend(other) - want)[-1].abs().max().item() > 3 * tol * want.abs().max().item()
        per = -(-L // page)
        table = torch.randperm(per + 2, generator=g)[:per].tolist()
        kc = torch.zeros(per + 2, page, G, D, dtype=_dt(dtype))
        vc = torch.zeros(per + 2, page, G, Dv, dtype=_dt(dtype))
        for p in range(L):
            kc[table[p // page], p % page], vc[table[p // page], p % page] = k[p], v[p]
        kc, vc = kc.to(device), vc.to(device)
        qd = q.reshape(L, H * D).to(_dt(dtype)).to(device)

        def run(step, rows, what):
            got = mix_ops.window_pool_attention(qd[rows].contiguous(), kc, vc, None, None, None, step, H, G, D, Dv, 1 << 30, 0, scale,
                                                has_sink=False, softcap=cap)
            _near(got, want[rows], tol, (what, H, G, D, Dv, page, cap))

        every = list(range(L))
        run(K.make_step([L], [0], [0], [table], device), every, "prompt")
        idx = sorted({i for j in beacons for i in (j - 1, j, j + 1) if 0 <= i < L} | set(range(L - 5, L)))
        run(K.make_step([1] * len(idx), idx, [0] * len(idx), [table] * len(idx), device), idx, "decode")
        run(K.make_step([1], [L - 1], [0], [table], device), [L - 1], "one sequence")
        rows = list(range(page - 1, L - 20)) + list(range(5)) + list(range(L - 19, L))
        run(K.make_step([L - 20 - page + 1, 5, 19], [page - 1, 0, L - 19], [0, 1, 2], [table] * 3, device), rows, "portions")


# ----------------------------------------------------------------------------------------- engine
def _model(tmp_path, cfg, seed):
    weights = oracle.random_weights(cfg, seed)
    return K.write_model(tmp_path / f"m{seed}", cfg, weights), weights


def _oracle_runs(cfg, weights, prompts):
    return {i: oracle.forward(t, weights, cfg)[0] for i, t in prompts.items()}


def case_checkpoint_placement(tmp_path):
    """Every tensor of a checkpoint lands where the oracle reads it: parts of merged projections, filters of q, k and v side by
    side, batched projections input first, the head on the token table; sizes that only the tensors give; what is missing,
    unknown or of another shape is refused."""
    import json
    import os
    from light_vllm_amd.models.feditar import FeditarConfig, FeditarForCausalLM
    from light_vllm_amd.models.registry import load_config, model_class
    cfg = K.CFG_MAIN
    weights = oracle.random_weights(cfg, 3)
    model_dir = K.write_model(tmp_path / "m", cfg, weights)
    config = load_config(model_dir)
    assert isinstance(config, FeditarConfig) and model_class(config) is FeditarForCausalLM
    assert config.layers[2]["mixer"]["right"]["decay_rank"] == 5 and config.layers[5]["mixer"]["right"]["decay_rank"] == 3
    assert config.max_position_embeddings == 192 and config.pair == (31, 7, 3)
    old = torch.get_default_dtype()
    torch.set_default_dtype(torch.float32)
    try:
        model = FeditarForCausalLM(config)
    finally:
        torch.set_default_dtype(old)
    model.load_weights(weights.items())
    assert sorted(model.weight_targets()) == sorted(weights)
    assert model.lm_head.weight is model.embed.weight
    mem, left, right = model.layers[0].mix, model.layers[2].mix.left, model.layers[2].mix.right
    at = mem.offsets
    for j, nm in enumerate(("q", "k", "v", "g", "i", "f")):
        assert torch.equal(mem.in_proj.weight[at[j]:at[j + 1]].double(), weights["l0.mix." + nm])
    assert torch.equal(left.conv_weight[48:48 + 24].double(), weights["l2.mix.left.k.conv"])
    assert torch.equal(right.proj_weight[2].t().double(), weights["l2.mix.right.v"])
    assert torch.equal(right.mix_weight[4].double(), weights["l2.mix.right.mu.w"])
    short = dict(weights)
    del short["l2.mix.right.u"]
    for broken, error in ((short, KeyError), ({**weights, "l0.mix.extra": torch.zeros(1)}, KeyError),
                          ({**weights, "pos": torch.zeros(3, 48)}, ValueError)):
        try:
            model.load_weights(broken.items())
            raise AssertionError("a wrong checkpoint went unnoticed")
        except error:
            pass
    for change in (lambda c: c["layers"][0].update(type="recurrent"), lambda c: c["layers"][1]["mixer"].pop("state"),
                   lambda c: c["layers"][0]["mlp"].update(kind="moe"), lambda c: c.pop("max_positions"),
                   lambda c: c["layers"][2]["mixer"]["left"]["q_temp"].update(every=0)):
        bad = json.load(open(os.path.join(model_dir, "config.json")))
        change(bad)
        try:
            FeditarConfig.from_dict(bad, {"l2.mix.right.w1": (5, 48)})
            raise AssertionError("a wrong configuration went unnoticed")
        except ValueError:
            pass


def case_layer_by_layer(device, tmp_path, cfg=None):
    """The f32 residual after every layer of a whole prompt, against the oracle: names the first layer that differs."""
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
    assert len(got) == len(want) == len(cfg["layers"])
    for i, (a, b) in enumerate(zip(got, want)):
        assert (a.to(F64) - b).abs().max().item() <= 3e-4 * b.abs().max().item(), f"layer {i}"


def case_engine_schedules(device, dtype, tmp_path, cfg=None, seed=5):
    """Whole prompts, token-by-token decoding, portions down to two tokens and mixed batches of unequal requests give the logits
    of the whole-sequence oracle at every position: the first tokens, every page border (pages of 16 tokens), portions shorter
    than a filter and cuts inside it."""
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
    """Attention over several pages and key tiles, states over hundreds of tokens: a prompt of 330 tokens whole, cut at odd
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
    """One token changed at the start of a prompt changes the logits hundreds of positions later by what the oracle says, through
    the attention's far keys and the states alike; a model that forgot it would give the unchanged prompt's logits."""
    cfg = K.CFG_LONG
    model_dir, weights = _model(tmp_path, cfg, 12)
    a = K.tokens_for(cfg, 300, 51)
    b = [(a[0] + 1) % cfg["vocab"]] + a[1:]
    wa, wb = (oracle.forward(t, weights, cfg)[0][-1] for t in (a, b))
    moved = (wb - wa).abs().max().item() / wa.std().item()
    assert moved > 3e-3, "the test's weights forget: pick another seed"
    got = {}
    for schedule in ([[("a", 300)], [("b", 300)]], [[("a", 250), ("b", 20)], [("b", 230)]] + [[("a", 1), ("b", 1)]] * 50):
        got = K.replay(model_dir, "float32", device, {"a": a, "b": b}, schedule, max_tokens=640, page=64, slots=2)
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


def case_position_limit(device, tmp_path):
    """A sequence may fill the position table to its last row; one token more is refused before anything runs."""
    cfg = K.CFG_ODD
    model_dir, weights = _model(tmp_path, cfg, 13)
    tokens = K.tokens_for(cfg, 65, 61)
    want = oracle.forward(tokens[:64], weights, cfg)[0]
    got = K.replay(model_dir, "float32", device, {"a": tokens[:64]}, [[("a", 60)], [("a", 4)]], max_tokens=128, page=16, slots=1)
    K.assert_close(got["a"], want, "float32", "full table")
    try:
        K.replay(model_dir, "float32", device, {"a": tokens}, [[("a", 60)], [("a", 5)]], max_tokens=128, page=16, slots=1)
        raise AssertionError("a position outside the table went unnoticed")
    except IndexError:
        pass


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
