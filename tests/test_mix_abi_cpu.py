"""liblvmix.so loads without a GPU, exports exactly what include/lv_mixers.h declares with the argument counts the
ctypes table binds, and rejects bad arguments on the host before any launch."""
import ctypes
import os
import re

ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
HEADER = os.path.join(ROOT, "include", "lv_mixers.h")


def declared():
    """name -> number of parameters of every function the header declares."""
    text = re.sub(r"/\*.*?\*/", "", open(HEADER).read(), flags=re.S)
    out = {}
    for name, args in re.findall(r"\b(lv_[a-z0-9_]+)\s*\(([^;{]*?)\)\s*;", text, flags=re.S):
        args = args.strip()
        out[name] = 0 if args in ("", "void") else args.count(",") + 1
    return out


def test_header_and_ctypes_table_agree():
    from light_vllm_amd import _mixlib
    decl = declared()
    assert sorted(decl) == sorted(_mixlib.SIGNATURES)
    for name, (_, args) in _mixlib.SIGNATURES.items():
        assert len(args) == decl[name], name
    lib = _mixlib.load()
    for name in decl:
        assert hasattr(lib, name), f"{name} missing from liblvmix.so"
    assert lib.lv_mix_abi_version() == _mixlib.ABI_VERSION
    version = int(re.search(r"#define LV_MIX_ABI_VERSION (\d+)", open(HEADER).read()).group(1))
    assert version == _mixlib.ABI_VERSION


def test_argument_validation_happens_before_any_launch():
    from light_vllm_amd import _mixlib
    lib = _mixlib.load()
    buf = ctypes.create_string_buffer(256)
    p = (ctypes.addressof(buf) + 15) & ~15
    # zero tokens: nothing to do, whatever else is passed
    assert lib.lv_sandwich_add_norm(None, None, None, None, None, None, 1.0, None, 0, 64, 1e-6, 0, None) == 0
    assert lib.lv_rotary_store(None, 0, 0, 0, 0, None, None, None, None, None, None, None, None, None, 1, 0, 4, 2, 8, 8, 4, 16, 0, None) == 0
    assert lib.lv_polynorm(None, 0, None, None, 0, 8, 1e-6, 0, None) == 0
    assert lib.lv_expert_glu(None, 0, None, None, 0, None, 0, 0, 2, 8, 1.0, 1.702, 0, None) == 0
    # a sublayer output without its norm weight; an output without a norm weight
    assert lib.lv_sandwich_add_norm(p, p, None, None, None, p, 1.0, p, 1, 8, 1e-6, 0, None) == -1
    assert lib.lv_sandwich_add_norm(p, None, None, None, None, None, 1.0, p, 1, 8, 1e-6, 0, None) == -1
    assert lib.lv_sandwich_add_norm(p, None, None, None, None, p, 1.0, p, 1, 1 << 20, 1e-6, 0, None) == -2     # row above the LDS
    # an odd number of rotated entries, more of them than the head has, heads that do not divide, columns past the row
    args = lambda **kw: [p, kw.get("ld", 64), 0, 32, 48, p, None, p, p, p, p, p, p, p, 1, 1, kw.get("H", 4), kw.get("G", 2), 8, 8,  # noqa: E731
                         kw.get("rot", 4), 16, 0, None]
    assert lib.lv_rotary_store(*args(rot=3)) == -1
    assert lib.lv_rotary_store(*args(rot=10)) == -1
    assert lib.lv_rotary_store(*args(H=3)) == -1
    assert lib.lv_rotary_store(*args(ld=40)) == -1 and b"lv_rotary_store" in lib.lv_mix_last_error()
    assert lib.lv_polynorm(p, 4, p, p, 1, 8, 1e-6, 0, None) == -1                      # row stride below the row
    assert lib.lv_polynorm(p, 8, p, p, 1, 8, 1e-6, 7, None) == -1                      # unknown dtype
    assert lib.lv_expert_glu(p, 8, None, None, 0, p, 8, 1, 2, 8, 1.0, 1.702, 0, None) == -1     # two experts need 32 columns
    assert lib.lv_moe_route(p, None, p, p, None, 1, 4, 5, 1, 1, 0, None) == -1                 # more choices than experts
    assert lib.lv_router_logits(p, 4, p, p, 1, 8, 4, 0, None) == -1                            # row stride below the row
    assert lib.lv_moe_grouped_glu_ff(p, p, p, p, p, 0, p, p, 1, 48, 32, 4, 2, 1.0, 1.702, None) == -1     # width no multiple of 32
    assert lib.lv_moe_grouped_glu_ff(p, p, p, p, p, 100, p, p, 1, 64, 32, 4, 2, 1.0, 1.702, None) == -1   # down rows shorter than E*F
    assert lib.lv_window_pool_attn(p, p, p, None, None, p, 4, p, p, p, p, p, 1, 1, 4, 2, 8, 8, 16, 64, 0, 0.5, 0, 0, 0, 5, 0, None) == -1   # gate kind
    # scans, convolutions and the steps around them
    assert lib.lv_causal_conv(None, 0, None, None, None, None, None, None, None, 0, 5, 8, 4, 1, 0, None) == 0           # no sequence
    conv = lambda **kw: [p, kw.get("ld", 8), p, None, kw.get("state", p), p, p, p, p, 1, 1, 8, kw.get("taps", 4), 1, kw.get("dt", 0), None]  # noqa: E731
    assert lib.lv_causal_conv(*conv(ld=7)) == -1 and lib.lv_causal_conv(*conv(taps=0)) == -1
    assert lib.lv_causal_conv(*conv(state=None)) == -1 and lib.lv_causal_conv(*conv(dt=9)) == -1
    qkv = lambda **kw: [p, kw.get("ld", 64), p, p, p, p, p, p, p, p, p, 1, 1, 1, kw.get("H", 4), kw.get("G", 2), 8, 8, 3, kw.get("coef", 0.5),  # noqa: E731
                        kw.get("every", 4), 16, 0, None]
    assert lib.lv_conv_qkv_store(*qkv(H=3)) == -1 and lib.lv_conv_qkv_store(*qkv(ld=63)) == -1 and lib.lv_conv_qkv_store(*qkv(every=0)) == -1
    scan = lambda **kw: [kw.get("kind", 0), p, kw.get("ldq", 16), p, 16, p, 16, p, kw.get("a2", p), kw.get("lda", 16), p, p, kw.get("p2", p), 1.0,  # noqa: E731
                         kw.get("cap", 1.0), p, kw.get("ns", p), p, p, p, p, p, p, 1, kw.get("H", 2), kw.get("G", 2), kw.get("D", 8), 8, 0, None]
    assert lib.lv_gated_scan(*scan(kind=5)) == -1 and lib.lv_gated_scan(*scan(p2=None)) == -1
    assert lib.lv_gated_scan(*scan(kind=1, ns=None)) == -1 and lib.lv_gated_scan(*scan(kind=1, cap=0.0)) == -1
    assert lib.lv_gated_scan(*scan(kind=2, G=1)) == -1 and lib.lv_gated_scan(*scan(kind=2, lda=15)) == -1
    assert lib.lv_gated_scan(*scan(ldq=15)) == -1 and lib.lv_gated_scan(*scan(H=3)) == -1
    assert lib.lv_gated_scan(*scan(G=1, D=257, ldq=512)) in (-1, -2)
    assert lib.lv_token_shift(p, p, None, p, p, p, p, p, 1, 8, 5, 0, None) == -1
    assert lib.lv_grouped_gate_norm(p, p, 8, p, p, 1, 8, 3, 1e-6, 0, None) == -1                                      # parts that do not divide
    assert lib.lv_scaled_head_norm_gate(p, None, p, 16, p, 5, p, 1, 2, 8, 1e-6, 0, 0, None) == -1                      # weight stride
    assert lib.lv_residual_pair_norm(p, p, p, p, None, 0.5, 1e-6, p, 1.0, p, 1, 8, 1e-6, 0, None) == -1
    assert lib.lv_embed_norm(p, p, 8, 1.0, p, 0, 1, 1, p, None, 0, p, p, 1.0, 1e-6, p, p, p, p, p, p, 1, 8, 0, None) == -1   # no buckets
    assert lib.lv_embed_norm(p, p, 8, 1.0, None, 0, 0, 0, None, p, 0, p, p, 1.0, 1e-6, p, p, p, p, p, p, 1, 8, 0, None) == -1   # empty position table
    assert lib.lv_unary_act(p, p, 8, 17, 0, None) == -1
    assert lib.lv_masked_attn(p, p, p, None, None, None, 0, p, p, p, p, p, 1, 1, 4, 2, 8, 8, 16, 64, 0, 0, 0, 0.5, -1.0, 0, None, 0, 0, 1, None, 0, None) == -1   # cap
    # the gated linear recurrence, stored norms, split residuals, extended attention
    assert lib.lv_gated_linear_recurrence(None, 0, None, 0, None, None, None, None, None, None, None, None, 0, 0, 0, 0, 8, 2, 1, None, 0, 0, None) == 0
    lru = lambda **kw: [p, kw.get("ldu", 64), p, kw.get("ldy", 64), p, p, p, p, p, p, p, p, 64, 1, 1, 1, 64, kw.get("blocks", 2), kw.get("nsplit", 1),  # noqa: E731
                        kw.get("ws"), kw.get("mfma", 1), kw.get("dt", 0), None]
    assert lib.lv_gated_linear_recurrence(*lru(blocks=3)) == -1 and lib.lv_gated_linear_recurrence(*lru(ldu=63)) == -1
    assert lib.lv_gated_linear_recurrence(*lru(nsplit=2)) == -1 and lib.lv_gated_linear_recurrence(*lru(nsplit=2, ws=p, mfma=0)) == -1    # no workspace; no parts
    assert lib.lv_gated_linear_recurrence(*lru(blocks=4)) == -1 and lib.lv_gated_linear_recurrence(*lru(dt=1)) == -1     # blocks of 16, f32: not the matrix cores
    assert lib.lv_gated_linear_recurrence(*lru(ldu=68)) == -1 and lib.lv_gated_linear_recurrence(*lru(ldy=60)) == -1
    hn = lambda **kw: [p, kw.get("ld", 64), 0, 32, p, p, p, kw.get("ks", p), p, p, p, p, 1, 1, kw.get("H", 4), kw.get("G", 2), 8, 16, 1e-6, 0, None]  # noqa: E731
    assert lib.lv_head_norm_store(*hn(ld=40)) == -1 and lib.lv_head_norm_store(*hn(H=3)) == -1 and lib.lv_head_norm_store(*hn(ks=None)) == -1
    ls = lambda **kw: [p, kw.get("ld", 64), 0, 48, p, p, 1.0, p, p, p, p, p, p, 1, 1, 4, 8, 4, kw.get("R", 12), kw.get("rot", 4), 1, 16, 1e-6, 0, None]  # noqa: E731
    assert lib.lv_latent_store(*ls(R=13)) == -1 and lib.lv_latent_store(*ls(rot=3)) == -1 and lib.lv_latent_store(*ls(rot=6)) == -1
    assert lib.lv_scaled_embedding(p, p, 0, 1.0, p, None, None, 1, 8, 0, None) == -1 and lib.lv_residual_split(p, None, None, 1, 8, None) == -1
    assert lib.lv_glu_act(p, 16, p, 7, 1, 8, 4, 0, None) == -1 and lib.lv_glu_act(p, 16, p, 8, 1, 8, 5, 0, None) == -1              # short output rows; unknown act
    ext = lambda **kw: ctypes.byref(_mixlib.AttnExtras(p, p, kw.get("n", 4), kw.get("ld", 0)))  # noqa: E731
    for ex, P, cap in ((ext(), 4, 0.0), (ext(), 0, 2.0), (ext(n=0), 0, 0.0), (ext(ld=31), 0, 0.0)):     # pools, a softcap, an empty table, short rows
        assert lib.lv_masked_attn(p, p, p, p, p, None, 0, p, p, p, p, p, 1, 1, 4, 2, 8, 8, 16, 64, 0, 0, P, 0.5, cap, 0, None, 0, 0, 1, ex, 0, None) == -1
