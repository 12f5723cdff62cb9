// Real-gated linear recurrent unit (Griffin): per channel S <- a S + sqrt(1 - a^2) i u, log a = rate r, with the gates r and i from
// block-diagonal matrices of u, and the read-out S gelu(y). Gates, decays and state never leave f32 and never reach memory.
//
//   lru_tile_kernel    bf16. One workgroup = 64 channels of one block, walking a sequence (or a part of it) in tiles of 64 tokens.
//                      A wave owns 16 channels: both gates of 64 tokens as 16x16x32 MFMAs straight from the rows of u and of the gate
//                      matrices; in the result a lane holds 4 neighbouring tokens of one channel, whose decays and inputs it folds into
//                      one (decay, sum) pair; the pairs of 16 tokens meet in two shuffles, the 16-token groups and the tiles follow one
//                      another through a running state in registers. States go through LDS so that y is read and the output
//                      written in whole rows.
//                      AGG: only the (decay, sum) pair of a part of the sequence, for the parts behind it. A few long prompts do
//                      not fill the chip with a workgroup per 64 channels, so the sequence is cut into parts: a first launch
//                      computes every part's pair, a second one starts each part from the pairs before it. Computing the gates
//                      twice moves 2 bytes a channel and token once more; keeping decays and inputs in f32 between launches
//                      would move 16.
//   lru_step_kernel    bf16, single tokens: 16 channels x 16 sequences a workgroup, the four waves share the inner dimension.
//   lru_plain_kernel   f32, and sizes the matrix cores do not take: a lane per channel, 16 tokens at a time.
#include "mix_common.h"

namespace lvmix {

typedef __attribute__((ext_vector_type(8))) __bf16 bf16x8_t;
typedef __attribute__((ext_vector_type(4))) float f32x4_t;

struct LruParams {
  const void *u, *y;
  int64_t ldu, ldy;
  const void* gw;                  // act [blocks, 2, n, n]
  const float *gb, *rate;          // [blocks, 2, n], [N]
  float* state;                    // [slots, N]
  const int32_t *cu_q, *ctx_lens, *slots;
  void* out;
  int64_t ldo;
  int N, n, B, nsplit, rows16;     // rows16: y and out rows allow 16-byte accesses
  int64_t T;
  float* ws;                       // [B, nsplit, 2, N] decay and sum of each part; the last part's sum holds the starting state
};

// Hardware exponential, reciprocal and square root (about one unit in the last place of f32 each) for the bf16 kernels.
__device__ __forceinline__ float fast_sigmoid(float x) { return __builtin_amdgcn_rcpf(1.0f + __expf(-x)); }
__device__ __forceinline__ float fast_gelu_tanh(float z) {               // z (1 + tanh(w)) / 2 = z sigmoid(2 w)
  return z * fast_sigmoid(1.5957691216057308f * (z + 0.044715f * z * z * z));
}
// (a, sqrt(1 - a^2)) from log a <= 0; near a = 1 the difference is taken as the series of -expm1(2 log a).
__device__ __forceinline__ void decay_pair(float log_a, float& a, float& root) {
  a = __expf(log_a);
  const float z = 2.0f * log_a;
  const float series = -z * (1.0f + z * (1.0f / 2) * (1.0f + z * (1.0f / 3) * (1.0f + z * (1.0f / 4) * (1.0f + z * (1.0f / 5) * (1.0f + z * (1.0f / 6))))));
  root = __builtin_amdgcn_sqrtf(z > -0.25f ? series : 1.0f - a * a);
}

constexpr int kLruTile = 64;
constexpr int kLruLd = 68;         // f32 row stride of the state tile: rows stay 16-byte aligned

template <bool AGG>
__global__ __launch_bounds__(256, 4) void lru_tile_kernel(LruParams p) {
  __shared__ __attribute__((aligned(16))) float s_lds[AGG ? 4 : kLruTile * kLruLd];
  const int wave = threadIdx.x / kWave, lane = threadIdx.x % kWave;
  const int ln = lane & 15, lg = lane >> 4;
  const int n = p.n, ctiles = (n + 63) / 64;
  const int blk = blockIdx.x / ctiles, c0 = (blockIdx.x - blk * ctiles) * 64;
  const int split = blockIdx.y, b = blockIdx.z;
  const int q0 = p.cu_q[b], cnt = p.cu_q[b + 1] - q0;
  if (cnt <= 0) return;
  const int tiles = (cnt + kLruTile - 1) / kLruTile;
  const int per = (tiles + p.nsplit - 1) / p.nsplit;
  const int t_begin = split * per, t_end = min(tiles, t_begin + per);
  const int cw = c0 + 16 * wave;
  const bool active = cw < n;                                   // n is a multiple of 32
  const int cl = min(cw, n - 16) + ln;                          // this lane's channel within the block
  const int ch = blk * n + cl;
  const uint16_t* u = static_cast<const uint16_t*>(p.u) + static_cast<int64_t>(q0) * p.ldu + blk * n;
  const uint16_t* wr = static_cast<const uint16_t*>(p.gw) + (static_cast<int64_t>(blk) * 2 * n + cl) * n;
  const uint16_t* wi = wr + static_cast<int64_t>(n) * n;
  const float br = p.gb[blk * 2 * n + cl], bi = p.gb[blk * 2 * n + n + cl], rate = p.rate[ch];
  float* ws = p.ws + static_cast<int64_t>(b) * p.nsplit * 2 * p.N + ch;
  float* sstate = p.state + static_cast<int64_t>(p.slots[b]) * p.N + ch;
  float run = 0.0f, arun = 1.0f;                                // state ahead of the tile; AGG: the part's sum and decay so far
  if (AGG) {
    // the parts of the second launch must not read the state that the last of them replaces: it is handed on through the workspace
    if (split == 0 && active && lg == 0) ws[static_cast<int64_t>(2 * (p.nsplit - 1) + 1) * p.N] = p.ctx_lens[b] > 0 ? *sstate : 0.0f;
  } else if (p.nsplit > 1) {
    if (t_begin >= t_end) return;
    run = ws[static_cast<int64_t>(2 * (p.nsplit - 1) + 1) * p.N];
    for (int s = 0; s < split; ++s) run = ws[static_cast<int64_t>(2 * s) * p.N] * run + ws[static_cast<int64_t>(2 * s + 1) * p.N];
  } else if (p.ctx_lens[b] > 0) {
    run = *sstate;
  }
  for (int tile = t_begin; tile < t_end; ++tile) {
    const int t0 = tile * kLruTile;
    if (active) {
      f32x4_t ar[4], ai[4];
      const uint16_t* arow[4];
#pragma unroll
      for (int mb = 0; mb < 4; ++mb) {
        ar[mb] = f32x4_t{0.0f, 0.0f, 0.0f, 0.0f};
        ai[mb] = ar[mb];
        arow[mb] = u + static_cast<int64_t>(min(t0 + 16 * mb + ln, cnt - 1)) * p.ldu + 8 * lg;
      }
#pragma unroll 2
      for (int k = 0; k < n; k += 32) {
        const bf16x8_t fr = *reinterpret_cast<const bf16x8_t*>(wr + k + 8 * lg);
        const bf16x8_t fi = *reinterpret_cast<const bf16x8_t*>(wi + k + 8 * lg);
#pragma unroll
        for (int mb = 0; mb < 4; ++mb) {
          const bf16x8_t fu = *reinterpret_cast<const bf16x8_t*>(arow[mb] + k);
          ar[mb] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(fu, fr, ar[mb], 0, 0, 0);
          ai[mb] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(fu, fi, ai[mb], 0, 0, 0);
        }
      }
#pragma unroll
      for (int mb = 0; mb < 4; ++mb) {                          // result row 4 * lg + i: token, column ln: channel
        float a[4], x[4];
#pragma unroll
        for (int i = 0; i < 4; ++i) {
          const int tok = t0 + 16 * mb + 4 * lg + i;
          const float uv = __builtin_bit_cast(float, static_cast<uint32_t>(u[static_cast<int64_t>(min(tok, cnt - 1)) * p.ldu + cl]) << 16);
          float root;
          decay_pair(rate * fast_sigmoid(ar[mb][i] + br), a[i], root);
          x[i] = root * fast_sigmoid(ai[mb][i] + bi) * uv;
          if (tok >= cnt) {
            a[i] = 1.0f;
            x[i] = 0.0f;
          }
        }
        float da = (a[0] * a[1]) * (a[2] * a[3]);
        float sx = ((x[0] * a[1] + x[1]) * a[2] + x[2]) * a[3] + x[3];
#pragma unroll
        for (int o = 16; o <= 32; o <<= 1) {                    // over the four lane groups: the earlier pair first
          const float pa = __shfl_up(da, o, kWave), px = __shfl_up(sx, o, kWave);
          if (lane >= o) {
            sx = da * px + sx;
            da *= pa;
          }
        }
        const float ta = __shfl(da, 48 + ln, kWave), tx = __shfl(sx, 48 + ln, kWave);
        if (!AGG) {
          const float ea = __shfl_up(da, 16, kWave), ex = __shfl_up(sx, 16, kWave);
          float s = lg == 0 ? run : ea * run + ex;
#pragma unroll
          for (int i = 0; i < 4; ++i) {
            s = a[i] * s + x[i];
            s_lds[(16 * mb + 4 * lg + i) * kLruLd + 16 * wave + ln] = s;
          }
        } else {
          arun *= ta;
        }
        run = ta * run + tx;
      }
    }
    if (!AGG) {
      __syncthreads();
      const uint16_t* y = static_cast<const uint16_t*>(p.y) + static_cast<int64_t>(q0 + t0) * p.ldy + blk * n + c0;
      uint16_t* out = static_cast<uint16_t*>(p.out) + static_cast<int64_t>(q0 + t0) * p.ldo + blk * n + c0;
      const int rows = min(kLruTile, cnt - t0), cols = min(64, n - c0);
#pragma unroll
      for (int pass = 0; pass < 2; ++pass) {
        const int tok = (threadIdx.x >> 3) + 32 * pass, c = 8 * (threadIdx.x & 7);
        if (tok < rows && c < cols) {
          const float* srow = s_lds + tok * kLruLd + c;
          float v[8];
          *reinterpret_cast<float4*>(v) = *reinterpret_cast<const float4*>(srow);
          *reinterpret_cast<float4*>(v + 4) = *reinterpret_cast<const float4*>(srow + 4);
          uint16_t yy[8];
          if (p.rows16) {
            *reinterpret_cast<uint4*>(yy) = *reinterpret_cast<const uint4*>(y + static_cast<int64_t>(tok) * p.ldy + c);
          } else {
#pragma unroll
            for (int e = 0; e < 8; ++e) yy[e] = y[static_cast<int64_t>(tok) * p.ldy + c + e];
          }
          bf16_t o[8];
#pragma unroll
          for (int e = 0; e < 8; ++e) stf(o + e, v[e] * fast_gelu_tanh(__builtin_bit_cast(float, static_cast<uint32_t>(yy[e]) << 16)));
          uint16_t* dst = out + static_cast<int64_t>(tok) * p.ldo + c;
          if (p.rows16) {
            *reinterpret_cast<uint4*>(dst) = *reinterpret_cast<const uint4*>(o);
          } else {
#pragma unroll
            for (int e = 0; e < 8; ++e) dst[e] = o[e].bits;
          }
        }
      }
      __syncthreads();                                          // the next tile overwrites the states read above
    }
  }
  if (!active || lg != 0) return;
  if (AGG) {
    ws[static_cast<int64_t>(2 * split) * p.N] = arun;
    ws[static_cast<int64_t>(2 * split + 1) * p.N] = run;
  } else if (t_end == tiles) {
    *sstate = run;
  }
}

__global__ __launch_bounds__(256) void lru_step_kernel(LruParams p) {
  __shared__ float red[4][2][16][17];
  const int wave = threadIdx.x / kWave, lane = threadIdx.x % kWave;
  const int ln = lane & 15, lg = lane >> 4;
  const int n = p.n, b0 = blockIdx.y * 16;
  const int blk = blockIdx.x / (n / 16), c0 = (blockIdx.x - blk * (n / 16)) * 16;
  const uint16_t* u = static_cast<const uint16_t*>(p.u) + blk * n;
  const uint16_t* arow = u + min(static_cast<int64_t>(p.cu_q[min(b0 + ln, p.B - 1)]), p.T - 1) * p.ldu + 8 * lg;
  const uint16_t* wr = static_cast<const uint16_t*>(p.gw) + (static_cast<int64_t>(blk) * 2 * n + c0 + ln) * n + 8 * lg;
  const uint16_t* wi = wr + static_cast<int64_t>(n) * n;
  f32x4_t ar = f32x4_t{0.0f, 0.0f, 0.0f, 0.0f}, ai = ar;
#pragma unroll 2
  for (int k = 32 * wave; k < n; k += 128) {
    const bf16x8_t fu = *reinterpret_cast<const bf16x8_t*>(arow + k);
    ar = __builtin_amdgcn_mfma_f32_16x16x32_bf16(fu, *reinterpret_cast<const bf16x8_t*>(wr + k), ar, 0, 0, 0);
    ai = __builtin_amdgcn_mfma_f32_16x16x32_bf16(fu, *reinterpret_cast<const bf16x8_t*>(wi + k), ai, 0, 0, 0);
  }
#pragma unroll
  for (int i = 0; i < 4; ++i) {
    red[wave][0][4 * lg + i][ln] = ar[i];
    red[wave][1][4 * lg + i][ln] = ai[i];
  }
  __syncthreads();
  const int tok = threadIdx.x / 16, c = threadIdx.x % 16, b = b0 + tok;
  if (b >= p.B) return;
  const int64_t t = p.cu_q[b];
  if (p.cu_q[b + 1] <= t) return;
  const int ch = blk * n + c0 + c;
  float r = p.gb[blk * 2 * n + c0 + c], g = p.gb[blk * 2 * n + n + c0 + c];
#pragma unroll
  for (int w = 0; w < 4; ++w) {
    r += red[w][0][tok][c];
    g += red[w][1][tok][c];
  }
  float a, root;
  decay_pair(p.rate[ch] * fast_sigmoid(r), a, root);
  const float uv = ldf(reinterpret_cast<const bf16_t*>(u) + t * p.ldu + c0 + c);
  float* sstate = p.state + static_cast<int64_t>(p.slots[b]) * p.N + ch;
  const float s = (p.ctx_lens[b] > 0 ? a * *sstate : 0.0f) + root * fast_sigmoid(g) * uv;
  *sstate = s;
  stf(static_cast<bf16_t*>(p.out) + t * p.ldo + ch, s * fast_gelu_tanh(ldf(static_cast<const bf16_t*>(p.y) + t * p.ldy + ch)));
}

constexpr int kPlainTok = 16, kPlainK = 256;

template <typename T>
__global__ __launch_bounds__(64) void lru_plain_kernel(LruParams p) {
  __shared__ float u_lds[kPlainTok * kPlainK];
  const int lane = threadIdx.x, n = p.n, ctiles = (n + 63) / 64;
  const int blk = blockIdx.x / ctiles, c = (blockIdx.x - blk * ctiles) * 64 + lane, b = blockIdx.y;
  const bool active = c < n;
  const int cl = min(c, n - 1), ch = blk * n + cl;
  const int q0 = p.cu_q[b], cnt = p.cu_q[b + 1] - q0;
  if (cnt <= 0) return;
  const T* u = static_cast<const T*>(p.u) + static_cast<int64_t>(q0) * p.ldu + blk * n;
  const T* y = static_cast<const T*>(p.y) + static_cast<int64_t>(q0) * p.ldy + ch;
  T* out = static_cast<T*>(p.out) + static_cast<int64_t>(q0) * p.ldo + ch;
  const T* wr = static_cast<const T*>(p.gw) + (static_cast<int64_t>(blk) * 2 * n + cl) * n;
  const T* wi = wr + static_cast<int64_t>(n) * n;
  const float br = p.gb[blk * 2 * n + cl], bi = p.gb[blk * 2 * n + n + cl], rate = p.rate[ch];
  float* sstate = p.state + static_cast<int64_t>(p.slots[b]) * p.N + ch;
  float s = p.ctx_lens[b] > 0 ? *sstate : 0.0f;
  for (int t0 = 0; t0 < cnt; t0 += kPlainTok) {
    const int m = min(kPlainTok, cnt - t0);
    float r[kPlainTok], g[kPlainTok];
#pragma unroll
    for (int i = 0; i < kPlainTok; ++i) {
      r[i] = br;
      g[i] = bi;
    }
    for (int k0 = 0; k0 < n; k0 += kPlainK) {
      const int kn = min(kPlainK, n - k0);
      __syncthreads();                                          // the previous piece is used up
      for (int i = 0; i < kPlainTok; ++i)
        for (int k = lane; k < kn; k += kWave)
          u_lds[i * kPlainK + k] = i < m ? ldf(u + static_cast<int64_t>(t0 + i) * p.ldu + k0 + k) : 0.0f;
      __syncthreads();
      for (int k = 0; k < kn; ++k) {
        const float w0 = ldf(wr + k0 + k), w1 = ldf(wi + k0 + k);
#pragma unroll
        for (int i = 0; i < kPlainTok; ++i) {
          const float uv = u_lds[i * kPlainK + k];
          r[i] += w0 * uv;
          g[i] += w1 * uv;
        }
      }
    }
#pragma unroll
    for (int i = 0; i < kPlainTok; ++i) {
      if (i < m) {
        const float log_a = rate * sigmoidf_(r[i]);
        const float x = sqrtf(-expm1f(2.0f * log_a)) * sigmoidf_(g[i]) * ldf(u + static_cast<int64_t>(t0 + i) * p.ldu + cl);
        s = expf(log_a) * s + x;
        if (active)
          stf(out + static_cast<int64_t>(t0 + i) * p.ldo, s * gelu_tanh_(ldf(y + static_cast<int64_t>(t0 + i) * p.ldy)));
      }
    }
  }
  if (active) *sstate = s;
}

}  // namespace lvmix

using namespace lvmix;

extern "C" int lv_gated_linear_recurrence(const void* u, int64_t ldu, const void* y, int64_t ldy, const void* gate_w,
                                          const void* gate_b, const void* rate, void* state, const int32_t* cu_q,
                                          const int32_t* ctx_lens, const int32_t* slots, void* out, int64_t ldo, int B, int64_t T,
                                          int max_new_tokens, int N, int blocks, int nsplit, void* workspace, int mfma, int dtype,
                                          void* stream) {
  if (B == 0 || T == 0 || max_new_tokens == 0) return 0;
  if (!u || !y || !gate_w || !gate_b || !rate || !state || !cu_q || !ctx_lens || !slots || !out)
    return fail(-1, "lv_gated_linear_recurrence: null pointer");
  if (B < 0 || T < 0 || max_new_tokens < 0 || N <= 0 || blocks <= 0 || N % blocks != 0 || ldu < N || ldy < N || ldo < N || nsplit < 1 ||
      (nsplit > 1 && (!mfma || workspace == nullptr)))
    return fail(-1, "lv_gated_linear_recurrence: bad sizes");
  if (dtype != LV_MIX_BF16 && dtype != LV_MIX_F32) return fail(-1, "lv_gated_linear_recurrence: dtype %d", dtype);
  const int n = N / blocks;
  auto a16 = [](const void* q) { return (reinterpret_cast<uintptr_t>(q) & 15) == 0; };
  if (mfma && (dtype != LV_MIX_BF16 || n % 32 != 0 || ldu % 8 != 0 || !a16(u) || !a16(gate_w)))
    return fail(-1, "lv_gated_linear_recurrence: the matrix cores take bf16 blocks in multiples of 32 on aligned rows");
  LruParams p{u, y, ldu, ldy, gate_w, static_cast<const float*>(gate_b), static_cast<const float*>(rate), static_cast<float*>(state),
              cu_q, ctx_lens, slots, out, ldo, N, n, B, nsplit, ldy % 8 == 0 && ldo % 8 == 0 && a16(y) && a16(out),
              T, static_cast<float*>(workspace)};
  hipStream_t st = as_stream(stream);
  if (!mfma) {
    dim3 grid(blocks * ((n + 63) / 64), B), block(64);
    if (dtype == LV_MIX_BF16) lru_plain_kernel<bf16_t><<<grid, block, 0, st>>>(p);
    else lru_plain_kernel<float><<<grid, block, 0, st>>>(p);
  } else if (max_new_tokens == 1) {
    lru_step_kernel<<<dim3(blocks * (n / 16), (B + 15) / 16), dim3(256), 0, st>>>(p);
  } else {
    const int columns = blocks * ((n + 63) / 64);
    if (nsplit > 1) lru_tile_kernel<true><<<dim3(columns, nsplit - 1, B), dim3(256), 0, st>>>(p);
    lru_tile_kernel<false><<<dim3(columns, nsplit, B), dim3(256), 0, st>>>(p);
  }
  return launched("lv_gated_linear_recurrence");
}
