// Matrix-core form of the windowed pooled attention for bf16 activations and caches.
//
// One workgroup = one tile of 16 consecutive new tokens of one sequence, one kv head, up to four of its
// query heads (one per wave). Keys are walked in tiles of 64 entries, first the pooled blocks that any
// query of the tile may see, then the tokens from the first window start to the last query; what a
// query does not see (outside its window, a block not yet wholly before it, the future) is masked.
//
// Everything is computed transposed so that no operand changes layout between the two products:
//   S^T = K Q^T   v_mfma_f32_16x16x32_bf16, A = 16 keys x 32 of D read straight from the cache rows with 16-byte loads, B = the
//                 wave's Q fragments (registers, loaded once); a lane ends up with 4 keys of ONE query, so the softmax
//                 statistics of a query live in 4 lanes (two shuffles) and
//   O^T += V^T P^T  takes the probabilities of two 16-key blocks as its B operand exactly as they lie (keys x
//                 queries), with A = V^T from transposing LDS reads of the 64-entry V tile that the four waves stage
//                 together, rows as they are.
// Fragment counts are compile-time bounds and nothing in the tile loop branches on the head sizes: a step past the end of D reads
// the last entries of the row again against zeros in Q, a block past Dv reads the last block of V and is not stored. (With a
// branch around every load and its MFMA the loads could not be issued together, and the kernel ran at one memory latency per
// MFMA.)
// The sink is the initial state of the running softmax: maximum 0 (or the head's learned number), sum 1.
// Extended form: a tile's key factors (norms kept beside unnormed keys) and the heads' distance biases sit in LDS; a score becomes
// product * scale * factor + bias before the softmax.
#include "mix_common.h"

namespace lvmix {

typedef __attribute__((ext_vector_type(4))) __bf16 bf16x4v_t;
typedef __attribute__((address_space(3))) __bf16 lds_bf16;
typedef __attribute__((address_space(3))) bf16x4v_t lds_bf16x4;
typedef __attribute__((ext_vector_type(8))) __bf16 bf16x8_t;
typedef __attribute__((ext_vector_type(4))) float f32x4_t;
typedef __attribute__((ext_vector_type(4))) uint32_t u32x4_t;

struct WindowMfmaParams {
  const uint16_t *q, *k_cache, *v_cache, *kp, *vp, *gate;
  int64_t ld_gate;
  int gate_dv;         // entries of a gate row per head: Dv (one per output channel) or 1 (one per head)
  uint16_t* out;
  const int32_t *cu_q, *ctx_lens, *block_tables;
  int bt_stride, H, G, D, Dv, page, window, P, PP, ngroups;
  float scale, sink;
  uint32_t m_page, m_P, m_nseg;   // floor(2^32 / d) of the three divisors the tile loop divides by (see fdiv)
  int nsplit;          // > 1 (launches of at most one query tile per sequence): grid.x = split of the key tiles
  float* ws;           // [T, H, nsplit, Dv + 4] partial read-outs, running maximum and sum
  int64_t k_ld, v_ld;  // elements between the rows of two cached tokens (G*D, G*Dv unless the caches are views of wider rows)
  float m0;            // start of the running maximum: the sink's score 0, or far below any score without a sink
  int keep_first;      // positions below this are seen from everywhere; they take the place of the pooled tiles (P == 0)
  int chunk;           // > 0: a query sees its own chunk of that many positions (counted from 0) up to itself; no window
  const float* sinks;  // [H] or NULL: a learned score per query head in place of the sink's 0
  float cap_in, cap;   // kCapped: scores pass cap * tanh(product * cap_in), cap_in = scale / cap
  const float* key_scale;   // kExtended: [pages, page, G] or NULL, a factor on the score of every cached key
  const float* dist_bias;   // kExtended: [H, bias_len] or NULL, added to the score at distance min(pos - key, bias_len - 1)
  int bias_len;
  int64_t out_ld;      // elements between the output rows of two tokens
};

enum ScoreForm { kPlain = 0, kCapped = 1, kExtended = 2 };

constexpr int kTileQ = 16;
constexpr int kTileK = 64;
constexpr int kMaxK32 = 8;     // D <= 256: 32-wide steps over D (template K32: 2, 4 or 8)
// Row stride of the V tile: an odd multiple of 16 entries, so that the 16 rows a transposed read touches lie in all banks.
__host__ __device__ constexpr int v_row(int Dv) { return Dv % 32 == 0 ? Dv + 16 : Dv; }
constexpr int kMaxDvb = 16;    // Dv <= 256
constexpr int kBiasLds = 1024; // distance biases of a head up to this many are copied to LDS (longer tables are read from memory)
constexpr int kBtCache = 2048; // page ids of a sequence kept in LDS (longer sequences look them up in memory)

// n / d for 0 <= n < 2^31 with magic = floor(2^32 / d) (0xffffffff for d = 1): the estimate is the quotient or one
// less. The tile loop divides by the page size, the pool size and the row's segment count for every row address;
// the compiler's general 32-bit division is some forty instructions each and dominated the kernel.
__device__ __forceinline__ int fdiv(int n, int d, uint32_t magic) {
  const uint32_t q = __umulhi(static_cast<uint32_t>(n), magic);
  const uint32_t r = static_cast<uint32_t>(n) - q * static_cast<uint32_t>(d);
  return static_cast<int>(r >= static_cast<uint32_t>(d) ? q + 1 : q);
}

__device__ __forceinline__ short bf16_bits(float x) {
  __bf16 b = static_cast<__bf16>(x);
  return __builtin_bit_cast(short, b);
}

// tanh through the exponential: the absolute error stays at a few 1e-7, which is what a score multiplied by the cap needs.
__device__ __forceinline__ float fast_tanh(float x) { return 1.0f - 2.0f * __builtin_amdgcn_rcpf(1.0f + __expf(2.0f * x)); }

// AHEAD: the next tile's V rows, key-row addresses and (once the current scores are done) K fragments are fetched while
// the current tile is computed. That pays when a launch has few workgroups per compute unit (decoded tokens). A prompt's
// many tiles hide latency by occupancy instead, and every register counts there: with the 32 registers of a V tile held
// ahead the kernel fell from two waves a SIMD to one and ran 1.7x slower; K32 and DVB size the fragment arrays for the
// head sizes at hand for the same reason.
template <bool AHEAD, int K32, int DVB, int FORM>
__global__ __launch_bounds__(256, AHEAD ? 1 : (DVB > 8 ? 2 : (DVB > 4 ? 3 : 4))) void window_pool_mfma_kernel(WindowMfmaParams p) {
  extern __shared__ __attribute__((aligned(16))) uint16_t vs[];             // V tile [kTileK][ldv]
  const int wave = threadIdx.x / kWave, lane = threadIdx.x % kWave;
  const int ln = lane & 15, lg = lane >> 4;
  const int b = blockIdx.z;
  const int g = blockIdx.y / p.ngroups, hg = blockIdx.y % p.ngroups;
  const int q0 = p.cu_q[b], n = p.cu_q[b + 1] - q0;
  const int split = p.nsplit > 1 ? blockIdx.x : 0;
  const int r0 = p.nsplit > 1 ? 0 : blockIdx.x * kTileQ;
  if (r0 >= n) return;
  const int ctx = p.ctx_lens[b];
  const int nvalid = min(kTileQ, n - r0);
  const int i0 = ctx + r0, i1 = i0 + nvalid - 1;
  const bool qvalid = ln < nvalid;
  const int r = r0 + min(ln, nvalid - 1);
  const int pos = ctx + r;
  const int64_t t = q0 + r;
  const int rep = p.H / p.G;
  const int hloc = hg * 4 + wave;
  const bool active = hloc < rep;
  const int h = g * rep + min(hloc, rep - 1);
  const int D = p.D, Dv = p.Dv, page = p.page, P = p.P, W = p.window;
  const int ndvb = Dv / 16, ldv = v_row(Dv);
  // transposed reads: of every 4 keys x 16 columns, lane 4 q + r of 16 names key q, columns 4r .. 4r + 3, and gets column 4 q + r of all four
  const lds_bf16* vt0 = (const lds_bf16*)vs + (4 * lg + (ln >> 2)) * ldv + 4 * (ln & 3);
  const int64_t GD = static_cast<int64_t>(p.G) * D, GDv = static_cast<int64_t>(p.G) * Dv;
  const int32_t* bt_global = p.block_tables + static_cast<int64_t>(b) * p.bt_stride;
  // the sequence's page ids up to the last query's page, once, so that no row address waits for a second trip to memory
  __shared__ int32_t bt_lds[kBtCache];
  const int nbt = (ctx + r0 + nvalid - 1) / page + 1;
  const bool bt_cached = nbt <= kBtCache;
  if (bt_cached) {
    for (int x = threadIdx.x; x < nbt; x += blockDim.x) bt_lds[x] = bt_global[x];
    __syncthreads();
  }
  auto bt = [&](int idx) { return bt_cached ? bt_lds[idx] : bt_global[idx]; };
  // kExtended: the tile's key factors and the distance biases of the workgroup's heads, behind the V tile
  float* ks_lds = reinterpret_cast<float*>(vs + kTileK * ldv);             // [kTileK]
  float* bias_lds = ks_lds + kTileK;                                       // [4][bias_len]
  const float* bias_h = nullptr;
  float bias_reg[4] = {0.0f, 0.0f, 0.0f, 0.0f};
  bool bias_cached = false;
  if constexpr (FORM == kExtended) {
    if (p.dist_bias != nullptr) {
      bias_cached = p.bias_len <= kBiasLds;
      bias_h = p.dist_bias + static_cast<int64_t>(h) * p.bias_len;
#pragma unroll
      for (int x = 0; x < 4; ++x) bias_reg[x] = bias_h[min(lane + x * kWave, p.bias_len - 1)];     // stored behind the first tile's requests
    }
    if (p.key_scale == nullptr && threadIdx.x < kTileK) ks_lds[threadIdx.x] = 1.0f;                 // read behind the first barrier
  }

  bf16x8_t qf[K32];
  int koff[K32];                                        // this lane's entries of a key or query row in step kk
  {
    const uint16_t* qrow = p.q + (t * p.H + h) * D;
#pragma unroll
    for (int kk = 0; kk < K32; ++kk) {
      koff[kk] = min(32 * kk + 8 * lg, D - 8);
      qf[kk] = *reinterpret_cast<const bf16x8_t*>(qrow + koff[kk]);
      if (32 * kk + 8 * lg >= D) qf[kk] = __builtin_bit_cast(bf16x8_t, u32x4_t{0, 0, 0, 0});
    }
  }
  f32x4_t acc_o[DVB];
#pragma unroll
  for (int d = 0; d < DVB; ++d) acc_o[d] = f32x4_t{0.0f, 0.0f, 0.0f, 0.0f};
  float m = p.sinks != nullptr ? p.sinks[h] : p.m0, l = split == 0 ? p.sink : 0.0f;

  const int chunk = p.chunk, keep = p.keep_first;
  const int jlo = chunk > 0 ? (i0 / chunk) * chunk : max(0, i0 - W + 1);
  const int cstart = chunk > 0 ? (pos / chunk) * chunk : 0;                // first position of this lane's query's chunk
  // entries of the first phase: pooled blocks the last query sees, or (without a pool) kept first tokens before the token tiles
  const int nbmax = P > 0 ? ((chunk == 0 && i1 - W + 1 > 0) ? (i1 - W + 1) / P : 0) : min(keep, jlo);

  // The tiles of both phases as one list: [pooled tiles | token tiles]. The V rows of the next tile and the
  // addresses of its key rows are fetched while the current tile is computed; they meet LDS behind a barrier.
  const int npt = (nbmax + kTileK - 1) / kTileK;
  const int ntt = (i1 + 1 - jlo + kTileK - 1) / kTileK;
  const int ntiles = npt + ntt;
  const int nseg = Dv / 8;                                                // 16-byte segments of a row

  auto tile_start = [&](int tile) { return tile < npt ? tile * kTileK : jlo + (tile - npt) * kTileK; };

  // Cache row of entry `lane` of a tile: every wave finds its 64 rows once, a lane each, and hands them round by shuffles.
  auto tile_slot = [&](int tile) {
    const int e = tile_start(tile) + lane;
    if (tile < npt && P > 0) {
      const int ec = min(e, nbmax - 1);
      const int pj = fdiv(ec * P + P - 1, page, p.m_page);
      return bt(pj) * p.PP + (ec - fdiv(page * pj, P, p.m_P));
    }
    const int ec = min(e, tile < npt ? nbmax - 1 : i1);
    const int pj = fdiv(ec, page, p.m_page);
    return bt(pj) * page + (ec - pj * page);
  };
  // V rows of a tile: consecutive threads take consecutive 16-byte segments of a row (whole cache lines per load instruction),
  // all of a thread's loads are issued together. AHEAD: one tile ahead of their use, and they wait in registers.
  constexpr int NV = DVB / 2;
  const bool keyed = FORM == kExtended && p.key_scale != nullptr && threadIdx.x < kTileK;
  float ksreg = 1.0f;
  u32x4_t vreg[NV];
  const uint16_t* knext[4];
  auto fetch_rows = [&](int tile) {
    const int slot = tile_slot(tile);
    const bool pooled = tile < npt && P > 0;
    const uint16_t* kbase = (pooled ? p.kp : p.k_cache) + g * D;
    const uint16_t* vbase = (pooled ? p.vp : p.v_cache) + g * Dv;
    const int64_t kld = pooled ? GD : p.k_ld, vld = pooled ? GDv : p.v_ld;
#pragma unroll
    for (int x = 0; x < NV; ++x) {
      const int c = min(static_cast<int>(threadIdx.x) + 256 * x, kTileK * nseg - 1);
      const int row = fdiv(c, nseg, p.m_nseg), seg = c - row * nseg;
      vreg[x] = *reinterpret_cast<const u32x4_t*>(vbase + __shfl(slot, row, kWave) * vld + seg * 8);
    }
#pragma unroll
    for (int kb = 0; kb < 4; ++kb) knext[kb] = kbase + __shfl(slot, kb * 16 + ln, kWave) * kld;
    if (keyed) ksreg = p.key_scale[static_cast<int64_t>(slot) * p.G + g];    // the first wave: lane = entry
  };
  // Only LDS traffic meets at the barriers of the tile loop. The fetch-ahead variant waits for that alone, so that the
  // vector loads of the next tile stay in flight across them (a full __syncthreads would drain them every tile).
  auto tile_barrier = [&]() {
    if (AHEAD) asm volatile("s_waitcnt lgkmcnt(0)\n\ts_barrier" ::: "memory");
    else __syncthreads();
  };
  bf16x8_t kdata[AHEAD ? 4 : 1][K32];
  auto fetch_k = [&]() {                                                    // the K fragments of the tile knext points to
#pragma unroll
    for (int kb = 0; kb < (AHEAD ? 4 : 0); ++kb) {
#pragma unroll
      for (int kk = 0; kk < K32; ++kk) kdata[kb][kk] = *reinterpret_cast<const bf16x8_t*>(knext[kb] + koff[kk]);
    }
  };
  // a split takes a contiguous share of the tiles
  const int per_split = p.nsplit > 1 ? (ntiles + p.nsplit - 1) / p.nsplit : ntiles;
  const int t_begin = split * per_split, t_end = min(ntiles, t_begin + per_split);
  if (AHEAD && t_begin < t_end) {
    fetch_rows(t_begin);
    if (active) fetch_k();
  }
  if (bias_cached) {                                                       // read by this wave alone
#pragma unroll
    for (int x = 0; x < 4; ++x)
      if (lane + x * kWave < p.bias_len) bias_lds[wave * p.bias_len + lane + x * kWave] = bias_reg[x];
    for (int x = lane + 4 * kWave; x < p.bias_len; x += kWave) bias_lds[wave * p.bias_len + x] = bias_h[x];
  }
  for (int tile = t_begin; tile < t_end; ++tile) {
    const int phase = tile < npt ? 0 : 1;
    const int e0 = tile_start(tile);
    const int e_end = phase == 0 ? nbmax : i1 + 1;
    const uint16_t* kcur[4];
    tile_barrier();                                                         // the previous tile's V reads are done
    if constexpr (!AHEAD) fetch_rows(tile);
#pragma unroll
    for (int x = 0; x < NV; ++x) {
      const int c = threadIdx.x + 256 * x;
      if (c < kTileK * nseg) {
        const int row = fdiv(c, nseg, p.m_nseg), seg = c - row * nseg;
        *reinterpret_cast<u32x4_t*>(vs + row * ldv + seg * 8) = vreg[x];
      }
    }
#pragma unroll
    for (int kb = 0; kb < 4; ++kb) kcur[kb] = knext[kb];
    if (keyed) ks_lds[threadIdx.x] = ksreg;
    tile_barrier();
    if (AHEAD && tile + 1 < t_end) fetch_rows(tile + 1);
    if (!active) continue;
    {
      f32x4_t s[4];
#pragma unroll
      for (int kb = 0; kb < 4; ++kb) {
        const uint16_t* krow = kcur[kb];
        s[kb] = f32x4_t{0.0f, 0.0f, 0.0f, 0.0f};
#pragma unroll
        for (int kk = 0; kk < K32; ++kk)
          s[kb] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(
              AHEAD ? kdata[AHEAD ? kb : 0][kk] : *reinterpret_cast<const bf16x8_t*>(krow + koff[kk]), qf[kk], s[kb], 0, 0, 0);
      }
      if (AHEAD && tile + 1 < t_end) fetch_k();                            // in flight across the softmax, PV and the barriers
      // result row 4*lg + i of key block kb: key e0 + 16 kb + 4 lg + i
      if constexpr (FORM == kExtended) {
        const bool far = bias_h != nullptr && i0 - (e0 + kTileK - 1) >= p.bias_len - 1;      // all of the tile at the last bias
        const float bias_far = far ? (bias_cached ? bias_lds[wave * p.bias_len + p.bias_len - 1] : bias_h[p.bias_len - 1]) : 0.0f;
#pragma unroll
        for (int kb = 0; kb < 4; ++kb) {
          const f32x4_t ks = *reinterpret_cast<const f32x4_t*>(ks_lds + kb * 16 + 4 * lg);
          s[kb] = s[kb] * (ks * p.scale) + bias_far;
        }
        if (bias_h != nullptr && !far) {
#pragma unroll
          for (int kb = 0; kb < 4; ++kb)
#pragma unroll
            for (int i = 0; i < 4; ++i) {
              const int dist = min(max(pos - (e0 + kb * 16 + 4 * lg + i), 0), p.bias_len - 1);
              s[kb][i] += bias_cached ? bias_lds[wave * p.bias_len + dist] : bias_h[dist];
            }
        }
      } else {
#pragma unroll
        for (int kb = 0; kb < 4; ++kb)
#pragma unroll
          for (int i = 0; i < 4; ++i) s[kb][i] = FORM == kCapped ? p.cap * fast_tanh(s[kb][i] * p.cap_in) : s[kb][i] * p.scale;
      }
      // a tile of tokens that every query of the workgroup sees whole needs no mask
      const bool whole = phase == 1 && e0 + kTileK - 1 <= i0 && (chunk > 0 ? e0 >= i1 - i1 % chunk : i1 - e0 < W);
      if (!whole) {
#pragma unroll
        for (int kb = 0; kb < 4; ++kb)
#pragma unroll
          for (int i = 0; i < 4; ++i) {
            const int ke = e0 + kb * 16 + 4 * lg + i;
            bool vis = ke < e_end;
            if (phase == 0) vis = vis && (P == 0 || ke * P + P - 1 <= pos - W);
            else vis = vis && ke <= pos && ((chunk > 0 ? ke >= cstart : pos - ke < W) || ke < keep);
            s[kb][i] = vis ? s[kb][i] : -INFINITY;
          }
      }
      float mx = -INFINITY;
#pragma unroll
      for (int kb = 0; kb < 4; ++kb)
#pragma unroll
        for (int i = 0; i < 4; ++i) mx = fmaxf(mx, s[kb][i]);
      mx = fmaxf(mx, __shfl_xor(mx, 16, kWave));
      mx = fmaxf(mx, __shfl_xor(mx, 32, kWave));
      const float nm = fmaxf(m, mx);
      const float corr = __expf(m - nm);
      float rs = 0.0f;
      bf16x8_t pb[2];                                                       // key blocks (0, 1) and (2, 3) side by side
#pragma unroll
      for (int kb = 0; kb < 4; ++kb) {
#pragma unroll
        for (int i = 0; i < 4; ++i) {
          const float e = __expf(s[kb][i] - nm);                            // exp(-inf) = 0 for what is not seen
          rs += e;
          pb[kb >> 1][(kb & 1) * 4 + i] = static_cast<__bf16>(e);
        }
      }
      rs += __shfl_xor(rs, 16, kWave);
      rs += __shfl_xor(rs, 32, kWave);
      l = l * corr + rs;
      m = nm;
#pragma unroll
      for (int d = 0; d < DVB; ++d) acc_o[d] *= corr;
#pragma unroll
      for (int c = 0; c < 2; ++c) {                                         // key blocks 2c and 2c + 1
#pragma unroll
        for (int d = 0; d < DVB; ++d) {
          const lds_bf16* vt = vt0 + 32 * c * ldv + 16 * min(d, ndvb - 1);
          const bf16x4v_t lo = __builtin_amdgcn_ds_read_tr16_b64_v4bf16((lds_bf16x4*)vt);
          const bf16x4v_t hi = __builtin_amdgcn_ds_read_tr16_b64_v4bf16((lds_bf16x4*)(vt + 16 * ldv));
          acc_o[d] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(__builtin_shufflevector(lo, hi, 0, 1, 2, 3, 4, 5, 6, 7), pb[c], acc_o[d], 0, 0, 0);
        }
      }
    }
  }
  if (!active || !qvalid) return;
  if (p.nsplit > 1) {                                                       // unnormalised partials; window_pool_merge_kernel ends the job
    float* w = p.ws + ((t * p.H + h) * p.nsplit + split) * (Dv + 4);
#pragma unroll
    for (int d = 0; d < DVB; ++d)
      if (d < ndvb)
        *reinterpret_cast<f32x4_t*>(w + 16 * d + 4 * lg) = acc_o[d];
    if (lg == 0) {
      w[Dv] = m;
      w[Dv + 1] = l;
    }
    return;
  }
  const float inv = l > 0.0f ? 1.0f / l : 0.0f;
  uint16_t* orow = p.out + t * p.out_ld + static_cast<int64_t>(h) * Dv;
  const uint16_t* grow = p.gate != nullptr ? p.gate + t * p.ld_gate + static_cast<int64_t>(h) * p.gate_dv : nullptr;
  const int gstep = p.gate_dv > 1 ? 1 : 0;
#pragma unroll
  for (int d = 0; d < DVB; ++d) {
    if (d < ndvb) {
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        const int dv = 16 * d + 4 * lg + i;
        float val = acc_o[d][i] * inv;
        if (grow != nullptr) val *= sigmoidf_(__builtin_bit_cast(float, static_cast<uint32_t>(grow[dv * gstep]) << 16));
        orow[dv] = static_cast<uint16_t>(bf16_bits(val));
      }
    }
  }
}

// One wave per (token, query head): combines the splits' partials (each with its own running maximum), applies the gate.
__global__ __launch_bounds__(256) void window_pool_merge_kernel(const float* __restrict__ ws, const uint16_t* __restrict__ gate,
                                                                int64_t ld_gate, int gate_dv, uint16_t* __restrict__ out,
                                                                int64_t items, int H, int Dv, int nsplit, int64_t out_ld, float m0,
                                                                const float* __restrict__ sinks) {
  const int wave = threadIdx.x / kWave, lane = threadIdx.x % kWave;
  const int64_t item = static_cast<int64_t>(blockIdx.x) * (blockDim.x / kWave) + wave;
  if (item >= items) return;
  const int64_t t = item / H;
  const int h = static_cast<int>(item - t * H);
  const float* w = ws + item * nsplit * (Dv + 4);
  // lane s holds split s (at most kWave of them): its maximum and sum, then the factor that brings it to the common maximum
  const float m0h = sinks != nullptr ? sinks[h] : m0;
  const bool in = lane < nsplit;
  const float ms = in ? w[lane * (Dv + 4) + Dv] : -INFINITY, ls = in ? w[lane * (Dv + 4) + Dv + 1] : 0.0f;
  const float mm = fmaxf(m0h, wave_max(ms));
  const float f = in ? expf(ms - mm) : 0.0f;
  const float ll = wave_sum(ls * f);
  const float inv = ll > 0.0f ? 1.0f / ll : 0.0f;
  for (int dv0 = 0; dv0 < Dv; dv0 += kWave) {                               // the same trip count for every lane: the factors are shuffled
    const int dv = dv0 + lane;
    const float* col = w + min(dv, Dv - 1);
    float acc = 0.0f;
#pragma unroll 4
    for (int s = 0; s < nsplit; ++s) acc += col[s * (Dv + 4)] * __shfl(f, s, kWave);
    float val = acc * inv;
    if (dv >= Dv) continue;
    if (gate != nullptr)
      val *= sigmoidf_(__builtin_bit_cast(float, static_cast<uint32_t>(gate[t * ld_gate + static_cast<int64_t>(h) * gate_dv +
                                                                            (gate_dv > 1 ? dv : 0)]) << 16));
    out[t * out_ld + static_cast<int64_t>(h) * Dv + dv] = static_cast<uint16_t>(bf16_bits(val));
  }
}

}  // namespace lvmix

using namespace lvmix;

static uint32_t magic(int d) { return d <= 1 ? 0xffffffffu : static_cast<uint32_t>((1ull << 32) / static_cast<uint64_t>(d)); }

extern "C" int lv_window_pool_attn_mfma(const void* q, const void* k_cache, const void* v_cache, const void* kp,
                                        const void* vp, const void* gate, int64_t ld_gate, void* out, const int32_t* cu_q,
                                        const int32_t* ctx_lens, const int32_t* block_tables, int bt_stride, int B,
                                        int max_new_tokens, int H, int G, int D, int Dv, int page, int window, int P,
                                        float scale, int has_sink, int nsplit, void* workspace, int64_t T, int64_t k_ld,
                                        int64_t v_ld, int gate_kind, void* stream) {
  return lv_masked_attn_mfma(q, k_cache, v_cache, kp, vp, gate, ld_gate, out, cu_q, ctx_lens, block_tables, bt_stride, B,
                             max_new_tokens, H, G, D, Dv, page, window, 0, 0, P, scale, 0.0f, has_sink, nullptr, nsplit, workspace, T,
                             k_ld, v_ld, gate_kind, nullptr, stream);
}

extern "C" int lv_masked_attn_mfma(const void* q, const void* k_cache, const void* v_cache, const void* kp, const void* vp,
                                   const void* gate, int64_t ld_gate, void* out, const int32_t* cu_q, const int32_t* ctx_lens,
                                   const int32_t* block_tables, int bt_stride, int B, int max_new_tokens, int H, int G, int D,
                                   int Dv, int page, int window, int keep_first, int chunk, int P, float scale, float softcap, int has_sink,
                                   const void* sinks, int nsplit, void* workspace, int64_t T, int64_t k_ld, int64_t v_ld,
                                   int gate_kind, const lv_attn_extras* extras, void* stream) {
  if (B == 0 || max_new_tokens <= 0) return 0;
  if (keep_first < 0 || chunk < 0 || (P > 0 && (keep_first > 0 || chunk > 0)))
    return fail(-1, "lv_masked_attn_mfma: kept first tokens and chunks do not combine with pooled blocks");
  if (!(softcap >= 0.0f)) return fail(-1, "lv_masked_attn_mfma: softcap");
  if (sinks != nullptr) has_sink = 1;
  if (!q || !k_cache || !v_cache || !out || !cu_q || !ctx_lens || !block_tables)
    return fail(-1, "lv_window_pool_attn_mfma: null pointer");
  if (P > 0 && (!kp || !vp)) return fail(-1, "lv_window_pool_attn_mfma: pooled blocks without their cache");
  if (B < 0 || H <= 0 || G <= 0 || H % G != 0 || page <= 0 || window <= 0 || bt_stride <= 0)
    return fail(-1, "lv_window_pool_attn_mfma: bad sizes");
  if (D % 16 != 0 || Dv % 16 != 0 || D <= 0 || Dv <= 0 || D > 32 * kMaxK32 || Dv > 16 * kMaxDvb)
    return fail(-2, "lv_window_pool_attn_mfma: head sizes %d / %d (multiples of 16 up to 256)", D, Dv);
  if (gate_kind != LV_MIX_GATE_PER_HEAD && gate_kind != LV_MIX_GATE_PER_CHANNEL)
    return fail(-1, "lv_window_pool_attn_mfma: gate kind %d", gate_kind);
  const int gate_dv = gate_kind == LV_MIX_GATE_PER_HEAD ? 1 : Dv;
  if (gate != nullptr && ld_gate < static_cast<int64_t>(H) * gate_dv) return fail(-1, "lv_window_pool_attn_mfma: gate stride");
  if (k_ld <= 0) k_ld = static_cast<int64_t>(G) * D;
  if (v_ld <= 0) v_ld = static_cast<int64_t>(G) * Dv;
  if (k_ld < static_cast<int64_t>(G) * D || v_ld < static_cast<int64_t>(G) * Dv || k_ld % 8 != 0 || v_ld % 8 != 0 ||
      (reinterpret_cast<uintptr_t>(k_cache) & 15) != 0 || (reinterpret_cast<uintptr_t>(v_cache) & 15) != 0)
    return fail(-1, "lv_window_pool_attn_mfma: row strides or alignment of the caches");
  const bool extended = extras != nullptr && (extras->key_scale != nullptr || extras->dist_bias != nullptr);
  if (extended && (P > 0 || softcap > 0.0f || (extras->dist_bias != nullptr && extras->bias_len <= 0)))
    return fail(-1, "lv_masked_attn_mfma: key factors and distance biases combine with neither pooled blocks nor a softcap");
  const int64_t out_ld = extras != nullptr && extras->out_ld > 0 ? extras->out_ld : static_cast<int64_t>(H) * Dv;
  if (out_ld < static_cast<int64_t>(H) * Dv) return fail(-1, "lv_masked_attn_mfma: output stride");
  const float m0 = has_sink ? 0.0f : -1e30f;
  const int rep = H / G;
  const int ngroups = (rep + 3) / 4;
  WindowMfmaParams p{static_cast<const uint16_t*>(q), static_cast<const uint16_t*>(k_cache),
                     static_cast<const uint16_t*>(v_cache), static_cast<const uint16_t*>(kp),
                     static_cast<const uint16_t*>(vp), static_cast<const uint16_t*>(gate), ld_gate, gate_dv,
                     static_cast<uint16_t*>(out), cu_q, ctx_lens, block_tables, bt_stride, H, G, D, Dv, page, window, P,
                     P > 0 ? (page + P - 1) / P : 0, ngroups, scale, has_sink ? 1.0f : 0.0f,
                     magic(page), magic(P > 0 ? P : 1), magic(Dv / 8), nsplit > 1 ? nsplit : 1, static_cast<float*>(workspace),
                     k_ld, v_ld, m0, keep_first, chunk, static_cast<const float*>(sinks), softcap > 0.0f ? scale / softcap : 0.0f,
                     softcap, extended ? static_cast<const float*>(extras->key_scale) : nullptr,
                     extended ? static_cast<const float*>(extras->dist_bias) : nullptr, extended ? extras->bias_len : 0, out_ld};
  if (nsplit > 1 && (max_new_tokens > kTileQ || workspace == nullptr || T <= 0 || nsplit > kWave))
    return fail(-1, "lv_window_pool_attn_mfma: key splits need one query tile per sequence and a workspace");
  size_t shm = static_cast<size_t>(kTileK) * v_row(Dv) * sizeof(uint16_t);
  if (extended) shm += sizeof(float) * (kTileK + (p.dist_bias != nullptr && p.bias_len <= kBiasLds ? 4 * static_cast<size_t>(p.bias_len) : 0));
  dim3 grid(nsplit > 1 ? nsplit : (max_new_tokens + kTileQ - 1) / kTileQ, G * ngroups, B), block(256);
  hipStream_t st = as_stream(stream);
  const bool tiny = D <= 64 && Dv <= 64, small = D <= 128 && Dv <= 128;
#define LVMIX_ATT_FORM(AHEAD, FORM)                                                               \
  do {                                                                                            \
    if (tiny) window_pool_mfma_kernel<AHEAD, 2, 4, FORM><<<grid, block, shm, st>>>(p);            \
    else if (small) window_pool_mfma_kernel<AHEAD, 4, 8, FORM><<<grid, block, shm, st>>>(p);      \
    else window_pool_mfma_kernel<AHEAD, kMaxK32, kMaxDvb, FORM><<<grid, block, shm, st>>>(p);     \
  } while (0)
#define LVMIX_ATT(AHEAD)                                     \
  do {                                                       \
    if (softcap > 0.0f) LVMIX_ATT_FORM(AHEAD, kCapped);      \
    else if (extended) LVMIX_ATT_FORM(AHEAD, kExtended);     \
    else LVMIX_ATT_FORM(AHEAD, kPlain);                      \
  } while (0)
  if (max_new_tokens <= kTileQ) LVMIX_ATT(true);
  else LVMIX_ATT(false);
#undef LVMIX_ATT
#undef LVMIX_ATT_FORM
  if (nsplit > 1) {
    const int64_t items = T * H;
    window_pool_merge_kernel<<<dim3(static_cast<unsigned>((items + 3) / 4)), block, 0, st>>>(
        static_cast<const float*>(workspace), static_cast<const uint16_t*>(gate), ld_gate, gate_dv,
        static_cast<uint16_t*>(out), items, H, Dv, nsplit, out_ld, m0, static_cast<const float*>(sinks));
  }
  return launched("lv_window_pool_attn_mfma");
}
