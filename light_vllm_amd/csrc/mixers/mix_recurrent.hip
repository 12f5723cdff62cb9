// Recurrent mixers that share one form of state update, and the small steps around them.
//
//   causal_conv_kernel        short causal convolution over columns of a projection: one thread walks a tile of a sequence's
//                             new tokens for one or four channels with the last inputs in registers, adds a bias, applies
//                             silu, and carries the sequence's last inputs in the same launch. A second form hands the
//                             result to attention: queries times a factor of their position, keys and values into the
//                             paged caches. Long filters read their taps from memory instead.
//   token_shift_kernel        every token's input mixed with its predecessor's by several weight vectors at once; prompts take
//                             tiles of tokens with the weights in registers.
//   gated_scan_kernel         S <- decay S + write k v^T, o = S^T q per head over the new tokens of every sequence. What decays
//                             and what is written are computed in f32 as the inputs are staged, from one of three rules:
//                             step sizes of a state-space layer, log gates under a running maximum with a normaliser
//                             vector beside the state, or a decay per row of the state with a bonus for the current token.
//                             A lane owns a block of rows by four columns of the state.
//   grouped_gate_norm_kernel  o silu(z), RMS norm in equal parts of the row, weight.
//   residual_pair_norm_kernel the f32 residual receives the scaled sum of two RMS-normed and weighted sublayer outputs and
//                             is normed for the next sublayer.
//   embed_norm_kernel         token row times a constant + hashed pair row + position row, norm, first sublayer's norm.
//   unary_act_kernel          activation without a gate.
#include "mix_common.h"

namespace lvmix {

__device__ __forceinline__ float log_sigmoidf_(float x) { return x < 0.0f ? x - log1pf(expf(x)) : -log1pf(expf(-x)); }

__device__ __forceinline__ float read_lane(float x, int i) {           // i uniform over the wave
  return __builtin_bit_cast(float, __builtin_amdgcn_readlane(__builtin_bit_cast(int, x), i));
}

__device__ __forceinline__ float block_sum(float a, float* red) {      // over the workgroup's waves (at most four)
  a = wave_sum(a);
  const int waves = blockDim.x / kWave;
  if (waves == 1) return a;
  __syncthreads();
  if (threadIdx.x % kWave == 0) red[threadIdx.x / kWave] = a;
  __syncthreads();
  a = red[0];
  for (int w = 1; w < waves; ++w) a += red[w];
  return a;
}

template <int VEC, typename T>
__device__ __forceinline__ void ldv(const T* p, float (&v)[VEC]) {
  if constexpr (VEC == 4) {
    const float4 x = ld4(p);
    v[0] = x.x; v[1] = x.y; v[2] = x.z; v[3] = x.w;
  } else {
    v[0] = ldf(p);
  }
}
template <int VEC, typename T>
__device__ __forceinline__ void stv(T* p, const float (&v)[VEC]) {
  if constexpr (VEC == 4) st4(p, float4{v[0], v[1], v[2], v[3]});
  else stf(p, v[0]);
}

// ------------------------------------------------------------------------------------------------
struct ConvParams {
  const void* in;           // act [T, ld], the C channels start at the pointer
  int64_t ld;
  const float *w, *bias;    // [C, taps] (last column: the current token), [C] or NULL
  void* state;              // act [slots, taps - 1, C]
  const int32_t *cu_q, *ctx_lens, *slots;
  int C, taps, silu;
  void* out;                // act [T, C]; in the attention form the queries, act [T, HD]
  // attention form: channels [queries HD | keys GD | values GDv]
  void *k_cache, *v_cache;
  const int32_t* block_tables;
  int bt_stride, HD, GD, GDv, page;
  float temp_coef;          // queries times 1 + temp_coef * ln(floor((pos + 1) / temp_every) + 1); 0: as they are
  int temp_every;
};

constexpr int kConvTile = 32;
constexpr int kMaxTaps = 8;       // longer filters take the form that reads its taps from memory

template <typename T, int VEC, bool ATT>
__device__ __forceinline__ void conv_emit(const ConvParams& p, int64_t t, int b, int pos, int c, float (&y)[VEC]) {
  if constexpr (!ATT) {
    if (p.silu) {
#pragma unroll
      for (int e = 0; e < VEC; ++e) y[e] = siluf_(y[e]);
    }
    stv<VEC>(static_cast<T*>(p.out) + t * p.C + c, y);
  } else {
    if (c < p.HD) {
      if (p.temp_coef != 0.0f) {
        const float f = 1.0f + p.temp_coef * logf(static_cast<float>((pos + 1) / p.temp_every + 1));
#pragma unroll
        for (int e = 0; e < VEC; ++e) y[e] *= f;
      }
      stv<VEC>(static_cast<T*>(p.out) + t * p.HD + c, y);
    } else {
      const int64_t slot = static_cast<int64_t>(p.block_tables[static_cast<int64_t>(b) * p.bt_stride + pos / p.page]) * p.page + pos % p.page;
      if (c < p.HD + p.GD) stv<VEC>(static_cast<T*>(p.k_cache) + slot * p.GD + (c - p.HD), y);
      else stv<VEC>(static_cast<T*>(p.v_cache) + slot * p.GDv + (c - p.HD - p.GD), y);
    }
  }
}

// grid: (channel blocks, token tiles, sequences). The first tile of a sequence reads the carried inputs and, being their only
// reader, writes the new ones when it is done.
template <typename T, int TAPS, int VEC, bool ATT>
__global__ __launch_bounds__(128) void causal_conv_kernel(ConvParams p) {
  const int b = blockIdx.z;
  const int c = (blockIdx.x * blockDim.x + threadIdx.x) * VEC;
  if (c >= p.C) return;
  const int q0 = p.cu_q[b], n = p.cu_q[b + 1] - q0;
  const int r0 = blockIdx.y * kConvTile;
  if (r0 >= n) return;
  const int ctx = p.ctx_lens[b];
  constexpr int HIST = TAPS > 1 ? TAPS - 1 : 1;
  const T* in = static_cast<const T*>(p.in) + static_cast<int64_t>(q0) * p.ld + c;
  T* state = static_cast<T*>(p.state) + static_cast<int64_t>(p.slots[b]) * (TAPS - 1) * p.C + c;
  float w[TAPS][VEC], hist[HIST][VEC], bias[VEC];
#pragma unroll
  for (int e = 0; e < VEC; ++e) {
    bias[e] = p.bias != nullptr ? p.bias[c + e] : 0.0f;
#pragma unroll
    for (int j = 0; j < TAPS; ++j) w[j][e] = p.w[static_cast<int64_t>(c + e) * TAPS + j];
  }
#pragma unroll
  for (int j = 0; j < TAPS - 1; ++j) {
    const int rr = r0 - (TAPS - 1) + j;            // a tile is longer than the filter: only the first one looks behind row 0
    if (rr >= 0) ldv<VEC>(in + static_cast<int64_t>(rr) * p.ld, hist[j]);
    else if (ctx > 0) ldv<VEC>(state + static_cast<int64_t>(TAPS - 1 + rr) * p.C, hist[j]);
    else {
#pragma unroll
      for (int e = 0; e < VEC; ++e) hist[j][e] = 0.0f;
    }
  }
  const int r1 = min(n, r0 + kConvTile);
  for (int r = r0; r < r1; ++r) {
    float u[VEC], y[VEC];
    ldv<VEC>(in + static_cast<int64_t>(r) * p.ld, u);
#pragma unroll
    for (int e = 0; e < VEC; ++e) {
      y[e] = bias[e];
#pragma unroll
      for (int j = 0; j < TAPS - 1; ++j) y[e] += w[j][e] * hist[j][e];
      y[e] += w[TAPS - 1][e] * u[e];
#pragma unroll
      for (int j = 0; j + 1 < TAPS - 1; ++j) hist[j][e] = hist[j + 1][e];
      if (TAPS > 1) hist[HIST - 1][e] = u[e];
    }
    conv_emit<T, VEC, ATT>(p, q0 + r, b, ctx + r, c, y);
  }
  if (r0 == 0 && TAPS > 1) {
#pragma unroll
    for (int j = 0; j < TAPS - 1; ++j) {
      if (n > kConvTile) ldv<VEC>(in + static_cast<int64_t>(n - (TAPS - 1) + j) * p.ld, hist[j]);   // all of them are rows of this step
      stv<VEC>(state + static_cast<int64_t>(j) * p.C, hist[j]);
    }
  }
}

// Filters of any length: one thread per (token, channel), taps read from the step's rows or the carried inputs. The carried
// inputs are moved by a launch of their own (lv_conv_state_update).
template <typename T, bool ATT>
__global__ __launch_bounds__(128) void causal_conv_long_kernel(ConvParams p) {
  const int b = blockIdx.z;
  const int c = blockIdx.x * blockDim.x + threadIdx.x;
  if (c >= p.C) return;
  const int q0 = p.cu_q[b], n = p.cu_q[b + 1] - q0, ctx = p.ctx_lens[b], taps = p.taps;
  const T* in = static_cast<const T*>(p.in) + static_cast<int64_t>(q0) * p.ld + c;
  const T* state = static_cast<const T*>(p.state) + static_cast<int64_t>(p.slots[b]) * (taps - 1) * p.C + c;
  const int r1 = min(n, (static_cast<int>(blockIdx.y) + 1) * kConvTile);
  for (int r = blockIdx.y * kConvTile; r < r1; ++r) {
    float y[1] = {p.bias != nullptr ? p.bias[c] : 0.0f};
    for (int j = 0; j < taps; ++j) {
      const int rr = r - (taps - 1) + j;
      float u = 0.0f;
      if (rr >= 0) u = ldf(in + static_cast<int64_t>(rr) * p.ld);
      else if (ctx + rr >= 0) u = ldf(state + static_cast<int64_t>(taps - 1 + rr) * p.C);
      y[0] += p.w[static_cast<int64_t>(c) * taps + j] * u;
    }
    conv_emit<T, 1, ATT>(p, q0 + r, b, ctx + r, c, y);
  }
}

template <typename T, bool ATT>
static int conv_dispatch(const ConvParams& p, int B, int max_new, bool vec4, hipStream_t s) {
  const int vec = vec4 ? 4 : 1;
  dim3 grid((p.C / vec + 127) / 128, (max_new + kConvTile - 1) / kConvTile, B), block(128);
  if (vec4) {
    switch (p.taps) {
      case 1: causal_conv_kernel<T, 1, 4, ATT><<<grid, block, 0, s>>>(p); return 0;
      case 2: causal_conv_kernel<T, 2, 4, ATT><<<grid, block, 0, s>>>(p); return 0;
      case 3: causal_conv_kernel<T, 3, 4, ATT><<<grid, block, 0, s>>>(p); return 0;
      case 4: causal_conv_kernel<T, 4, 4, ATT><<<grid, block, 0, s>>>(p); return 0;
      default: break;
    }
  }
  grid.x = (p.C + 127) / 128;
  switch (p.taps) {
    case 1: causal_conv_kernel<T, 1, 1, ATT><<<grid, block, 0, s>>>(p); return 0;
    case 2: causal_conv_kernel<T, 2, 1, ATT><<<grid, block, 0, s>>>(p); return 0;
    case 3: causal_conv_kernel<T, 3, 1, ATT><<<grid, block, 0, s>>>(p); return 0;
    case 4: causal_conv_kernel<T, 4, 1, ATT><<<grid, block, 0, s>>>(p); return 0;
    case 5: causal_conv_kernel<T, 5, 1, ATT><<<grid, block, 0, s>>>(p); return 0;
    case 6: causal_conv_kernel<T, 6, 1, ATT><<<grid, block, 0, s>>>(p); return 0;
    case 7: causal_conv_kernel<T, 7, 1, ATT><<<grid, block, 0, s>>>(p); return 0;
    case 8: causal_conv_kernel<T, 8, 1, ATT><<<grid, block, 0, s>>>(p); return 0;
    default: break;
  }
  causal_conv_long_kernel<T, ATT><<<grid, block, 0, s>>>(p);
  return 1;                       // the carried inputs still have to move
}

// ------------------------------------------------------------------------------------------------
// out [M, T, W] = h + (h' - h) * mu[m], h' the previous token's row of the sequence. The workgroup of a sequence's first new
// token is the only reader of the carried row and replaces it (each thread reads an element before it writes it).
// Few tokens (decoded ones): a workgroup per token. Many, and M at most kShiftMax: below.
template <typename T, int VEC>
__global__ __launch_bounds__(256) void token_shift_kernel(const T* __restrict__ h, const float* __restrict__ mu, T* state,
                                                          T* __restrict__ out, const int32_t* __restrict__ cu_q,
                                                          const int32_t* __restrict__ ctx_lens, const int32_t* __restrict__ slots,
                                                          const int32_t* __restrict__ tok_seq, int64_t Tn, int W, int M) {
  const int64_t t = blockIdx.x;
  const int b = tok_seq[t];
  const int q0 = cu_q[b], q1 = cu_q[b + 1];
  const bool first = t == q0;
  T* srow = state + static_cast<int64_t>(slots[b]) * W;
  const bool carry = ctx_lens[b] > 0;
  for (int i = threadIdx.x * VEC; i < W; i += blockDim.x * VEC) {
    float cur[VEC], prev[VEC];
    ldv<VEC>(h + t * W + i, cur);
    if (!first) ldv<VEC>(h + (t - 1) * W + i, prev);
    else if (carry) ldv<VEC>(srow + i, prev);
    else {
#pragma unroll
      for (int e = 0; e < VEC; ++e) prev[e] = 0.0f;
    }
    for (int m = 0; m < M; ++m) {
      float f[VEC], y[VEC];
      ldv<VEC>(mu + static_cast<int64_t>(m) * W + i, f);
#pragma unroll
      for (int e = 0; e < VEC; ++e) y[e] = cur[e] + (prev[e] - cur[e]) * f[e];
      stv<VEC>(out + (static_cast<int64_t>(m) * Tn + t) * W + i, y);
    }
    if (first) {
      float last[VEC];
      ldv<VEC>(h + static_cast<int64_t>(q1 - 1) * W + i, last);
      stv<VEC>(srow + i, last);
    }
  }
}

constexpr int kShiftMax = 5;
constexpr int kShiftTile = 16;

// Prompts: a thread keeps the weights of its four channels in registers and walks kShiftTile packed tokens, each row read once.
template <typename T>
__global__ __launch_bounds__(256) void token_shift_tile_kernel(const T* __restrict__ h, const float* __restrict__ mu, T* state,
                                                               T* __restrict__ out, const int32_t* __restrict__ cu_q,
                                                               const int32_t* __restrict__ ctx_lens,
                                                               const int32_t* __restrict__ slots,
                                                               const int32_t* __restrict__ tok_seq, int64_t Tn, int W, int M) {
  const int i = (blockIdx.y * blockDim.x + threadIdx.x) * 4;
  if (i >= W) return;
  float f[kShiftMax][4];
#pragma unroll
  for (int m = 0; m < kShiftMax; ++m)
    if (m < M) ldv<4>(mu + static_cast<int64_t>(m) * W + i, f[m]);
  const int64_t t0 = static_cast<int64_t>(blockIdx.x) * kShiftTile, t1 = min(t0 + kShiftTile, Tn);
  float prev[4] = {0.0f, 0.0f, 0.0f, 0.0f};
  if (t0 > 0) ldv<4>(h + (t0 - 1) * W + i, prev);
  for (int64_t t = t0; t < t1; ++t) {
    float cur[4];
    ldv<4>(h + t * W + i, cur);
    const int b = tok_seq[t];
    if (t == cu_q[b]) {
      T* srow = state + static_cast<int64_t>(slots[b]) * W + i;
      if (ctx_lens[b] > 0) ldv<4>(srow, prev);
      else prev[0] = prev[1] = prev[2] = prev[3] = 0.0f;
      float last[4];
      ldv<4>(h + static_cast<int64_t>(cu_q[b + 1] - 1) * W + i, last);
      stv<4>(srow, last);
    }
#pragma unroll
    for (int m = 0; m < kShiftMax; ++m) {
      if (m < M) {
        float y[4];
#pragma unroll
        for (int e = 0; e < 4; ++e) y[e] = cur[e] + (prev[e] - cur[e]) * f[m][e];
        stv<4>(out + (static_cast<int64_t>(m) * Tn + t) * W + i, y);
      }
    }
#pragma unroll
    for (int e = 0; e < 4; ++e) prev[e] = cur[e];
  }
}

// ------------------------------------------------------------------------------------------------
enum ScanKind { kScanStep = LV_MIX_SCAN_STEP, kScanLogGates = LV_MIX_SCAN_LOG_GATES, kScanRowDecay = LV_MIX_SCAN_ROW_DECAY };

struct ScanParams {
  const void *q, *k, *v;           // act rows of stride ldq, ldk, ldv: query/key group h / (H/G) of D, value head h of Dv
  int64_t ldq, ldk, ldv;
  const void *a, *a2;              // act rows of stride lda, see the staging code of each kind
  int64_t lda;
  const float *p0, *p1, *p2;
  float q_scale, cap;
  float *state, *norm_state, *max_state;
  const int32_t *cu_q, *ctx_lens, *slots;
  float *o, *den;
  int H, G, D, Dv;
};

// N consecutive f32 values from LDS, N = 1, 2 or a multiple of 4 (aligned to as many).
template <int N>
__device__ __forceinline__ void lds_rows(const float* p, float (&v)[N]) {
  if constexpr (N % 4 == 0) {
#pragma unroll
    for (int r = 0; r < N; r += 4) {
      const float4 x = *reinterpret_cast<const float4*>(p + r);
      v[r] = x.x; v[r + 1] = x.y; v[r + 2] = x.z; v[r + 3] = x.w;
    }
  } else if constexpr (N == 2) {
    const float2 x = *reinterpret_cast<const float2*>(p);
    v[0] = x.x; v[1] = x.y;
  } else {
    v[0] = p[0];
  }
}

template <int CTRL>
__device__ __forceinline__ float quad_perm(float x) {
  return __builtin_bit_cast(float, __builtin_amdgcn_update_dpp(0, __builtin_bit_cast(int, x), CTRL, 0xf, 0xf, true));
}
// Four lanes hold shares of four columns each; lane rl of the four is left with the sum of column rl.
__device__ __forceinline__ float quad_columns(const float (&p)[4], int rl) {
  const bool odd = rl & 1, high = rl & 2;
  const float a = (odd ? p[1] : p[0]) + quad_perm<0xb1>(odd ? p[0] : p[1]);     // columns 0 | 1 over lanes rl, rl ^ 1
  const float b = (odd ? p[3] : p[2]) + quad_perm<0xb1>(odd ? p[2] : p[3]);     // columns 2 | 3
  return (high ? b : a) + quad_perm<0x4e>(high ? a : b);
}

// NW waves a workgroup on 64 value columns, DR = rows of the state each wave owns (NW * DR >= D; rows beyond D stay zero). A lane
// holds a block of DR / 4 rows by 4 columns: four neighbouring lanes share the columns and divide the wave's rows, so that a
// token costs a lane DR / 4 keys, DR / 4 queries and 4 values from LDS for DR entries (with a lane per column every lane reads
// all DR keys and queries, and the kernel ran at the speed of those reads), and the four lanes' read-outs meet in the ALU.
// A chunk of tokens is fetched into registers one chunk ahead and staged in LDS; every wave then walks the chunk alone (its
// rows of S need nobody else's) and leaves its share of each read-out in LDS; the shares are added when the chunk is done.
//
// Where a head has one decay per token, S is held as F S' with a number F that takes the decays: S' <- S' + (write / F) k v^T,
// o = F S'^T q, two multiply-adds per entry and token instead of a multiply more. Before F would fall below kMinFactor it is
// multiplied into S' and starts again at 1, so nothing but exponents differs from the plain recurrence.
constexpr float kMinFactor = 1.0f / (1 << 30);

template <int KIND, int DR, int NW>
struct ScanShape {
  static constexpr int kDP = NW * DR;
  static constexpr int kChunk = kDP >= 256 ? 8 : 16;
  static constexpr int kSeg = kDP > kWave ? kDP / kWave : 1;         // partial sums of a token's bonus
  static constexpr int kExtra = KIND == kScanStep ? 0 : (KIND == kScanRowDecay ? kChunk * kDP : kChunk * kDP / 16);
  static constexpr size_t kLds = sizeof(float) * (2 * kChunk * kDP + kChunk * kWave + kChunk * NW * kWave + kExtra + 8 * kChunk +
                                                  kChunk * kSeg);
};

template <typename T, int KIND, int DR, int NW>
__global__ __launch_bounds__(NW * 64, DR > 32 ? 2 : (KIND == kScanRowDecay && DR == 32 ? 3 : 4)) void gated_scan_kernel(ScanParams p) {
  extern __shared__ __attribute__((aligned(16))) float sl[];
  using Shape = ScanShape<KIND, DR, NW>;
  constexpr int DP = Shape::kDP, NT = NW * kWave, CH = Shape::kChunk, SEG = Shape::kSeg;
  float* k_lds = sl;                               // [CH][DP]
  float* q_lds = k_lds + CH * DP;                  // [CH][DP]
  float* x_lds = q_lds + CH * DP;                  // [CH][DP] row decays, or [CH][DP / 16] normaliser shares
  float* v_lds = x_lds + Shape::kExtra;            // [CH][64]
  float* part_o = v_lds + CH * kWave;              // [CH][NW][64]
  float* sc_all = part_o + CH * NW * kWave;        // [2][CH][4]: what S' is multiplied by, write / F, F, floor of the normaliser
  float* bon_lds = sc_all + 8 * CH;                // [CH][SEG]
  const int lane = threadIdx.x % kWave, rp = threadIdx.x / kWave;
  constexpr int RL = DR / 4;                       // rows of a lane's block
  const int rl = lane & 3;
  const int col0 = blockIdx.x * kWave + (lane & ~3);
  const int h = blockIdx.y, b = blockIdx.z;
  const int g = h / (p.H / p.G);
  const int q0 = p.cu_q[b], n = p.cu_q[b + 1] - q0;
  if (n <= 0) return;
  const int row0 = rp * DR, own0 = row0 + rl * RL;
  const int64_t head = static_cast<int64_t>(p.slots[b]) * p.H + h;
  float* sbase = p.state + head * p.D * p.Dv;
  const bool carry = p.ctx_lens[b] > 0;
  float s[RL][4];
  const bool whole = (p.Dv & 3) == 0 && col0 + 3 < p.Dv;               // the block's rows are aligned and inside
#pragma unroll
  for (int r = 0; r < RL; ++r)
#pragma unroll
    for (int c = 0; c < 4; ++c) s[r][c] = 0.0f;
  if (carry && whole) {                            // all of a lane's loads in flight at once
#pragma unroll
    for (int r = 0; r < RL; ++r) {
      const float4 x = ld4(sbase + static_cast<int64_t>(min(own0 + r, p.D - 1)) * p.Dv + col0);
      const bool in = own0 + r < p.D;
      s[r][0] = in ? x.x : 0.0f; s[r][1] = in ? x.y : 0.0f; s[r][2] = in ? x.z : 0.0f; s[r][3] = in ? x.w : 0.0f;
    }
  } else if (carry) {
#pragma unroll
    for (int r = 0; r < RL; ++r)
#pragma unroll
      for (int c = 0; c < 4; ++c)
        if (own0 + r < p.D && col0 + c < p.Dv) s[r][c] = sbase[static_cast<int64_t>(own0 + r) * p.Dv + col0 + c];
  }
  // kScanLogGates: the first workgroup of a head keeps the normaliser, a row a thread of its last waves. The running maximum is a
  // copy per workgroup (its place in max_state), so that none waits for another.
  const bool owner = KIND == kScanLogGates && blockIdx.x == 0;
  const int nr = static_cast<int>(threadIdx.x) - (NT - DP);
  const bool nrow = owner && nr >= 0 && nr < p.D;
  float nstate = (nrow && carry) ? p.norm_state[head * p.D + nr] : 0.0f;
  float* mplace = KIND == kScanLogGates ? p.max_state + head * gridDim.x + blockIdx.x : nullptr;
  float m = (KIND == kScanLogGates && carry) ? *mplace : 0.0f;

  float factor = 1.0f, last_factor = 1.0f;         // F: the first wave's running value, and what it ends with

  const T* qp = static_cast<const T*>(p.q) + static_cast<int64_t>(g) * p.D;
  const T* kp = static_cast<const T*>(p.k) + static_cast<int64_t>(g) * p.D;
  const T* vp = static_cast<const T*>(p.v) + static_cast<int64_t>(h) * p.Dv;
  const T* ap = static_cast<const T*>(p.a);
  const int d_own = threadIdx.x % DP;              // DP divides the workgroup: a thread stages one row index of every token
  const bool d_in = d_own < p.D;
  const int tok_own = threadIdx.x / DP;
  const uint32_t koff = static_cast<uint32_t>(tok_own * static_cast<int>(p.ldk) + d_own);
  const uint32_t qoff = static_cast<uint32_t>(tok_own * static_cast<int>(p.ldq) + d_own);
  const uint32_t aoff = static_cast<uint32_t>(tok_own * static_cast<int>(p.lda) + d_own);
  float u_own = 0.0f, w0_own = 0.0f, gate_a = 0.0f, gate_b = 0.0f, skip = 0.0f;
  if (KIND == kScanRowDecay && d_in) {
    w0_own = p.p0[h * p.D + d_own];
    u_own = p.p1[h * p.D + d_own];
  }
  if (KIND == kScanStep) {
    gate_a = p.p0[h];                              // bias of the step size
    gate_b = -expf(p.p1[h]);                       // minus the rate
    skip = p.p2[h];
  }
  if (KIND == kScanLogGates) {
    gate_a = p.p0[h];
    gate_b = p.p1[h];
  }
  constexpr int NKQ = CH * DP / NT, NV = (CH * kWave + NT - 1) / NT;
  static_assert(NT % DP == 0 && CH * DP % NT == 0, "a thread stages one row index of every token");
  float kreg[NKQ], qreg[NKQ], wreg[KIND == kScanRowDecay ? NKQ : 1], vreg[NV], areg = 0.0f, breg = 0.0f;
  auto fetch = [&](int c0) {
    const int cn = min(CH, n - c0);
    const int64_t tb = static_cast<int64_t>(q0) + c0;
#pragma unroll
    for (int it = 0; it < NKQ; ++it) {             // uniform part of the address per step, a thread's own part once
      constexpr int per = NT / DP;
      const int64_t t = tb + it * per;
      const bool in = tok_own + it * per < cn && d_in;
      kreg[it] = in ? ldf(kp + t * p.ldk + koff) : 0.0f;
      qreg[it] = in ? ldf(qp + t * p.ldq + qoff) : 0.0f;
      if (KIND == kScanRowDecay) wreg[it] = in ? ldf(ap + h * p.D + t * p.lda + aoff) : 0.0f;
    }
#pragma unroll
    for (int it = 0; it < NV; ++it) {
      const int x = threadIdx.x + it * NT;
      const int tok = x / kWave, cc = blockIdx.x * kWave + (x % kWave);
      vreg[it] = (tok < cn && cc < p.Dv) ? ldf(vp + (tb + tok) * p.ldv + cc) : 0.0f;
    }
    if (KIND != kScanRowDecay && static_cast<int>(threadIdx.x) < cn) {
      const int64_t t = tb + threadIdx.x;
      areg = ldf(ap + t * p.lda + h);
      if (KIND == kScanLogGates) breg = ldf(static_cast<const T*>(p.a2) + t * p.lda + h);
    }
  };
  // Decays and writes of a chunk of cn tokens, lane = token: the first wave's job, done for the next chunk while the last waves are
  // at the normaliser.
  auto scalars = [&](int cn, float* sc) {
    float dec, write, floor_ = 0.0f;
    if (KIND == kScanStep) {
      write = softplusf_(areg + gate_a);
      dec = expf(gate_b * write);
    } else {
      const float li = p.cap * tanhf((areg + gate_a) / p.cap);
      const float lf = log_sigmoidf_(p.cap * tanhf((breg + gate_b) / p.cap));
      float before = 0.0f, after = 0.0f;         // the running maximum on either side of this lane's token
      for (int i = 0; i < cn; ++i) {
        const float nm = fmaxf(read_lane(lf, i) + m, read_lane(li, i));
        if (lane == i) {
          before = m;
          after = nm;
        }
        m = nm;
      }
      dec = expf(lf + before - after);
      write = expf(li - after);
      floor_ = expf(-after);
    }
    float mul = 1.0f, fac = 1.0f;
    for (int i = 0; i < cn; ++i) {
      const float nf = factor * read_lane(dec, i);
      const bool fold = nf < kMinFactor;
      factor = fold ? 1.0f : nf;
      if (lane == i) {
        mul = fold ? nf : 1.0f;
        fac = factor;
      }
    }
    if (lane < CH) *reinterpret_cast<float4*>(sc + lane * 4) = float4{mul, write / fac, fac, floor_};
  };
  fetch(0);
  if (KIND != kScanRowDecay && rp == 0) scalars(min(CH, n), sc_all);
  int buf = 0;
  for (int c0 = 0; c0 < n; c0 += CH, buf ^= 1) {
    const int cn = min(CH, n - c0);
    const float* sc_lds = sc_all + buf * 4 * CH;
    // every wave is past the previous chunk's use of what is written here: behind the barrier that followed its token loop
#pragma unroll
    for (int it = 0; it < NKQ; ++it) {
      const int x = threadIdx.x + it * NT;
      const float qs = KIND == kScanRowDecay ? qreg[it] : qreg[it] * p.q_scale;
      k_lds[x] = kreg[it];
      q_lds[x] = qs;
      if (KIND == kScanRowDecay) {
        x_lds[x] = d_in ? expf(-expf(wreg[it] + w0_own)) : 1.0f;
        float bon = kreg[it] * qreg[it] * u_own;   // summed over the rows of a token below
        constexpr int width = DP < kWave ? DP : kWave;
#pragma unroll
        for (int off = width / 2; off > 0; off >>= 1) bon += __shfl_xor(bon, off, kWave);
        if (lane % width == 0) bon_lds[(x / DP) * SEG + (x % DP) / kWave] = bon;
      }
    }
#pragma unroll
    for (int it = 0; it < NV; ++it)
      if (threadIdx.x + it * NT < CH * kWave) v_lds[threadIdx.x + it * NT] = vreg[it];
    __syncthreads();
    if (c0 + CH < n) fetch(c0 + CH);
    for (int i = 0; i < cn; ++i) {
      float4 vv = *reinterpret_cast<const float4*>(v_lds + i * kWave + (lane & ~3));
      if (KIND != kScanRowDecay) {
        const float2 mw = *reinterpret_cast<const float2*>(sc_lds + i * 4);
        if (__builtin_amdgcn_readfirstlane(__builtin_bit_cast(int, mw.x)) != __builtin_bit_cast(int, 1.0f)) {
#pragma unroll
          for (int r = 0; r < RL; ++r)
#pragma unroll
            for (int c = 0; c < 4; ++c) s[r][c] *= mw.x;
        }
        vv.x *= mw.y; vv.y *= mw.y; vv.z *= mw.y; vv.w *= mw.y;
      }
      float kr[RL], qr[RL], wr[KIND == kScanRowDecay ? RL : 1];
      lds_rows<RL>(k_lds + i * DP + own0, kr);
      lds_rows<RL>(q_lds + i * DP + own0, qr);
      if constexpr (KIND == kScanRowDecay) lds_rows<RL>(x_lds + i * DP + own0, wr);
      const float v4[4] = {vv.x, vv.y, vv.z, vv.w};
      float po[4] = {0.0f, 0.0f, 0.0f, 0.0f};
#pragma unroll
      for (int r = 0; r < RL; ++r) {
#pragma unroll
        for (int c = 0; c < 4; ++c) {
          if constexpr (KIND == kScanRowDecay) {   // read before this token decays and writes
            po[c] += s[r][c] * qr[r];
            s[r][c] = wr[r] * s[r][c] + kr[r] * v4[c];
          } else {
            s[r][c] += kr[r] * v4[c];
            po[c] += s[r][c] * qr[r];
          }
        }
      }
      part_o[(i * NW + rp) * kWave + lane] = quad_columns(po, rl);
    }
    if (owner && nr >= 0)
      for (int i = 0; i < cn; ++i) {
        const float2 mw = *reinterpret_cast<const float2*>(sc_lds + i * 4);
        nstate = nstate * mw.x + mw.y * k_lds[i * DP + nr];
        const float share = row16_sum(nstate * q_lds[i * DP + nr]);
        if ((lane & 15) == 0) x_lds[i * (DP / 16) + nr / 16] = share;
      }
    if (KIND != kScanRowDecay && rp == 0 && c0 + CH < n) scalars(min(CH, n - c0 - CH), sc_all + (buf ^ 1) * 4 * CH);
    __syncthreads();
    for (int x = threadIdx.x; x < cn * kWave; x += NT) {
      const int tok = x / kWave, ln = x % kWave, cc = blockIdx.x * kWave + ln;
      const float* po = part_o + tok * NW * kWave + ln;
      float sum = 0.0f;
#pragma unroll
      for (int w = 0; w < NW; w += 2) sum += po[w * kWave] + po[(w + 1) * kWave];
      if (KIND != kScanRowDecay) sum *= sc_lds[tok * 4 + 2];
      if (KIND == kScanStep) sum += skip * v_lds[x];
      if (KIND == kScanRowDecay) {
        float bon = bon_lds[tok * SEG];
#pragma unroll
        for (int e = 1; e < SEG; ++e) bon += bon_lds[tok * SEG + e];
        sum += bon * v_lds[x];
      }
      if (cc < p.Dv) p.o[((static_cast<int64_t>(q0) + c0 + tok) * p.H + h) * p.Dv + cc] = sum;
    }
    if (owner && threadIdx.x < cn) {
      const float* sh = x_lds + threadIdx.x * (DP / 16);
      float nq = 0.0f;
      for (int e = 0; e < DP / 16; ++e) nq += sh[e];
      p.den[(static_cast<int64_t>(q0) + c0 + threadIdx.x) * p.H + h] =
          fmaxf(fabsf(nq) * sc_lds[threadIdx.x * 4 + 2], sc_lds[threadIdx.x * 4 + 3]) + 1e-6f;
    }
    if (KIND != kScanRowDecay && c0 + CH >= n) last_factor = sc_lds[(cn - 1) * 4 + 2];
    __syncthreads();                               // the next chunk overwrites the values and scalars read above
  }
#pragma unroll
  for (int r = 0; r < RL; ++r) {
    float* dst = sbase + static_cast<int64_t>(own0 + r) * p.Dv + col0;
    if (own0 + r >= p.D) continue;
    if (whole) {
      st4(dst, float4{s[r][0] * last_factor, s[r][1] * last_factor, s[r][2] * last_factor, s[r][3] * last_factor});
    } else {
#pragma unroll
      for (int c = 0; c < 4; ++c)
        if (col0 + c < p.Dv) dst[c] = s[r][c] * last_factor;
    }
  }
  if (nrow) p.norm_state[head * p.D + nr] = nstate * last_factor;
  if (KIND == kScanLogGates && threadIdx.x == 0) *mplace = m;
}

template <typename T, int KIND, int DR, int NW>
static void scan_launch(const ScanParams& p, dim3 grid, hipStream_t s) {
  static_assert(ScanShape<KIND, DR, NW>::kLds <= 64 * 1024, "LDS of a workgroup");
  gated_scan_kernel<T, KIND, DR, NW><<<grid, dim3(NW * kWave), ScanShape<KIND, DR, NW>::kLds, s>>>(p);
}

template <typename T, int KIND>
static void scan_dispatch(const ScanParams& p, int B, hipStream_t s) {
  dim3 grid((p.Dv + kWave - 1) / kWave, p.H, B);
  // fewer than four workgroups a compute unit: eight waves each, so that a SIMD still holds four
  const bool eight = static_cast<int64_t>(grid.x) * grid.y * grid.z < 4 * 256 && p.D > 16 && p.D <= 128;
  if (eight) {
    if (p.D <= 32) scan_launch<T, KIND, 4, 8>(p, grid, s);
    else if (p.D <= 64) scan_launch<T, KIND, 8, 8>(p, grid, s);
    else scan_launch<T, KIND, 16, 8>(p, grid, s);
  } else {
    if (p.D <= 32) scan_launch<T, KIND, 8, 4>(p, grid, s);
    else if (p.D <= 64) scan_launch<T, KIND, 16, 4>(p, grid, s);
    else if (p.D <= 128) scan_launch<T, KIND, 32, 4>(p, grid, s);
    else scan_launch<T, KIND, 64, 4>(p, grid, s);
  }
}

template <typename T>
static void scan_kind(const ScanParams& p, int kind, int B, hipStream_t s) {
  if (kind == kScanStep) scan_dispatch<T, kScanStep>(p, B, s);
  else if (kind == kScanLogGates) scan_dispatch<T, kScanLogGates>(p, B, s);
  else scan_dispatch<T, kScanRowDecay>(p, B, s);
}

// ------------------------------------------------------------------------------------------------
// Parts of at most 4 * 64 * kPartRegs entries, aligned: a wave per (token, part), the gated values in registers.
constexpr int kPartRegs = 4;
template <typename T>
__global__ __launch_bounds__(256) void part_gate_norm_kernel(const float* __restrict__ o, const T* __restrict__ z, int64_t ldz,
                                                             const float* __restrict__ w, T* __restrict__ out, int64_t items, int N,
                                                             int groups, float eps) {
  const int64_t item = static_cast<int64_t>(blockIdx.x) * (blockDim.x / kWave) + threadIdx.x / kWave;
  if (item >= items) return;
  const int64_t t = item / groups;
  const int gs = N / groups, c0 = static_cast<int>(item - t * groups) * gs, i0 = 4 * (threadIdx.x % kWave);
  float y[kPartRegs][4], ss = 0.0f;
#pragma unroll
  for (int x = 0; x < kPartRegs; ++x) {
    const int i = i0 + x * 4 * kWave;
    if (i < gs) {
      float g[4];
      ldv<4>(o + t * N + c0 + i, y[x]);
      ldv<4>(z + t * ldz + c0 + i, g);
#pragma unroll
      for (int e = 0; e < 4; ++e) {
        y[x][e] *= siluf_(g[e]);
        ss += y[x][e] * y[x][e];
      }
    }
  }
  const float inv = 1.0f / sqrtf(wave_sum(ss) / static_cast<float>(gs) + eps);
#pragma unroll
  for (int x = 0; x < kPartRegs; ++x) {
    const int i = i0 + x * 4 * kWave;
    if (i < gs) {
      float ww[4];
      ldv<4>(w + c0 + i, ww);
#pragma unroll
      for (int e = 0; e < 4; ++e) y[x][e] *= inv * ww[e];
      stv<4>(out + t * N + c0 + i, y[x]);
    }
  }
}

// One workgroup (64 or 256 threads) per (token, part of the row): y = o * silu(z), y / rms(part) * w.
template <typename T, int VEC>
__global__ __launch_bounds__(256) void grouped_gate_norm_kernel(const float* __restrict__ o, const T* __restrict__ z, int64_t ldz,
                                                                const float* __restrict__ w, T* __restrict__ out, int N, int groups,
                                                                float eps) {
  __shared__ float red[4];
  const int64_t t = blockIdx.x / groups;
  const int gs = N / groups, c0 = static_cast<int>(blockIdx.x % groups) * gs;
  const float* orow = o + t * N + c0;
  const T* zrow = z + t * ldz + c0;
  float ss = 0.0f;
  for (int i = threadIdx.x * VEC; i < gs; i += blockDim.x * VEC) {
    float a[VEC], g[VEC];
    ldv<VEC>(orow + i, a);
    ldv<VEC>(zrow + i, g);
#pragma unroll
    for (int e = 0; e < VEC; ++e) {
      const float y = a[e] * siluf_(g[e]);
      ss += y * y;
    }
  }
  const float inv = 1.0f / sqrtf(block_sum(ss, red) / static_cast<float>(gs) + eps);
  for (int i = threadIdx.x * VEC; i < gs; i += blockDim.x * VEC) {
    float a[VEC], g[VEC], ww[VEC], y[VEC];
    ldv<VEC>(orow + i, a);
    ldv<VEC>(zrow + i, g);
    ldv<VEC>(w + c0 + i, ww);
#pragma unroll
    for (int e = 0; e < VEC; ++e) y[e] = a[e] * siluf_(g[e]) * inv * ww[e];
    stv<VEC>(out + t * N + c0 + i, y);
  }
}

// ------------------------------------------------------------------------------------------------
template <typename T, int VEC>
__global__ __launch_bounds__(256) void residual_pair_norm_kernel(float* __restrict__ x, const T* __restrict__ y1,
                                                                 const float* __restrict__ pw1, const T* __restrict__ y2,
                                                                 const float* __restrict__ pw2, float pair_scale, float pair_eps,
                                                                 const float* __restrict__ w, float w_offset,
                                                                 T* __restrict__ out, int W, float eps) {
  extern __shared__ __attribute__((aligned(16))) float row[];          // [W] the updated row
  __shared__ float red[4];
  const int64_t t = blockIdx.x;
  const int first = threadIdx.x * VEC, stride = blockDim.x * VEC;
  float s1 = 0.0f, s2 = 0.0f;
  for (int i = first; i < W; i += stride) {
    float a[VEC], b[VEC];
    ldv<VEC>(y1 + t * W + i, a);
    ldv<VEC>(y2 + t * W + i, b);
#pragma unroll
    for (int e = 0; e < VEC; ++e) {
      s1 += a[e] * a[e];
      s2 += b[e] * b[e];
    }
  }
  const float f1 = pair_scale / sqrtf(block_sum(s1, red) / static_cast<float>(W) + pair_eps);
  const float f2 = pair_scale / sqrtf(block_sum(s2, red) / static_cast<float>(W) + pair_eps);
  float ss = 0.0f;
  for (int i = first; i < W; i += stride) {
    float a[VEC], b[VEC], g1[VEC], g2[VEC], xv[VEC];
    ldv<VEC>(y1 + t * W + i, a);
    ldv<VEC>(y2 + t * W + i, b);
    ldv<VEC>(pw1 + i, g1);
    ldv<VEC>(pw2 + i, g2);
    ldv<VEC>(x + t * W + i, xv);
#pragma unroll
    for (int e = 0; e < VEC; ++e) {
      xv[e] += a[e] * f1 * g1[e] + b[e] * f2 * g2[e];
      ss += xv[e] * xv[e];
    }
    stv<VEC>(x + t * W + i, xv);
    stv<VEC>(row + i, xv);
  }
  if (out == nullptr) return;
  const float inv = 1.0f / sqrtf(block_sum(ss, red) / static_cast<float>(W) + eps);
  for (int i = first; i < W; i += stride) {                    // each thread reads back what it wrote itself
    float xv[VEC], g[VEC], y[VEC];
    ldv<VEC>(row + i, xv);
    ldv<VEC>(w + i, g);
#pragma unroll
    for (int e = 0; e < VEC; ++e) y[e] = xv[e] * inv * (w_offset + g[e]);
    stv<VEC>(out + t * W + i, y);
  }
}

// ------------------------------------------------------------------------------------------------
struct EmbedParams {
  const int64_t* ids;
  const void *table, *pair_table, *pos_table;    // act [vocab, W], [buckets + 1, W] or NULL, [max_pos, W] or NULL
  float scale;
  int64_t mul_prev, mul_cur;
  int buckets, vocab, max_pos, W;
  int32_t* prev_state;                           // [slots] each sequence's last token
  const int32_t *cu_q, *ctx_lens, *slots, *tok_seq;
  const float *w_embed, *w_next;
  float w_offset, eps;
  float* x;
  void* out;
};

template <typename T, int VEC>
__global__ __launch_bounds__(256) void embed_norm_kernel(EmbedParams p) {
  extern __shared__ __attribute__((aligned(16))) float row[];          // [W]
  __shared__ float red[4];
  __shared__ int64_t prev_sh;
  const int64_t t = blockIdx.x;
  const int b = p.tok_seq[t], W = p.W;
  const int q0 = p.cu_q[b], r = static_cast<int>(t) - q0, ctx = p.ctx_lens[b];
  auto token = [&](int64_t at) {                                       // a row of the table whatever the caller passed
    const int64_t id = p.ids[at];
    return id < 0 ? 0 : (id >= p.vocab ? static_cast<int64_t>(p.vocab) - 1 : id);
  };
  if (threadIdx.x == 0 && p.prev_state != nullptr) {
    // the workgroup of a sequence's first new token is the only one that reads the carried token, and replaces it
    int64_t prev = -1;
    if (r > 0) prev = token(t - 1);
    else {
      int32_t* place = p.prev_state + p.slots[b];
      if (ctx > 0) prev = *place;
      *place = static_cast<int32_t>(token(p.cu_q[b + 1] - 1));
    }
    prev_sh = prev;
  }
  __syncthreads();
  const int64_t tok = token(t);
  const T* e_row = static_cast<const T*>(p.table) + tok * W;
  const T* b_row = nullptr;
  if (p.pair_table != nullptr) {
    const int64_t idx = prev_sh < 0 ? p.buckets : (prev_sh * p.mul_prev + tok * p.mul_cur) % p.buckets;
    b_row = static_cast<const T*>(p.pair_table) + idx * W;
  }
  const T* p_row = p.pos_table != nullptr ? static_cast<const T*>(p.pos_table) + static_cast<int64_t>(min(ctx + r, p.max_pos - 1)) * W : nullptr;
  float ss = 0.0f;
  for (int i = threadIdx.x * VEC; i < W; i += blockDim.x * VEC) {
    float v[VEC], a[VEC];
    ldv<VEC>(e_row + i, v);
#pragma unroll
    for (int e = 0; e < VEC; ++e) v[e] *= p.scale;
    if (b_row != nullptr) {
      ldv<VEC>(b_row + i, a);
#pragma unroll
      for (int e = 0; e < VEC; ++e) v[e] += a[e];
    }
    if (p_row != nullptr) {
      ldv<VEC>(p_row + i, a);
#pragma unroll
      for (int e = 0; e < VEC; ++e) v[e] += a[e];
    }
#pragma unroll
    for (int e = 0; e < VEC; ++e) ss += v[e] * v[e];
    stv<VEC>(row + i, v);
  }
  const float inv = 1.0f / sqrtf(block_sum(ss, red) / static_cast<float>(W) + p.eps);
  float s2 = 0.0f;
  for (int i = threadIdx.x * VEC; i < W; i += blockDim.x * VEC) {      // each thread reads back what it wrote itself
    float v[VEC], g[VEC];
    ldv<VEC>(row + i, v);
    ldv<VEC>(p.w_embed + i, g);
#pragma unroll
    for (int e = 0; e < VEC; ++e) {
      v[e] *= inv * (p.w_offset + g[e]);
      s2 += v[e] * v[e];
    }
    stv<VEC>(row + i, v);
    stv<VEC>(p.x + t * W + i, v);
  }
  const float inv2 = 1.0f / sqrtf(block_sum(s2, red) / static_cast<float>(W) + p.eps);
  for (int i = threadIdx.x * VEC; i < W; i += blockDim.x * VEC) {
    float v[VEC], g[VEC];
    ldv<VEC>(row + i, v);
    ldv<VEC>(p.w_next + i, g);
#pragma unroll
    for (int e = 0; e < VEC; ++e) v[e] *= inv2 * (p.w_offset + g[e]);
    stv<VEC>(static_cast<T*>(p.out) + t * W + i, v);
  }
}

// ------------------------------------------------------------------------------------------------
template <typename T, int VEC>
__global__ __launch_bounds__(256) void unary_act_kernel(const T* __restrict__ in, T* __restrict__ out, int64_t n, int act) {
  const int64_t i = (static_cast<int64_t>(blockIdx.x) * blockDim.x + threadIdx.x) * VEC;
  if (i >= n) return;
  float v[VEC];
  ldv<VEC>(in + i, v);
#pragma unroll
  for (int e = 0; e < VEC; ++e) v[e] = mix_act(v[e], act);
  stv<VEC>(out + i, v);
}

static bool aligned16(const void* q) { return (reinterpret_cast<uintptr_t>(q) & 15) == 0; }
static bool aligned8(const void* q) { return (reinterpret_cast<uintptr_t>(q) & 7) == 0; }

template <bool ATT>
static int conv_entry(const char* what, ConvParams& p, int B, int max_new, int dtype, void* stream) {
  // four channels a thread: every row it touches starts on its access size
  const bool f32 = dtype == LV_MIX_F32;
  auto ok = [&](const void* q) { return f32 ? aligned16(q) : aligned8(q); };
  bool vec4 = p.C % 4 == 0 && p.ld % 4 == 0 && ok(p.in) && ok(p.out) && (p.taps == 1 || ok(p.state));
  if (ATT) vec4 = vec4 && p.HD % 4 == 0 && p.GD % 4 == 0 && p.GDv % 4 == 0 && ok(p.k_cache) && ok(p.v_cache);
  int more;
  if (dtype == LV_MIX_BF16) more = conv_dispatch<bf16_t, ATT>(p, B, max_new, vec4, as_stream(stream));
  else if (f32) more = conv_dispatch<float, ATT>(p, B, max_new, vec4, as_stream(stream));
  else return fail(-1, "%s: dtype %d", what, dtype);
  const int rc = launched(what);
  if (rc != 0 || more == 0) return rc;
  return lv_conv_state_update(p.in, p.ld, p.state, p.cu_q, p.ctx_lens, p.slots, B, p.C, p.taps, dtype, stream);
}

}  // namespace lvmix

using namespace lvmix;

extern "C" {

int lv_causal_conv(const void* in, int64_t ld, const void* w, const void* bias, void* state, const int32_t* cu_q,
                   const int32_t* ctx_lens, const int32_t* slots, void* out, int B, int max_new_tokens, int C, int taps, int silu,
                   int dtype, void* stream) {
  if (B == 0 || max_new_tokens == 0) return 0;
  if (!in || !w || (!state && taps > 1) || !cu_q || !ctx_lens || !slots || !out) return fail(-1, "lv_causal_conv: null pointer");
  if (B < 0 || max_new_tokens < 0 || C <= 0 || taps < 1 || ld < C) return fail(-1, "lv_causal_conv: bad sizes");
  ConvParams p{};
  p.in = in; p.ld = ld; p.w = static_cast<const float*>(w); p.bias = static_cast<const float*>(bias); p.state = state;
  p.cu_q = cu_q; p.ctx_lens = ctx_lens; p.slots = slots; p.C = C; p.taps = taps; p.silu = silu; p.out = out;
  return conv_entry<false>("lv_causal_conv", p, B, max_new_tokens, dtype, stream);
}

int lv_conv_qkv_store(const void* in, int64_t ld, const void* w, void* state, void* q_out, void* k_cache, void* v_cache,
                      const int32_t* cu_q, const int32_t* ctx_lens, const int32_t* slots, const int32_t* block_tables,
                      int bt_stride, int B, int max_new_tokens, int H, int G, int D, int Dv, int taps, float temp_coef,
                      int temp_every, int page, int dtype, void* stream) {
  if (B == 0 || max_new_tokens == 0) return 0;
  if (!in || !w || (!state && taps > 1) || !q_out || !k_cache || !v_cache || !cu_q || !ctx_lens || !slots || !block_tables)
    return fail(-1, "lv_conv_qkv_store: null pointer");
  const int64_t C = static_cast<int64_t>(H) * D + static_cast<int64_t>(G) * (D + Dv);
  if (B < 0 || max_new_tokens < 0 || H <= 0 || G <= 0 || H % G != 0 || D <= 0 || Dv <= 0 || taps < 1 || ld < C || page <= 0 ||
      bt_stride <= 0 || (temp_coef != 0.0f && temp_every < 1))
    return fail(-1, "lv_conv_qkv_store: bad sizes");
  ConvParams p{};
  p.in = in; p.ld = ld; p.w = static_cast<const float*>(w); p.state = state; p.cu_q = cu_q; p.ctx_lens = ctx_lens;
  p.slots = slots; p.C = static_cast<int>(C); p.taps = taps; p.out = q_out; p.k_cache = k_cache; p.v_cache = v_cache;
  p.block_tables = block_tables; p.bt_stride = bt_stride; p.HD = H * D; p.GD = G * D; p.GDv = G * Dv; p.page = page;
  p.temp_coef = temp_coef; p.temp_every = temp_every > 0 ? temp_every : 1;
  return conv_entry<true>("lv_conv_qkv_store", p, B, max_new_tokens, dtype, stream);
}

int lv_token_shift(const void* h, const void* mu, void* state, void* out, const int32_t* cu_q, const int32_t* ctx_lens,
                   const int32_t* slots, const int32_t* tok_seq, int64_t T, int W, int M, int dtype, void* stream) {
  if (T == 0) return 0;
  if (!h || !mu || !state || !out || !cu_q || !ctx_lens || !slots || !tok_seq || T < 0 || W <= 0 || M <= 0)
    return fail(-1, "lv_token_shift: bad arguments");
  dim3 grid(static_cast<unsigned>(T)), block(256);
  const bool vec4 = W % 4 == 0 && aligned16(h) && aligned16(mu) && aligned16(state) && aligned16(out);
  const bool tiled = vec4 && M <= kShiftMax && T >= 128 * kShiftTile;
  if (tiled) {
    dim3 tgrid(static_cast<unsigned>((T + kShiftTile - 1) / kShiftTile), (W / 4 + 255) / 256);
    if (dtype == LV_MIX_BF16)
      token_shift_tile_kernel<bf16_t><<<tgrid, block, 0, as_stream(stream)>>>(
          static_cast<const bf16_t*>(h), static_cast<const float*>(mu), static_cast<bf16_t*>(state), static_cast<bf16_t*>(out), cu_q,
          ctx_lens, slots, tok_seq, T, W, M);
    else if (dtype == LV_MIX_F32)
      token_shift_tile_kernel<float><<<tgrid, block, 0, as_stream(stream)>>>(
          static_cast<const float*>(h), static_cast<const float*>(mu), static_cast<float*>(state), static_cast<float*>(out), cu_q,
          ctx_lens, slots, tok_seq, T, W, M);
    else
      return fail(-1, "lv_token_shift: dtype %d", dtype);
    return launched("lv_token_shift");
  }
#define LVMIX_SHIFT(TT, VV)                                                                                               \
  token_shift_kernel<TT, VV><<<grid, block, 0, as_stream(stream)>>>(static_cast<const TT*>(h), static_cast<const float*>(mu), \
                                                                   static_cast<TT*>(state), static_cast<TT*>(out), cu_q,  \
                                                                   ctx_lens, slots, tok_seq, T, W, M)
  if (dtype == LV_MIX_BF16) {
    if (vec4) LVMIX_SHIFT(bf16_t, 4); else LVMIX_SHIFT(bf16_t, 1);
  } else if (dtype == LV_MIX_F32) {
    if (vec4) LVMIX_SHIFT(float, 4); else LVMIX_SHIFT(float, 1);
  } else {
    return fail(-1, "lv_token_shift: dtype %d", dtype);
  }
#undef LVMIX_SHIFT
  return launched("lv_token_shift");
}

int lv_gated_scan(int kind, const void* q, int64_t ldq, const void* k, int64_t ldk, const void* v, int64_t ldv, const void* a,
                  const void* a2, int64_t lda, const void* p0, const void* p1, const void* p2, float q_scale, float cap,
                  void* state, void* norm_state, void* max_state, const int32_t* cu_q, const int32_t* ctx_lens,
                  const int32_t* slots, void* o, void* den, int B, int H, int G, int D, int Dv, int dtype, void* stream) {
  if (B == 0) return 0;
  if (!q || !k || !v || !a || !p0 || !p1 || !state || !cu_q || !ctx_lens || !slots || !o)
    return fail(-1, "lv_gated_scan: null pointer");
  if (kind != LV_MIX_SCAN_STEP && kind != LV_MIX_SCAN_LOG_GATES && kind != LV_MIX_SCAN_ROW_DECAY)
    return fail(-1, "lv_gated_scan: kind %d", kind);
  if (kind == LV_MIX_SCAN_STEP && !p2) return fail(-1, "lv_gated_scan: step sizes without the skip factors");
  if (kind == LV_MIX_SCAN_LOG_GATES && (!a2 || !norm_state || !max_state || !den || !(cap > 0.0f)))
    return fail(-1, "lv_gated_scan: log gates need both gates, their cap, the normaliser's state and its output");
  if (B < 0 || H <= 0 || G <= 0 || H % G != 0 || D <= 0 || Dv <= 0 || ldq < static_cast<int64_t>(G) * D ||
      ldk < static_cast<int64_t>(G) * D || ldv < static_cast<int64_t>(H) * Dv ||
      lda < (kind == LV_MIX_SCAN_ROW_DECAY ? static_cast<int64_t>(H) * D : H) || (kind == LV_MIX_SCAN_ROW_DECAY && G != H))
    return fail(-1, "lv_gated_scan: bad sizes");
  if (D > 256) return fail(-2, "lv_gated_scan: key size %d above 256", D);
  ScanParams p{q, k, v, ldq, ldk, ldv, a, a2, lda, static_cast<const float*>(p0), static_cast<const float*>(p1),
               static_cast<const float*>(p2), q_scale, cap, static_cast<float*>(state), static_cast<float*>(norm_state),
               static_cast<float*>(max_state), cu_q, ctx_lens, slots, static_cast<float*>(o), static_cast<float*>(den), H, G, D, Dv};
  if (dtype == LV_MIX_BF16) scan_kind<bf16_t>(p, kind, B, as_stream(stream));
  else if (dtype == LV_MIX_F32) scan_kind<float>(p, kind, B, as_stream(stream));
  else return fail(-1, "lv_gated_scan: dtype %d", dtype);
  return launched("lv_gated_scan");
}

int lv_grouped_gate_norm(const void* o, const void* z, int64_t ldz, const void* w, void* out, int64_t T, int N, int groups,
                         float eps, int dtype, void* stream) {
  if (T == 0) return 0;
  if (!o || !z || !w || !out || T < 0 || N <= 0 || groups <= 0 || N % groups != 0 || ldz < N)
    return fail(-1, "lv_grouped_gate_norm: bad arguments");
  const int gs = N / groups;
  const bool vec4 = gs % 4 == 0 && ldz % 4 == 0 && aligned16(o) && aligned8(z) && aligned16(w) && aligned16(out) &&
                    (dtype == LV_MIX_BF16 || aligned16(z));
  if (vec4 && gs <= 4 * kWave * kPartRegs && (dtype == LV_MIX_BF16 || dtype == LV_MIX_F32)) {
    const int64_t items = T * groups;
    dim3 pgrid(static_cast<unsigned>((items + 3) / 4)), pblock(256);
    if (dtype == LV_MIX_BF16)
      part_gate_norm_kernel<bf16_t><<<pgrid, pblock, 0, as_stream(stream)>>>(
          static_cast<const float*>(o), static_cast<const bf16_t*>(z), ldz, static_cast<const float*>(w), static_cast<bf16_t*>(out),
          items, N, groups, eps);
    else
      part_gate_norm_kernel<float><<<pgrid, pblock, 0, as_stream(stream)>>>(
          static_cast<const float*>(o), static_cast<const float*>(z), ldz, static_cast<const float*>(w), static_cast<float*>(out),
          items, N, groups, eps);
    return launched("lv_grouped_gate_norm");
  }
  dim3 grid(static_cast<unsigned>(T * groups)), block(gs > 512 ? 256 : 64);
#define LVMIX_GGN(TT, VV)                                                                                                   \
  grouped_gate_norm_kernel<TT, VV><<<grid, block, 0, as_stream(stream)>>>(static_cast<const float*>(o), static_cast<const TT*>(z), ldz, \
                                                                         static_cast<const float*>(w), static_cast<TT*>(out), N,  \
                                                                         groups, eps)
  if (dtype == LV_MIX_BF16) {
    if (vec4) LVMIX_GGN(bf16_t, 4); else LVMIX_GGN(bf16_t, 1);
  } else if (dtype == LV_MIX_F32) {
    if (vec4) LVMIX_GGN(float, 4); else LVMIX_GGN(float, 1);
  } else {
    return fail(-1, "lv_grouped_gate_norm: dtype %d", dtype);
  }
#undef LVMIX_GGN
  return launched("lv_grouped_gate_norm");
}

int lv_residual_pair_norm(void* x, const void* y1, const void* post_w1, const void* y2, const void* post_w2, float pair_scale,
                          float pair_eps, const void* w, float w_offset, void* out, int64_t T, int W, float eps, int dtype,
                          void* stream) {
  if (T == 0) return 0;
  if (!x || !y1 || !y2 || !post_w1 || !post_w2 || T < 0 || W <= 0 || (out != nullptr && w == nullptr))
    return fail(-1, "lv_residual_pair_norm: bad arguments");
  const size_t shm = static_cast<size_t>(W) * sizeof(float);
  if (shm > 60 * 1024) return fail(-2, "lv_residual_pair_norm: width %d too large", W);
  dim3 grid(static_cast<unsigned>(T)), block(256);
  const bool vec4 = W % 4 == 0 && aligned16(x) && aligned16(y1) && aligned16(y2) && aligned16(post_w1) && aligned16(post_w2) &&
                    aligned16(w) && aligned16(out);
#define LVMIX_RPN(TT, VV)                                                                                                    \
  residual_pair_norm_kernel<TT, VV><<<grid, block, shm, as_stream(stream)>>>(                                               \
      static_cast<float*>(x), static_cast<const TT*>(y1), static_cast<const float*>(post_w1), static_cast<const TT*>(y2),    \
      static_cast<const float*>(post_w2), pair_scale, pair_eps, static_cast<const float*>(w), w_offset, static_cast<TT*>(out), W, eps)
  if (dtype == LV_MIX_BF16) {
    if (vec4) LVMIX_RPN(bf16_t, 4); else LVMIX_RPN(bf16_t, 1);
  } else if (dtype == LV_MIX_F32) {
    if (vec4) LVMIX_RPN(float, 4); else LVMIX_RPN(float, 1);
  } else {
    return fail(-1, "lv_residual_pair_norm: dtype %d", dtype);
  }
#undef LVMIX_RPN
  return launched("lv_residual_pair_norm");
}

int lv_embed_norm(const void* ids, const void* table, int vocab, float scale, const void* pair_table, int buckets,
                  int64_t mul_prev, int64_t mul_cur, void* prev_state, const void* pos_table, int max_pos, const void* w_embed,
                  const void* w_next, float w_offset, float eps, const int32_t* cu_q, const int32_t* ctx_lens,
                  const int32_t* slots, const int32_t* tok_seq, void* x, void* out, int64_t T, int W, int dtype, void* stream) {
  if (T == 0) return 0;
  if (!ids || !table || !w_embed || !w_next || !cu_q || !ctx_lens || !slots || !tok_seq || !x || !out)
    return fail(-1, "lv_embed_norm: null pointer");
  if (T < 0 || W <= 0 || vocab <= 0 || (pair_table != nullptr && (buckets <= 0 || mul_prev < 0 || mul_cur < 0 || !prev_state)) ||
      (pos_table != nullptr && max_pos <= 0))
    return fail(-1, "lv_embed_norm: bad sizes");
  const size_t shm = static_cast<size_t>(W) * sizeof(float);
  if (shm > 60 * 1024) return fail(-2, "lv_embed_norm: width %d too large", W);
  EmbedParams p{static_cast<const int64_t*>(ids), table, pair_table, pos_table, scale, mul_prev, mul_cur, buckets, vocab, max_pos, W,
                static_cast<int32_t*>(prev_state), cu_q, ctx_lens, slots, tok_seq, static_cast<const float*>(w_embed),
                static_cast<const float*>(w_next), w_offset, eps, static_cast<float*>(x), out};
  dim3 grid(static_cast<unsigned>(T)), block(256);
  const bool vec4 = W % 4 == 0 && aligned16(table) && aligned16(pair_table) && aligned16(pos_table) && aligned16(w_embed) &&
                    aligned16(w_next) && aligned16(x) && aligned16(out);
  if (dtype == LV_MIX_BF16) {
    if (vec4) embed_norm_kernel<bf16_t, 4><<<grid, block, shm, as_stream(stream)>>>(p);
    else embed_norm_kernel<bf16_t, 1><<<grid, block, shm, as_stream(stream)>>>(p);
  } else if (dtype == LV_MIX_F32) {
    if (vec4) embed_norm_kernel<float, 4><<<grid, block, shm, as_stream(stream)>>>(p);
    else embed_norm_kernel<float, 1><<<grid, block, shm, as_stream(stream)>>>(p);
  } else {
    return fail(-1, "lv_embed_norm: dtype %d", dtype);
  }
  return launched("lv_embed_norm");
}

int lv_unary_act(const void* in, void* out, int64_t n, int act, int dtype, void* stream) {
  if (n == 0) return 0;
  if (!in || !out || n < 0 || act < 0 || act > LV_MIX_ACT_MAX) return fail(-1, "lv_unary_act: bad arguments");
  const bool vec4 = n % 4 == 0 && aligned16(in) && aligned16(out);
  dim3 grid(static_cast<unsigned>((n / (vec4 ? 4 : 1) + 255) / 256)), block(256);
  if (dtype == LV_MIX_BF16) {
    if (vec4) unary_act_kernel<bf16_t, 4><<<grid, block, 0, as_stream(stream)>>>(static_cast<const bf16_t*>(in), static_cast<bf16_t*>(out), n, act);
    else unary_act_kernel<bf16_t, 1><<<grid, block, 0, as_stream(stream)>>>(static_cast<const bf16_t*>(in), static_cast<bf16_t*>(out), n, act);
  } else if (dtype == LV_MIX_F32) {
    if (vec4) unary_act_kernel<float, 4><<<grid, block, 0, as_stream(stream)>>>(static_cast<const float*>(in), static_cast<float*>(out), n, act);
    else unary_act_kernel<float, 1><<<grid, block, 0, as_stream(stream)>>>(static_cast<const float*>(in), static_cast<float*>(out), n, act);
  } else {
    return fail(-1, "lv_unary_act: dtype %d", dtype);
  }
  return launched("lv_unary_act");
}

}  // extern "C"
