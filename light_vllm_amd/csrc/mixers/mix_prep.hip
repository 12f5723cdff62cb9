// Steps ahead of the paged attention kernels and of the matrix products, memory-bound, one launch each.
//
//   head_norm_store_kernel    per-head RMS norm of the queries; keys go to the cache as projected, with 1 / rms of each head beside
//                             them, so that one cached row is key (the attention kernel multiplies its score) and value.
//   latent_store_kernel       RMS norm of the key/value latent and rotation of the shared positional key part into the cache row,
//                             rotation of every query's positional part into the row the attention kernel reads.
//   scaled_embedding_kernel   token rows times a constant as the f32 residual, on request the rows and the split residual as well.
//   residual_split_kernel     residual update; the residual as two bf16 numbers side by side, operands of a matrix product.
#include "mix_common.h"

namespace lvmix {

struct HeadNormParams {
  const void* proj;
  int64_t ld;
  int off_q, off_k;
  const float* q_w;
  void *q_out, *cache;
  float* key_scale;
  const int32_t *cu_q, *ctx_lens, *tok_seq, *block_tables;
  int bt_stride, H, G, D, page;
  float eps;
};

// One workgroup per token. VEC: four entries per lane, a head of D <= 256 entries in P lanes (the power of two at or above D / 4),
// 64 / P heads a wave at once, every value read once. Otherwise a wave per head, entries in turns of 64.
template <typename T, bool VEC>
__global__ __launch_bounds__(256) void head_norm_store_kernel(HeadNormParams p, int P) {
  const int64_t t = blockIdx.x;
  const int wave = threadIdx.x / kWave, lane = threadIdx.x % kWave;
  const int b = p.tok_seq[t], D = p.D;
  const int pos = p.ctx_lens[b] + static_cast<int>(t) - p.cu_q[b];
  const int64_t slot = static_cast<int64_t>(p.block_tables[static_cast<int64_t>(b) * p.bt_stride + pos / p.page]) * p.page + pos % p.page;
  const T* row = static_cast<const T*>(p.proj) + t * p.ld;
  T* q_out = static_cast<T*>(p.q_out) + t * p.H * D;
  T* k_out = static_cast<T*>(p.cache) + slot * p.G * D;
  float* ks_out = p.key_scale + slot * p.G;
  const int heads = p.H + p.G;                                   // query heads, then key heads
  if constexpr (VEC) {
    const int per_wave = kWave / P, sub = lane / P, j = 4 * (lane % P);
    const float4 w = j < D ? ld4(p.q_w + j) : float4{0.0f, 0.0f, 0.0f, 0.0f};
    for (int hd0 = 0; hd0 < heads; hd0 += 4 * per_wave) {        // the same trip count for every lane: the sums below shuffle
      const int hd = hd0 + wave * per_wave + sub;
      const bool live = hd < heads && j < D, is_q = hd < p.H;
      const T* head = row + (is_q ? p.off_q + hd * D : p.off_k + (hd - p.H) * D);
      const float4 v = live ? ld4(head + j) : float4{0.0f, 0.0f, 0.0f, 0.0f};
      float ss = (v.x * v.x + v.y * v.y) + (v.z * v.z + v.w * v.w);
      for (int o = P >> 1; o > 0; o >>= 1) ss += __shfl_xor(ss, o, kWave);
      const float f = 1.0f / sqrtf(ss / static_cast<float>(D) + p.eps);
      if (!live) continue;
      if (is_q) {
        st4(q_out + hd * D + j, float4{v.x * f * w.x, v.y * f * w.y, v.z * f * w.z, v.w * f * w.w});
      } else {
        st4(k_out + (hd - p.H) * D + j, v);
        if (j == 0) ks_out[hd - p.H] = f;
      }
    }
  } else {
    for (int hd = wave; hd < heads; hd += 4) {
      const bool is_q = hd < p.H;
      const T* head = row + (is_q ? p.off_q + hd * D : p.off_k + (hd - p.H) * D);
      float ss = 0.0f;
      for (int j = lane; j < D; j += kWave) {
        const float v = ldf(head + j);
        ss += v * v;
      }
      const float f = 1.0f / sqrtf(wave_sum(ss) / static_cast<float>(D) + p.eps);
      for (int j = lane; j < D; j += kWave) {
        if (is_q) stf(q_out + hd * D + j, ldf(head + j) * f * p.q_w[j]);
        else k_out[(hd - p.H) * D + j] = head[j];
      }
      if (!is_q && lane == 0) ks_out[hd - p.H] = f;
    }
  }
}

// ------------------------------------------------------------------------------------------------
struct LatentStoreParams {
  const void* proj;
  int64_t ld;
  int off_q, off_kv;
  const float *kv_w, *inv_freq;
  float magnitude;
  void *q_out, *cache;
  const int32_t *cu_q, *ctx_lens, *tok_seq, *block_tables;
  int bt_stride, H, Dn, Dr, R, rot_dims, interleaved, page;
  float eps;
};

// One workgroup per token; VEC: four entries per access (rotated pairs lie side by side).
template <typename T, bool VEC>
__global__ __launch_bounds__(256) void latent_store_kernel(LatentStoreParams p) {
  extern __shared__ __attribute__((aligned(16))) float cs[];     // [rot_dims/2] cosines | [rot_dims/2] sines
  __shared__ float red[4];
  const int64_t t = blockIdx.x;
  const int b = p.tok_seq[t], R = p.R, Dr = p.Dr, half = p.rot_dims / 2;
  const int pos = p.ctx_lens[b] + static_cast<int>(t) - p.cu_q[b];
  const int64_t slot = static_cast<int64_t>(p.block_tables[static_cast<int64_t>(b) * p.bt_stride + pos / p.page]) * p.page + pos % p.page;
  const T* row = static_cast<const T*>(p.proj) + t * p.ld;
  for (int i = threadIdx.x; i < half; i += blockDim.x) {
    float s, c;
    sincosf(static_cast<float>(pos) * p.inv_freq[i], &s, &c);
    cs[i] = p.magnitude * c;
    cs[half + i] = p.magnitude * s;
  }
  const T* lat = row + p.off_kv;
  float ss = 0.0f;
  if constexpr (VEC) {
    for (int i = threadIdx.x * 4; i < R; i += blockDim.x * 4) {
      const float4 v = ld4(lat + i);
      ss += (v.x * v.x + v.y * v.y) + (v.z * v.z + v.w * v.w);
    }
  } else {
    for (int i = threadIdx.x; i < R; i += blockDim.x) {
      const float v = ldf(lat + i);
      ss += v * v;
    }
  }
  ss = wave_sum(ss);
  if (threadIdx.x % kWave == 0) red[threadIdx.x / kWave] = ss;
  __syncthreads();
  const float inv = 1.0f / sqrtf(((red[0] + red[1]) + (red[2] + red[3])) / static_cast<float>(R) + p.eps);
  T* crow = static_cast<T*>(p.cache) + slot * (R + Dr);
  T* q_out = static_cast<T*>(p.q_out) + t * p.H * (R + Dr);
  if constexpr (VEC) {
    for (int i = threadIdx.x * 4; i < R; i += blockDim.x * 4) {
      const float4 v = ld4(lat + i), w = ld4(p.kv_w + i);
      st4(crow + i, float4{v.x * inv * w.x, v.y * inv * w.y, v.z * inv * w.z, v.w * inv * w.w});
    }
    const int per = Dr / 4;                                      // the query heads' positional parts, then the key's
    for (int x = threadIdx.x; x < (p.H + 1) * per; x += blockDim.x) {
      const int hd = x / per, j = 4 * (x - hd * per);
      const T* src = hd < p.H ? row + p.off_q + hd * (p.Dn + Dr) + p.Dn : lat + R;
      float4 v = ld4(src + j);
      if (j < p.rot_dims) {
        const int i = j >> 1;
        const float c0 = cs[i], s0 = cs[half + i], c1 = cs[i + 1], s1 = cs[half + i + 1];
        v = float4{v.x * c0 - v.y * s0, v.y * c0 + v.x * s0, v.z * c1 - v.w * s1, v.w * c1 + v.z * s1};
      }
      st4((hd < p.H ? q_out + hd * (R + Dr) + R : crow + R) + j, v);
    }
  } else {
    for (int i = threadIdx.x; i < R; i += blockDim.x) stf(crow + i, ldf(lat + i) * inv * p.kv_w[i]);
    for (int x = threadIdx.x; x < (p.H + 1) * Dr; x += blockDim.x) {
      const int hd = x / Dr, j = x - hd * Dr;
      const T* src = hd < p.H ? row + p.off_q + hd * (p.Dn + Dr) + p.Dn : lat + R;
      float v = ldf(src + j);
      if (j < p.rot_dims) {
        int i, other;
        bool lead;
        if (p.interleaved) { i = j >> 1; lead = (j & 1) == 0; other = j ^ 1; }
        else { lead = j < half; i = lead ? j : j - half; other = lead ? j + half : j - half; }
        const float u = ldf(src + other);
        v = lead ? v * cs[i] - u * cs[half + i] : v * cs[i] + u * cs[half + i];
      }
      stf((hd < p.H ? q_out + hd * (R + Dr) + R : crow + R) + j, v);
    }
  }
}

// ------------------------------------------------------------------------------------------------
// x = high + low + (what 16 bits of mantissa do not hold)
__device__ __forceinline__ void split_store(bf16_t* high, bf16_t* low, float x) {
  bf16_t hi;
  stf(&hi, x);
  *high = hi;
  stf(low, x - ldf(&hi));
}
__device__ __forceinline__ void split_store4(bf16_t* high, bf16_t* low, float4 x) {
  bf16_t h[4];
  stf(&h[0], x.x); stf(&h[1], x.y); stf(&h[2], x.z); stf(&h[3], x.w);
  const float4 hf = float4{ldf(&h[0]), ldf(&h[1]), ldf(&h[2]), ldf(&h[3])};
  st4(high, hf);                                   // exact: already bf16 numbers
  st4(low, float4{x.x - hf.x, x.y - hf.y, x.z - hf.z, x.w - hf.w});
}

template <typename T, int VEC>
__global__ __launch_bounds__(256) void scaled_embedding_kernel(const int64_t* __restrict__ ids, const T* __restrict__ table, int vocab,
                                                               float scale, float* __restrict__ x, T* __restrict__ rows,
                                                               bf16_t* __restrict__ split, int W) {
  const int64_t t = blockIdx.x;
  int64_t id = ids[t];
  id = id < 0 ? 0 : (id >= vocab ? static_cast<int64_t>(vocab) - 1 : id);      // a row of the table whatever the caller passed
  const T* src = table + id * W;
  for (int i = (blockIdx.y * blockDim.x + threadIdx.x) * VEC; i < W; i += gridDim.y * blockDim.x * VEC) {
    if constexpr (VEC == 4) {
      const float4 e = ld4(src + i);
      const float4 v = float4{e.x * scale, e.y * scale, e.z * scale, e.w * scale};
      st4(x + t * W + i, v);
      if (rows != nullptr) st4(rows + t * W + i, e);
      if (split != nullptr) split_store4(split + t * 2 * W + i, split + t * 2 * W + W + i, v);
    } else {
      const float e = ldf(src + i);
      x[t * W + i] = e * scale;
      if (rows != nullptr) stf(rows + t * W + i, e);
      if (split != nullptr) split_store(split + t * 2 * W + i, split + t * 2 * W + W + i, e * scale);
    }
  }
}

template <int VEC>
__global__ __launch_bounds__(256) void residual_split_kernel(float* __restrict__ x, const bf16_t* __restrict__ y,
                                                             bf16_t* __restrict__ out, int W) {
  const int64_t t = blockIdx.x;
  for (int i = (blockIdx.y * blockDim.x + threadIdx.x) * VEC; i < W; i += gridDim.y * blockDim.x * VEC) {
    if constexpr (VEC == 4) {
      float4 v = ld4(x + t * W + i);
      if (y != nullptr) {
        const float4 a = ld4(y + t * W + i);
        v.x += a.x; v.y += a.y; v.z += a.z; v.w += a.w;
        st4(x + t * W + i, v);
      }
      split_store4(out + t * 2 * W + i, out + t * 2 * W + W + i, v);
    } else {
      float v = x[t * W + i];
      if (y != nullptr) {
        v += ldf(y + t * W + i);
        x[t * W + i] = v;
      }
      split_store(out + t * 2 * W + i, out + t * 2 * W + W + i, v);
    }
  }
}

static bool aligned16(const void* q) { return (reinterpret_cast<uintptr_t>(q) & 15) == 0; }

}  // namespace lvmix

using namespace lvmix;

extern "C" {

int lv_head_norm_store(const void* proj, int64_t ld, int off_q, int off_k, const void* q_w, void* q_out, void* cache, void* key_scale,
                       const int32_t* cu_q, const int32_t* ctx_lens, const int32_t* tok_seq, const int32_t* block_tables, int bt_stride,
                       int64_t T, int H, int G, int D, int page, float eps, int dtype, void* stream) {
  if (T == 0) return 0;
  if (!proj || !q_w || !q_out || !cache || !key_scale || !cu_q || !ctx_lens || !tok_seq || !block_tables)
    return fail(-1, "lv_head_norm_store: null pointer");
  if (T < 0 || H <= 0 || G <= 0 || H % G != 0 || D <= 0 || page <= 0 || bt_stride <= 0 || off_q < 0 || off_k < 0 ||
      off_q + static_cast<int64_t>(H) * D > ld || off_k + static_cast<int64_t>(G) * D > ld)
    return fail(-1, "lv_head_norm_store: bad sizes");
  if (dtype != LV_MIX_BF16 && dtype != LV_MIX_F32) return fail(-1, "lv_head_norm_store: dtype %d", dtype);
  HeadNormParams p{proj, ld, off_q, off_k, static_cast<const float*>(q_w), q_out, cache, static_cast<float*>(key_scale), cu_q, ctx_lens,
                   tok_seq, block_tables, bt_stride, H, G, D, page, eps};
  dim3 grid(static_cast<unsigned>(T)), block(256);
  const bool vec4 = D % 4 == 0 && D <= 4 * kWave && ld % 4 == 0 && off_q % 4 == 0 && off_k % 4 == 0 && aligned16(proj) &&
                    aligned16(q_w) && aligned16(q_out) && aligned16(cache);
  int P = 1;
  while (4 * P < D && P < kWave) P <<= 1;          // lanes that hold one head
  hipStream_t st = as_stream(stream);
  if (dtype == LV_MIX_BF16) {
    if (vec4) head_norm_store_kernel<bf16_t, true><<<grid, block, 0, st>>>(p, P);
    else head_norm_store_kernel<bf16_t, false><<<grid, block, 0, st>>>(p, P);
  } else {
    if (vec4) head_norm_store_kernel<float, true><<<grid, block, 0, st>>>(p, P);
    else head_norm_store_kernel<float, false><<<grid, block, 0, st>>>(p, P);
  }
  return launched("lv_head_norm_store");
}

int lv_latent_store(const void* proj, int64_t ld, int off_q, int off_kv, const void* kv_w, const void* inv_freq, float magnitude,
                    void* q_out, void* cache, const int32_t* cu_q, const int32_t* ctx_lens, const int32_t* tok_seq,
                    const int32_t* block_tables, int bt_stride, int64_t T, int H, int Dn, int Dr, int R, int rot_dims, int interleaved,
                    int page, float eps, int dtype, void* stream) {
  if (T == 0) return 0;
  if (!proj || !kv_w || !q_out || !cache || !cu_q || !ctx_lens || !tok_seq || !block_tables)
    return fail(-1, "lv_latent_store: null pointer");
  if (T < 0 || H <= 0 || Dn < 0 || Dr < 0 || R <= 0 || rot_dims < 0 || rot_dims > Dr || rot_dims % 2 != 0 || page <= 0 ||
      bt_stride <= 0 || off_q < 0 || off_kv < 0 || off_q + static_cast<int64_t>(H) * (Dn + Dr) > ld || off_kv + R + Dr > ld ||
      (rot_dims > 0 && !inv_freq))
    return fail(-1, "lv_latent_store: bad sizes");
  if (dtype != LV_MIX_BF16 && dtype != LV_MIX_F32) return fail(-1, "lv_latent_store: dtype %d", dtype);
  const size_t shm = sizeof(float) * static_cast<size_t>(rot_dims > 0 ? rot_dims : 4);
  if (shm > 60 * 1024) return fail(-2, "lv_latent_store: %d rotated entries", rot_dims);
  LatentStoreParams p{proj, ld, off_q, off_kv, static_cast<const float*>(kv_w), static_cast<const float*>(inv_freq), magnitude, q_out,
                      cache, cu_q, ctx_lens, tok_seq, block_tables, bt_stride, H, Dn, Dr, R, rot_dims, interleaved != 0, page, eps};
  dim3 grid(static_cast<unsigned>(T)), block(256);
  const bool vec4 = (interleaved != 0 || rot_dims == 0) && R % 4 == 0 && Dr % 4 == 0 && Dn % 4 == 0 && rot_dims % 4 == 0 && ld % 4 == 0 &&
                    off_q % 4 == 0 && off_kv % 4 == 0 && aligned16(proj) && aligned16(kv_w) && aligned16(q_out) && aligned16(cache);
  hipStream_t st = as_stream(stream);
  if (dtype == LV_MIX_BF16) {
    if (vec4) latent_store_kernel<bf16_t, true><<<grid, block, shm, st>>>(p);
    else latent_store_kernel<bf16_t, false><<<grid, block, shm, st>>>(p);
  } else {
    if (vec4) latent_store_kernel<float, true><<<grid, block, shm, st>>>(p);
    else latent_store_kernel<float, false><<<grid, block, shm, st>>>(p);
  }
  return launched("lv_latent_store");
}

int lv_scaled_embedding(const void* ids, const void* table, int vocab, float scale, void* x, void* rows, void* split, int64_t T, int W,
                        int dtype, void* stream) {
  if (T == 0) return 0;
  if (!ids || !table || !x || T < 0 || W <= 0 || vocab <= 0) return fail(-1, "lv_scaled_embedding: bad arguments");
  if (dtype != LV_MIX_BF16 && dtype != LV_MIX_F32) return fail(-1, "lv_scaled_embedding: dtype %d", dtype);
  const bool vec4 = W % 4 == 0 && aligned16(table) && aligned16(x) && aligned16(rows) && aligned16(split);
  const int parts = (W / (vec4 ? 4 : 1) + 255) / 256;
  dim3 grid(static_cast<unsigned>(T), T < 256 ? parts : 1), block(256);
#define LVMIX_EMB(TT, VV)                                                                                                       \
  scaled_embedding_kernel<TT, VV><<<grid, block, 0, as_stream(stream)>>>(static_cast<const int64_t*>(ids), static_cast<const TT*>(table), \
                                                                        vocab, scale, static_cast<float*>(x), static_cast<TT*>(rows), \
                                                                        static_cast<bf16_t*>(split), W)
  if (dtype == LV_MIX_BF16) {
    if (vec4) LVMIX_EMB(bf16_t, 4); else LVMIX_EMB(bf16_t, 1);
  } else {
    if (vec4) LVMIX_EMB(float, 4); else LVMIX_EMB(float, 1);
  }
#undef LVMIX_EMB
  return launched("lv_scaled_embedding");
}

int lv_residual_split(void* x, const void* y, void* out, int64_t T, int W, void* stream) {
  if (T == 0) return 0;
  if (!x || !out || T < 0 || W <= 0) return fail(-1, "lv_residual_split: bad arguments");
  const bool vec4 = W % 4 == 0 && aligned16(x) && aligned16(y) && aligned16(out);
  const int parts = (W / (vec4 ? 4 : 1) + 255) / 256;
  dim3 grid(static_cast<unsigned>(T), T < 256 ? parts : 1), block(256);
  if (vec4)
    residual_split_kernel<4><<<grid, block, 0, as_stream(stream)>>>(static_cast<float*>(x), static_cast<const bf16_t*>(y),
                                                                    static_cast<bf16_t*>(out), W);
  else
    residual_split_kernel<1><<<grid, block, 0, as_stream(stream)>>>(static_cast<float*>(x), static_cast<const bf16_t*>(y),
                                                                    static_cast<bf16_t*>(out), W);
  return launched("lv_residual_split");
}

}  // extern "C"
