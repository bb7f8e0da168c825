// Attention over a shared low-rank latent kept in pages: every cached token is one row
// [c (kv_rank) | k_r (rot_dim)] that all heads read, as key (all of it) and as value (c).
// Queries arrive already carried into that space, q' = [U_k^T q_n | rot(q_r)], and the
// result leaves as sum_t p_t c_t per head, for the value up-projection behind it.
//
// Kernels: the preparation of a step's rows (norms of the two latents, rotation of the
// shared key part, the write into the pages), the rotation of the queries' rotated part in
// place, both of these in one kernel where queries and latent come out of one product, and
// attention (with, where a layer has one, a sink per head in the softmax's denominator).  (Carrying queries into the latent's space and results out of it
// are plain products over weights folded at load.)
// Scores, softmax, rotation angles, norms: float32.  The rotation pairs dimension 2i with
// 2i+1 and turns them by position * freq[i]; cosine and sine are computed here, at the
// position, so there is no table and no longest position.
#include "common.h"

typedef __attribute__((ext_vector_type(4))) float f32x4_l;
typedef __attribute__((ext_vector_type(4))) __bf16 bf16x4_l;
__device__ __forceinline__ f32x4_l load4_l(const float* p) { return *(const f32x4_l*)p; }
__device__ __forceinline__ f32x4_l load4_l(const bf16_t* p) {
  const bf16x4_l v = *(const bf16x4_l*)p;
  return f32x4_l{(float)v[0], (float)v[1], (float)v[2], (float)v[3]};
}

__device__ __forceinline__ void rotate_pair(float u, float v, int pos, float freq, float* ou,
                                            float* ov) {
  float sn, cs;
  sincosf((float)pos * freq, &sn, &cs);
  *ou = u * cs - v * sn;
  *ov = v * cs + u * sn;
}

// ---------------------------------------------------------------- preparation
// proj row: [q latent (q_rank) | kv latent (kv_rank) | shared key part (rot_dim)], float32.
// cq = q latent / rms * q_norm -> out (the up-projection's input);
// c = kv latent / rms * kv_norm and the rotated key part -> the token's row in the pages.
template <typename TO, typename TC>
__global__ __launch_bounds__(256) void latent_prepare_kernel(
    const float* __restrict__ proj, const float* __restrict__ q_norm,
    const float* __restrict__ kv_norm, const float* __restrict__ freqs, TO* __restrict__ cq,
    TC* __restrict__ pages, const int* __restrict__ positions,
    const int* __restrict__ entry_of_token, const int* __restrict__ table, int table_width,
    int page_size, int q_rank, int kv_rank, int rot_dim, int rot_dims, float eps) {
  __shared__ float scratch[16];
  const int t = blockIdx.x;
  const int ld = q_rank + kv_rank + rot_dim, dl = kv_rank + rot_dim;
  const float* row = proj + (int64_t)t * ld;
  float sq = 0.f, sc = 0.f;
  for (int i = threadIdx.x; i < q_rank; i += blockDim.x) sq += row[i] * row[i];
  for (int i = threadIdx.x; i < kv_rank; i += blockDim.x) sc += row[q_rank + i] * row[q_rank + i];
  const float rq = 1.0f / sqrtf(block_sum(sq, scratch) / (float)q_rank + eps);
  const float rc = 1.0f / sqrtf(block_sum(sc, scratch) / (float)kv_rank + eps);
  TO* o = cq + (int64_t)t * q_rank;
  for (int i = threadIdx.x; i < q_rank; i += blockDim.x) o[i] = from_f32<TO>(row[i] * rq * q_norm[i]);
  const int pos = positions[t];
  const int page = table[(int64_t)entry_of_token[t] * table_width + pos / page_size];
  if (page < 0) return;     // an idle lane of a fixed-size batch: nothing to keep
  TC* dst = pages + ((int64_t)page * page_size + pos % page_size) * dl;
  for (int i = threadIdx.x; i < kv_rank; i += blockDim.x)
    dst[i] = from_f32<TC>(row[q_rank + i] * rc * kv_norm[i]);
  const float* kr = row + q_rank + kv_rank;
  for (int i = threadIdx.x; i < rot_dim / 2 + rot_dim % 2; i += blockDim.x) {
    if (2 * i + 1 < rot_dims) {
      float u, v;
      rotate_pair(kr[2 * i], kr[2 * i + 1], pos, freqs[i], &u, &v);
      dst[kv_rank + 2 * i] = from_f32<TC>(u);
      dst[kv_rank + 2 * i + 1] = from_f32<TC>(v);
    } else {
      dst[kv_rank + 2 * i] = from_f32<TC>(kr[2 * i]);
      if (2 * i + 1 < rot_dim) dst[kv_rank + 2 * i + 1] = from_f32<TC>(kr[2 * i + 1]);
    }
  }
}

extern "C" int ts_latent_prepare(const float* proj, const float* q_norm, const float* kv_norm,
                                 const float* freqs, void* cq, int out_type, void* pages,
                                 int cache_type, const int* positions,
                                 const int* entry_of_token, const int* table, int table_width,
                                 int page_size, int num_tokens, int q_rank, int kv_rank,
                                 int rot_dim, int rot_dims, float eps, hipStream_t stream) {
  if (num_tokens <= 0) return 0;
  if (q_rank <= 0 || kv_rank <= 0 || rot_dim < 0 || rot_dims % 2 || rot_dims > rot_dim ||
      page_size <= 0 || table_width <= 0)
    TS_FAIL("latent_prepare: bad sizes q_rank=%d kv_rank=%d rot_dim=%d rot_dims=%d", q_rank,
            kv_rank, rot_dim, rot_dims);
  TS_DISPATCH_TYPE(out_type, TO, TS_DISPATCH_TYPE(cache_type, TC,
      hipLaunchKernelGGL((latent_prepare_kernel<TO, TC>), dim3(num_tokens), dim3(256), 0, stream,
                         proj, q_norm, kv_norm, freqs, (TO*)cq, (TC*)pages, positions,
                         entry_of_token, table, table_width, page_size, q_rank, kv_rank, rot_dim,
                         rot_dims, eps)));
  TS_CHECK_LAUNCH("latent_prepare");
  return 0;
}

// ---------------------------------------------------------------- rotation in place
// x [T, heads, width]: the pairs (offset + 2i, offset + 2i + 1), i < dims / 2, of every
// head's vector are turned by positions[t] * freqs[i].
template <typename T>
__global__ __launch_bounds__(256) void rotate_interleaved_kernel(
    T* __restrict__ x, const int* __restrict__ positions, const float* __restrict__ freqs,
    int64_t total, int heads, int width, int offset, int half) {
  const int64_t idx = (int64_t)blockIdx.x * blockDim.x + threadIdx.x;
  if (idx >= total) return;
  const int i = (int)(idx % half);
  const int64_t th = idx / half;                      // token * heads + head
  T* v = x + th * width + offset + 2 * i;
  float a, b;
  rotate_pair(to_f32(v[0]), to_f32(v[1]), positions[th / heads], freqs[i], &a, &b);
  v[0] = from_f32<T>(a);
  v[1] = from_f32<T>(b);
}

extern "C" int ts_rotate_interleaved(void* x, int type, const int* positions, const float* freqs,
                                     int num_tokens, int heads, int width, int offset, int dims,
                                     hipStream_t stream) {
  if (num_tokens <= 0 || dims == 0) return 0;
  if (heads <= 0 || dims % 2 || offset < 0 || offset + dims > width)
    TS_FAIL("rotate_interleaved: bad sizes heads=%d width=%d offset=%d dims=%d", heads, width,
            offset, dims);
  const int64_t total = (int64_t)num_tokens * heads * (dims / 2);
  TS_DISPATCH_TYPE(type, T,
                   hipLaunchKernelGGL(rotate_interleaved_kernel<T>,
                                      dim3((unsigned)((total + 255) / 256)), dim3(256), 0, stream,
                                      (T*)x, positions, freqs, total, heads, width, offset,
                                      dims / 2));
  TS_CHECK_LAUNCH("rotate_interleaved");
  return 0;
}

// ---------------------------------------------------------------- rows of one product
// x [T, ld] float32: the queries, heads x (kv_rank + rot_dim), then (`own`) the token's
// latent (kv_rank) and shared key part (rot_dim).  The queries' rotated parts are turned in
// place; the latent over its root mean square times kv_norm and the turned key part go to
// the token's row of the pages.  One workgroup a token, which works out the position's
// cosines and sines once.
constexpr int kMaxRotPairs = 512;
template <typename TC>
__global__ __launch_bounds__(256) void latent_rows_kernel(
    float* __restrict__ x, const float* __restrict__ kv_norm, const float* __restrict__ freqs,
    TC* __restrict__ pages, const int* __restrict__ positions,
    const int* __restrict__ entry_of_token, const int* __restrict__ table, int table_width,
    int page_size, int ld, int heads, int own, int kv_rank, int rot_dim, int half, float eps) {
  __shared__ float scratch[16], cos_s[kMaxRotPairs], sin_s[kMaxRotPairs];
  const int t = blockIdx.x, dl = kv_rank + rot_dim;
  float* row = x + (int64_t)t * ld;
  const float* kv = row + heads * dl;
  const int pos = positions[t];
  for (int i = threadIdx.x; i < half; i += blockDim.x)
    sincosf((float)pos * freqs[i], &sin_s[i], &cos_s[i]);
  float rc = 0.f;
  if (own) {
    float ss = 0.f;
    for (int i = threadIdx.x; i < kv_rank; i += blockDim.x) ss += kv[i] * kv[i];
    rc = 1.0f / sqrtf(block_sum(ss, scratch) / (float)kv_rank + eps);
  }
  __syncthreads();
  for (int idx = threadIdx.x; idx < heads * half; idx += blockDim.x) {
    const int h = idx / half, i = idx % half;
    float* v = row + h * dl + kv_rank + 2 * i;
    const float a = v[0], b = v[1];
    v[0] = a * cos_s[i] - b * sin_s[i];
    v[1] = b * cos_s[i] + a * sin_s[i];
  }
  if (!own) return;
  const int page = table[(int64_t)entry_of_token[t] * table_width + pos / page_size];
  if (page < 0) return;     // an idle lane of a fixed-size batch: nothing to keep
  TC* dst = pages + ((int64_t)page * page_size + pos % page_size) * dl;
  for (int i = threadIdx.x; i < dl; i += blockDim.x) {
    float v;
    if (i < kv_rank) {
      v = kv[i] * rc * kv_norm[i];
    } else {
      const int d = i - kv_rank;
      v = kv[i];
      if (d < 2 * half) {
        const float o = kv[kv_rank + (d ^ 1)];
        v = d & 1 ? v * cos_s[d / 2] + o * sin_s[d / 2] : v * cos_s[d / 2] - o * sin_s[d / 2];
      }
    }
    dst[i] = from_f32<TC>(v);
  }
}

extern "C" int ts_latent_rows(float* x, const float* kv_norm, const float* freqs, void* pages,
                              int cache_type, const int* positions, const int* entry_of_token,
                              const int* table, int table_width, int page_size, int num_tokens,
                              int ld, int heads, int own, int kv_rank, int rot_dim, int rot_dims,
                              float eps, hipStream_t stream) {
  if (num_tokens <= 0) return 0;
  const int dl = kv_rank + rot_dim;
  if (heads <= 0 || kv_rank <= 0 || rot_dim < 0 || rot_dims < 0 || rot_dims % 2 ||
      rot_dims > rot_dim || rot_dims / 2 > kMaxRotPairs || page_size <= 0 || table_width <= 0)
    TS_FAIL("latent_rows: bad sizes heads=%d kv_rank=%d rot_dim=%d rot_dims=%d (at most %d turned)",
            heads, kv_rank, rot_dim, rot_dims, 2 * kMaxRotPairs);
  if (ld != heads * dl + (own ? dl : 0)) TS_FAIL("latent_rows: rows of %d", ld);
  if (own && !kv_norm) TS_FAIL("latent_rows: no norm weight");
  TS_DISPATCH_TYPE(cache_type, TC,
      hipLaunchKernelGGL(latent_rows_kernel<TC>, dim3(num_tokens), dim3(256), 0, stream, x,
                         kv_norm, freqs, (TC*)pages, positions, entry_of_token, table,
                         table_width, page_size, ld, heads, own, kv_rank, rot_dim, rot_dims / 2,
                         eps));
  TS_CHECK_LAUNCH("latent_rows");
  return 0;
}

// A head's sink in units of the softmax's weights relative to `m`; cut off where the output
// has long become zero, so nothing overflows.
__device__ __forceinline__ float sink_weight(float sink, float m) {
  return expf(fminf(sink - m, 69.f));
}

// ---------------------------------------------------------------- attention
// One wavefront per (token, head), four heads of a token to a workgroup (they read the same
// rows).  Keys are cut into tiles of 64 starting at the first visible key, so the partition
// and with it the rounding depends only on the token's position and the window.  In a
// tile, lane j scores key j (a dot product over the whole row); then the lanes turn to the
// columns of c and add the tile's weighted rows, key by key in order.
constexpr int kMaxLatent = 2048;              // kv_rank + rot_dim
constexpr int kLatentWaves = 4;
constexpr int kMaxRankPerLane = 16;           // kv_rank <= 1024

template <typename TC, typename TO>
__global__ __launch_bounds__(kLatentWaves* kWave) void latent_attention_kernel(
    const float* __restrict__ qa, const TC* __restrict__ pages, TO* __restrict__ out,
    const int* __restrict__ positions, const int* __restrict__ entry_of_token,
    const int* __restrict__ table, int table_width, int page_size, int heads, int kv_rank,
    int rot_dim, int window, float scale, int q_ld, const float* __restrict__ sink) {
  extern __shared__ float lds[];      // per wave: q [dl], p [64], row numbers [64]
  const int wave = threadIdx.x / kWave, lane = threadIdx.x % kWave;
  const int dl = kv_rank + rot_dim;
  const int per_wave = dl + 2 * kWave;
  float* q_s = lds + (size_t)wave * per_wave;
  float* p_s = q_s + dl;
  int* row_s = (int*)(p_s + kWave);
  const int t = blockIdx.x;
  const int h = blockIdx.y * kLatentWaves + wave;
  if (h >= heads) return;             // waves are independent: no workgroup barrier below
  const int pos = positions[t];
  const int lo = window > 0 ? max(0, pos - window + 1) : 0;
  const int* tab = table + (int64_t)entry_of_token[t] * table_width;
  const float* q = qa + (int64_t)t * q_ld + h * dl;
  for (int d = lane; d < dl; d += kWave) q_s[d] = q[d];
  __builtin_amdgcn_wave_barrier();
  const bool by4 = dl % 4 == 0 && ((uintptr_t)pages & 15) == 0;

  float m = -INFINITY, l = 0.f;
  float acc[kMaxRankPerLane] = {};
  for (int j0 = lo; j0 <= pos; j0 += kWave) {
    const int j = j0 + lane;
    float s = -INFINITY;
    int row = -1;               // the token's row in the pages
    if (j <= pos) {
      const int page = tab[j / page_size];
      if (page >= 0) {
        row = page * page_size + j % page_size;
        const TC* kr = pages + (int64_t)row * dl;
        float dot = 0.f;
        if (by4) {
          for (int d = 0; d < dl; d += 4) {
            const f32x4_l k4 = load4_l(kr + d);
#pragma unroll
            for (int e = 0; e < 4; ++e) dot = fmaf(q_s[d + e], k4[e], dot);
          }
        } else {
          for (int d = 0; d < dl; ++d) dot = fmaf(q_s[d], to_f32(kr[d]), dot);
        }
        s = dot * scale;
      }
    }
    const float m_new = fmaxf(m, wave_max(s));
    const float corr = m_new == -INFINITY ? 1.f : expf(m - m_new);
    const float p = (row >= 0 && m_new != -INFINITY) ? expf(s - m_new) : 0.f;
    l = l * corr + wave_sum(p);
    m = m_new;
    p_s[lane] = p;
    row_s[lane] = row;
    __builtin_amdgcn_wave_barrier();
#pragma unroll
    for (int r = 0; r < kMaxRankPerLane; ++r) acc[r] *= corr;
    const int n = min(kWave, pos - j0 + 1);
    for (int jj = 0; jj < n; ++jj) {
      if (row_s[jj] < 0) continue;
      const int64_t vr = (int64_t)row_s[jj] * dl;
      const float pj = p_s[jj];
#pragma unroll
      for (int r = 0; r < kMaxRankPerLane; ++r) {
        const int d = lane + r * kWave;
        if (d < kv_rank) acc[r] = fmaf(pj, to_f32(pages[vr + d]), acc[r]);
      }
    }
    __builtin_amdgcn_wave_barrier();
  }
  if (sink) l += sink_weight(sink[h], m);
  TO* o = out + ((int64_t)t * heads + h) * kv_rank;
  const float inv = l > 0.f ? 1.0f / l : 0.f;
#pragma unroll
  for (int r = 0; r < kMaxRankPerLane; ++r) {
    const int d = lane + r * kWave;
    if (d < kv_rank) o[d] = from_f32<TO>(acc[r] * inv);
  }
}

extern "C" int ts_latent_attention(const float* qa, const void* pages, int cache_type, void* out,
                                   int out_type, const int* positions, const int* entry_of_token,
                                   const int* table, int table_width, int page_size,
                                   int num_tokens, int heads, int kv_rank, int rot_dim,
                                   int window, float scale, int q_ld, const float* sink,
                                   hipStream_t stream) {
  if (num_tokens <= 0) return 0;
  const int dl = kv_rank + rot_dim;
  if (q_ld < heads * dl) TS_FAIL("latent_attention: query rows of %d", q_ld);
  if (heads <= 0 || kv_rank <= 0 || rot_dim < 0 || page_size <= 0 || table_width <= 0)
    TS_FAIL("latent_attention: bad sizes heads=%d kv_rank=%d rot_dim=%d", heads, kv_rank, rot_dim);
  if (kv_rank > kMaxRankPerLane * kWave || dl > kMaxLatent)
    TS_FAIL("latent_attention: latent of %d + %d elements, at most %d + %d are built", kv_rank,
            rot_dim, kMaxRankPerLane * kWave, kMaxLatent - kMaxRankPerLane * kWave);
  const size_t lds = (size_t)kLatentWaves * (dl + 2 * kWave) * sizeof(float);
  const dim3 grid(num_tokens, (heads + kLatentWaves - 1) / kLatentWaves);
  TS_DISPATCH_TYPE(cache_type, TC, TS_DISPATCH_TYPE(out_type, TO,
      hipLaunchKernelGGL((latent_attention_kernel<TC, TO>), grid, dim3(kLatentWaves * kWave), lds,
                         stream, qa, (const TC*)pages, (TO*)out, positions, entry_of_token, table,
                         table_width, page_size, heads, kv_rank, rot_dim, window, scale, q_ld,
                         sink)));
  TS_CHECK_LAUNCH("latent_attention");
  return 0;
}


// ---------------------------------------------------------------- attention on the matrix cores
// bfloat16 pages.  A tile is 16 consecutive rows of the step's (token, head) rows that
// belong to one entry: every head reads the same cached rows, so a decode step's token is
// one tile of its heads, and a prompt's tile a few tokens with all their heads.  One
// wavefront per (tile, share of the keys):
//     S^T = K Q'^T        v_mfma_f32_16x16x32_bf16, reduction over the latent row
//     O^T += C^T P^T      the same instruction, reduction over 32 keys
// Lane (r, g) = (lane % 16, lane / 16) owns query row r: its scores come out as
// S^T[key 4g + t][row r], which is, in place, its part of the second product's B operand;
// its softmax statistics are shared with lanes r + 16, r + 32, r + 48; its part of O^T is
// [columns 16 db + 4g + t][row r], so rescaling needs nothing from other lanes.
// Keys are walked in blocks of 32 at absolute multiples of 32, staged in LDS, from where both
// operands come: the K operand as 16 bytes of a row, the C^T operand by the transposing read.
// Where a step has few tiles, a tile's keys are shared out in runs of `keys_per_split` over
// several workgroups, whose unnormalised results and statistics (the largest score in units
// of log2) a second kernel merges.
typedef __attribute__((ext_vector_type(8))) __bf16 bf16x8_l;

struct LatentMfmaArgs {
  const float* qa;          // [tokens, q_ld]: the heads' rows of dl side by side (and, where
                            // q_ld is larger, something else behind them)
  const bf16_t* pages;      // [pages, page_size, dl]
  void* out;                // [rows, kv_rank]
  const int* tiles;         // [num_tiles, 3]: first row, rows (1..16), entry
  const int* positions;     // [tokens]
  const int* table;
  float* part_o;            // [num_tiles, splits, 16, kv_rank]
  float* part_ml;           // [num_tiles, splits, 16, 2]
  int table_width, page_size, heads, kv_rank, rot_dim, window, keys_per_split, splits;
  float scale;
  int q_ld;
  const float* sink;        // [heads] or null: a score that joins a row's denominator once
};

constexpr int kLatentPad = 8;     // elements between staged rows: operand reads spread over banks

// The query operand of a row: elements 32 s + 8 g .. + 7.  (The row's length is a multiple of
// 8: eight elements are there together or not at all.)
template <int KS>
__device__ __forceinline__ void load_query_row(bf16x8_l (&q)[KS], const float* qr, int dl, int g) {
#pragma unroll
  for (int s = 0; s < KS; ++s) {
    const int d0 = 32 * s + 8 * g;
    const float* src = qr + min(d0, dl - 8);
    const f32x4_l lo4 = *(const f32x4_l*)src, hi4 = *(const f32x4_l*)(src + 4);
    const bool there = d0 < dl;
#pragma unroll
    for (int j = 0; j < 4; ++j) {
      q[s][j] = (__bf16)(there ? lo4[j] : 0.f);
      q[s][4 + j] = (__bf16)(there ? hi4[j] : 0.f);
    }
  }
}

// Scores, in units of log2, of row r with keys kb + 16 (e / 4) + 4 g + e % 4, the keys staged
// as rows of `stride` elements at k_s; -inf where the row does not see a key.  Returns the
// largest of the row's 32.
template <int KS>
__device__ __forceinline__ float score_block(float (&sc)[8], const bf16x8_l (&q)[KS],
                                             const bf16_t* k_s, int stride, int kb, int dl,
                                             float scale_log2, int pos, int lo, int r, int g) {
  // two blocks of 16 keys, the reduction over the row in two chains each
  f32x4_l st[2][2];
#pragma unroll
  for (int c = 0; c < 4; ++c) st[c / 2][c % 2] = f32x4_l{0.f, 0.f, 0.f, 0.f};
  const bf16_t* kr = k_s + r * stride + 8 * g;
#pragma unroll
  for (int s = 0; s < KS; ++s) {
    if (32 * s < dl) {
      // (past the row's end the query's elements are zeros: the row's last eight stand in)
      const int d0 = min(32 * s, dl - 8 - 8 * g);
#pragma unroll
      for (int blk = 0; blk < 2; ++blk) {
        const bf16x8_l kop = *(const bf16x8_l*)(kr + 16 * blk * stride + d0);
        st[blk][s & 1] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(kop, q[s], st[blk][s & 1], 0, 0, 0);
      }
    }
  }
  float mx = -INFINITY;
#pragma unroll
  for (int e = 0; e < 8; ++e) {
    const int key = kb + 16 * (e / 4) + 4 * g + e % 4;
    const float dot = st[e / 4][0][e % 4] + st[e / 4][1][e % 4];
    sc[e] = (key <= pos && key >= lo) ? dot * scale_log2 : -INFINITY;
    mx = fmaxf(mx, sc[e]);
  }
  mx = fmaxf(mx, __shfl_xor(mx, 16, kWave));
  return fmaxf(mx, __shfl_xor(mx, 32, kWave));
}

// Weights of the block's scores relative to m_use; returns this lane's share of their sum.
__device__ __forceinline__ float weigh_block(bf16x8_l& pv, const float (&sc)[8], float m_use) {
  float sum = 0.f;
#pragma unroll
  for (int e = 0; e < 8; ++e) {
    const float p = __builtin_amdgcn_exp2f(sc[e] - m_use);
    sum += p;
    pv[e] = (__bf16)p;
  }
  return sum;
}

// O^T += C^T P^T for `DB` blocks of 16 columns from `db0` on.  A lane's column of four keys
// comes out of LDS by the transposing read (sixteen lanes name four rows' runs of sixteen
// elements, four elements a lane, and each gets one column of the four rows; columns from
// kv_rank on, which belong to the key part or the padding, give results that nobody stores).
template <int DB>
__device__ __forceinline__ void value_block(f32x4_l (&o)[DB], bf16x8_l pv, const bf16_t* k_s,
                                            int stride, int kv_rank, int db0, int r, int g) {
  typedef short s16x4 __attribute__((ext_vector_type(4)));
  typedef __attribute__((address_space(3))) s16x4* Lds4;
  const bf16_t* vrow = k_s + (4 * g + r / 4) * stride + 4 * (r % 4) + 16 * db0;
#pragma unroll
  for (int db = 0; db < DB; ++db) {
    if (16 * (db0 + db) < kv_rank) {
      const s16x4 a = __builtin_amdgcn_ds_read_tr16_b64_v4i16((Lds4)(vrow + 16 * db));
      const s16x4 b = __builtin_amdgcn_ds_read_tr16_b64_v4i16((Lds4)(vrow + 16 * stride + 16 * db));
      const auto both = __builtin_shufflevector(a, b, 0, 1, 2, 3, 4, 5, 6, 7);
      o[db] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(__builtin_bit_cast(bf16x8_l, both), pv,
                                                      o[db], 0, 0, 0);
    }
  }
}

// The four lanes r, r + 16, r + 32, r + 48 hold a row: the sum of their shares.
__device__ __forceinline__ float row_total(float v) {
  v += __shfl_xor(v, 16, kWave);
  return v + __shfl_xor(v, 32, kWave);
}

// A sink's weight relative to `m_log2`, a largest score in units of log2.
__device__ __forceinline__ float sink_weight_log2(float sink, float m_log2) {
  return __builtin_amdgcn_exp2f(fminf(sink * 1.44269504088896f - m_log2, 100.f));
}

// Many tiles: the four wavefronts of a workgroup take four tiles of one entry (the last of an
// entry's may be empty: such a wavefront only helps load) and walk the union of their keys
// together.  Each block of 32 cached rows passes through registers into one of two LDS
// buffers, eight threads a row, sent for while the block before it is worked on; the page of
// the block after that is looked up meanwhile.
template <int KS, int DB, typename TO>
__global__ __launch_bounds__(4 * kWave) void latent_attention_mfma_kernel(LatentMfmaArgs a) {
  constexpr int PIECES = (4 * KS + 7) / 8;                // 16-byte pieces of a row a thread brings
  extern __shared__ __attribute__((aligned(16))) unsigned char lds_raw[];
  const int dl = a.kv_rank + a.rot_dim, P = a.page_size;
  const int stride = dl + kLatentPad;
  bf16_t* bufs = (bf16_t*)lds_raw;                        // [2][32][stride]
  const int wave = threadIdx.x / kWave, lane = threadIdx.x % kWave, r = lane % 16, g = lane / 16;
  const int tile0 = blockIdx.x * 4, tile = tile0 + wave;
  const int row0 = a.tiles[3 * tile], nrows = a.tiles[3 * tile + 1];
  const int* tab = a.table + (int64_t)a.tiles[3 * tile0 + 2] * a.table_width;
  const bool row_ok = r < nrows;
  const int my_row = row0 + max(0, min(r, nrows - 1));
  const int my_head = my_row % a.heads, my_token = my_row / a.heads;
  const int pos_r = a.positions[my_token];
  const int my_pos = row_ok ? pos_r : -1;
  const int lo_r = a.window > 0 ? max(0, pos_r - a.window + 1) : 0;
  // the keys of the whole workgroup: from the first tile's first token to the last token
  const int pos_first = a.positions[a.tiles[3 * tile0] / a.heads];
  const int lo_t = a.window > 0 ? max(0, pos_first - a.window + 1) : 0;
  int hi_t = pos_first;
  for (int w = 0; w < 4; ++w) {
    const int n = a.tiles[3 * (tile0 + w) + 1];
    if (n > 0) hi_t = max(hi_t, a.positions[(a.tiles[3 * (tile0 + w)] + n - 1) / a.heads]);
  }
  const int k_begin = (lo_t / 32) * 32, k_end = hi_t + 1;
  // the wavefront's own first and last visible keys: blocks outside are not its business
  const int tile_last = __builtin_amdgcn_readfirstlane(nrows) > 0
      ? a.positions[(row0 + nrows - 1) / a.heads] : -1;
  const int tile_lo = __builtin_amdgcn_readfirstlane(a.window > 0
      ? max(0, a.positions[row0 / a.heads] - a.window + 1) : 0);

  const int key_l = threadIdx.x / 8, piece = threadIdx.x % 8;
  const int parts = dl / 8;
  auto look_up = [&](int kb) {
    const int j = kb + key_l;
    return (j >= lo_t && j <= hi_t) ? tab[j / P] : -1;
  };
  bf16x8_l held[PIECES];
  auto fetch = [&](int kb, int page) {
    const bf16_t* row = a.pages + ((int64_t)max(page, 0) * P + (kb + key_l) % P) * dl;
#pragma unroll
    for (int i = 0; i < PIECES; ++i) held[i] = *(const bf16x8_l*)(row + 8 * min(piece + 8 * i, parts - 1));
  };
  auto commit = [&](bf16_t* buf, int page) {
    const bf16x8_l zero = {0, 0, 0, 0, 0, 0, 0, 0};
#pragma unroll
    for (int i = 0; i < PIECES; ++i)
      if (piece + 8 * i < parts)
        *(bf16x8_l*)(buf + key_l * stride + 8 * (piece + 8 * i)) = page >= 0 ? held[i] : zero;
  };
  int page = look_up(k_begin), page_next = look_up(k_begin + 32);
  fetch(k_begin, page);
  bf16x8_l q[KS];
  load_query_row<KS>(q, a.qa + (int64_t)my_token * a.q_ld + my_head * dl, dl, g);
  f32x4_l o[DB];
#pragma unroll
  for (int db = 0; db < DB; ++db) o[db] = f32x4_l{0.f, 0.f, 0.f, 0.f};
  float m = -INFINITY, l = 0.f;            // l: this lane's share of the row's sum
  commit(bufs, page);
  __syncthreads();
  const float scale_log2 = a.scale * 1.44269504088896341f;
  int which = 0;
  for (int kb = k_begin; kb < k_end; kb += 32, which ^= 1) {
    const bool more = kb + 32 < k_end;
    if (more) {
      page = page_next;
      fetch(kb + 32, page);
      page_next = look_up(kb + 64);
    }
    if (kb <= tile_last && kb + 31 >= tile_lo) {
      const bf16_t* k_s = bufs + which * 32 * stride;
      float sc[8];
      bf16x8_l pv;
      const float m_new = fmaxf(m, score_block<KS>(sc, q, k_s, stride, kb, dl, scale_log2, my_pos, lo_r, r, g));
      // (a finite stand-in while the row has seen no key makes every exponential zero)
      const float m_use = fmaxf(m_new, -1e30f);
      const float corr = __builtin_amdgcn_exp2f(m - m_use);
      l = l * corr + weigh_block(pv, sc, m_use);
      m = m_new;
      if (__builtin_amdgcn_ballot_w64(corr != 1.f) != 0) {
#pragma unroll
        for (int db = 0; db < DB; ++db) o[db] = o[db] * corr;
      }
      value_block<DB>(o, pv, k_s, stride, a.kv_rank, 0, r, g);
    }
    if (more) commit(bufs + (which ^ 1) * 32 * stride, page);
    __syncthreads();
  }
  l = row_total(l);
  if (!row_ok) return;
  if (a.sink) l += sink_weight_log2(a.sink[my_head], m);
  const float inv = l > 0.f ? 1.0f / l : 0.f;
  TO* orow = (TO*)a.out + (int64_t)my_row * a.kv_rank;
#pragma unroll
  for (int db = 0; db < DB; ++db)
#pragma unroll
    for (int e = 0; e < 4; ++e) {
      const int d = 16 * db + 4 * g + e;
      if (d < a.kv_rank) orow[d] = from_f32<TO>(o[db][e] * inv);
    }
}

// Few tiles: a workgroup per (tile, share of its keys).  Of every 32 NW keys each of the NW
// wavefronts stages and scores 32; with the rows' largest scores and the weights exchanged
// through LDS, each then adds up its share of the columns over all of them.  With one share
// of the keys the rows are finished here, else the share's results go to the merge kernel.
template <int KS, int DB, int NW, typename TO>
__global__ __launch_bounds__(NW* kWave) void latent_attention_split_kernel(LatentMfmaArgs a) {
  constexpr int PIECES = (4 * KS + 7) / 8, OWN = (DB + NW - 1) / NW;
  // rows a lane's loads are in flight for at once: as many as registers allow
  constexpr int ROWS = KS > 10 ? 2 : 4;
  extern __shared__ __attribute__((aligned(16))) unsigned char lds_raw[];   // [NW][32][stride]
  __shared__ bf16x8_l p_s[NW][kWave];
  __shared__ float m_s[NW][16], l_s[NW][16];
  const int dl = a.kv_rank + a.rot_dim, P = a.page_size;
  const int stride = dl + kLatentPad;
  const int wave = threadIdx.x / kWave, lane = threadIdx.x % kWave, r = lane % 16, g = lane / 16;
  bf16_t* all_s = (bf16_t*)lds_raw;
  bf16_t* k_s = all_s + wave * 32 * stride;
  const int tile = blockIdx.x, split = blockIdx.y;
  const int row0 = a.tiles[3 * tile], nrows = a.tiles[3 * tile + 1];
  const int* tab = a.table + (int64_t)a.tiles[3 * tile + 2] * a.table_width;
  const bool row_ok = r < nrows;
  const int my_row = row0 + max(0, min(r, nrows - 1));
  const int my_head = my_row % a.heads, my_token = my_row / a.heads;
  const int pos_r = a.positions[my_token];
  const int my_pos = row_ok ? pos_r : -1;
  const int lo_r = a.window > 0 ? max(0, pos_r - a.window + 1) : 0;
  const int pos_first = a.positions[row0 / a.heads];
  const int hi_t = a.positions[(row0 + nrows - 1) / a.heads];
  const int lo_t = a.window > 0 ? max(0, pos_first - a.window + 1) : 0;
  const int k_begin = (lo_t / 32) * 32 + split * a.keys_per_split;
  const int k_end = min(k_begin + a.keys_per_split, hi_t + 1);
  const int64_t slot = ((int64_t)tile * a.splits + split) * 16 + r;
  if (k_begin >= k_end) {        // more shares than keys: a neutral result, no data touched
    if (threadIdx.x < 16) {
      a.part_ml[2 * slot] = -INFINITY;
      a.part_ml[2 * slot + 1] = 0.f;
    }
    return;
  }
  const int parts = dl / 8, key8 = lane / 8, piece = lane % 8;
  const float scale_log2 = a.scale * 1.44269504088896341f;
  bf16x8_l q[KS];
  f32x4_l o[OWN];
#pragma unroll
  for (int db = 0; db < OWN; ++db) o[db] = f32x4_l{0.f, 0.f, 0.f, 0.f};
  float m = -INFINITY, l = 0.f;            // l: this lane's share of its wavefront's keys
  for (int kb0 = k_begin; kb0 < k_end; kb0 += 32 * NW) {
    const int kb = kb0 + 32 * wave;
#pragma unroll 1
    for (int c0 = 0; c0 < 4; c0 += ROWS) {
      int page[ROWS];
#pragma unroll
      for (int c = 0; c < ROWS; ++c) {
        const int j = kb + 8 * (c0 + c) + key8;
        page[c] = (j >= lo_t && j < k_end) ? tab[j / P] : -1;
      }
      bf16x8_l held[ROWS][PIECES];
#pragma unroll
      for (int c = 0; c < ROWS; ++c) {
        const bf16_t* row = a.pages + ((int64_t)max(page[c], 0) * P + (kb + 8 * (c0 + c) + key8) % P) * dl;
#pragma unroll
        for (int i = 0; i < PIECES; ++i)
          held[c][i] = *(const bf16x8_l*)(row + 8 * min(piece + 8 * i, parts - 1));
      }
      const bf16x8_l zero = {0, 0, 0, 0, 0, 0, 0, 0};
#pragma unroll
      for (int c = 0; c < ROWS; ++c)
#pragma unroll
        for (int i = 0; i < PIECES; ++i)
          if (piece + 8 * i < parts)
            *(bf16x8_l*)(k_s + (8 * (c0 + c) + key8) * stride + 8 * (piece + 8 * i)) =
                page[c] >= 0 ? held[c][i] : zero;
    }
    if (kb0 == k_begin) load_query_row<KS>(q, a.qa + (int64_t)my_token * a.q_ld + my_head * dl, dl, g);
    // (a wavefront's LDS accesses are carried out in order: its own rows need no barrier)
    float sc[8];
    const float mx = score_block<KS>(sc, q, k_s, stride, kb, dl, scale_log2, my_pos, lo_r, r, g);
    if (g == 0) m_s[wave][r] = mx;
    __syncthreads();                       // every wavefront's rows and largest scores are there
    float m_new = m;
#pragma unroll
    for (int w = 0; w < NW; ++w) m_new = fmaxf(m_new, m_s[w][r]);
    const float m_use = fmaxf(m_new, -1e30f);
    const float corr = __builtin_amdgcn_exp2f(m - m_use);
    bf16x8_l pv;
    l = l * corr + weigh_block(pv, sc, m_use);
    m = m_new;
    p_s[wave][lane] = pv;
    __syncthreads();                       // and every wavefront's weights
#pragma unroll
    for (int db = 0; db < OWN; ++db) o[db] = o[db] * corr;
#pragma unroll 1
    for (int w = 0; w < NW; ++w)
      value_block<OWN>(o, p_s[w][lane], all_s + w * 32 * stride, stride, a.kv_rank, wave * OWN, r, g);
    __syncthreads();                       // before the areas are written again
  }
  const float share = row_total(l);
  if (g == 0) l_s[wave][r] = share;
  __syncthreads();
  if (!row_ok) return;
  float sum = 0.f;
#pragma unroll
  for (int w = 0; w < NW; ++w) sum += l_s[w][r];
  float inv = 1.f;
  if (a.splits > 1) {
    if (wave == 0 && g == 0) {
      a.part_ml[2 * slot] = m;
      a.part_ml[2 * slot + 1] = sum;
    }
  } else {
    if (a.sink) sum += sink_weight_log2(a.sink[my_head], m);
    inv = sum > 0.f ? 1.0f / sum : 0.f;
  }
#pragma unroll
  for (int db = 0; db < OWN; ++db)
#pragma unroll
    for (int e = 0; e < 4; ++e) {
      const int d = 16 * (wave * OWN + db) + 4 * g + e;
      if (d < a.kv_rank) {
        if (a.splits > 1) a.part_o[slot * a.kv_rank + d] = o[db][e];
        else ((TO*)a.out)[(int64_t)my_row * a.kv_rank + d] = from_f32<TO>(o[db][e] * inv);
      }
    }
}

// One workgroup per (tile, row): the shares' results weighted by exp(m_s - max m) and
// divided by the summed weights of their l, shares in index order.  The first wavefront
// turns the shares' statistics into weights (in LDS); then every thread adds its columns
// over the shares, eight loads at a time.
template <typename TO>
__global__ __launch_bounds__(128) void latent_attention_merge_kernel(LatentMfmaArgs a) {
  extern __shared__ float w_s[];            // [splits] weights, then the reciprocal of their sum
  const int tile = blockIdx.x, r = blockIdx.y;
  if (r >= a.tiles[3 * tile + 1]) return;
  const int64_t base = (int64_t)tile * a.splits * 16 + r;
  if (threadIdx.x < kWave) {
    float mx = -INFINITY;
    for (int s = threadIdx.x; s < a.splits; s += kWave)
      mx = fmaxf(mx, a.part_ml[2 * (base + 16 * s)]);
    mx = wave_max(mx);
    float total = 0.f;
    for (int s = threadIdx.x; s < a.splits; s += kWave) {
      const float ms = a.part_ml[2 * (base + 16 * s)];
      const float w = ms == -INFINITY ? 0.f : __builtin_amdgcn_exp2f(ms - mx);
      w_s[s] = w;
      total += a.part_ml[2 * (base + 16 * s) + 1] * w;
    }
    total = wave_sum(total);
    if (a.sink) total += sink_weight_log2(a.sink[(a.tiles[3 * tile] + r) % a.heads], mx);
    if (threadIdx.x == 0) w_s[a.splits] = total > 0.f ? 1.0f / total : 0.f;
  }
  __syncthreads();
  const float inv = w_s[a.splits];
  // shares beyond the row's keys are empty and wrote no values: what is there is dropped
  int used = a.splits;
  while (used > 1 && w_s[used - 1] == 0.f) --used;
  TO* orow = (TO*)a.out + (int64_t)(a.tiles[3 * tile] + r) * a.kv_rank;
  for (int d = threadIdx.x; d < a.kv_rank; d += blockDim.x) {
    float acc = 0.f;
    int s = 0;
    for (; s + 8 <= used; s += 8) {
      float v[8];
#pragma unroll
      for (int u = 0; u < 8; ++u) v[u] = a.part_o[(base + 16 * (s + u)) * a.kv_rank + d];
#pragma unroll
      for (int u = 0; u < 8; ++u) acc = w_s[s + u] == 0.f ? acc : fmaf(v[u], w_s[s + u], acc);
    }
    for (; s < used; ++s)
      if (w_s[s] != 0.f) acc = fmaf(a.part_o[(base + 16 * s) * a.kv_rank + d], w_s[s], acc);
    orow[d] = from_f32<TO>(acc * inv);
  }
}

// An LDS size above the default has to be allowed per kernel, once.
static int allow_lds(const void* kernel, size_t bytes, size_t* allowed) {
  if (bytes <= *allowed) return 0;
  if (hipFuncSetAttribute(kernel, hipFuncAttributeMaxDynamicSharedMemorySize, (int)bytes) != hipSuccess)
    TS_FAIL("latent_attention_mfma: cannot raise the LDS limit to %zu bytes", bytes);
  *allowed = bytes;
  return 0;
}

constexpr size_t kLatentLds = 154 * 1024;      // of a compute unit's 160 KB, beside weights and statistics

template <int KS, int DB, typename TO>
static int launch_latent_typed(const LatentMfmaArgs& a, int num_tiles, int waves, hipStream_t stream) {
  const size_t block = (size_t)32 * (a.kv_rank + a.rot_dim + kLatentPad) * sizeof(bf16_t);
  if (waves == 4) {
    static size_t allowed = 48 * 1024;         // per instantiation, here and below
    auto kernel = latent_attention_mfma_kernel<KS, DB, TO>;
    if (allow_lds((const void*)kernel, 2 * block, &allowed)) return -1;
    hipLaunchKernelGGL(kernel, dim3(num_tiles / 4), dim3(4 * kWave), 2 * block, stream, a);
    return 0;
  }
  // four wavefronts' rows in LDS at once where a row is short enough, else two's
  constexpr int NW = (size_t)4 * 32 * (32 * KS + kLatentPad) * sizeof(bf16_t) <= kLatentLds ? 4 : 2;
  static size_t allowed = 48 * 1024;
  auto kernel = latent_attention_split_kernel<KS, DB, NW, TO>;
  if (allow_lds((const void*)kernel, NW * block, &allowed)) return -1;
  hipLaunchKernelGGL(kernel, dim3(num_tiles, a.splits), dim3(NW * kWave), NW * block, stream, a);
  if (a.splits > 1)
    hipLaunchKernelGGL(latent_attention_merge_kernel<TO>, dim3(num_tiles, 16), dim3(128),
                       (size_t)(a.splits + 1) * sizeof(float), stream, a);
  return 0;
}

template <int KS, int DB>
static int launch_latent_mfma(const LatentMfmaArgs& a, int num_tiles, int waves, int out_type,
                              hipStream_t stream) {
  TS_DISPATCH_TYPE(out_type, TO, return (launch_latent_typed<KS, DB, TO>(a, num_tiles, waves, stream)));
  return 0;
}

// 1 if the matrix-core kernel serves these sizes (bfloat16 pages are the caller's to check).
extern "C" int ts_latent_attention_mfma_fits(int kv_rank, int rot_dim) {
  const int dl = kv_rank + rot_dim;
  return dl % 8 == 0 && dl <= 640 && kv_rank <= 512;
}

// `waves` 4: `tiles` comes in groups of four tiles of one entry, a group's last tiles possibly
// empty (0 rows), `num_tiles` counts them all and keys are not shared out; 1: every tile has
// rows and its keys are shared out in `splits` runs.
extern "C" int ts_latent_attention_mfma(const float* qa, const void* pages, void* out,
                                        int out_type, const int* tiles, int num_tiles, int waves,
                                        const int* positions, const int* table, int table_width,
                                        int page_size, int heads, int kv_rank, int rot_dim,
                                        int window, float scale, int keys_per_split, int splits,
                                        float* part_o, float* part_ml, int q_ld,
                                        const float* sink, hipStream_t stream) {
  if (num_tiles <= 0) return 0;
  if (q_ld < heads * (kv_rank + rot_dim)) TS_FAIL("latent_attention_mfma: query rows of %d", q_ld);
  if (!ts_latent_attention_mfma_fits(kv_rank, rot_dim) || heads <= 0 || page_size <= 0)
    TS_FAIL("latent_attention_mfma: sizes kv_rank=%d rot_dim=%d are not served", kv_rank, rot_dim);
  if (splits < 1 || keys_per_split < 32 || keys_per_split % 32)
    TS_FAIL("latent_attention_mfma: bad split of the keys (%d runs of %d)", splits, keys_per_split);
  if (splits > 1 && (!part_o || !part_ml)) TS_FAIL("latent_attention_mfma: no scratch for the shares");
  if ((waves != 1 && waves != 4) || num_tiles % waves || (waves == 4 && splits != 1))
    TS_FAIL("latent_attention_mfma: %d tiles in groups of %d", num_tiles, waves);
  if ((((uintptr_t)pages | (uintptr_t)qa) & 15) != 0 || q_ld % 4)
    TS_FAIL("latent_attention_mfma: pages and query rows must start on 16 bytes");
  LatentMfmaArgs a{qa, (const bf16_t*)pages, out, tiles, positions, table, part_o, part_ml,
                   table_width, page_size, heads, kv_rank, rot_dim, window, keys_per_split, splits,
                   scale, q_ld, sink};
  const int dl = kv_rank + rot_dim;
  int rc;
  if (dl <= 96 && kv_rank <= 64) rc = launch_latent_mfma<3, 4>(a, num_tiles, waves, out_type, stream);
  else if (dl <= 160 && kv_rank <= 128) rc = launch_latent_mfma<5, 8>(a, num_tiles, waves, out_type, stream);
  else if (dl <= 320 && kv_rank <= 256) rc = launch_latent_mfma<10, 16>(a, num_tiles, waves, out_type, stream);
  else if (dl <= 576) rc = launch_latent_mfma<18, 32>(a, num_tiles, waves, out_type, stream);
  else rc = launch_latent_mfma<20, 32>(a, num_tiles, waves, out_type, stream);
  if (rc) return rc;
  TS_CHECK_LAUNCH("latent_attention_mfma");
  return 0;
}
