// Row-wise kernels of layers that norm a sub-layer's output before adding it to the
// residual stream, and of what such models put in front of the stream: a bigram-hashed
// embedding with its norm, the add of a normalised output (alone, with the next
// sub-layer's norm, or with the new stream's rows for a sub-layer that reads it as it is),
// the gate of a token's own input to a layer, the norm with a token shift behind it, and the
// PolyNorm activation.
// One workgroup per row; every sum, root and product in float32.
//
// Per-request state (the previous token, the previous row of a token shift) lives in
// [slots, ...] arrays indexed by the entry's slot id.  A step reads a request's state for
// the first token of its portion only, and only if that token is not at position 0; the
// workgroup of that first token is also the one that writes the state the portion leaves
// (from the portion's last token), so within a launch every state element is read and then
// written by one thread.
#include "common.h"

__device__ __forceinline__ float inv_rms(float sumsq, int n, float eps) {
  return 1.0f / sqrtf(sumsq / (float)n + eps);
}

// A thread keeps the first kRowItems elements of its share of a row in registers between
// the passes over the row (sum of squares, then the scaled values), so a row of up to
// kRowItems x threads elements is read once; what lies beyond is read again.  A step of
// few rows is a chain of trips to memory and barriers, and this halves the trips.
constexpr int kRowItems = 8;

// Threads for a row of `width` elements: eight elements a thread, 64 to 1024 threads.
static int row_threads(int width) {
  int t = ((width + kRowItems - 1) / kRowItems + 63) / 64 * 64;
  return t < 64 ? 64 : (t > 1024 ? 1024 : t);
}

// ---------------------------------------------------------------- bigram embedding
template <typename TW>
__global__ __launch_bounds__(256) void bigram_embed_kernel(
    const TW* __restrict__ table, const TW* __restrict__ bigram, const float* __restrict__ norm_w,
    const int* __restrict__ ids, const int* __restrict__ positions,
    const int* __restrict__ entry_of_token, const int* __restrict__ q_start,
    const int* __restrict__ slot_ids, int* __restrict__ prev_state, float* __restrict__ out,
    int width, float scale, int buckets, int mul_prev, int mul_cur, float eps) {
  __shared__ float scratch[16];
  __shared__ int row_s;
  const int t = blockIdx.x;
  const int id = ids[t];
  if (threadIdx.x == 0) {
    const int e = entry_of_token[t];
    const int first = q_start[e];
    int prev = -1;
    if (t > first) {
      prev = ids[t - 1];
    } else {
      const int slot = slot_ids[e];
      if (positions[t] > 0) prev = prev_state[slot];
      prev_state[slot] = ids[q_start[e + 1] - 1];
    }
    int row = buckets;
    if (prev >= 0) {
      int64_t v = ((int64_t)prev * mul_prev + (int64_t)id * mul_cur) % buckets;
      if (v < 0) v += buckets;
      row = (int)v;
    }
    row_s = row;
  }
  __syncthreads();
  const TW* er = table + (int64_t)id * width;
  const TW* br = bigram + (int64_t)row_s * width;
  float* o = out + (int64_t)t * width;
  float ss = 0.f;
  for (int i = threadIdx.x; i < width; i += blockDim.x) {
    const float v = to_f32(er[i]) * scale + to_f32(br[i]);
    o[i] = v;
    ss += v * v;
  }
  const float r = inv_rms(block_sum(ss, scratch), width, eps);
  for (int i = threadIdx.x; i < width; i += blockDim.x) o[i] = o[i] * r * norm_w[i];
}

extern "C" int ts_bigram_embed(const void* table, const void* bigram, int table_type,
                               const float* norm_w, const int* ids, const int* positions,
                               const int* entry_of_token, const int* q_start,
                               const int* slot_ids, int* prev_state, float* out, int num_tokens,
                               int width, float scale, int buckets, int mul_prev, int mul_cur,
                               float eps, hipStream_t stream) {
  if (num_tokens <= 0) return 0;
  if (width <= 0 || buckets <= 0) TS_FAIL("bigram_embed: bad sizes width=%d buckets=%d", width, buckets);
  TS_DISPATCH_TYPE(table_type, TW,
                   hipLaunchKernelGGL(bigram_embed_kernel<TW>, dim3(num_tokens), dim3(256), 0,
                                      stream, (const TW*)table, (const TW*)bigram, norm_w, ids,
                                      positions, entry_of_token, q_start, slot_ids, prev_state,
                                      out, width, scale, buckets, mul_prev, mul_cur, eps));
  TS_CHECK_LAUNCH("bigram_embed");
  return 0;
}

// ---------------------------------------------------------------- add of a normalised output
// resid += delta / rms(delta) * post_w; then, by THEN, nothing more, or also
// out = resid / rms(resid) * norm_w, or out = resid itself (rounded to out's type, for a
// sub-layer that reads the stream as it is).
constexpr int kThenNothing = 0, kThenNorm = 1, kThenRows = 2;

template <typename TD, typename TO, int THEN>
__global__ __launch_bounds__(1024) void postnorm_add_kernel(
    float* __restrict__ resid, const TD* __restrict__ delta, const float* __restrict__ post_w,
    const float* __restrict__ norm_w, TO* __restrict__ out, int width, float post_eps,
    float norm_eps) {
  __shared__ float scratch[16];
  const int64_t row = blockIdx.x;
  const int nt = blockDim.x;
  float* x = resid + row * width;
  const TD* d = delta + row * width;
  TO* o = out + row * width;
  // (the weights are asked for with the row, not behind the sum that they wait for)
  float dc[kRowItems], xc[kRowItems], pc[kRowItems], nc[kRowItems];
  float ss = 0.f;
#pragma unroll
  for (int k = 0; k < kRowItems; ++k) {
    const int i = threadIdx.x + k * nt;
    dc[k] = i < width ? to_f32(d[i]) : 0.f;
    xc[k] = i < width ? x[i] : 0.f;
    pc[k] = i < width ? post_w[i] : 0.f;
    nc[k] = THEN == kThenNorm && i < width ? norm_w[i] : 0.f;
  }
#pragma unroll
  for (int k = 0; k < kRowItems; ++k) ss += dc[k] * dc[k];
  for (int i = threadIdx.x + kRowItems * nt; i < width; i += nt) {
    const float v = to_f32(d[i]);
    ss += v * v;
  }
  const float r = inv_rms(block_sum(ss, scratch), width, post_eps);
  float ss2 = 0.f;
#pragma unroll
  for (int k = 0; k < kRowItems; ++k) {
    const int i = threadIdx.x + k * nt;
    if (i < width) {
      xc[k] = xc[k] + dc[k] * r * pc[k];
      x[i] = xc[k];
      if (THEN == kThenRows) o[i] = from_f32<TO>(xc[k]);
      ss2 += xc[k] * xc[k];
    }
  }
  for (int i = threadIdx.x + kRowItems * nt; i < width; i += nt) {
    const float v = x[i] + to_f32(d[i]) * r * post_w[i];
    x[i] = v;
    if (THEN == kThenRows) o[i] = from_f32<TO>(v);
    ss2 += v * v;
  }
  if (THEN == kThenNorm) {
    const float r2 = inv_rms(block_sum(ss2, scratch), width, norm_eps);
#pragma unroll
    for (int k = 0; k < kRowItems; ++k) {
      const int i = threadIdx.x + k * nt;
      if (i < width) o[i] = from_f32<TO>(xc[k] * r2 * nc[k]);
    }
    // each thread reads back the elements it wrote itself
    for (int i = threadIdx.x + kRowItems * nt; i < width; i += nt)
      o[i] = from_f32<TO>(x[i] * r2 * norm_w[i]);
  }
}

// With `norm_w` the norm of the new stream goes to `out`; with `out` alone the new stream.
extern "C" int ts_postnorm_add(float* resid, const void* delta, int delta_type,
                               const float* post_w, float post_eps, const float* norm_w,
                               float norm_eps, void* out, int out_type, int rows, int width,
                               hipStream_t stream) {
  if (rows <= 0) return 0;
  if (width <= 0) TS_FAIL("postnorm_add: bad width %d", width);
  if (norm_w && !out) TS_FAIL("postnorm_add: a norm without an output");
  const dim3 grid(rows), block(row_threads(width));
  TS_DISPATCH_TYPE(delta_type, TD, {
    if (!out) {
      hipLaunchKernelGGL((postnorm_add_kernel<TD, float, kThenNothing>), grid, block, 0, stream,
                         resid, (const TD*)delta, post_w, nullptr, nullptr, width, post_eps, 0.f);
    } else if (norm_w) {
      TS_DISPATCH_TYPE(out_type, TO,
                       hipLaunchKernelGGL((postnorm_add_kernel<TD, TO, kThenNorm>), grid, block, 0,
                                          stream, resid, (const TD*)delta, post_w, norm_w,
                                          (TO*)out, width, post_eps, norm_eps));
    } else {
      TS_DISPATCH_TYPE(out_type, TO,
                       hipLaunchKernelGGL((postnorm_add_kernel<TD, TO, kThenRows>), grid, block, 0,
                                          stream, resid, (const TD*)delta, post_w, nullptr,
                                          (TO*)out, width, post_eps, 0.f));
    }
  });
  TS_CHECK_LAUNCH("postnorm_add");
  return 0;
}

// ---------------------------------------------------------------- two outputs, one sum
// d = a / rms(a) * wa + b / rms(b) * wb, the outputs of two sub-layers that run side by
// side, each normed by itself; then, where there is a stream, resid += d / rms(d) * post_w and
// THEN as above; without one d itself goes to `out`.  A row's values of a, b and resid wait in
// registers between the sums (up to kRowItems a thread; what lies beyond is read again).
__device__ __forceinline__ float2 block_sum2(float a, float b, float* scratch) {
  a = wave_sum(a);
  b = wave_sum(b);
  const int wave = threadIdx.x / kWave, lane = threadIdx.x % kWave;
  const int nwaves = (blockDim.x + kWave - 1) / kWave;
  __syncthreads();
  if (lane == 0) scratch[2 * wave] = a, scratch[2 * wave + 1] = b;
  __syncthreads();
  float2 total = make_float2(0.f, 0.f);
  for (int w = 0; w < nwaves; ++w) total.x += scratch[2 * w], total.y += scratch[2 * w + 1];
  return total;
}

template <typename TA, typename TB, typename TO, int THEN, bool STREAM>
__global__ __launch_bounds__(1024) void pair_add_kernel(
    float* __restrict__ resid, const TA* __restrict__ a, const float* __restrict__ wa,
    const TB* __restrict__ b, const float* __restrict__ wb, float pair_eps,
    const float* __restrict__ post_w, float post_eps, const float* __restrict__ norm_w,
    float norm_eps, TO* __restrict__ out, int width) {
  __shared__ float scratch[32];
  const int64_t row = blockIdx.x;
  const int nt = blockDim.x;
  const TA* ar = a + row * width;
  const TB* br = b + row * width;
  float* x = STREAM ? resid + row * width : nullptr;
  TO* o = out ? out + row * width : nullptr;
  float dc[kRowItems], bc[kRowItems], xc[kRowItems], wac[kRowItems], wbc[kRowItems];
  float pc[STREAM ? kRowItems : 1], nc[THEN == kThenNorm ? kRowItems : 1];
  float sa = 0.f, sb = 0.f;
#pragma unroll
  for (int k = 0; k < kRowItems; ++k) {
    const int i = threadIdx.x + k * nt;
    const bool in = i < width;
    dc[k] = in ? to_f32(ar[i]) : 0.f;
    bc[k] = in ? to_f32(br[i]) : 0.f;
    wac[k] = in ? wa[i] : 0.f;
    wbc[k] = in ? wb[i] : 0.f;
    if (STREAM) {
      xc[k] = in ? x[i] : 0.f;
      pc[k] = in ? post_w[i] : 0.f;
    }
    if (THEN == kThenNorm) nc[k] = in ? norm_w[i] : 0.f;
  }
#pragma unroll
  for (int k = 0; k < kRowItems; ++k) sa = fmaf(dc[k], dc[k], sa), sb = fmaf(bc[k], bc[k], sb);
  for (int i = threadIdx.x + kRowItems * nt; i < width; i += nt) {
    const float va = to_f32(ar[i]), vb = to_f32(br[i]);
    sa = fmaf(va, va, sa), sb = fmaf(vb, vb, sb);
  }
  const float2 ss = block_sum2(sa, sb, scratch);
  const float ra = inv_rms(ss.x, width, pair_eps), rb = inv_rms(ss.y, width, pair_eps);
  auto beyond = [&](int i) { return to_f32(ar[i]) * ra * wa[i] + to_f32(br[i]) * rb * wb[i]; };
  float sd = 0.f;
#pragma unroll
  for (int k = 0; k < kRowItems; ++k) {
    dc[k] = dc[k] * ra * wac[k] + bc[k] * rb * wbc[k];
    sd = fmaf(dc[k], dc[k], sd);
  }
  for (int i = threadIdx.x + kRowItems * nt; i < width; i += nt) {
    const float v = beyond(i);
    sd = fmaf(v, v, sd);
  }
  if constexpr (!STREAM) {
#pragma unroll
    for (int k = 0; k < kRowItems; ++k) {
      const int i = threadIdx.x + k * nt;
      if (i < width) o[i] = from_f32<TO>(dc[k]);
    }
    for (int i = threadIdx.x + kRowItems * nt; i < width; i += nt) o[i] = from_f32<TO>(beyond(i));
  } else {
    const float r = inv_rms(block_sum(sd, scratch), width, post_eps);
    float sx = 0.f;
#pragma unroll
    for (int k = 0; k < kRowItems; ++k) {
      const int i = threadIdx.x + k * nt;
      if (i < width) {
        xc[k] += dc[k] * r * pc[k];
        x[i] = xc[k];
        if (THEN == kThenRows) o[i] = from_f32<TO>(xc[k]);
        sx = fmaf(xc[k], xc[k], sx);
      }
    }
    for (int i = threadIdx.x + kRowItems * nt; i < width; i += nt) {
      const float v = x[i] + beyond(i) * r * post_w[i];
      x[i] = v;
      if (THEN == kThenRows) o[i] = from_f32<TO>(v);
      sx = fmaf(v, v, sx);
    }
    if constexpr (THEN == kThenNorm) {
      const float r2 = inv_rms(block_sum(sx, scratch), width, norm_eps);
#pragma unroll
      for (int k = 0; k < kRowItems; ++k) {
        const int i = threadIdx.x + k * nt;
        if (i < width) o[i] = from_f32<TO>(xc[k] * r2 * nc[k]);
      }
      // each thread reads back the elements it wrote itself
      for (int i = threadIdx.x + kRowItems * nt; i < width; i += nt)
        o[i] = from_f32<TO>(x[i] * r2 * norm_w[i]);
    }
  }
}

// `resid` null: the pair's sum goes to `out`.  Else with `norm_w` the norm of the new stream
// goes to `out`, with `out` alone the new stream's rows, and without it nothing more.
extern "C" int ts_pair_add(float* resid, const void* a, int a_type, const float* wa, const void* b,
                           int b_type, const float* wb, float pair_eps,
                           const float* post_w, float post_eps, const float* norm_w,
                           float norm_eps, void* out, int out_type, int rows, int width,
                           hipStream_t stream) {
  if (rows <= 0) return 0;
  if (width <= 0) TS_FAIL("pair_add: bad width %d", width);
  if (!a || !b || !wa || !wb) TS_FAIL("pair_add: two outputs with a norm weight each");
  if (resid ? !post_w : (!out || post_w || norm_w))
    TS_FAIL("pair_add: a stream comes with a norm weight, and without one the sum needs an output");
  if (norm_w && !out) TS_FAIL("pair_add: a norm without an output");
  const dim3 grid(rows), block(row_threads(width));
#define TS_PAIR_LAUNCH(TO, THEN, STREAM)                                                         \
  hipLaunchKernelGGL((pair_add_kernel<TA, TB, TO, THEN, STREAM>), grid, block, 0, stream, resid, \
                     (const TA*)a, wa, (const TB*)b, wb, pair_eps, post_w, post_eps,             \
                     norm_w, norm_eps, (TO*)out, width)
  TS_DISPATCH_TYPE(a_type, TA, TS_DISPATCH_TYPE(b_type, TB, {
    if (!resid) {
      TS_DISPATCH_TYPE(out_type, TO, TS_PAIR_LAUNCH(TO, kThenNothing, false));
    } else if (!out) {
      TS_PAIR_LAUNCH(float, kThenNothing, true);
    } else if (norm_w) {
      TS_DISPATCH_TYPE(out_type, TO, TS_PAIR_LAUNCH(TO, kThenNorm, true));
    } else {
      TS_DISPATCH_TYPE(out_type, TO, TS_PAIR_LAUNCH(TO, kThenRows, true));
    }
  }));
#undef TS_PAIR_LAUNCH
  TS_CHECK_LAUNCH("pair_add");
  return 0;
}

// ---------------------------------------------------------------- a token's own input
// out[t, j] = gelu_tanh(z[t, j]) * table[ids[t], col + j], j < dim: the gate of what a
// token's row of a table brings into a layer.  z float32 [T, dim], table [V, ld].
template <typename TW, typename TO>
__global__ __launch_bounds__(256) void token_gate_kernel(
    const float* __restrict__ z, const TW* __restrict__ table, const int* __restrict__ ids,
    TO* __restrict__ out, int64_t total, int dim, int ld, int col) {
  const int64_t idx = (int64_t)blockIdx.x * blockDim.x + threadIdx.x;
  if (idx >= total) return;
  const int64_t t = idx / dim;
  const int j = (int)(idx - t * dim);
  out[idx] = from_f32<TO>(gelu_tanh(z[idx]) * to_f32(table[(int64_t)ids[t] * ld + col + j]));
}

extern "C" int ts_token_gate(const float* z, const void* table, int table_type, const int* ids,
                             void* out, int out_type, int num_tokens, int dim, int ld, int col,
                             hipStream_t stream) {
  if (num_tokens <= 0) return 0;
  if (dim <= 0 || col < 0 || col + dim > ld)
    TS_FAIL("token_gate: columns [%d, %d) of rows of %d", col, col + dim, ld);
  const int64_t total = (int64_t)num_tokens * dim;
  TS_DISPATCH_TYPE(table_type, TW, TS_DISPATCH_TYPE(out_type, TO,
      hipLaunchKernelGGL((token_gate_kernel<TW, TO>), dim3((unsigned)((total + 255) / 256)),
                         dim3(256), 0, stream, z, (const TW*)table, ids, (TO*)out, total, dim, ld,
                         col)));
  TS_CHECK_LAUNCH("token_gate");
  return 0;
}

// The same gate inside the product that leads back to the stream, for few rows (bfloat16
// table and weight, bfloat16 gated values as the kernel above writes them):
// out[t, n] = sum_j (gelu_tanh(z[t, j]) * table[ids[t], col + j]) w[n, j], float32.
// A workgroup makes the gated values of 16 tokens in LDS and each of its wavefronts owns 16
// columns of the result.
typedef __attribute__((ext_vector_type(8))) __bf16 bf16x8_side;
typedef __attribute__((ext_vector_type(4))) float f32x4_side;
constexpr int kSideDim = 512;

__global__ __launch_bounds__(256) void token_gate_product_kernel(
    const float* __restrict__ z, const bf16_t* __restrict__ table, const int* __restrict__ ids,
    const bf16_t* __restrict__ w, float* __restrict__ out, int num_tokens, int width, int dim,
    int ld, int col) {
  extern __shared__ __attribute__((aligned(16))) unsigned char lds_raw[];
  bf16_t* act = (bf16_t*)lds_raw;                  // [16][stride]
  const int stride = (dim + 31) / 32 * 32 + 8;
  const int t0 = blockIdx.y * 16;
  const int wave = threadIdx.x / kWave, lane = threadIdx.x % kWave, r = lane % 16, g = lane / 16;
  const int n0 = (blockIdx.x * 4 + wave) * 16, n = min(n0 + r, width - 1);
  const bf16x8_side zero = {0, 0, 0, 0, 0, 0, 0, 0};
  // The first four steps' weights are asked for before the gated values' chain of loads (a
  // token's id, then its row of the table) begins.
  constexpr int kEarly = 4;
  bf16x8_side early[kEarly];
#pragma unroll
  for (int i = 0; i < kEarly; ++i)
    early[i] = *(const bf16x8_side*)(w + (int64_t)n * dim + min(32 * i + 8 * g, dim - 8));
  const bool wide = ld % 8 == 0 && col % 8 == 0 && ((uintptr_t)table & 15) == 0;
  const int units = (stride - 8) / 8;              // runs of eight values a token, padding included
  for (int u = threadIdx.x; u < 16 * units; u += blockDim.x) {
    const int row = u / units, j0 = (u - row * units) * 8;
    const int t = min(t0 + row, num_tokens - 1);
    bf16x8_side v = zero;
    if (t0 + row < num_tokens && j0 < dim) {
      const float* zr = z + (int64_t)t * dim + j0;
      const bf16_t* er = table + (int64_t)ids[t] * ld + col + j0;
      bf16x8_side e;
      if (wide) {
        e = *(const bf16x8_side*)er;
      } else {
#pragma unroll
        for (int j = 0; j < 8; ++j) e[j] = er[j];
      }
      const f32x4_side a = *(const f32x4_side*)zr, b = *(const f32x4_side*)(zr + 4);
#pragma unroll
      for (int j = 0; j < 8; ++j) v[j] = (bf16_t)(gelu_tanh(j < 4 ? a[j] : b[j - 4]) * (float)e[j]);
    }
    *(bf16x8_side*)(act + row * stride + j0) = v;
  }
  __syncthreads();
  f32x4_side acc = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
  for (int i = 0; i < kEarly; ++i) {
    if (32 * i < dim) {            // (past the last column the gated values are zeros)
      const bf16x8_side av = *(const bf16x8_side*)(act + r * stride + 32 * i + 8 * g);
      acc = __builtin_amdgcn_mfma_f32_16x16x32_bf16(early[i], av, acc, 0, 0, 0);
    }
  }
  for (int k = 32 * kEarly; k < dim; k += 32) {
    const int at = k + 8 * g;
    const bf16x8_side wv = *(const bf16x8_side*)(w + (int64_t)n * dim + min(at, dim - 8));
    const bf16x8_side av = *(const bf16x8_side*)(act + r * stride + at);
    acc = __builtin_amdgcn_mfma_f32_16x16x32_bf16(wv, av, acc, 0, 0, 0);
  }
  // lane (r, g) holds columns n0 + 4 g .. + 3 of token r
  if (t0 + r >= num_tokens) return;
  float* o = out + (int64_t)(t0 + r) * width + n0 + 4 * g;
#pragma unroll
  for (int e = 0; e < 4; ++e)
    if (n0 + 4 * g + e < width) o[e] = acc[e];
}

extern "C" int ts_token_gate_product_fits(int num_tokens, int dim) {
  return num_tokens <= 64 && dim % 8 == 0 && dim <= kSideDim;
}

extern "C" int ts_token_gate_product(const float* z, const void* table, const int* ids,
                                     const void* w, float* out, int num_tokens, int width,
                                     int dim, int ld, int col, hipStream_t stream) {
  if (num_tokens <= 0) return 0;
  if (width <= 0 || dim <= 0 || !ts_token_gate_product_fits(num_tokens, dim))
    TS_FAIL("token_gate_product: %d tokens of %d values are not taken", num_tokens, dim);
  if (col < 0 || col + dim > ld) TS_FAIL("token_gate_product: columns [%d, %d) of rows of %d", col, col + dim, ld);
  if (((uintptr_t)w | (uintptr_t)z) & 15) TS_FAIL("token_gate_product: weight and values must start on 16 bytes");
  const size_t lds = (size_t)16 * ((dim + 31) / 32 * 32 + 8) * sizeof(bf16_t);
  hipLaunchKernelGGL(token_gate_product_kernel, dim3((width + 63) / 64, (num_tokens + 15) / 16),
                     dim3(256), lds, stream, z, (const bf16_t*)table, ids, (const bf16_t*)w, out,
                     num_tokens, width, dim, ld, col);
  TS_CHECK_LAUNCH("token_gate_product");
  return 0;
}

// ---------------------------------------------------------------- norm and token shift
// h_t = resid_t / rms(resid_t) * w;  out_t = h_t + (h_(t-1) - h_t) * shift.
// h_(t-1) is recomputed from the row before inside a portion, read from the request's
// state at a portion's first token, and zero at position 0.
template <typename TO>
__global__ __launch_bounds__(1024) void norm_token_shift_kernel(
    const float* __restrict__ resid, const float* __restrict__ norm_w,
    const float* __restrict__ shift_w, float* __restrict__ state, TO* __restrict__ out,
    const int* __restrict__ positions, const int* __restrict__ entry_of_token,
    const int* __restrict__ q_start, const int* __restrict__ slot_ids, int width, float eps) {
  __shared__ float scratch[16];
  const int t = blockIdx.x, nt = blockDim.x;
  const int e = entry_of_token[t];
  const int first = q_start[e], last = q_start[e + 1] - 1;
  const bool is_first = t == first;
  const bool from_state = is_first && positions[t] > 0;
  const bool other_last = is_first && last != t;
  const float* x = resid + (int64_t)t * width;
  const float* xp = resid + (int64_t)(t - 1) * width;
  const float* xl = resid + (int64_t)last * width;
  float* st = state + (int64_t)slot_ids[e] * width;
  // the row, and the one other row this workgroup needs (the row before, or the portion's
  // last row whose norm goes into the state), both kept in registers
  const float* y = !is_first ? xp : xl;
  const bool need_y = !is_first || other_last;
  float xc[kRowItems], yc[kRowItems];
  float ss = 0.f, ssy = 0.f;
#pragma unroll
  for (int k = 0; k < kRowItems; ++k) {
    const int i = threadIdx.x + k * nt;
    xc[k] = i < width ? x[i] : 0.f;
    yc[k] = (need_y && i < width) ? y[i] : 0.f;
    ss += xc[k] * xc[k];
    ssy += yc[k] * yc[k];
  }
  for (int i = threadIdx.x + kRowItems * nt; i < width; i += nt) {
    ss += x[i] * x[i];
    if (need_y) ssy += y[i] * y[i];
  }
  const float r = inv_rms(block_sum(ss, scratch), width, eps);
  float ry = r;
  if (need_y) ry = inv_rms(block_sum(ssy, scratch), width, eps);
  TO* o = out + (int64_t)t * width;
  auto finish = [&](int i, float xv, float yv) {
    const float w = norm_w[i];
    const float h = xv * r * w;
    float prev = 0.f;
    if (!is_first) prev = yv * ry * w;
    else if (from_state) prev = st[i];
    o[i] = from_f32<TO>(h + (prev - h) * shift_w[i]);
    if (is_first) st[i] = other_last ? yv * ry * w : h;
  };
#pragma unroll
  for (int k = 0; k < kRowItems; ++k) {
    const int i = threadIdx.x + k * nt;
    if (i < width) finish(i, xc[k], yc[k]);
  }
  for (int i = threadIdx.x + kRowItems * nt; i < width; i += nt)
    finish(i, x[i], need_y ? y[i] : 0.f);
}

extern "C" int ts_norm_token_shift(const float* resid, const float* norm_w, float eps,
                                   const float* shift_w, float* state, void* out, int out_type,
                                   const int* positions, const int* entry_of_token,
                                   const int* q_start, const int* slot_ids, int num_tokens,
                                   int width, hipStream_t stream) {
  if (num_tokens <= 0) return 0;
  if (width <= 0) TS_FAIL("norm_token_shift: bad width %d", width);
  TS_DISPATCH_TYPE(out_type, TO,
                   hipLaunchKernelGGL(norm_token_shift_kernel<TO>, dim3(num_tokens),
                                      dim3(row_threads(width)), 0, stream, resid, norm_w, shift_w,
                                      state, (TO*)out, positions, entry_of_token, q_start,
                                      slot_ids, width, eps));
  TS_CHECK_LAUNCH("norm_token_shift");
  return 0;
}

// ---------------------------------------------------------------- PolyNorm
// out = a z/rms(z) + b z^2/rms(z^2) + c z^3/rms(z^3) + e, powers element by element.
template <typename TO>
__global__ __launch_bounds__(1024) void polynorm_kernel(const float* __restrict__ z,
                                                        const float* __restrict__ coef,
                                                        TO* __restrict__ out, int width,
                                                        float eps) {
  __shared__ float scratch[16];
  const int64_t row = blockIdx.x;
  const int nt = blockDim.x;
  const float* x = z + row * width;
  float zc[kRowItems];
  float s2 = 0.f, s4 = 0.f, s6 = 0.f;
  auto add = [&](float v) {
    const float v2 = v * v, v3 = v2 * v;
    s2 += v2;
    s4 += v2 * v2;
    s6 += v3 * v3;
  };
#pragma unroll
  for (int k = 0; k < kRowItems; ++k) {
    const int i = threadIdx.x + k * nt;
    zc[k] = i < width ? x[i] : 0.f;
    add(zc[k]);
  }
  for (int i = threadIdx.x + kRowItems * nt; i < width; i += nt) add(x[i]);
  const float r1 = inv_rms(block_sum(s2, scratch), width, eps);
  const float r2 = inv_rms(block_sum(s4, scratch), width, eps);
  const float r3 = inv_rms(block_sum(s6, scratch), width, eps);
  const float a = coef[0], b = coef[1], c = coef[2], e = coef[3];
  TO* o = out + row * width;
  auto value = [&](float v) {
    const float v2 = v * v;
    return a * (v * r1) + b * (v2 * r2) + c * (v2 * v * r3) + e;
  };
#pragma unroll
  for (int k = 0; k < kRowItems; ++k) {
    const int i = threadIdx.x + k * nt;
    if (i < width) o[i] = from_f32<TO>(value(zc[k]));
  }
  for (int i = threadIdx.x + kRowItems * nt; i < width; i += nt) o[i] = from_f32<TO>(value(x[i]));
}

extern "C" int ts_polynorm(const float* z, const float* coef, void* out, int out_type, int rows,
                           int width, float eps, hipStream_t stream) {
  if (rows <= 0) return 0;
  if (width <= 0) TS_FAIL("polynorm: bad width %d", width);
  TS_DISPATCH_TYPE(out_type, TO,
                   hipLaunchKernelGGL(polynorm_kernel<TO>, dim3(rows), dim3(row_threads(width)), 0,
                                      stream, z, coef, (TO*)out, width, eps));
  TS_CHECK_LAUNCH("polynorm");
  return 0;
}
