// Paged causal attention on the matrix cores for bfloat16: decode tokens and portions
// of prompts in one launch, any head grouping, head sizes in steps of 16 up to 256.
//
// One wavefront owns a tile of 16 query rows: up to 16 query heads of one key/value
// head for 16/rows_per_token consecutive tokens of one batch entry (a decode token
// gives one token per tile).  Everything is computed transposed,
//     S^T = K Q^T          (v_mfma_f32_16x16x32_bf16, reduction over the head size)
//     O^T = V^T P^T        (reduction over 32 keys)
// so that a lane holds one query's scores for 8 of the 32 keys: these 8 numbers are,
// in place, the B operand of the second product, and the softmax statistics of a query
// live in the four lanes that share its column.  K rows (contiguous along the head
// size) and V columns (contiguous along positions, the cache stores values transposed
// inside a page) are both read from global memory in operand layout: no LDS, no
// transposes.  The key range of a tile is cut into chunks of kChunk keys at fixed
// positions; a launch either lets a wave walk all its chunks or spreads them over
// `num_splits` waves whose partial results a second kernel merges.
#include "attention_mfma_kernel.h"

// Merge the splits of every tile: out = sum_s o_s e^(m_s - M) / sum_s l_s e^(m_s - M),
// splits taken in order.  One workgroup per item, thread (row, column group).  A split
// without keys has left m = -inf and is skipped.  Splits are taken eight at a time: the
// loads of the eight, statistics and values, are all asked for before the first is used,
// none under a condition, and the first eight do not wait for the position either (it
// says how many splits hold keys at all, which ends the loop early when a short context
// has been given many splits), so a merge of up to eight splits costs one trip to memory.
template <int HD>
__global__ __launch_bounds__(256) void attention_merge_kernel(AttentionMfmaArgs args) {
  constexpr int kGroup = 8, DC = HD / 16;
  const AttentionArgs& a = args.base;
  const int item = blockIdx.x;
  const int tile = item / (a.nkv * args.head_blocks);
  const int kvh = (item / args.head_blocks) % a.nkv;
  const int hb = item % args.head_blocks;
  const int tok0 = args.tiles ? args.tiles[tile * 3 + 1] : tile,
            ntok = args.tiles ? args.tiles[tile * 3 + 2] : 1;
  const int group = a.nq / a.nkv;
  const int r = threadIdx.x / 16, dc = threadIdx.x % 16;
  const int ti = r / args.rows_per_token, hh = hb * 16 + r % args.rows_per_token;
  if (ti >= ntok || hh >= group) return;
  const int S = args.num_splits;
  const int64_t base = (int64_t)item * S * 16 + r;
  // splits beyond the tile's chunks hold nothing: same arithmetic as the first kernel
  const int pos_first = a.positions[tok0], pos_last = pos_first + ntok - 1;
  float M = -INFINITY, L = 0.f;
  float acc[DC] = {};
  int used = S;                              // known after the first group's loads
  for (int s0 = 0; s0 < used; s0 += kGroup) {
    float ms[kGroup], ls[kGroup], part[kGroup][DC];
#pragma unroll
    for (int j = 0; j < kGroup; ++j) {
      const int64_t slot = base + (int64_t)min(s0 + j, S - 1) * 16;   // past the end: the last again
      ms[j] = args.partial_ml[slot * 2];
      ls[j] = args.partial_ml[slot * 2 + 1];
#pragma unroll
      for (int i = 0; i < DC; ++i) part[j][i] = args.partial_o[slot * HD + i * 16 + dc];
    }
    if (s0 == 0) {
      const int origin = key_walk<32>(a, first_visible(a, pos_first)).origin;
      const int nchunks = pos_last / kChunk - origin / kChunk + 1;
      const int per = (nchunks - 1 + S) / S;
      used = min(S, (nchunks + per - 1) / per);
    }
    float Mg = M;
#pragma unroll
    for (int j = 0; j < kGroup; ++j) Mg = (s0 + j < S) ? fmaxf(Mg, ms[j]) : Mg;
    if (Mg == -INFINITY) continue;            // nothing but empty splits so far
    const float keep = __builtin_amdgcn_exp2f(M - Mg);     // M = -inf gives 0
    L *= keep;
#pragma unroll
    for (int i = 0; i < DC; ++i) acc[i] *= keep;
#pragma unroll
    for (int j = 0; j < kGroup; ++j) {
      // an empty split wrote no values: what is there is dropped, not multiplied by 0
      const bool live = s0 + j < S && ms[j] != -INFINITY;
      const float w = live ? __builtin_amdgcn_exp2f(ms[j] - Mg) : 0.f;
      L += live ? ls[j] * w : 0.f;
#pragma unroll
      for (int i = 0; i < DC; ++i) acc[i] += live ? part[j][i] * w : 0.f;
    }
    M = Mg;
  }
  L = sum_with_sink(L, M, a.sink, kvh * group + hh);
  const float inv = L > 0.f ? 1.f / L : 0.f;
  bf16_t* out = (bf16_t*)a.out + ((int64_t)(tok0 + ti) * a.nq + kvh * group + hh) * HD;
#pragma unroll
  for (int i = 0; i < DC; ++i) out[i * 16 + dc] = (bf16_t)(acc[i] * inv);
}

int ts_check_attention_args(const AttentionArgs& a, const char* who);
int launch_attention_mfma_scores(const AttentionMfmaArgs& args, hipStream_t stream);

// The merge alone, for the decode kernel's splits.
int launch_attention_merge(const AttentionMfmaArgs& args, hipStream_t stream) {
  const int items = args.num_tiles * args.base.nkv * args.head_blocks;
  switch (args.base.hd) {
#define TS_CASE(HD) case HD: hipLaunchKernelGGL(attention_merge_kernel<HD>, dim3(items), dim3(256), 0, stream, args); break;
    TS_CASE(16) TS_CASE(32) TS_CASE(48) TS_CASE(64) TS_CASE(80) TS_CASE(96) TS_CASE(112)
    TS_CASE(128) TS_CASE(144) TS_CASE(160) TS_CASE(176) TS_CASE(192) TS_CASE(208) TS_CASE(224)
    TS_CASE(240) TS_CASE(256)
#undef TS_CASE
    default: TS_FAIL("attention_merge: head_dim=%d not built", args.base.hd);
  }
  return 0;
}

// The merge of a decode step's key splits that ts_attention_decode was told to leave.
extern "C" int ts_attention_merge(const AttentionMfmaArgs* p, hipStream_t stream) {
  const AttentionMfmaArgs& args = *p;
  if (args.num_tiles <= 0 || args.num_splits <= 1) return 0;
  if (!args.partial_o || !args.partial_ml) TS_FAIL("attention_merge: no partial results");
  if (launch_attention_merge(args, stream)) return -1;
  TS_CHECK_LAUNCH("attention_merge");
  return 0;
}

extern "C" int ts_attention_mfma_chunk() { return kChunk; }

int ts_check_attention_mfma_args(const AttentionMfmaArgs& args, const char* who) {
  const AttentionArgs& a = args.base;
  if (ts_check_attention_args(a, who)) return -1;
  if (a.hd % 16) TS_FAIL("%s: head_dim=%d must be a multiple of 16", who, a.hd);
  if (a.page_size % 4) TS_FAIL("%s: page_size=%d must be a multiple of 4", who, a.page_size);
  const int group = a.nq / a.nkv;
  if (args.rows_per_token != (group < 16 ? group : 16) ||
      args.head_blocks != (group + 15) / 16)
    TS_FAIL("%s: rows_per_token/head_blocks do not fit a group of %d", who, group);
  if (!args.tiles && args.num_tiles != a.num_entries)
    TS_FAIL("%s: without a tile list there is one tile per entry", who);
  if (((uintptr_t)a.q | (uintptr_t)a.out | (uintptr_t)a.k_pages | (uintptr_t)a.v_pages) & 15)
    TS_FAIL("%s: tensors must be 16-byte aligned", who);
  return 0;
}

extern "C" int ts_attention_mfma(const AttentionMfmaArgs* p, hipStream_t stream) {
  AttentionMfmaArgs args = *p;
  const AttentionArgs& a = args.base;
  if (a.num_tokens <= 0 || args.num_tiles <= 0) return 0;
  if (ts_check_attention_mfma_args(args, "attention_mfma")) return -1;
  if (args.num_splits < 1 || args.num_splits > 65535) TS_FAIL("attention_mfma: num_splits=%d", args.num_splits);
  if (args.num_splits > 1 && (!args.partial_o || !args.partial_ml))
    TS_FAIL("attention_mfma: splits need partial buffers");
  if (has_score_extras(a)) {
    if (launch_attention_mfma_scores(args, stream)) return -1;
    TS_CHECK_LAUNCH("attention_mfma");
    return 0;
  }
  switch (a.hd) {
#define TS_CASE(HD) case HD: if (launch_mfma<HD, false>(args, stream)) return -1; break;
    TS_CASE(16) TS_CASE(32) TS_CASE(48) TS_CASE(64) TS_CASE(80) TS_CASE(96) TS_CASE(112)
    TS_CASE(128) TS_CASE(144) TS_CASE(160) TS_CASE(176) TS_CASE(192) TS_CASE(208) TS_CASE(224)
    TS_CASE(240) TS_CASE(256)
#undef TS_CASE
    default: TS_FAIL("attention_mfma: head_dim=%d not built", a.hd);
  }
  TS_CHECK_LAUNCH("attention_mfma");
  return 0;
}
