// Attention over paged rows that are wider than the matrix-unit kernels take (a key row of more than 256 entries, as a large
// latent beside its rotated part gives): the same function of (positions, window, sink) computed with vector arithmetic.
//
// A workgroup takes one row of one query head.  Keys are walked in tiles of 64 at absolute positions, ascending; a tile's 64
// scores are shared through LDS, the running maximum moves when a tile's is larger, and every thread owns the output columns
// t, t + 256, ....  All sums are in 32-bit and their order is a function of absolute positions, so the result does not depend
// on how a sequence was cut into steps.  Score = q.k * scale; exp(sinks[head]) joins the denominator.
#include "common.h"
#include "vec.h"

#define WIDE_THREADS 256
#define WIDE_TILE 64
#define WIDE_COLS 4            // output columns a thread may own: rows of up to 1024 entries

struct WideArgs {
  const elem_t* q;             // [T, nq, d]
  elem_t* out;                 // [T, nq, d]
  const elem_t* kc;            // [pages, nkv, P, d]
  const elem_t* vc;            // [pages, nkv, d, P]
  const int32_t *block_table, *cu_q, *k_len, *items;
  const void* sinks;
  int bt_stride, nq, nkv, d, P, window, rows_per_item, sinks_f32;
  float scale;
};

__global__ __launch_bounds__(WIDE_THREADS) void attn_wide_kernel(WideArgs a) {
  __shared__ float q[WIDE_THREADS * WIDE_COLS];
  __shared__ float score[WIDE_TILE];
  const int item = blockIdx.x / a.rows_per_item;
  const int seq = a.items[2 * item], row = a.items[2 * item + 1] + blockIdx.x % a.rows_per_item;
  const int q_begin = a.cu_q[seq], q_len = a.cu_q[seq + 1] - q_begin;
  if (row >= q_len) return;                                   // the whole workgroup
  const int head = blockIdx.y, kvh = head / (a.nq / a.nkv);
  const int pos = a.k_len[seq] - q_len + row;
  const int lo = a.window > 0 ? max(0, pos - a.window + 1) : 0;
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
  const int lp = __builtin_ctz(a.P);
  const int32_t* bt = a.block_table + (int64_t)seq * a.bt_stride;
  const int64_t page_elems = (int64_t)a.P * a.d, page_stride = (int64_t)a.nkv * page_elems;
  const elem_t* kbase = a.kc + (int64_t)kvh * page_elems;
  const elem_t* vbase = a.vc + (int64_t)kvh * page_elems;
  const elem_t* qrow = a.q + ((int64_t)(q_begin + row) * a.nq + head) * a.d;
  for (int c = threadIdx.x; c < a.d; c += WIDE_THREADS) q[c] = to_f32(qrow[c]);

  float M = -INFINITY, L = 0.f, acc[WIDE_COLS];
#pragma unroll
  for (int j = 0; j < WIDE_COLS; ++j) acc[j] = 0.f;
  for (int t = lo / WIDE_TILE; t <= pos / WIDE_TILE; ++t) {
    __syncthreads();                                          // q is there; the tile before is done with `score`
    // Wave w: the tile's keys 16 w .. 16 w + 15, four lanes a key, each lane every fourth 16-byte vector of the row.
    {
      const int key = t * WIDE_TILE + wave * 16 + (lane >> 2);
      const bool seen = key >= lo && key <= pos;
      float s = 0.f;
      if (seen) {
        const elem_t* krow = kbase + (int64_t)bt[key >> lp] * page_stride + (int64_t)(key & (a.P - 1)) * a.d;
        for (int c = (lane & 3) * VK_VEC; c < a.d; c += 4 * VK_VEC) {
          float kv[VK_VEC];
          load_elems(krow + c, kv);
#pragma unroll
          for (int e = 0; e < VK_VEC; ++e) s = __builtin_fmaf(q[c + e], kv[e], s);
        }
      }
      s = group_sum<4>(s);
      if ((lane & 3) == 0) score[wave * 16 + (lane >> 2)] = seen ? s * a.scale : -INFINITY;
    }
    __syncthreads();
    const float m = wave_max_xor(score[lane]);                // every wave the same; a walked tile has a visible key
    const float Mn = fmaxf(M, m);
    const float keep = M > -INFINITY ? expf(M - Mn) : 0.f;
    const float p = expf(score[lane] - Mn);                   // 0 for a key that is not seen
    L = L * keep + wave_sum_xor(p);
    M = Mn;
#pragma unroll
    for (int j = 0; j < WIDE_COLS; ++j) {
      const int c = threadIdx.x + j * WIDE_THREADS;
      if (c >= a.d) continue;
      float sum = acc[j] * keep;
      for (int k = max(lo, t * WIDE_TILE) & ~(VK_VEC - 1); k <= min(pos, t * WIDE_TILE + WIDE_TILE - 1); k += VK_VEC) {
        // VK_VEC keys at a multiple of VK_VEC lie in one page.
        float v[VK_VEC];
        load_elems(vbase + (int64_t)bt[k >> lp] * page_stride + (int64_t)c * a.P + (k & (a.P - 1)), v);
#pragma unroll
        for (int e = 0; e < VK_VEC; ++e)
          if (k + e >= lo && k + e <= pos) sum = __builtin_fmaf(expf(score[k + e - t * WIDE_TILE] - Mn), v[e], sum);
      }
      acc[j] = sum;
    }
  }
  if (a.sinks != nullptr) L = L + expf(load_weight(a.sinks, a.sinks_f32, head) - M);
  elem_t* orow = a.out + ((int64_t)(q_begin + row) * a.nq + head) * a.d;
#pragma unroll
  for (int j = 0; j < WIDE_COLS; ++j) {
    const int c = threadIdx.x + j * WIDE_THREADS;
    if (c < a.d) orow[c] = from_f32<elem_t>(acc[j] / L);
  }
}

extern "C" {

// The widest row that vk_attention_wide takes.
int vk_attention_wide_limit(void) { return WIDE_THREADS * WIDE_COLS; }

// items: n_items pairs (sequence, first row); every item stands for rows_per_item consecutive rows of the sequence's new
// tokens (rows beyond the last are skipped): vk_attn_item_rows() for prompt items, 1 for decoded tokens.
int vk_attention_wide(elem_t* out, const elem_t* q, const elem_t* kc, const elem_t* vc, const int32_t* block_table, int bt_stride, const int32_t* cu_q,
                      const int32_t* k_len, const int32_t* items, int n_items, int rows_per_item, int nq, int nkv, int d, int P, int window, float scale,
                      const void* sinks, int sinks_f32, hipStream_t st) {
  VK_REQUIRE(nq > 0 && nkv > 0 && nq % nkv == 0 && nq <= 65535, "wide attention: %d q heads are not a multiple of %d kv heads", nq, nkv);
  VK_REQUIRE(d >= 16 && d <= WIDE_THREADS * WIDE_COLS && d % 16 == 0, "wide attention: row size %d must be a multiple of 16 in 16..%d", d,
             WIDE_THREADS * WIDE_COLS);
  VK_REQUIRE(P >= 8 && (P & (P - 1)) == 0, "wide attention: page size %d must be a power of two >= 8", P);
  VK_REQUIRE(window >= 0 && scale > 0.f && rows_per_item > 0, "wide attention: bad window %d or scale", window);
  VK_REQUIRE((int64_t)n_items * rows_per_item < (1ll << 31), "wide attention: too many items");
  if (n_items <= 0) return 0;
  WideArgs a;
  a.q = q; a.out = out; a.kc = kc; a.vc = vc; a.block_table = block_table; a.cu_q = cu_q; a.k_len = k_len; a.items = items; a.sinks = sinks;
  a.sinks_f32 = sinks_f32; a.bt_stride = bt_stride; a.nq = nq; a.nkv = nkv; a.d = d; a.P = P; a.window = window; a.rows_per_item = rows_per_item;
  a.scale = scale;
  attn_wide_kernel<<<dim3(n_items * rows_per_item, nq), WIDE_THREADS, 0, st>>>(a);
  return vk_check_launch("attention (wide rows)");
}

}  // extern "C"
