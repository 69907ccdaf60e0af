// What stands between the projections of q, k and v and attention, for designs that qkv_post.hip does not cover: norms of q and k
// in three kinds, a rotation, values blended with an earlier layer's, and the write of k and v into their pages, in one launch.
//
// For every token, with nq q heads, nkv k heads and nkv v heads of `size` entries (in rows of d >= size, zero beyond):
//   norm 1  every q and k head  <- x / sqrt(mean(x^2) + eps) * w, a weight [size] for all heads, before the rotation
//   norm 2  every q and k head  <- x / sqrt(mean(x^2) + eps), after the rotation
//   norm 3  all q heads' entries together <- x / sqrt(mean(x^2) + eps) * w, a weight [nq * size] (k alike), before the rotation
//   turn    pair c of a head's first 2 rot_half entries (c and c + rot_half) by position * inv_freq[c]
//   blend   v <- (1 - share) v + share v0, v0 the entries that an earlier layer projected for the same token
// all in 32-bit; a q, k or v entry is rounded to the element type once, where it is stored.
//
// A lane owns 16 bytes of a row, LPH lanes (a power of two, the last ones idle for sizes that are none) a head, a wave
// 64 / LPH heads.  A sum of squares runs over a lane's entries in order and then as a butterfly over the head's lanes (norm 3:
// over the workgroup, each thread its vectors in steps of the workgroup's size, a butterfly, the four waves in order), so its
// order depends on the sizes alone.
#include "common.h"
#include "vec.h"

#define PREP_THREADS 256
#define PREP_MAX_HALF 128

struct PrepareArgs {
  const elem_t* x;          // [T, row]: nq q heads, nkv k heads, nkv v heads, d each
  int64_t row;
  elem_t* q_out;            // [T, nq, d]
  elem_t *kc, *vc;          // [pages, nkv, P, d], [pages, nkv, d, P]
  const void *q_w, *k_w;    // norms 1 and 3
  const float* inv_freq;    // [rot_half] or null
  const int32_t *positions, *slots;
  const elem_t* v0;         // [T, v0_row]: v0's heads of v0_d entries, of which v0_size count; or null
  int64_t v0_row;
  const void* share;        // [1]
  int w_is_f32, share_is_f32, norm, nq, nkv, d, size, vsize, P, rot_half, v0_d, v0_size;
  float eps;
};

template <int LPH>
__global__ __launch_bounds__(PREP_THREADS) void qkv_prepare_kernel(PrepareArgs a, int per_wave) {
  constexpr int HPW = 64 / LPH;
  __shared__ float cs[PREP_MAX_HALF], sn[PREP_MAX_HALF];
  __shared__ float red[2][4];
  __shared__ float rows[4][64 * VK_VEC];         // a wave's heads while they turn
  const int tok = blockIdx.x, lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
  const int d = a.d, heads = a.nq + 2 * a.nkv, vecs = d / VK_VEC, rh = a.rot_half;
  const elem_t* xrow = a.x + tok * a.row;
  if (a.inv_freq != nullptr) {
    const float p = (float)a.positions[tok];
    for (int c = threadIdx.x; c < rh; c += PREP_THREADS) {
      const float angle = p * a.inv_freq[c];
      cs[c] = cosf(angle);
      sn[c] = sinf(angle);
    }
  }
  float whole[2] = {0.f, 0.f};                   // norm 3: 1 / root mean square of q and of k
  if (a.norm == 3) {
    float part[2];
#pragma unroll
    for (int s = 0; s < 2; ++s) {
      part[s] = 0.f;
      const int n = (s == 0 ? a.nq : a.nkv) * vecs, first = s == 0 ? 0 : a.nq * vecs;
      for (int i = threadIdx.x; i < n; i += PREP_THREADS) {
        float v[VK_VEC];
        load_elems(xrow + (int64_t)(first + i) * VK_VEC, v);
#pragma unroll
        for (int e = 0; e < VK_VEC; ++e) part[s] = part[s] + v[e] * v[e];
      }
      part[s] = wave_sum_xor(part[s]);
      if (lane == 0) red[s][wave] = part[s];
    }
    __syncthreads();
#pragma unroll
    for (int s = 0; s < 2; ++s) {
      float t = red[s][0];
      t = t + red[s][1];
      t = t + red[s][2];
      t = t + red[s][3];
      whole[s] = rsqrtf(t / (float)((s == 0 ? a.nq : a.nkv) * a.size) + a.eps);
    }
  } else if (a.inv_freq != nullptr) {
    __syncthreads();
  }
  const int slot = a.slots[tok];
  const int page = slot >= 0 ? slot / a.P : 0, off = slot >= 0 ? slot - page * a.P : 0;
  const float share = a.v0 != nullptr ? load_weight(a.share, a.share_is_f32, 0) : 0.f;
  const int j = lane % LPH, hsub = lane / LPH, c0 = j * VK_VEC;
  const bool inside = j < vecs;
  for (int it = 0; it < per_wave; ++it) {
    const int hh = ((blockIdx.y * per_wave + it) * 4 + wave) * HPW + hsub;
    const bool live = hh < heads && inside;
    const int kind = hh < a.nq ? 0 : (hh < a.nq + a.nkv ? 1 : 2);   // q, k, v
    const int head = kind == 0 ? hh : (kind == 1 ? hh - a.nq : hh - a.nq - a.nkv);
    float v[VK_VEC];
#pragma unroll
    for (int e = 0; e < VK_VEC; ++e) v[e] = 0.f;
    if (live) load_elems(xrow + (int64_t)hh * d + c0, v);
    if (a.norm == 1 || a.norm == 3) {
      float rr = whole[kind & 1];
      if (a.norm == 1) {
        float part = 0.f;
#pragma unroll
        for (int e = 0; e < VK_VEC; ++e) part = part + v[e] * v[e];
#pragma unroll
        for (int m = 1; m < LPH; m <<= 1) part = part + __shfl_xor(part, m, VK_WAVE);
        rr = rsqrtf(part / (float)a.size + a.eps);
      }
      if (live && kind != 2) {
        const void* w = kind == 0 ? a.q_w : a.k_w;
        const int w0 = a.norm == 1 ? c0 : head * a.size + c0;
#pragma unroll
        for (int e = 0; e < VK_VEC; ++e)
          if (c0 + e < a.size) v[e] = (v[e] * rr) * load_weight(w, a.w_is_f32, w0 + e);
      }
    }
    if (a.inv_freq != nullptr) {
      // A head's row goes through LDS; the lanes of a wave read what the same wave wrote.
      float* y = rows[wave] + hsub * LPH * VK_VEC;
#pragma unroll
      for (int e = 0; e < VK_VEC; ++e) y[c0 + e] = v[e];
      __builtin_amdgcn_fence(__ATOMIC_ACQ_REL, "wavefront");
      __builtin_amdgcn_wave_barrier();
      if (live && kind != 2) {
#pragma unroll
        for (int e = 0; e < VK_VEC; ++e) {
          const int c = c0 + e;
          if (c < rh) v[e] = v[e] * cs[c] - y[c + rh] * sn[c];
          else if (c < 2 * rh) v[e] = v[e] * cs[c - rh] + y[c - rh] * sn[c - rh];
        }
      }
      __builtin_amdgcn_fence(__ATOMIC_ACQ_REL, "wavefront");
      __builtin_amdgcn_wave_barrier();                              // y is free for the next heads
    }
    if (a.norm == 2) {
      float part = 0.f;
#pragma unroll
      for (int e = 0; e < VK_VEC; ++e) part = part + v[e] * v[e];
#pragma unroll
      for (int m = 1; m < LPH; m <<= 1) part = part + __shfl_xor(part, m, VK_WAVE);
      const float rr = rsqrtf(part / (float)a.size + a.eps);
      if (kind != 2) {
#pragma unroll
        for (int e = 0; e < VK_VEC; ++e) v[e] = v[e] * rr;
      }
    }
    if (!live) continue;
    if (kind == 2 && a.v0 != nullptr) {
      const elem_t* first = a.v0 + tok * a.v0_row;
      float u[VK_VEC];
      if (a.v0_size == a.vsize && a.v0_size % VK_VEC == 0) {
#pragma unroll
        for (int e = 0; e < VK_VEC; ++e) u[e] = 0.f;
        if (c0 < a.vsize) load_elems(first + (int64_t)head * a.v0_d + c0, u);
      } else {
#pragma unroll
        for (int e = 0; e < VK_VEC; ++e) {
          const int entry = head * a.vsize + c0 + e;                // its place among all heads' entries side by side
          u[e] = c0 + e < a.vsize ? to_f32(first[(int64_t)(entry / a.v0_size) * a.v0_d + entry % a.v0_size]) : 0.f;
        }
      }
#pragma unroll
      for (int e = 0; e < VK_VEC; ++e) v[e] = (1.f - share) * v[e] + share * u[e];
    }
    if (kind == 0) {
      store_elems(a.q_out + ((int64_t)tok * a.nq + head) * d + c0, v);
    } else if (slot >= 0) {
      if (kind == 1) {
        store_elems(a.kc + (((int64_t)page * a.nkv + head) * a.P + off) * d + c0, v);
      } else {
        elem_t* o = a.vc + (((int64_t)page * a.nkv + head) * d + c0) * a.P + off;
#pragma unroll
        for (int e = 0; e < VK_VEC; ++e) o[(int64_t)e * a.P] = from_f32<elem_t>(v[e]);
      }
    }
  }
}

extern "C" {

// x [T, row] with (nq + 2 nkv) heads of d from column 0.  norm: 0 none, 1, 2, 3 as above; size: the q and k heads' own entries,
// vsize: the v heads'.  inv_freq null: no rotation.  v0 null: no blend.  Slots (-1: nothing is stored) must lie inside the cache
// and positions be what the angles are meant for; the caller checks both on the host.
int vk_qkv_prepare(const elem_t* x, int64_t row, elem_t* q_out, elem_t* kc, elem_t* vc, int norm, const void* q_w, const void* k_w, int w_is_f32, int size,
                   int vsize, float eps, const float* inv_freq, int rot_half, const int32_t* positions, const int32_t* slots, const elem_t* v0,
                   int64_t v0_row, int v0_d, int v0_size, const void* share, int share_is_f32, int T, int nq, int nkv, int d, int P, hipStream_t st) {
  VK_REQUIRE(T >= 0 && nq > 0 && nkv > 0 && nq + 2 * nkv <= 65535, "qkv_prepare: bad sizes T=%d nq=%d nkv=%d", T, nq, nkv);
  VK_REQUIRE(d >= 16 && d <= 256 && d % 16 == 0 && size > 0 && size <= d && vsize > 0 && vsize <= d,
             "qkv_prepare: heads of %d and %d entries in rows of %d (multiples of 16, 16..256)", size, vsize, d);
  VK_REQUIRE(row >= (int64_t)(nq + 2 * nkv) * d && row % VK_VEC == 0, "qkv_prepare: row stride %lld", (long long)row);
  VK_REQUIRE(norm >= 0 && norm <= 3 && eps >= 0.f, "qkv_prepare: norm kind %d", norm);
  VK_REQUIRE((norm != 1 && norm != 3) || (q_w != nullptr && k_w != nullptr), "qkv_prepare: the norms' weights are missing");
  VK_REQUIRE(inv_freq == nullptr || (rot_half > 0 && 2 * rot_half <= size && rot_half <= PREP_MAX_HALF && positions != nullptr),
             "qkv_prepare: a rotation of %d entries of %d", 2 * rot_half, size);
  VK_REQUIRE(q_out != nullptr && kc != nullptr && vc != nullptr && slots != nullptr && P > 0, "qkv_prepare: caches and slots are missing");
  VK_REQUIRE(v0 == nullptr || (share != nullptr && v0_size > 0 && v0_size <= v0_d && v0_d % VK_VEC == 0 && (nkv * vsize) % v0_size == 0 &&
                               (int64_t)(nkv * vsize / v0_size) * v0_d <= v0_row && v0_row % VK_VEC == 0),
             "qkv_prepare: %d values a token cannot be blended with heads of %d", nkv * vsize, v0_size);
  VK_REQUIRE(((uintptr_t)x % 16) == 0 && ((uintptr_t)q_out % 16) == 0 && ((uintptr_t)kc % 16) == 0 && ((uintptr_t)v0 % 16) == 0,
             "qkv_prepare: operands must be 16-byte aligned");
  if (T == 0) return 0;
  PrepareArgs a;
  a.x = x; a.row = row; a.q_out = q_out; a.kc = kc; a.vc = vc; a.q_w = q_w; a.k_w = k_w; a.inv_freq = inv_freq; a.positions = positions; a.slots = slots;
  a.v0 = v0; a.v0_row = v0_row; a.share = share; a.w_is_f32 = w_is_f32; a.share_is_f32 = share_is_f32; a.norm = norm; a.nq = nq; a.nkv = nkv; a.d = d;
  a.size = size; a.vsize = vsize; a.P = P; a.rot_half = inv_freq != nullptr ? rot_half : 0; a.v0_d = v0_d; a.v0_size = v0_size; a.eps = eps;
  const int vecs = d / VK_VEC, heads = nq + 2 * nkv;
  int lph = 4;
  while (lph < vecs) lph *= 2;
  // Few tokens: a workgroup for every round of heads; many: all heads of a token in one.
  const int per_wg = 4 * (64 / lph);
  const int per_wave = T >= 512 ? (heads + per_wg - 1) / per_wg : 1;
  const dim3 grid(T, (heads + per_wg * per_wave - 1) / (per_wg * per_wave));
  if (lph == 4) qkv_prepare_kernel<4><<<grid, PREP_THREADS, 0, st>>>(a, per_wave);
  else if (lph == 8) qkv_prepare_kernel<8><<<grid, PREP_THREADS, 0, st>>>(a, per_wave);
  else if (lph == 16) qkv_prepare_kernel<16><<<grid, PREP_THREADS, 0, st>>>(a, per_wave);
  else if (lph == 32) qkv_prepare_kernel<32><<<grid, PREP_THREADS, 0, st>>>(a, per_wave);
  else qkv_prepare_kernel<64><<<grid, PREP_THREADS, 0, st>>>(a, per_wave);
  return vk_check_launch("qkv_prepare");
}

}  // extern "C"
