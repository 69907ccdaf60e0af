// A residual that is kept as several streams in 32-bit, read and written through learned coefficients around every
// sublayer (hyper-connections), and the embedding that opens such a stream with a norm.
//
// Around sublayer q with the coefficients a (S numbers), b (S numbers) and M (S x S, [from, to]):
//   u = sum over s of a[s] x_s;   y = sublayer(norm(u));   x_t <- sum over s of M[s, t] x_s + b[t] y   (all t at once)
// Writing one sublayer's output back and reading the next sublayer's input pass over the same streams, so they are one
// launch (vk_hyper_step): the streams are read once, mixed, written in place, their next mixture u is normed and leaves as
// elements.  At the start all streams are one row (stream stride 0); at the end vk_hyper_close adds the last output and sums
// the streams of the rows that are asked for.
//
// A workgroup takes a row; thread t owns the elements (or 16-byte vectors) t, t + 256, ... of every stream.  Sums over
// streams run in ascending order from the first product; the sum of squares has the order of this library's other norms
// over a row (a thread's elements in order, a butterfly over a wave, the four waves in order), so the result depends on
// the row alone.
#include "common.h"
#include "vec.h"

#define HYPER_THREADS 256

struct HyperArgs {
  const float* x;          // row r's stream s: x + r * x_row + s * x_stream
  int64_t x_row, x_stream; // x_stream 0: all streams are the one row
  float* x_out;            // [rows, S, W], or null: the streams stay as they are
  const void* y;           // [rows, W] the sublayer's output to write back (floats or elements), or null
  const float* back;       // that sublayer's coefficients: [a: S | b: S | M: S x S]
  const float* take;       // the next sublayer's coefficients (its a), or null: all ones
  elem_t* h;               // norm(u) * w as elements, or null
  float* u;                // u itself as floats, or null
  const void* w;
  const int32_t* rows;     // the rows to take (x and y), or null: row r is block r
  int w_is_f32, y_is_f32, W, S;
  float eps;
};

__device__ __forceinline__ float hyper_block_sum(float v, float* red) {
  v = wave_sum_xor(v);
  if ((threadIdx.x & 63) == 0) red[threadIdx.x >> 6] = v;
  __syncthreads();
  return ((red[0] + red[1]) + red[2]) + red[3];
}

// S streams of whole 16-byte vectors whose mixture fits a workgroup's registers (NV vectors a thread).
template <int S, int NV>
__global__ __launch_bounds__(HYPER_THREADS) void hyper_step_vec_kernel(HyperArgs a) {
  __shared__ float red[4];
  const int64_t src = a.rows != nullptr ? a.rows[blockIdx.x] : (int)blockIdx.x;
  const int nvec = a.W / 4;
  float take[S], out[S], mix[S][S];
#pragma unroll
  for (int s = 0; s < S; ++s) {
    take[s] = a.take != nullptr ? a.take[s] : 1.f;
    out[s] = a.y != nullptr ? a.back[S + s] : 0.f;
#pragma unroll
    for (int t = 0; t < S; ++t) mix[s][t] = a.y != nullptr ? a.back[2 * S + s * S + t] : 0.f;
  }
  const float* xr = a.x + src * a.x_row;
  f32x4 u[NV], w[NV];
  float part = 0.f;
  // The norm's weight is asked for together with the streams, so that nothing is waited for after the sum over the row.
#pragma unroll
  for (int j = 0; j < NV; ++j) {
    const int c = threadIdx.x + j * HYPER_THREADS;
    w[j] = f32x4{0.f, 0.f, 0.f, 0.f};
    if (c < nvec && a.h != nullptr) {
      if (a.w_is_f32) w[j] = *reinterpret_cast<const f32x4*>(static_cast<const float*>(a.w) + 4 * c);
      else w[j] = load_elems4(static_cast<const elem_t*>(a.w) + 4 * c);
    }
  }
#pragma unroll
  for (int j = 0; j < NV; ++j) {
    const int c = threadIdx.x + j * HYPER_THREADS;
    u[j] = f32x4{0.f, 0.f, 0.f, 0.f};
    if (c < nvec) {
      f32x4 x[S];
#pragma unroll
      for (int s = 0; s < S; ++s) x[s] = *reinterpret_cast<const f32x4*>(xr + s * a.x_stream + 4 * c);
      if (a.y != nullptr) {
        f32x4 y;
        if (a.y_is_f32) y = *reinterpret_cast<const f32x4*>(static_cast<const float*>(a.y) + src * a.W + 4 * c);
        else y = load_elems4(static_cast<const elem_t*>(a.y) + src * a.W + 4 * c);
        f32x4 n[S];
#pragma unroll
        for (int t = 0; t < S; ++t) {
#pragma unroll
          for (int e = 0; e < 4; ++e) {
            float v = mix[0][t] * x[0][e];
#pragma unroll
            for (int s = 1; s < S; ++s) v = v + mix[s][t] * x[s][e];
            n[t][e] = v + out[t] * y[e];
          }
        }
#pragma unroll
        for (int t = 0; t < S; ++t) {
          x[t] = n[t];
          if (a.x_out != nullptr) *reinterpret_cast<f32x4*>(a.x_out + ((int64_t)blockIdx.x * S + t) * a.W + 4 * c) = n[t];
        }
      }
#pragma unroll
      for (int e = 0; e < 4; ++e) {
        float v = take[0] * x[0][e];
#pragma unroll
        for (int s = 1; s < S; ++s) v = v + take[s] * x[s][e];
        u[j][e] = v;
      }
    }
    part = part + u[j].x * u[j].x;
    part = part + u[j].y * u[j].y;
    part = part + u[j].z * u[j].z;
    part = part + u[j].w * u[j].w;
  }
  if (a.u != nullptr) {
#pragma unroll
    for (int j = 0; j < NV; ++j) {
      const int c = threadIdx.x + j * HYPER_THREADS;
      if (c < nvec) *reinterpret_cast<f32x4*>(a.u + (int64_t)blockIdx.x * a.W + 4 * c) = u[j];
    }
  }
  if (a.h == nullptr) return;            // the same for the whole workgroup
  const float rr = rsqrtf(hyper_block_sum(part, red) / (float)a.W + a.eps);
#pragma unroll
  for (int j = 0; j < NV; ++j) {
    const int c = threadIdx.x + j * HYPER_THREADS;
    if (c < nvec) {
      f32x4 h;
#pragma unroll
      for (int e = 0; e < 4; ++e) h[e] = (u[j][e] * rr) * w[j][e];
      store_elems4(a.h + (int64_t)blockIdx.x * a.W + 4 * c, h);
    }
  }
}

// Any width and any number of streams.  x_out must not be x.  The mixture is computed a second time for the norm's output
// rather than kept.
__global__ __launch_bounds__(HYPER_THREADS) void hyper_step_kernel(HyperArgs a) {
  __shared__ float red[4];
  const int64_t src = a.rows != nullptr ? a.rows[blockIdx.x] : (int)blockIdx.x;
  const float* xr = a.x + src * a.x_row;
  // u at column c, the new streams stored on the way if `store` says so.
  auto mixture = [&](int c, bool store) {
    float y = 0.f;
    if (a.y != nullptr) y = a.y_is_f32 ? static_cast<const float*>(a.y)[src * a.W + c] : to_f32(static_cast<const elem_t*>(a.y)[src * a.W + c]);
    float u = 0.f;
    for (int t = 0; t < a.S; ++t) {
      float v;
      if (a.y != nullptr) {
        v = a.back[2 * a.S + t] * xr[c];
        for (int s = 1; s < a.S; ++s) v = v + a.back[2 * a.S + s * a.S + t] * xr[s * a.x_stream + c];
        v = v + a.back[a.S + t] * y;
        if (store && a.x_out != nullptr) a.x_out[((int64_t)blockIdx.x * a.S + t) * a.W + c] = v;
      } else {
        v = xr[t * a.x_stream + c];
      }
      const float p = (a.take != nullptr ? a.take[t] : 1.f) * v;
      u = t == 0 ? p : u + p;
    }
    return u;
  };
  float part = 0.f;
  for (int c = threadIdx.x; c < a.W; c += HYPER_THREADS) {
    const float u = mixture(c, true);
    part = part + u * u;
    if (a.u != nullptr) a.u[(int64_t)blockIdx.x * a.W + c] = u;
  }
  if (a.h == nullptr) return;            // the same for the whole workgroup
  const float rr = rsqrtf(hyper_block_sum(part, red) / (float)a.W + a.eps);
  for (int c = threadIdx.x; c < a.W; c += HYPER_THREADS)
    a.h[(int64_t)blockIdx.x * a.W + c] = from_f32<elem_t>((mixture(c, false) * rr) * load_weight(a.w, a.w_is_f32, c));
}

// out[t, :] = table[ids[t], :] / sqrt(mean(.^2) + eps) * w, as floats: a residual stream that starts with a normed embedding.
__global__ __launch_bounds__(HYPER_THREADS) void embed_normed_kernel(float* __restrict__ out, const elem_t* __restrict__ table,
                                                                     const int32_t* __restrict__ ids, const void* __restrict__ w, int w_is_f32,
                                                                     int W, float eps) {
  __shared__ float red[4];
  const elem_t* src = table + (int64_t)ids[blockIdx.x] * W;
  // Four elements a thread at a time where the rows are whole vectors (the table lies at a 16-byte address).
  const int nvec = W % 4 == 0 && ((uintptr_t)table % 16) == 0 && ((uintptr_t)out % 16) == 0 ? W / 4 : 0;
  float part = 0.f;
#pragma unroll 4
  for (int c = threadIdx.x; c < nvec; c += HYPER_THREADS) {
    const f32x4 v = load_elems4(src + 4 * c);
    part = part + v.x * v.x;
    part = part + v.y * v.y;
    part = part + v.z * v.z;
    part = part + v.w * v.w;
  }
  for (int c = 4 * nvec + threadIdx.x; c < W; c += HYPER_THREADS) {
    const float v = to_f32(src[c]);
    part = part + v * v;
  }
  const float rr = rsqrtf(hyper_block_sum(part, red) / (float)W + eps);
  float* dst = out + (int64_t)blockIdx.x * W;
#pragma unroll 4
  for (int c = threadIdx.x; c < nvec; c += HYPER_THREADS) {
    f32x4 v = load_elems4(src + 4 * c);
#pragma unroll
    for (int e = 0; e < 4; ++e) v[e] = (v[e] * rr) * load_weight(w, w_is_f32, 4 * c + e);
    *reinterpret_cast<f32x4*>(dst + 4 * c) = v;
  }
  for (int c = 4 * nvec + threadIdx.x; c < W; c += HYPER_THREADS) dst[c] = (to_f32(src[c]) * rr) * load_weight(w, w_is_f32, c);
}

static bool aligned16(const void* p) { return ((uintptr_t)p % 16) == 0; }

// Whether vk_hyper_step may write the new streams over the old ones for these sizes.
static bool hyper_vec_takes(int W, int S) { return W % 4 == 0 && W / 4 <= 8 * HYPER_THREADS && S >= 1 && S <= 4; }

static int hyper_launch(const HyperArgs& a, int rows, hipStream_t st) {
  const bool vec = hyper_vec_takes(a.W, a.S) && a.x_row % 4 == 0 && a.x_stream % 4 == 0 && aligned16(a.x) && aligned16(a.x_out) && aligned16(a.u) &&
                   aligned16(a.y) && aligned16(a.w) && aligned16(a.h);
  if (vec) {
    const int nv = (a.W / 4 + HYPER_THREADS - 1) / HYPER_THREADS;
#define HYPER_VEC(S, NV) hyper_step_vec_kernel<S, NV><<<rows, HYPER_THREADS, 0, st>>>(a)
#define HYPER_NV(S) do { if (nv <= 1) HYPER_VEC(S, 1); else if (nv <= 2) HYPER_VEC(S, 2); else if (nv <= 4) HYPER_VEC(S, 4); else HYPER_VEC(S, 8); } while (0)
    if (a.S == 1) HYPER_NV(1); else if (a.S == 2) HYPER_NV(2); else if (a.S == 3) HYPER_NV(3); else HYPER_NV(4);
#undef HYPER_NV
#undef HYPER_VEC
  } else {
    VK_REQUIRE(a.x_out != a.x, "hyper-connections: these sizes (width %d, %d streams) cannot be mixed in place", a.W, a.S);
    hyper_step_kernel<<<rows, HYPER_THREADS, 0, st>>>(a);
  }
  return vk_check_launch("hyper-connections");
}

extern "C" {

int vk_hyper_in_place(int W, int S) { return hyper_vec_takes(W, S) ? 1 : 0; }

// Writes a sublayer's output y [T, W] back (y null: nothing to write back) and reads the next sublayer's input.
// x: [T, S, W] floats, or (one_row) [T, W]: all streams are that row.  x_out [T, S, W] receives the new streams (null if y
// is null; it may be x where vk_hyper_in_place says so).  back / take: floats [a: S | b: S | M: S * S] of the sublayer that
// gave y and of the next one.  h [T, W] elements: norm(u) * w; without w (null) u [T, W] floats receives u.
int vk_hyper_step(const float* x, int one_row, float* x_out, const void* y, int y_is_f32, const float* back, const float* take, elem_t* h, float* u,
                  const void* w, int w_is_f32, float eps, int T, int W, int S, hipStream_t st) {
  VK_REQUIRE(T >= 0 && W > 0 && S > 0 && S <= 64 && eps >= 0.f && x != nullptr && take != nullptr, "hyper-connections: bad sizes T=%d W=%d S=%d", T, W, S);
  VK_REQUIRE((y == nullptr) == (x_out == nullptr) && (y == nullptr || back != nullptr), "hyper-connections: an output needs its coefficients and new streams");
  VK_REQUIRE((h != nullptr) == (w != nullptr) && (h != nullptr || u != nullptr), "hyper-connections: the next input has no memory");
  VK_REQUIRE(!one_row || x_out != x || S == 1, "hyper-connections: several streams do not fit the one row they start from");
  if (T == 0) return 0;
  HyperArgs a;
  a.x = x; a.x_row = one_row ? W : (int64_t)S * W; a.x_stream = one_row ? 0 : W; a.x_out = x_out; a.y = y; a.y_is_f32 = y_is_f32;
  a.back = back; a.take = take; a.h = h; a.u = u; a.w = w; a.w_is_f32 = w_is_f32; a.eps = eps; a.rows = nullptr; a.W = W; a.S = S;
  return hyper_launch(a, T, st);
}

// out [R, W] floats: the sum of the streams of the rows that `rows` names, after the last sublayer's output (y null: there
// is none).  Row numbers must lie below the streams': the caller checks them on the host.
int vk_hyper_close(float* out, const float* x, int one_row, const void* y, int y_is_f32, const float* back, const int32_t* rows, int R, int W, int S,
                   hipStream_t st) {
  VK_REQUIRE(R >= 0 && W > 0 && S > 0 && S <= 64 && out != nullptr && x != nullptr && rows != nullptr && (y == nullptr || back != nullptr),
             "hyper-connections (sum of the streams): bad sizes R=%d W=%d S=%d", R, W, S);
  if (R == 0) return 0;
  HyperArgs a;
  a.x = x; a.x_row = one_row ? W : (int64_t)S * W; a.x_stream = one_row ? 0 : W; a.x_out = nullptr; a.y = y; a.y_is_f32 = y_is_f32;
  a.back = back; a.take = nullptr; a.h = nullptr; a.u = out; a.w = nullptr; a.w_is_f32 = 0; a.eps = 0.f; a.rows = rows; a.W = W; a.S = S;
  return hyper_launch(a, R, st);
}

// ids must lie below V: the caller checks them on the host.
int vk_embed_normed(float* out, const elem_t* table, const int32_t* ids, const void* w, int w_is_f32, int T, int W, int V, float eps, hipStream_t st) {
  VK_REQUIRE(T >= 0 && W > 0 && V > 0 && eps >= 0.f && w != nullptr, "normed embedding: bad sizes T=%d W=%d V=%d", T, W, V);
  if (T == 0) return 0;
  embed_normed_kernel<<<T, HYPER_THREADS, 0, st>>>(out, table, ids, w, w_is_f32, W, eps);
  return vk_check_launch("normed embedding");
}

}  // extern "C"
