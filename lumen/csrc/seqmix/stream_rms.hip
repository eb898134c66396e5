// The fp32 residual stream of a pre-norm stack, with whatever joins it, and the next sublayer's
// input, in one pass over a row:
//
//   sm_stream_rms   x' = [x] + [table[token] * scale] + [y] + [f0] + [f1] + coef * [f2]   (given parts)
//                   then, of the new row,
//                     h = x' / sqrt(mean(x'^2) + eps) * w   in the compute dtype   (w given)
//                     or its two 16-bit parts hi = round(x'), lo = round(x' - hi)   (split): a
//                     GEMM over both keeps about 16 bits of the stream's mantissa
//                     or nothing but x' itself
//                 x, f0, f1, f2 are fp32; y and the embedding table are in the compute dtype.  With
//                 `rows` the token's table row is also copied out as it is (a GEMM's operand).
//
// One workgroup per row, four channels per lane; the new row stays in LDS between the sum of squares
// and the output.
#include "seqmix.h"

using namespace lumen;

namespace {

constexpr int kThreads = 256;

template <typename T>
struct StreamArgs {
  float* x; int keep;                                   // keep: x is one of the addends
  const T* table; const long long* tokens; int vocab; float scale; T* rows;
  const T* y;
  const float* f0; const float* f1; const float* f2; float coef;
  const float* w; T* h; int split;
  long long lo;                                         // split: offset of the low parts in h
  int W; float eps;
};

template <typename T, int V>
__device__ __forceinline__ void load_n(const T* p, float (&o)[V]) {
  if constexpr (V == 4) load4<T>(p, o);
  else o[0] = to_f32(p[0]);
}
template <typename T, int V>
__device__ __forceinline__ void store_n(T* p, const float (&o)[V]) {
  if constexpr (V == 4) store4<T>(p, o);
  else p[0] = from_f32<T>(o[0]);
}
template <typename T, int V>
__device__ __forceinline__ void add_n(const T* p, float k, float (&o)[V]) {
  float v[V];
  load_n<T, V>(p, v);
#pragma unroll
  for (int e = 0; e < V; ++e) o[e] += k * v[e];
}

template <typename T, int V>
__global__ void __launch_bounds__(kThreads) stream_rms_kernel(const StreamArgs<T> a) {
  extern __shared__ float s_row[];
  __shared__ float s_red[kThreads / 64];
  const int W = a.W;
  const long long base = (long long)blockIdx.x * W;
  const T* er = nullptr;
  if (a.table != nullptr) {
    long long tok = a.tokens[blockIdx.x];
    tok = tok < 0 ? 0 : (tok >= a.vocab ? a.vocab - 1 : tok);
    er = a.table + tok * W;
  }
  float sq = 0.f;
  for (int c = threadIdx.x * V; c < W; c += kThreads * V) {
    float v[V];
    if (a.keep) load_n<float, V>(a.x + base + c, v);
    else {
#pragma unroll
      for (int e = 0; e < V; ++e) v[e] = 0.f;
    }
    if (er != nullptr) {
      float ev[V];
      load_n<T, V>(er + c, ev);
      if (a.rows != nullptr) store_n<T, V>(a.rows + base + c, ev);      // exact: the table's own values
#pragma unroll
      for (int e = 0; e < V; ++e) v[e] += a.scale * ev[e];
    }
    if (a.y != nullptr) add_n<T, V>(a.y + base + c, 1.f, v);
    if (a.f0 != nullptr) add_n<float, V>(a.f0 + base + c, 1.f, v);
    if (a.f1 != nullptr) add_n<float, V>(a.f1 + base + c, 1.f, v);
    if (a.f2 != nullptr) add_n<float, V>(a.f2 + base + c, a.coef, v);
    store_n<float, V>(a.x + base + c, v);
    if (a.w != nullptr) {
#pragma unroll
      for (int e = 0; e < V; ++e) sq += v[e] * v[e];
      store_n<float, V>(s_row + c, v);
    } else if (a.split) {
      float lo[V];
#pragma unroll
      for (int e = 0; e < V; ++e) {
        const float hi = to_f32(from_f32<T>(v[e]));
        lo[e] = v[e] - hi;
        v[e] = hi;
      }
      store_n<T, V>(a.h + base + c, v);
      store_n<T, V>(a.h + a.lo + base + c, lo);
    }
  }
  if (a.w == nullptr) return;
  const float inv = 1.f / sqrtf(block_sum<kThreads>(sq, s_red) / (float)W + a.eps);
  for (int c = threadIdx.x * V; c < W; c += kThreads * V) {      // a thread re-reads its own entries
    float v[V], ww[V];
    load_n<float, V>(s_row + c, v);
    load_n<float, V>(a.w + c, ww);
#pragma unroll
    for (int e = 0; e < V; ++e) v[e] = v[e] * inv * ww[e];
    store_n<T, V>(a.h + base + c, v);
  }
}

}  // namespace

extern "C" {

// x fp32 [rows][W] (written; read with keep).  h [rows][W], or with split [2 rows][W]: the high parts
// of all rows, then the low parts.
hipError_t sm_stream_rms(int dt, float* x, int keep, const void* table, const long long* tokens,
                         int vocab, float scale, void* table_rows, const void* y, const float* f0,
                         const float* f1, const float* f2, float coef, const float* w, void* h,
                         int split, int rows, int W, float eps, hipStream_t st) {
  if (rows == 0) return hipSuccess;
  if (W < 1 || (w && (size_t)W * sizeof(float) > 65536 - 64)) return hipErrorInvalidValue;
  if (!x || (table && (!tokens || vocab < 1)) || (table_rows && !table) || (w && split) ||
      ((w || split) && !h))
    return hipErrorInvalidValue;
  const auto al = [](const void* p) { return (uintptr_t)p % 16 == 0; };
  const bool vec = W % 4 == 0 && al(x) && al(table) && al(table_rows) && al(y) && al(f0) &&
                   al(f1) && al(f2) && al(w) && al(h);
  const size_t lds = w != nullptr ? (size_t)W * sizeof(float) : 0;
#define CALL(T)                                                                                   \
  {                                                                                               \
    StreamArgs<T> a{x, keep, (const T*)table, tokens, vocab, scale, (T*)table_rows, (const T*)y,  \
                    f0, f1, f2, coef, w, (T*)h, split, (long long)rows * W, W, eps};              \
    if (vec) stream_rms_kernel<T, 4><<<rows, kThreads, lds, st>>>(a);                             \
    else stream_rms_kernel<T, 1><<<rows, kThreads, lds, st>>>(a);                                 \
  }
  SM_DISPATCH(dt, CALL)
#undef CALL
  return hipGetLastError();
}

}  // extern "C"
