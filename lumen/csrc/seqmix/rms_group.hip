// RMS norms in groups, fused with what surrounds them:
//   sm_group_rms   v = x / sqrt(mean_g(x^2) + eps) * w, the row split into `groups` equal
//                  consecutive parts that are each divided by their OWN root mean square
//                  (groups = 1: the ordinary RMS norm).  Without a residual the result is stored
//                  in the output dtype; with one, the fp32 residual row takes it in place,
//                  res += v, and -- optionally -- the new row is also stored rounded to the model
//                  dtype (the input of the next sublayer's GEMMs).
//   sm_gate_rows   out[t, d] = gelu_tanh(z[t, d]) * table[token[t], col0 + d]: a slice of a
//                  per-token embedding row gated by a projection of the stream.
//   sm_gated_rms   the read-out of a recurrence: the fp32 row, its group RMS norm and a gate from the
//                  layer's projection, stored in the model dtype.  The gate multiplies before the
//                  norm (x * act(g), then normed, times w) or after it (normed, times w, times
//                  act(g)); act is SiLU or the sigmoid; w is one weight per channel or one per
//                  group entry shared by the groups.
// One workgroup of four waves per row.  With four or more groups a wave owns a group (and walks
// the groups four at a time); with fewer, 4 / groups waves share one and add their partial sums in
// a fixed order, so the result never depends on timing.  Sums, roots and products are fp32.
#include "seqmix.h"

using namespace lumen;

namespace {

template <typename TI, typename TO, bool VEC>
__global__ void __launch_bounds__(256)
group_rms_kernel(const TI* __restrict__ x, long long ldx, const float* __restrict__ w,
                 float* __restrict__ res, TO* __restrict__ out, long long ldo, int W, int groups,
                 float eps) {
  const int r = blockIdx.x, lane = threadIdx.x & 63, wv = threadIdx.x >> 6;
  const int gs = W / groups;
  const int wpg = groups >= 4 ? 1 : groups == 1 ? 4 : groups == 2 ? 2 : 1;   // waves per group
  const int per_pass = 4 / wpg;
  const int slot = wv / wpg, sub = wv % wpg;
  const TI* xr = x + (long long)r * ldx;
  __shared__ float s_part[4];
  constexpr int V = VEC ? 4 : 1;
  for (int g0 = 0; g0 < groups; g0 += per_pass) {
    const int g = g0 + slot;
    const bool on = g < groups && slot < per_pass;
    float ss = 0.f;
    if (on) {
      for (int c = (sub * 64 + lane) * V; c < gs; c += wpg * 64 * V) {
        if (VEC) {
          float v[4];
          load4<TI>(xr + g * gs + c, v);
          ss += v[0] * v[0] + v[1] * v[1] + v[2] * v[2] + v[3] * v[3];
        } else {
          const float v = to_f32(xr[g * gs + c]);
          ss += v * v;
        }
      }
    }
    ss = wave_sum(ss);
    if (lane == 0) s_part[wv] = ss;
    __syncthreads();
    if (on) {
      float tot = 0.f;
      for (int k = 0; k < wpg; ++k) tot += s_part[slot * wpg + k];
      const float inv = 1.f / sqrtf(tot / (float)gs + eps);
      for (int c = (sub * 64 + lane) * V; c < gs; c += wpg * 64 * V) {
        const int col = g * gs + c;
        if (VEC) {
          float v[4], ww[4];
          load4<TI>(xr + col, v);
          load4<float>(w + col, ww);
#pragma unroll
          for (int e = 0; e < 4; ++e) v[e] = v[e] * inv * ww[e];
          if (res) {
            float a[4];
            load4<float>(res + (long long)r * W + col, a);
#pragma unroll
            for (int e = 0; e < 4; ++e) v[e] += a[e];
            store4<float>(res + (long long)r * W + col, v);
          }
          if (out) store4<TO>(out + (long long)r * ldo + col, v);
        } else {
          float v = to_f32(xr[col]) * inv * w[col];
          if (res) {
            v += res[(long long)r * W + col];
            res[(long long)r * W + col] = v;
          }
          if (out) out[(long long)r * ldo + col] = from_f32<TO>(v);
        }
      }
    }
    __syncthreads();
  }
}

// four or more groups: a wave per group, blockIdx.y naming the four a workgroup takes; fewer: one
// workgroup per row as above.  The entries (gated, when the gate comes first) stay in LDS between the
// two passes.
template <typename T, bool VEC>
__global__ void __launch_bounds__(256)
gated_rms_kernel(const float* __restrict__ x, const T* __restrict__ g, long long ldg,
                 const float* __restrict__ w, T* __restrict__ out, int W, int groups, int shared_w,
                 int gate_first, int sigmoid, float eps) {
  extern __shared__ float s_row[];
  __shared__ float s_part[4];
  const int r = blockIdx.x, lane = threadIdx.x & 63, wv = threadIdx.x >> 6;
  const int gs = W / groups;
  const int wpg = groups >= 4 ? 1 : groups == 1 ? 4 : groups == 2 ? 2 : 1;   // waves per group
  const int per_pass = 4 / wpg;
  const int slot = wv / wpg, sub = wv % wpg;
  const float* xr = x + (long long)r * W;
  const T* gr = g + (long long)r * ldg;
  T* orow = out + (long long)r * W;
  constexpr int V = VEC ? 4 : 1;
  const int gi = blockIdx.y * per_pass + slot;
  const bool on = gi < groups && slot < per_pass;
  float ss = 0.f;
  if (on) {
    for (int c = (sub * 64 + lane) * V; c < gs; c += wpg * 64 * V) {
      const int col = gi * gs + c;
      float v[V], z[V];
      if constexpr (VEC) load4<float>(xr + col, v);
      else v[0] = xr[col];
      if (gate_first) {
        if constexpr (VEC) load4<T>(gr + col, z);
        else z[0] = to_f32(gr[col]);
#pragma unroll
        for (int e = 0; e < V; ++e) v[e] *= sigmoid ? sigmoid_f(z[e]) : silu_f(z[e]);
      }
#pragma unroll
      for (int e = 0; e < V; ++e) {
        ss += v[e] * v[e];
        s_row[slot * gs + c + e] = v[e];
      }
    }
  }
  float tot = wave_sum(ss);
  if (wpg > 1) {                             // (uniform) waves sharing a group exchange their sums
    if (lane == 0) s_part[wv] = tot;
    __syncthreads();
    tot = 0.f;
    for (int k = 0; k < wpg; ++k) tot += s_part[slot * wpg + k];
  }
  if (on) {
    const float inv = 1.f / sqrtf(tot / (float)gs + eps);
    for (int c = (sub * 64 + lane) * V; c < gs; c += wpg * 64 * V) {   // its own entries again
      const int col = gi * gs + c;
      const float* wp = w + (shared_w ? c : col);
      float v[V], z[V];
#pragma unroll
      for (int e = 0; e < V; ++e) v[e] = s_row[slot * gs + c + e] * inv * wp[e];
      if (!gate_first) {
        if constexpr (VEC) load4<T>(gr + col, z);
        else z[0] = to_f32(gr[col]);
#pragma unroll
        for (int e = 0; e < V; ++e) v[e] *= sigmoid ? sigmoid_f(z[e]) : silu_f(z[e]);
      }
      if constexpr (VEC) store4<T>(orow + col, v);
      else orow[col] = from_f32<T>(v[0]);
    }
  }
}

// groups of at most 256 entries (heads): SG lanes of 4 entries each own a (row, group), in registers
template <typename T>
__global__ void __launch_bounds__(256)
gated_rms_small_kernel(const float* __restrict__ x, const T* __restrict__ g, long long ldg,
                       const float* __restrict__ w, T* __restrict__ out, int W, int groups, int gs,
                       int SG, long long items, int shared_w, int gate_first, int sigmoid,
                       float eps) {
  const long long item = (blockIdx.x * 256ll + threadIdx.x) / SG;
  const int c = 4 * (threadIdx.x & (SG - 1));
  const bool on = item < items && c < gs;
  const long long r = on ? item / groups : 0;
  const int col = on ? (int)(item - r * groups) * gs + c : 0;
  float v[4] = {0.f, 0.f, 0.f, 0.f}, z[4] = {0.f, 0.f, 0.f, 0.f};
  if (on) {
    load4<float>(x + r * W + col, v);
    load4<T>(g + r * ldg + col, z);
  }
#pragma unroll
  for (int e = 0; e < 4; ++e) z[e] = sigmoid ? sigmoid_f(z[e]) : silu_f(z[e]);
  if (gate_first) {
#pragma unroll
    for (int e = 0; e < 4; ++e) v[e] *= z[e];
  }
  float ss = (v[0] * v[0] + v[1] * v[1]) + (v[2] * v[2] + v[3] * v[3]);
  for (int m = 1; m < SG; m <<= 1) ss += __shfl_xor(ss, m, 64);
  if (!on) return;
  const float inv = 1.f / sqrtf(ss / (float)gs + eps);
  float ww[4];
  load4<float>(w + (shared_w ? c : col), ww);
#pragma unroll
  for (int e = 0; e < 4; ++e) v[e] = v[e] * inv * ww[e] * (gate_first ? 1.f : z[e]);
  store4<T>(out + r * W + col, v);
}

template <typename T>
__global__ void gate_rows_kernel(const T* __restrict__ z, long long ldz, const T* __restrict__ table,
                                 long long ldt, const long long* __restrict__ tokens, int col0,
                                 int dim, T* __restrict__ out, long long n) {
  for (long long i = blockIdx.x * (long long)blockDim.x + threadIdx.x; i < n;
       i += (long long)gridDim.x * blockDim.x) {
    const long long t = i / dim;
    const int d = (int)(i % dim);
    const float e = to_f32(table[tokens[t] * ldt + col0 + d]);
    out[i] = from_f32<T>(gelu_tanh_f(to_f32(z[t * ldz + d])) * e);
  }
}

template <typename TI, typename TO>
hipError_t launch_rms(const void* x, long long ldx, const float* w, float* res, void* out,
                      long long ldo, int rows, int W, int groups, float eps, hipStream_t st) {
  const int gs = W / groups;
  const bool vec = gs % 4 == 0 && ldx % 4 == 0 && ldo % 4 == 0 &&
                   ((uintptr_t)x % 16 == 0) && ((uintptr_t)out % 16 == 0);
  if (vec)
    group_rms_kernel<TI, TO, true><<<rows, 256, 0, st>>>((const TI*)x, ldx, w, res, (TO*)out, ldo,
                                                         W, groups, eps);
  else
    group_rms_kernel<TI, TO, false><<<rows, 256, 0, st>>>((const TI*)x, ldx, w, res, (TO*)out, ldo,
                                                          W, groups, eps);
  return hipGetLastError();
}

inline int grid_for(long long n, int block = 256) {
  const long long g = (n + block - 1) / block;
  return (int)(g < 1 ? 1 : g > 65535 ? 65535 : g);
}

}  // namespace

extern "C" {

// x [rows, W] (row stride ldx) in dtype dt_in (fp32 or the model dtype); out (nullable when res
// is given) [rows, W] (row stride ldo) in dtype dt_out; res (nullable) fp32 [rows, W] contiguous.
hipError_t sm_group_rms(int dt_in, int dt_out, const void* x, long long ldx, const float* w,
                        float* res, void* out, long long ldo, int rows, int W, int groups,
                        float eps, hipStream_t st) {
  if (rows == 0) return hipSuccess;
  if (groups < 1 || W % groups != 0 || (!res && !out)) return hipErrorInvalidValue;
#define CALL_O(TO)                                                                              \
  {                                                                                             \
    if (dt_in == kF32) return launch_rms<float, TO>(x, ldx, w, res, out, ldo, rows, W, groups,  \
                                                    eps, st);                                   \
    if (dt_in == kBF16) return launch_rms<bf16, TO>(x, ldx, w, res, out, ldo, rows, W, groups,  \
                                                    eps, st);                                   \
    if (dt_in == kF16) return launch_rms<fp16, TO>(x, ldx, w, res, out, ldo, rows, W, groups,   \
                                                   eps, st);                                    \
    return hipErrorInvalidValue;                                                                \
  }
  SM_DISPATCH(dt_out, CALL_O)
#undef CALL_O
  return hipGetLastError();
}

// x fp32 [rows][W] contiguous; g [rows][W] with row stride ldg; w fp32 [W], or [W / groups] with
// shared_w; out [rows][W] contiguous.
hipError_t sm_gated_rms(int dt, const float* x, const void* g, long long ldg, const float* w,
                        void* out, int rows, int W, int groups, int shared_w, int gate_first,
                        int sigmoid, float eps, hipStream_t st) {
  if (rows == 0) return hipSuccess;
  if (groups < 1 || W < 1 || W % groups) return hipErrorInvalidValue;
  const int per = groups < 4 ? groups : 4;     // groups of one workgroup
  const size_t lds = (size_t)(W / groups) * per * sizeof(float);
  if (lds > 65536 - 64) return hipErrorInvalidValue;
  const dim3 grid(rows, (groups + per - 1) / per);
  const bool vec = (W / groups) % 4 == 0 && ldg % 4 == 0 && (uintptr_t)x % 16 == 0 &&
                   (uintptr_t)g % 16 == 0 && (uintptr_t)out % 16 == 0;
  const int gs = W / groups;
  const bool small = vec && gs <= 256 && (uintptr_t)w % 16 == 0 && W % 4 == 0;
  int SG = 1;
  while (4 * SG < gs) SG <<= 1;
  const long long items = (long long)rows * groups;
  const unsigned blocks = (unsigned)((items * SG + 255) / 256);
#define CALL(TT)                                                                                \
  if (small)                                                                                    \
    gated_rms_small_kernel<TT><<<blocks, 256, 0, st>>>(x, (const TT*)g, ldg, w, (TT*)out, W,    \
                                groups, gs, SG, items, shared_w, gate_first, sigmoid, eps);     \
  else if (vec) gated_rms_kernel<TT, true><<<grid, 256, lds, st>>>(x, (const TT*)g, ldg, w, (TT*)out, \
                                                W, groups, shared_w, gate_first, sigmoid, eps); \
  else gated_rms_kernel<TT, false><<<grid, 256, lds, st>>>(x, (const TT*)g, ldg, w, (TT*)out, W, \
                                                groups, shared_w, gate_first, sigmoid, eps)
  SM_DISPATCH(dt, CALL)
#undef CALL
  return hipGetLastError();
}

hipError_t sm_gate_rows(int dt, const void* z, long long ldz, const void* table, long long ldt,
                        const long long* tokens, int col0, int dim, void* out, int T,
                        hipStream_t st) {
  const long long n = (long long)T * dim;
  if (n == 0) return hipSuccess;
#define CALL(TT) gate_rows_kernel<TT><<<grid_for(n), 256, 0, st>>>((const TT*)z, ldz, (const TT*)table, ldt, tokens, col0, dim, (TT*)out, n)
  SM_DISPATCH(dt, CALL)
#undef CALL
  return hipGetLastError();
}

}  // extern "C"
