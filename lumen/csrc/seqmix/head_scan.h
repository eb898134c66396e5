// Shared argument block of the matrix-state scans with ONE decay per (token, head)
// (head_scan_chunk.hip: prompt portions; head_scan_step.hip: decoded rows).
#pragma once
#include "seqmix.h"

namespace lumen {

template <typename T>
struct HeadScanArgs {
  const T* q; long long ldq;       // [T][>= (H / rep) * Dk]; head h reads block h / rep
  const T* k; long long ldk;
  const T* v; long long ldv;       // [T][>= H * Dv]
  const T* a; long long lda;       // decay logits [T][H]; null: constant decays
  const T* b; long long ldb;       // write-strength logits [T][H] (delta rule)
  const float* A_log; const float* dt_bias;   // [H], with a
  const float* log_decay;          // [H], without a
  const float* skip;               // [H] (nullable): + skip_h * v_t in the read-out
  float* state;                    // [slots][H][Dk][Dv]
  float* out;                      // [T][H * Dv]
  const int* cu; const int* slot; const int* start;
  int H, rep, Dk, Dv;
  int silu_in;                     // q, k, v pass through silu as they are read
  int vec;                         // rows can be read four elements at a time
  float key_eps, q_scale;          // delta rule: q, k -> unit vectors, q times q_scale
};

// log(1 + e^x); beyond 20 the difference to x is below fp32's last place
__device__ __forceinline__ float softplus_f(float x) { return x > 20.f ? x : log1pf(expf(x)); }

// a (token, head)'s log decay and step size (1 with constant decays).  A log decay below -1e4 is
// a decay of zero; the bound keeps differences of sums finite.
template <typename T>
__device__ __forceinline__ void head_decay(const HeadScanArgs<T>& s, long long row, int h,
                                           float& ld, float& dt) {
  if (s.a != nullptr) {
    dt = softplus_f(to_f32(s.a[row * s.lda + h]) + s.dt_bias[h]);
    ld = -expf(s.A_log[h]) * dt;
  } else {
    dt = 1.f;
    ld = s.log_decay[h];
  }
  ld = fmaxf(ld, -1e4f);
}

// silu of a value that is stored as T next: 16-bit types take the hardware exponential and
// reciprocal, whose last-place error disappears in the rounding
template <typename T> __device__ __forceinline__ float silu_as(float x) {
  return x * __builtin_amdgcn_rcpf(1.f + __expf(-x));
}
template <> __device__ __forceinline__ float silu_as<float>(float x) { return silu_f(x); }

// silu of a stored q or k element, rounded to its type again: what a projection with an activation
// stores, so that every kernel multiplies the same values
template <typename T> __device__ __forceinline__ float silu_stored(float x) {
  return to_f32(from_f32<T>(silu_f(x)));
}

// bf16 prompt portions (head_scan_chunk16.hip)
hipError_t head_scan_chunk16(const HeadScanArgs<bf16>& args, bool delta, int n_seg,
                             hipStream_t st);

}  // namespace lumen
