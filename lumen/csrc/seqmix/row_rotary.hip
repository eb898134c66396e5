// Whole-projection q / k norm, rotation and cache writes of an attention layer in one pass:
//
//   sm_row_norm_rotary  a fused projection's row [q heads | k heads | values]: q and k are RMS-normed
//                       over ALL their entries at once (every head together) with weights of that
//                       size and turned on the first `dims` entries of every head in the half layout
//                       (entry i with entry i + dims / 2) by position * inv_freq[i], cosine and sine
//                       carrying the factor `amp`; q in place, k and the values as projected into
//                       their paged caches.
//
// One workgroup of four waves per row.  The sums of squares of the two parts are reduced in a fixed
// order; the row's dims / 2 sines and cosines are computed once, in LDS, for all heads.  A work item is
// V consecutive entries and, where they turn, their V partners: it is read, normed, turned and stored
// by one lane, so nothing is exchanged and nothing is read after it was replaced.  Norms, angles and
// the rotation are fp32; only a stored q or k is rounded.
#include "seqmix.h"

using namespace lumen;

namespace {

constexpr int kThreads = 256;
constexpr int kMaxHead = 512;

template <typename T>
struct RowRotArgs {
  T* z; long long ld;
  const float* wq; const float* wk;
  const int* positions; const long long* slots;
  T* kc; T* vc;
  const float* inv_freq;
  int H, G, D, vw, dims;                     // vw: value columns (G * Dv)
  float amp, eps;
};

template <typename T, int V>
__device__ __forceinline__ void load_v(const T* p, float (&o)[V]) {
  if constexpr (V == 8) load8<T>(p, o);
  else if constexpr (V == 4) load4<T>(p, o);
  else o[0] = to_f32(p[0]);
}
template <typename T, int V>
__device__ __forceinline__ void store_v(T* p, const float (&o)[V]) {
  if constexpr (V == 8) store8<T>(p, o);
  else if constexpr (V == 4) store4<T>(p, o);
  else p[0] = from_f32<T>(o[0]);
}

template <typename T, int V>
__global__ void __launch_bounds__(kThreads) row_norm_rotary_kernel(const RowRotArgs<T> a) {
  __shared__ float s_cs[kMaxHead / 2], s_sn[kMaxHead / 2];
  __shared__ float s_red[2][kThreads / 64];
  const int t = blockIdx.x, lane = threadIdx.x & 63, w = threadIdx.x >> 6;
  const int half = a.dims / 2, HD = a.H * a.D, GD = a.G * a.D;
  const long long slot = a.slots[t];
  T* row = a.z + (long long)t * a.ld;
  const float pos = (float)a.positions[t];
  for (int i = threadIdx.x; i < half; i += kThreads) {
    float sn, cs;
    sincosf(pos * a.inv_freq[i], &sn, &cs);
    s_sn[i] = sn * a.amp;
    s_cs[i] = cs * a.amp;
  }
  float sq = 0.f, sk = 0.f;
  for (int c = threadIdx.x * V; c < HD; c += kThreads * V) {
    float v[V];
    load_v<T, V>(row + c, v);
#pragma unroll
    for (int e = 0; e < V; ++e) sq += v[e] * v[e];
  }
  for (int c = threadIdx.x * V; c < GD; c += kThreads * V) {
    float v[V];
    load_v<T, V>(row + HD + c, v);
#pragma unroll
    for (int e = 0; e < V; ++e) sk += v[e] * v[e];
  }
  sq = wave_sum(sq);
  sk = wave_sum(sk);
  if (lane == 0) {
    s_red[0][w] = sq;
    s_red[1][w] = sk;
  }
  __syncthreads();
  sq = (s_red[0][0] + s_red[0][1]) + (s_red[0][2] + s_red[0][3]);
  sk = (s_red[1][0] + s_red[1][1]) + (s_red[1][2] + s_red[1][3]);
  const float iq = 1.f / sqrtf(sq / (float)HD + a.eps), ik = 1.f / sqrtf(sk / (float)GD + a.eps);
  const int turning = half / V, per = turning + (a.D - a.dims) / V;     // items of a head
  for (int it = threadIdx.x; it < (a.H + a.G) * per; it += kThreads) {
    const int hd = it / per, j = it - hd * per;
    const bool is_q = hd < a.H, turns = j < turning;
    const int c = turns ? j * V : a.dims + (j - turning) * V;           // first entry in the head
    const T* src = row + hd * a.D + c;
    const float* wt = is_q ? a.wq + hd * a.D + c : a.wk + (hd - a.H) * a.D + c;
    const float inv = is_q ? iq : ik;
    T* dst = is_q ? row + hd * a.D + c
                  : (slot < 0 ? nullptr : a.kc + slot * GD + (hd - a.H) * a.D + c);
    float u[V], ww[V];
    load_v<T, V>(src, u);
    load_v<float, V>(wt, ww);
#pragma unroll
    for (int e = 0; e < V; ++e) u[e] = u[e] * inv * ww[e];
    if (turns) {
      float v[V];
      load_v<T, V>(src + half, v);
      load_v<float, V>(wt + half, ww);
#pragma unroll
      for (int e = 0; e < V; ++e) {
        const float y = v[e] * inv * ww[e], x = u[e], cs = s_cs[c + e], sn = s_sn[c + e];
        u[e] = x * cs - y * sn;
        v[e] = y * cs + x * sn;
      }
      if (dst != nullptr) store_v<T, V>(dst + half, v);
    }
    if (dst != nullptr) store_v<T, V>(dst, u);
  }
  if (slot < 0) return;
  const T* vs = row + HD + GD;
  T* vd = a.vc + slot * a.vw;
  for (int c = threadIdx.x * V; c < a.vw; c += kThreads * V) {
    if constexpr (V == 8 && sizeof(T) == 2) {
      *reinterpret_cast<uint4*>(vd + c) = *reinterpret_cast<const uint4*>(vs + c);
    } else {
#pragma unroll
      for (int e = 0; e < V; ++e) vd[c + e] = vs[c + e];
    }
  }
}

}  // namespace

extern "C" {

// z [T][>= (H + G) D + vw] (row stride ld); kc / vc rows of G D / vw entries by slot.
hipError_t sm_row_norm_rotary(int dt, void* z, long long ld, const float* wq, const float* wk,
                              const int* positions, const long long* slots, void* kc, void* vc,
                              const float* inv_freq, int T, int H, int G, int D, int vw, int dims,
                              float amp, float eps, hipStream_t st) {
  if (T == 0) return hipSuccess;
  if (H < 1 || G < 1 || D < 1 || D > kMaxHead || vw < 1 || dims < 0 || dims % 2 || dims > D ||
      (dims > 0 && !inv_freq) || ld < (long long)(H + G) * D + vw)
    return hipErrorInvalidValue;
  const auto al = [](const void* p) { return (uintptr_t)p % 16 == 0; };
  const int half = dims / 2;
  const auto fits = [&](int v) {
    return half % v == 0 && D % v == 0 && (D - dims) % v == 0 && vw % v == 0 && ld % v == 0 &&
           al(z) && al(kc) && al(vc) && al(wq) && al(wk);
  };
#define CALL(TT)                                                                                  \
  {                                                                                               \
    RowRotArgs<TT> a{(TT*)z, ld, wq, wk, positions, slots, (TT*)kc, (TT*)vc, inv_freq, H, G, D,   \
                     vw, dims, amp, eps};                                                         \
    if (fits(8)) row_norm_rotary_kernel<TT, 8><<<T, kThreads, 0, st>>>(a);                        \
    else if (fits(4)) row_norm_rotary_kernel<TT, 4><<<T, kThreads, 0, st>>>(a);                   \
    else row_norm_rotary_kernel<TT, 1><<<T, kThreads, 0, st>>>(a);                                \
  }
  SM_DISPATCH(dt, CALL)
#undef CALL
  return hipGetLastError();
}

}  // extern "C"
