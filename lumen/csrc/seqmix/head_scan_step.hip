// Matrix-state recurrences with one decay per (token, head), for decoded rows (the recurrences
// are those of head_scan_chunk.hip), and the short causal convolution in front of them.
//
//   sm_head_scan_step  one workgroup per (segment, head, 64 value columns) walks the segment's rows
//                      (one, when decoding) with its [Dk x 64] slice of the state in registers: the
//                      step reads and writes the state once, 16 bytes per lane, and everything else
//                      is small.  V consecutive columns per lane, the key channels dealt out to the
//                      256 / (64 / V) row groups; sums over channels are lane exchanges inside a
//                      wave and one LDS exchange between the four waves.
//   sm_short_conv      y_t = silu(sum_j w[:, taps - 1 - j] x_(t - j) (+ bias)) per channel, rows
//                      before a segment's first row from the slot's tail (zero below position 0)
//   sm_conv_tail       the tail moves on to the segment's last taps - 1 inputs
//   sm_conv_step       both at once for one-row segments
// The tail holds the projection's rows as they are, [slots][taps - 1][C] in the model dtype.
#include "head_scan.h"

using namespace lumen;

namespace {

// sums over all key channels of a per-thread partial for V columns; every thread gets the result
template <int V>
__device__ __forceinline__ void column_sum(float (&x)[V], float (*s_red)[64], int lane, int wv) {
  constexpr int CL = 64 / V;
#pragma unroll
  for (int m = CL; m < 64; m <<= 1)
#pragma unroll
    for (int e = 0; e < V; ++e) x[e] += __shfl_xor(x[e], m, 64);
  const int cl = lane % CL;
  if (lane < CL) {
#pragma unroll
    for (int e = 0; e < V; ++e) s_red[wv][cl * V + e] = x[e];
  }
  __syncthreads();
#pragma unroll
  for (int e = 0; e < V; ++e)
    x[e] = (s_red[0][cl * V + e] + s_red[1][cl * V + e]) +
           (s_red[2][cl * V + e] + s_red[3][cl * V + e]);
}

template <typename T, int KM, int V, bool DELTA>
__global__ void __launch_bounds__(256) head_scan_step_kernel(const HeadScanArgs<T> a) {
  constexpr int CL = 64 / V, RG = 256 / CL;          // lanes across columns, row groups
  __shared__ float s_q[256], s_k[256], s_n[8];
  __shared__ float s_red[2][4][64];
  const int sg = blockIdx.x, hd = blockIdx.y;
  const int r0 = a.cu[sg], r1 = a.cu[sg + 1];
  if (r1 <= r0) return;
  const int tid = threadIdx.x, lane = tid & 63, wv = tid >> 6;
  const int rg = tid / CL, col = blockIdx.z * 64 + (tid % CL) * V;
  const int Dk = a.Dk, Dv = a.Dv;
  const bool on = col < Dv;                          // V = 4 only with Dv a multiple of 4
  float* sp = a.state + ((long long)a.slot[sg] * a.H + hd) * Dk * Dv + col;
  const bool fresh = a.start[sg] == 0;
  float S[KM][V];
#pragma unroll
  for (int m = 0; m < KM; ++m) {
    const int row = rg + RG * m;
#pragma unroll
    for (int e = 0; e < V; ++e) S[m][e] = 0.f;
    if (!fresh && on && row < Dk) {
      if constexpr (V == 4) load4<float>(sp + (long long)row * Dv, S[m]);
      else S[m][0] = sp[(long long)row * Dv];
    }
  }
  const float skip = a.skip != nullptr ? a.skip[hd] : 0.f;
  for (long long r = r0; r < r1; ++r) {
    float qv = 0.f, kv = 0.f;
    if (tid < Dk) {
      const int qc = (hd / a.rep) * Dk + tid;
      qv = to_f32(a.q[r * a.ldq + qc]);
      kv = to_f32(a.k[r * a.ldk + qc]);
      if (a.silu_in) { qv = silu_stored<T>(qv); kv = silu_stored<T>(kv); }
    }
    float x[V], o[V];
#pragma unroll
    for (int e = 0; e < V; ++e) x[e] = 0.f;
    if (on) {
      const T* vp = a.v + r * a.ldv + (long long)hd * Dv + col;
#pragma unroll
      for (int e = 0; e < V; ++e) {
        x[e] = to_f32(vp[e]);
        if (a.silu_in) x[e] = silu_f(x[e]);
      }
    }
    float ld, dt;
    head_decay(a, r, hd, ld, dt);
    const float g = expf(ld);
    s_q[tid] = qv;
    s_k[tid] = kv;
    if (DELTA) {
      const float nq = wave_sum(qv * qv), nk = wave_sum(kv * kv);
      if (lane == 0) { s_n[wv] = nq; s_n[4 + wv] = nk; }
    }
    __syncthreads();
    float fq = 1.f, fk = 1.f;
    if (DELTA) {
      fq = a.q_scale / sqrtf((s_n[0] + s_n[1]) + (s_n[2] + s_n[3]) + a.key_eps);
      fk = 1.f / sqrtf((s_n[4] + s_n[5]) + (s_n[6] + s_n[7]) + a.key_eps);
    }
    float u[V];
    if (DELTA) {
#pragma unroll
      for (int e = 0; e < V; ++e) u[e] = 0.f;
#pragma unroll
      for (int m = 0; m < KM; ++m) {
        const float kk = s_k[rg + RG * m] * fk;
#pragma unroll
        for (int e = 0; e < V; ++e) {
          S[m][e] *= g;
          u[e] += S[m][e] * kk;
        }
      }
      column_sum<V>(u, s_red[0], lane, wv);
      const float beta = sigmoid_f(to_f32(a.b[r * a.ldb + hd]));
#pragma unroll
      for (int e = 0; e < V; ++e) u[e] = beta * (x[e] - u[e]);
    } else {
#pragma unroll
      for (int e = 0; e < V; ++e) u[e] = dt * x[e];
    }
#pragma unroll
    for (int e = 0; e < V; ++e) o[e] = 0.f;
#pragma unroll
    for (int m = 0; m < KM; ++m) {
      const float kk = s_k[rg + RG * m] * fk, qq = s_q[rg + RG * m] * fq;
#pragma unroll
      for (int e = 0; e < V; ++e) {
        S[m][e] = (DELTA ? S[m][e] : g * S[m][e]) + kk * u[e];
        o[e] += S[m][e] * qq;
      }
    }
    column_sum<V>(o, s_red[1], lane, wv);
    if (on && rg == 0) {
      float* op = a.out + r * ((long long)a.H * Dv) + (long long)hd * Dv + col;
#pragma unroll
      for (int e = 0; e < V; ++e) op[e] = o[e] + skip * x[e];
    }
    if (r + 1 < r1) __syncthreads();                 // s_q, s_k and s_red are written again
  }
  if (on) {
#pragma unroll
    for (int m = 0; m < KM; ++m) {
      const int row = rg + RG * m;
      if (row < Dk) {
        if constexpr (V == 4) store4<float>(sp + (long long)row * Dv, S[m]);
        else sp[(long long)row * Dv] = S[m][0];
      }
    }
  }
}

template <typename T, bool DELTA>
hipError_t launch_step(const HeadScanArgs<T>& a, int n_seg, hipStream_t st) {
  const dim3 grid(n_seg, a.H, (a.Dv + 63) / 64);
  const bool v4 = a.Dv % 4 == 0 && (uintptr_t)a.state % 16 == 0;
#define GO(KM, V) head_scan_step_kernel<T, KM, V, DELTA><<<grid, 256, 0, st>>>(a)
  if (v4) {
    if (a.Dk <= 32) GO(2, 4);
    else if (a.Dk <= 64) GO(4, 4);
    else if (a.Dk <= 128) GO(8, 4);
    else GO(16, 4);
  } else {
    if (a.Dk <= 64) GO(16, 1);
    else GO(64, 1);
  }
#undef GO
  return hipGetLastError();
}

// ---- short causal convolution ---------------------------------------------------------------------
constexpr int kMaxTaps = 16;
constexpr int kStrip = 16;         // rows per workgroup

template <typename T>
struct ConvArgs {
  const T* x; long long ldx;       // [T][>= C] rows
  const float* w; const float* bias;          // [C][taps], [C] (nullable)
  T* tail;                         // [slots][taps - 1][C]
  T* out;                          // [T][C]
  const int* cu; const int* slot; const int* start; const int* row_seg;
  int rows, C, taps;
};

template <typename T, int V>
__device__ __forceinline__ void load_v(const T* p, float (&o)[V]) {
  if constexpr (V == 4) load4<T>(p, o);
  else o[0] = to_f32(p[0]);
}
template <typename T, int V>
__device__ __forceinline__ void store_v(T* p, const float (&o)[V]) {
  if constexpr (V == 4) store4<T>(p, o);
  else p[0] = from_f32<T>(o[0]);
}

// a thread walks a strip of rows of V channels with the last TAPS - 1 inputs in registers
template <typename T, int V, int TAPS>
__global__ void __launch_bounds__(64) short_conv_kernel(const ConvArgs<T> a) {
  constexpr int K = TAPS - 1;
  const int c = V * (blockIdx.x * 64 + threadIdx.x);
  if (c >= a.C) return;
  float wv[V][TAPS], bv[V];
#pragma unroll
  for (int j = 0; j < V; ++j) {
    bv[j] = a.bias != nullptr ? a.bias[c + j] : 0.f;
#pragma unroll
    for (int q = 0; q < TAPS; ++q) wv[j][q] = a.w[(long long)(c + j) * TAPS + q];
  }
  float win[K > 0 ? K : 1][V];                       // win[d - 1]: the input d positions back
  const int t0 = blockIdx.y * kStrip, t1 = min(a.rows, t0 + kStrip);
  // a whole strip of one segment: all its rows and the taps before them are loaded at once
  if (t1 - t0 == kStrip) {
    float x[kStrip + K][V];
#pragma unroll
    for (int i = 0; i < kStrip; ++i) load_v<T, V>(a.x + (long long)(t0 + i) * a.ldx + c, x[K + i]);
    const int sg = a.row_seg[t0];
    if (sg == a.row_seg[t1 - 1]) {
      const int local = t0 - a.cu[sg], p0 = a.start[sg];
#pragma unroll
      for (int d = 1; d <= K; ++d) {
#pragma unroll
        for (int j = 0; j < V; ++j) x[K - d][j] = 0.f;
        const int src = local - d;
        if (src >= 0) load_v<T, V>(a.x + (long long)(t0 - d) * a.ldx + c, x[K - d]);
        else if (p0 + src >= 0) load_v<T, V>(a.tail + ((long long)a.slot[sg] * K + (K + src)) * a.C + c, x[K - d]);
      }
#pragma unroll
      for (int i = 0; i < kStrip; ++i) {
        float o[V];
#pragma unroll
        for (int j = 0; j < V; ++j) {
          float acc = wv[j][K] * x[K + i][j] + bv[j];
#pragma unroll
          for (int d = 1; d <= K; ++d) acc += wv[j][K - d] * x[K + i - d][j];
          o[j] = silu_as<T>(acc);
        }
        store_v<T, V>(a.out + (long long)(t0 + i) * a.C + c, o);
      }
      return;
    }
  }
  int cur = -1;
  for (int t = t0; t < t1; ++t) {
    const int sg = a.row_seg[t];
    if (sg != cur) {                                 // strip start or a new segment
      cur = sg;
      const int local = t - a.cu[sg], p0 = a.start[sg];
#pragma unroll
      for (int d = 1; d <= K; ++d) {
        const int src = local - d;
        float h[V];
#pragma unroll
        for (int j = 0; j < V; ++j) h[j] = 0.f;
        if (src >= 0) load_v<T, V>(a.x + (long long)(t - d) * a.ldx + c, h);
        else if (p0 + src >= 0) load_v<T, V>(a.tail + ((long long)a.slot[sg] * K + (K + src)) * a.C + c, h);
#pragma unroll
        for (int j = 0; j < V; ++j) win[d - 1][j] = h[j];
      }
    }
    float h[V], o[V];
    load_v<T, V>(a.x + (long long)t * a.ldx + c, h);
#pragma unroll
    for (int j = 0; j < V; ++j) {
      float acc = wv[j][K] * h[j] + bv[j];
#pragma unroll
      for (int d = 1; d <= K; ++d) acc += wv[j][K - d] * win[d - 1][j];
      o[j] = silu_as<T>(acc);
    }
    store_v<T, V>(a.out + (long long)t * a.C + c, o);
#pragma unroll
    for (int d = K; d >= 2; --d)
#pragma unroll
      for (int j = 0; j < V; ++j) win[d - 1][j] = win[d - 2][j];
    if (K > 0) {
#pragma unroll
      for (int j = 0; j < V; ++j) win[0][j] = h[j];
    }
  }
}

// any number of taps, one element per thread
template <typename T>
__global__ void __launch_bounds__(256) short_conv_any_kernel(const ConvArgs<T> a) {
  const int K = a.taps - 1;
  const int c = blockIdx.x * 256 + threadIdx.x;
  if (c >= a.C) return;
  for (int t = blockIdx.y; t < a.rows; t += gridDim.y) {
    const int sg = a.row_seg[t];
    const int local = t - a.cu[sg], p0 = a.start[sg];
    float acc = a.bias != nullptr ? a.bias[c] : 0.f;
    for (int d = 0; d <= K; ++d) {
      const int src = local - d;
      float h = 0.f;
      if (src >= 0) h = to_f32(a.x[(long long)(t - d) * a.ldx + c]);
      else if (p0 + src >= 0) h = to_f32(a.tail[((long long)a.slot[sg] * K + (K + src)) * a.C + c]);
      acc += a.w[(long long)c * a.taps + (K - d)] * h;
    }
    a.out[(long long)t * a.C + c] = from_f32<T>(silu_as<T>(acc));
  }
}

// STEP: the convolution of a one-row segment in the same pass
template <typename T, bool STEP>
__global__ void __launch_bounds__(256) conv_tail_kernel(const ConvArgs<T> a) {
  const int K = a.taps - 1, sg = blockIdx.y;
  const int c = blockIdx.x * 256 + threadIdx.x;
  if (c >= a.C) return;
  const int r0 = a.cu[sg], L = a.cu[sg + 1] - r0;
  if (L <= 0) return;
  const int p0 = a.start[sg];
  T* tp = a.tail + (long long)a.slot[sg] * K * a.C + c;
  T old[kMaxTaps];
#pragma unroll
  for (int k = 0; k < kMaxTaps; ++k)
    old[k] = (k < K && p0 - K + k >= 0) ? tp[(long long)k * a.C] : from_f32<T>(0.f);
  if (STEP) {
    const T h = a.x[(long long)r0 * a.ldx + c];
    const float* w = a.w + (long long)c * a.taps;
    float acc = w[K] * to_f32(h) + (a.bias != nullptr ? a.bias[c] : 0.f);
#pragma unroll
    for (int k = 0; k < kMaxTaps; ++k)
      if (k < K) acc += w[k] * to_f32(old[k]);
    a.out[(long long)r0 * a.C + c] = from_f32<T>(silu_as<T>(acc));
#pragma unroll
    for (int k = 0; k < kMaxTaps - 1; ++k)
      if (k < K) tp[(long long)k * a.C] = k == K - 1 ? h : old[k + 1];
    return;
  }
  for (int k = 0; k < K; ++k) {                      // new tail row k is local row L - K + k
    const int src = L - K + k;
    T h = from_f32<T>(0.f);
    if (src >= 0) {
      h = a.x[(long long)(r0 + src) * a.ldx + c];
    } else {
#pragma unroll
      for (int q = 0; q < kMaxTaps; ++q)
        if (q == k + L) h = old[q];                  // zero below position 0
    }
    tp[(long long)k * a.C] = h;
  }
}

}  // namespace

extern "C" {

hipError_t sm_head_scan_step(int dt, int delta, const void* q, long long ldq, const void* k,
                             long long ldk, const void* v, long long ldv, const void* al,
                             long long lda, const void* bl, long long ldb, const float* A_log,
                             const float* dt_bias, const float* log_decay, const float* skip,
                             float* state, float* out, const int* cu, const int* slot,
                             const int* start, int n_seg, int H, int rep, int Dk, int Dv,
                             int silu_in, float key_eps, float q_scale, hipStream_t st) {
  if (n_seg == 0) return hipSuccess;
  if (Dk < 1 || Dk > 256 || Dv < 1 || rep < 1 || H < 1 || H % rep) return hipErrorInvalidValue;
  if ((al == nullptr) == (log_decay == nullptr) || (al && (!A_log || !dt_bias)) ||
      (delta && (!bl || !al)))
    return hipErrorInvalidValue;
#define CALL(T)                                                                                 \
  {                                                                                             \
    HeadScanArgs<T> a{(const T*)q, ldq, (const T*)k, ldk, (const T*)v, ldv, (const T*)al, lda,  \
                      (const T*)bl, ldb, A_log, dt_bias, log_decay, skip, state, out, cu, slot, \
                      start, H, rep, Dk, Dv, silu_in, 0, key_eps, q_scale};                     \
    return delta ? launch_step<T, true>(a, n_seg, st) : launch_step<T, false>(a, n_seg, st);    \
  }
  SM_DISPATCH(dt, CALL)
#undef CALL
  return hipSuccess;
}

// rows [0, rows) of x; row_seg names each row's segment among cu / slot / start
hipError_t sm_short_conv(int dt, const void* x, long long ldx, const float* w, const float* bias,
                         const void* tail, void* out, const int* cu, const int* slot,
                         const int* start, const int* row_seg, int rows, int C, int taps,
                         hipStream_t st) {
  if (rows == 0) return hipSuccess;
  if (taps < 1 || taps > kMaxTaps || C < 1) return hipErrorInvalidValue;
  const bool v4 = C % 4 == 0 && ldx % 4 == 0 && (uintptr_t)x % 16 == 0 &&
                  (uintptr_t)tail % 16 == 0 && (uintptr_t)out % 16 == 0;
#define GO(TT, TP)                                                                              \
  if (v4) short_conv_kernel<TT, 4, TP><<<dim3((C / 4 + 63) / 64, strips), 64, 0, st>>>(a);      \
  else short_conv_kernel<TT, 1, TP><<<dim3((C + 63) / 64, strips), 64, 0, st>>>(a);             \
  break
#define CALL(TT)                                                                                \
  {                                                                                             \
    ConvArgs<TT> a{(const TT*)x, ldx, w, bias, (TT*)tail, (TT*)out, cu, slot, start, row_seg,   \
                   rows, C, taps};                                                              \
    const int strips = (rows + kStrip - 1) / kStrip;                                            \
    switch (taps) {                                                                             \
      case 1: GO(TT, 1);                                                                        \
      case 2: GO(TT, 2);                                                                        \
      case 3: GO(TT, 3);                                                                        \
      case 4: GO(TT, 4);                                                                        \
      default:                                                                                  \
        short_conv_any_kernel<TT>                                                               \
            <<<dim3((C + 255) / 256, rows < 65535 ? rows : 65535), 256, 0, st>>>(a);            \
    }                                                                                           \
  }
  SM_DISPATCH(dt, CALL)
#undef CALL
#undef GO
  return hipGetLastError();
}

// step = 0: the tails of n_seg segments move on; 1: one-row segments are convolved as well
hipError_t sm_conv_tail(int dt, int step, const void* x, long long ldx, const float* w,
                        const float* bias, void* tail, void* out, const int* cu, const int* slot,
                        const int* start, int n_seg, int C, int taps, hipStream_t st) {
  if (n_seg == 0 || (taps == 1 && !step)) return hipSuccess;
  if (taps < 1 || taps > kMaxTaps || C < 1 || n_seg > 65535) return hipErrorInvalidValue;
  const dim3 grid((C + 255) / 256, n_seg);
#define CALL(TT)                                                                                \
  {                                                                                             \
    ConvArgs<TT> a{(const TT*)x, ldx, w, bias, (TT*)tail, (TT*)out, cu, slot, start, nullptr,   \
                   0, C, taps};                                                                 \
    if (step) conv_tail_kernel<TT, true><<<grid, 256, 0, st>>>(a);                              \
    else conv_tail_kernel<TT, false><<<grid, 256, 0, st>>>(a);                                  \
  }
  SM_DISPATCH(dt, CALL)
#undef CALL
  return hipGetLastError();
}

}  // extern "C"
