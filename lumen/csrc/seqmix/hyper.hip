// A residual stream kept as several copies (hyper-connections), fused with what surrounds it:
//
//   sm_hyper_mix   one pass over a row between two sublayers
//                    y    = the sublayer's output, or -- two outputs side by side -- the sum of
//                           both, each RMS-normed over the row with its own weight
//                    x'_t = sum_s mix[s][t] x_s + out[t] y         (all copies from the old ones)
//                    u    = sum_t in[t] x'_t
//                    h    = LN(u) * w + b in the compute dtype, or u itself in fp32
//                  The copies of a row, [S][W] fp32, are read and written in place once.  The first
//                  call of a step takes them all from the embedding row (x_s = table[token]) and has
//                  no y.
//   sm_head_norm_rotary  the heads of a fused projection's row [q heads | k heads | v heads]: q and k
//                  RMS-normed per head with a weight shared by the heads and turned on their first
//                  `dims` entries (half layout), v optionally divided by its own root mean square; q
//                  in place, k and v into their paged caches.
// The copies, the norms, their sums and the rotation are fp32; only a stored h, q, k or v is rounded.
#include "seqmix.h"

using namespace lumen;

namespace {

constexpr int kThreads = 256;

template <typename T>
struct HyperArgs {
  float* x;                                  // [T][S][W]
  const T* table; const long long* tokens; int vocab;   // first call: rows of the embedding
  const T* ya; const T* yb;                  // [T][W]; yb: the second of two outputs
  const float* wa; const float* wb; float eps_y;        // with yb
  const float* mix; const float* out; const float* in;  // [S][S] (from, to), [S], [S]
  const float* w; const float* b; float eps;            // LN; null: u is stored
  T* h; float* u;
  int store_x, W;
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

// one workgroup per row; V consecutive channels per thread and step; the row u stays in LDS
// between the passes (sum, squared deviations from the mean, output)
template <typename T, int S, int V>
__global__ void __launch_bounds__(kThreads) hyper_mix_kernel(const HyperArgs<T> a) {
  extern __shared__ float s_u[];
  __shared__ float s_red[kThreads / 64];
  const int W = a.W;
  const long long row = blockIdx.x;
  float* xr = a.x + row * S * W;
  const T* er = nullptr;
  if (a.table != nullptr) {
    long long tok = a.tokens[row];
    tok = tok < 0 ? 0 : (tok >= a.vocab ? a.vocab - 1 : tok);
    er = a.table + tok * W;
  }
  float mx[S][S], ot[S], in[S];
#pragma unroll
  for (int t = 0; t < S; ++t) {
    in[t] = a.in[t];
    ot[t] = a.ya != nullptr ? a.out[t] : 0.f;
#pragma unroll
    for (int s = 0; s < S; ++s) mx[s][t] = a.ya != nullptr ? a.mix[s * S + t] : 0.f;
  }
  float ia = 1.f, ib = 0.f;
  if (a.yb != nullptr) {
    float sa = 0.f, sb = 0.f;
    for (int c = threadIdx.x * V; c < W; c += kThreads * V) {
      float p[V], q[V];
      load_n<T, V>(a.ya + row * W + c, p);
      load_n<T, V>(a.yb + row * W + c, q);
#pragma unroll
      for (int e = 0; e < V; ++e) { sa += p[e] * p[e]; sb += q[e] * q[e]; }
    }
    ia = 1.f / sqrtf(block_sum<kThreads>(sa, s_red) / (float)W + a.eps_y);
    ib = 1.f / sqrtf(block_sum<kThreads>(sb, s_red) / (float)W + a.eps_y);
  }
  float sum = 0.f;
  for (int c = threadIdx.x * V; c < W; c += kThreads * V) {
    float nx[S][V], u[V];
    if (er != nullptr) {
      load_n<T, V>(er + c, nx[0]);
#pragma unroll
      for (int t = 1; t < S; ++t)
#pragma unroll
        for (int e = 0; e < V; ++e) nx[t][e] = nx[0][e];
    } else {
      float ox[S][V], y[V];
#pragma unroll
      for (int s = 0; s < S; ++s) load_n<float, V>(xr + (long long)s * W + c, ox[s]);
      load_n<T, V>(a.ya + row * W + c, y);
      if (a.yb != nullptr) {
        float q[V], wa[V], wb[V];
        load_n<T, V>(a.yb + row * W + c, q);
        load_n<float, V>(a.wa + c, wa);
        load_n<float, V>(a.wb + c, wb);
#pragma unroll
        for (int e = 0; e < V; ++e) y[e] = y[e] * ia * wa[e] + q[e] * ib * wb[e];
      }
#pragma unroll
      for (int t = 0; t < S; ++t)
#pragma unroll
        for (int e = 0; e < V; ++e) {
          float v = ot[t] * y[e];
#pragma unroll
          for (int s = 0; s < S; ++s) v += mx[s][t] * ox[s][e];
          nx[t][e] = v;
        }
    }
    if (a.store_x) {
#pragma unroll
      for (int t = 0; t < S; ++t) store_n<float, V>(xr + (long long)t * W + c, nx[t]);
    }
#pragma unroll
    for (int e = 0; e < V; ++e) {
      float v = 0.f;
#pragma unroll
      for (int t = 0; t < S; ++t) v += in[t] * nx[t][e];
      u[e] = v;
      sum += v;
    }
    if (a.w == nullptr) store_n<float, V>(a.u + row * W + c, u);
    else store_n<float, V>(s_u + c, u);
  }
  if (a.w == nullptr) return;
  const float mean = block_sum<kThreads>(sum, s_red) / (float)W;
  float sq = 0.f;
  for (int c = threadIdx.x * V; c < W; c += kThreads * V) {      // a thread re-reads its own entries
#pragma unroll
    for (int e = 0; e < V; ++e) {
      const float d = s_u[c + e] - mean;
      sq += d * d;
    }
  }
  const float inv = 1.f / sqrtf(block_sum<kThreads>(sq, s_red) / (float)W + a.eps);
  for (int c = threadIdx.x * V; c < W; c += kThreads * V) {
    float v[V], ww[V], bb[V];
    load_n<float, V>(s_u + c, v);
    load_n<float, V>(a.w + c, ww);
    load_n<float, V>(a.b + c, bb);
#pragma unroll
    for (int e = 0; e < V; ++e) v[e] = (v[e] - mean) * inv * ww[e] + bb[e];
    store_n<T, V>(a.h + row * W + c, v);
  }
}

template <typename T>
struct HeadArgs {
  T* z; long long ld;
  const float* wq; const float* wk;
  const int* positions; const long long* slots;
  T* kc; T* vc;
  const float* inv_freq;
  int H, G, D, Dv, dims, vnorm;
  float eps;
};

constexpr int kMaxHead = 512;

// one workgroup per row.  The row's dims / 2 sines and cosines are computed once, in LDS, for all
// heads; a subgroup of SG lanes (a power of two, 4 entries per lane) owns a head, so that a
// wave works on 64 / SG heads at a time; the pair partner dims / 2 entries away is a lane exchange.
// A step with few rows deals a row's heads out to several workgroups (grid y).
template <typename T>
__global__ void __launch_bounds__(kThreads) head_norm_rotary_v4(const HeadArgs<T> a, int SG) {
  __shared__ float s_cs[kMaxHead / 2], s_sn[kMaxHead / 2];
  const int t = blockIdx.x, lane = threadIdx.x & 63;
  const long long slot = a.slots[t];
  T* row = a.z + (long long)t * a.ld;
  const int half = a.dims / 2;
  const float pos = (float)a.positions[t];
  for (int i = threadIdx.x; i < half; i += kThreads) sincosf(pos * a.inv_freq[i], &s_sn[i], &s_cs[i]);
  __syncthreads();
  const int sub = threadIdx.x / SG, nsub = kThreads / SG, sl = lane & (SG - 1), sb = lane & ~(SG - 1);
  const int items = a.H + 2 * a.G;
  // every lane of a wave runs the same number of rounds: the exchanges below need all of them
  for (int i0 = blockIdx.y * nsub; i0 < items; i0 += gridDim.y * nsub) {
    const int item = i0 + sub;
    const bool live = item < items;
    const bool is_v = item >= a.H + a.G, is_q = item < a.H;
    const int size = is_v ? a.Dv : a.D;
    const int c = 4 * sl;
    const bool on = live && c < size;
    T* src = row + (is_v ? (long long)(a.H + a.G) * a.D + (long long)(item - a.H - a.G) * a.Dv
                         : (long long)item * a.D);
    float v[4] = {0.f, 0.f, 0.f, 0.f};
    if (on) load4<T>(src + c, v);
    float ss = v[0] * v[0] + v[1] * v[1] + v[2] * v[2] + v[3] * v[3];
    for (int m = 1; m < SG; m <<= 1) ss += __shfl_xor(ss, m, 64);
    float inv = 1.f / sqrtf(ss / (float)size + a.eps);
    if (is_v && !a.vnorm) inv = 1.f;
    if (on && !is_v) {
      float ww[4];
      load4<float>((is_q ? a.wq : a.wk) + c, ww);
#pragma unroll
      for (int e = 0; e < 4; ++e) v[e] = v[e] * inv * ww[e];
    } else {
#pragma unroll
      for (int e = 0; e < 4; ++e) v[e] *= inv;
    }
    if (half > 0) {                                  // uniform: whole waves exchange
      const bool low = c < half;
      const int partner = sb + (low ? sl + half / 4 : sl - half / 4);
      float o[4];
#pragma unroll
      for (int e = 0; e < 4; ++e) o[e] = __shfl(v[e], partner & 63, 64);
      if (on && !is_v && c < a.dims) {
        const int p = low ? c : c - half;
#pragma unroll
        for (int e = 0; e < 4; ++e)
          v[e] = low ? v[e] * s_cs[p + e] - o[e] * s_sn[p + e]
                     : v[e] * s_cs[p + e] + o[e] * s_sn[p + e];
      }
    }
    if (!on) continue;
    if (is_q) store4<T>(src + c, v);
    else if (slot >= 0 && !is_v) store4<T>(a.kc + (slot * a.G + (item - a.H)) * a.D + c, v);
    else if (slot >= 0) store4<T>(a.vc + (slot * a.G + (item - a.H - a.G)) * a.Dv + c, v);
  }
}

// any sizes: a wave per head, the normed head in the wave's LDS row while it turns
template <typename T>
__global__ void __launch_bounds__(kThreads) head_norm_rotary_any(const HeadArgs<T> a) {
  __shared__ float s_v[kThreads / 64][kMaxHead];
  const int t = blockIdx.x, lane = threadIdx.x & 63, w = threadIdx.x >> 6;
  const long long slot = a.slots[t];
  T* row = a.z + (long long)t * a.ld;
  const int half = a.dims / 2;
  const float pos = (float)a.positions[t];
  for (int i0 = 0; i0 < a.H + 2 * a.G; i0 += kThreads / 64) {
    const int item = i0 + w;
    const bool live = item < a.H + 2 * a.G;
    const bool is_v = item >= a.H + a.G, is_q = item < a.H;
    const int size = live ? (is_v ? a.Dv : a.D) : 0;
    T* src = row + (is_v ? (long long)(a.H + a.G) * a.D + (long long)(item - a.H - a.G) * a.Dv
                         : (long long)item * a.D);
    float ss = 0.f;
    for (int c = lane; c < size; c += 64) {
      const float v = to_f32(src[c]);
      ss += v * v;
    }
    ss = wave_sum(ss);
    float inv = live ? 1.f / sqrtf(ss / (float)size + a.eps) : 0.f;
    if (is_v && !a.vnorm) inv = 1.f;
    const float* wt = is_q ? a.wq : a.wk;
    for (int c = lane; c < size; c += 64) s_v[w][c] = to_f32(src[c]) * inv * (is_v ? 1.f : wt[c]);
    __syncthreads();
    T* dst = is_q ? src
                  : (slot < 0 ? nullptr
                              : (is_v ? a.vc + (slot * a.G + (item - a.H - a.G)) * a.Dv
                                      : a.kc + (slot * a.G + (item - a.H)) * a.D));
    if (dst != nullptr) {
      for (int c = lane; c < size; c += 64) {
        float v = s_v[w][c];
        if (!is_v && c < a.dims) {
          float sn, cs;
          const bool low = c < half;
          sincosf(pos * a.inv_freq[low ? c : c - half], &sn, &cs);
          v = low ? v * cs - s_v[w][c + half] * sn : v * cs + s_v[w][c - half] * sn;
        }
        dst[c] = from_f32<T>(v);
      }
    }
    __syncthreads();
  }
}

template <typename T, int S>
hipError_t launch_hyper(const HyperArgs<T>& a, int rows, bool vec, hipStream_t st) {
  const size_t lds = a.w != nullptr ? (size_t)a.W * sizeof(float) : 0;
  if (vec) hyper_mix_kernel<T, S, 4><<<rows, kThreads, lds, st>>>(a);
  else hyper_mix_kernel<T, S, 1><<<rows, kThreads, lds, st>>>(a);
  return hipGetLastError();
}

template <typename T>
hipError_t launch_hyper_s(const HyperArgs<T>& a, int rows, int S, bool vec, hipStream_t st) {
  switch (S) {
    case 1: return launch_hyper<T, 1>(a, rows, vec, st);
    case 2: return launch_hyper<T, 2>(a, rows, vec, st);
    case 3: return launch_hyper<T, 3>(a, rows, vec, st);
    case 4: return launch_hyper<T, 4>(a, rows, vec, st);
    case 5: return launch_hyper<T, 5>(a, rows, vec, st);
    case 6: return launch_hyper<T, 6>(a, rows, vec, st);
    case 7: return launch_hyper<T, 7>(a, rows, vec, st);
    case 8: return launch_hyper<T, 8>(a, rows, vec, st);
    default: return hipErrorInvalidValue;
  }
}

}  // namespace

extern "C" {

// x fp32 [rows][S][W] (in place).  First call: table + tokens, no ya.  Later: ya (and yb with wa,
// wb), mix, out.  w (with b, h): LN into h; w null: u [rows][W] fp32 is stored.
hipError_t sm_hyper_mix(int dt, float* x, const void* table, const long long* tokens, int vocab,
                        const void* ya, const void* yb, const float* wa, const float* wb,
                        float eps_y, const float* mix, const float* out, const float* in,
                        const float* w, const float* b, float eps, void* h, float* u, int store_x,
                        int rows, int S, int W, hipStream_t st) {
  if (rows == 0) return hipSuccess;
  if (W < 1 || (size_t)W * sizeof(float) > 65536 - 64) return hipErrorInvalidValue;
  if ((table == nullptr) == (ya == nullptr) || (table && (!tokens || vocab < 1)) ||
      (ya && (!mix || !out)) || (yb && (!wa || !wb)) || !in || (w ? (!b || !h) : !u))
    return hipErrorInvalidValue;
  const auto al = [](const void* p) { return (uintptr_t)p % 16 == 0; };
  const bool vec = W % 4 == 0 && al(x) && al(table) && al(ya) && al(yb) && al(wa) && al(wb) &&
                   al(w) && al(b) && al(h) && al(u);
#define CALL(T)                                                                                 \
  {                                                                                             \
    HyperArgs<T> a{x, (const T*)table, tokens, vocab, (const T*)ya, (const T*)yb, wa, wb, eps_y, \
                   mix, out, in, w, b, eps, (T*)h, u, store_x, W};                              \
    return launch_hyper_s<T>(a, rows, S, vec, st);                                              \
  }
  SM_DISPATCH(dt, CALL)
#undef CALL
  return hipSuccess;
}

hipError_t sm_head_norm_rotary(int dt, void* z, long long ld, const float* wq, const float* wk,
                               const int* positions, const long long* slots, void* kc, void* vc,
                               const float* inv_freq, int T, int H, int G, int D, int Dv, int dims,
                               int vnorm, float eps, hipStream_t st) {
  if (T == 0) return hipSuccess;
  if (H < 1 || G < 1 || D < 1 || Dv < 1 || D > kMaxHead || Dv > kMaxHead || dims < 0 || dims % 2 ||
      dims > D || ld < (long long)(H + G) * D + (long long)G * Dv)
    return hipErrorInvalidValue;
  const int m = D > Dv ? D : Dv;
  const bool vec = D % 4 == 0 && Dv % 4 == 0 && dims % 8 == 0 && ld % 4 == 0 && m <= 256 &&
                   (uintptr_t)z % 16 == 0 && (uintptr_t)kc % 16 == 0 && (uintptr_t)vc % 16 == 0 &&
                   (uintptr_t)wq % 16 == 0 && (uintptr_t)wk % 16 == 0;
  int SG = 1;
  while (4 * SG < m) SG <<= 1;
  const int rounds = (H + 2 * G + kThreads / SG - 1) / (kThreads / SG);
  const dim3 grid(T, T <= 64 ? rounds : 1);
#define CALL(TT)                                                                                \
  {                                                                                             \
    HeadArgs<TT> a{(TT*)z, ld, wq, wk, positions, slots, (TT*)kc, (TT*)vc, inv_freq, H, G, D,   \
                   Dv, dims, vnorm, eps};                                                       \
    if (vec) head_norm_rotary_v4<TT><<<grid, kThreads, 0, st>>>(a, SG);                         \
    else head_norm_rotary_any<TT><<<T, kThreads, 0, st>>>(a);                                   \
  }
  SM_DISPATCH(dt, CALL)
#undef CALL
  return hipGetLastError();
}

}  // extern "C"
