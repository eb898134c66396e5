// Matrix-state recurrences with one decay per (token, head), over a step's prompt portions:
//
//   linear   S_t = e^{l_t} S_(t-1) + k_t (dt_t v_t)^T           o_t = S_t^T q_t (+ skip_h v_t)
//   delta    S  <- e^{l_t} S;  u_t = beta_t (v_t - S^T k_t);  S <- S + k_t u_t^T;  o_t = S^T q_t
//
// A segment is walked in chunks of 32 tokens; within a chunk everything is a matrix product.  With
// L_i the sum of the chunk's log decays up to token i, S_0 the state before the chunk and
// G_ij = e^{L_i - L_j} (j <= i):
//   U   = dt * V                                                   (linear)
//   U   = (I + strict_lower(beta_i G_ij k_i.k_j))^-1 (beta (V - e^L K S_0))       (delta)
//   O   = e^L (Q S_0) + (G . Q K^T) U
//   S_C = e^{L_C} S_0 + K^T (e^{L_C - L} U)
// One workgroup per (segment, head, 32 * NW value columns); a wave owns 32 value columns and keeps
// its [Dk x 32] slice of the state in accumulator registers for the whole segment.  Every product
// above has a per-wave right operand whose inner index lies on accumulator ROWS (S_0, U), and the
// 32x32 products' accumulator register r of lane half hi holds row 8 (r >> 2) + 4 hi + (r & 3):
// register r IS the right operand of one k = 2 product over the inner pair {a, a + 4}, when the
// left operand is read as [row][a + 4 hi].  So state and U never pass through LDS; the left
// operands (Q, K, the two chunk matrices) are staged there once for all waves and read 16 bytes at
// a time.  The products are fp32 matrix instructions (fp32 in, fp32 accumulate); bf16 models take
// head_scan_chunk16.hip instead.  Log-decay sums and their differences are fp64, so
// G is accurate however far a chunk decays.
// State in HBM: [slot][head][Dk][Dv] fp32; a segment that starts at position 0 starts from zero.
#include "head_scan.h"

using namespace lumen;

namespace {

typedef float f32x16 __attribute__((ext_vector_type(16)));
typedef float f32x4 __attribute__((ext_vector_type(4)));

constexpr int kC = 32;             // tokens per chunk
constexpr int LP = kC + 4;         // row stride of the chunk matrices in LDS

__device__ __forceinline__ f32x16 mma32(float a, float b, f32x16 c) {
  return __builtin_amdgcn_mfma_f32_32x32x2f32(a, b, c, 0, 0, 0);
}
__device__ __forceinline__ f32x4 mma16(float a, float b, f32x4 c) {
  return __builtin_amdgcn_mfma_f32_16x16x4f32(a, b, c, 0, 0, 0);
}

// acc += X[32 rows][32 inner] * B, X at p (row stride ld) already offset to the lane's row and
// half, B's inner index on accumulator rows
__device__ __forceinline__ f32x16 mma_rows(const float* p, const f32x16& b, f32x16 acc) {
#pragma unroll
  for (int m = 0; m < 4; ++m) {
    const float4 x = *reinterpret_cast<const float4*>(p + 8 * m);
    acc = mma32(x.x, b[4 * m], acc);
    acc = mma32(x.y, b[4 * m + 1], acc);
    acc = mma32(x.z, b[4 * m + 2], acc);
    acc = mma32(x.w, b[4 * m + 3], acc);
  }
  return acc;
}

__device__ __forceinline__ void wave_lds_fence() {
  __builtin_amdgcn_fence(__ATOMIC_RELEASE, "wavefront");
  __builtin_amdgcn_wave_barrier();
  __builtin_amdgcn_fence(__ATOMIC_ACQUIRE, "wavefront");
}

template <typename T, int KT, int NW, bool DELTA>
__global__ void __launch_bounds__(64 * NW)
head_scan_chunk_kernel(const HeadScanArgs<T> a) {
  constexpr int DKP = 32 * KT, LK = DKP + 4, NT = 64 * NW, TPR = NT / kC;
  __shared__ __align__(16) float s_q[kC * LK], s_k[kC * LK];
  __shared__ __align__(16) float s_p[kC * LP], s_a[DELTA ? kC * LP : 4];
  __shared__ double s_L[kC];
  __shared__ float s_g[kC], s_e[kC], s_w[kC];        // e^{L_i}, e^{L_C - L_i}, dt_i or beta_i
  __shared__ float s_gc;                             // e^{L_C}
  const int sg = blockIdx.x, hd = blockIdx.y;
  const int r0 = a.cu[sg], len = a.cu[sg + 1] - r0;
  if (len <= 0) return;
  const int tid = threadIdx.x, lane = tid & 63, w = tid >> 6, c = lane & 31, hi = lane >> 5;
  const int Dk = a.Dk, Dv = a.Dv;
  const int col = (blockIdx.z * NW + w) * 32 + c;
  const bool on = col < Dv;
  const bool wave_on = (blockIdx.z * NW + w) * 32 < Dv;
  const int qcol = (hd / a.rep) * Dk;

  f32x16 S[KT];
  float* sp = a.state + ((long long)a.slot[sg] * a.H + hd) * Dk * Dv + col;
  const bool fresh = a.start[sg] == 0;
#pragma unroll
  for (int kt = 0; kt < KT; ++kt)
#pragma unroll
    for (int r = 0; r < 16; ++r) {
      const int row = 32 * kt + 8 * (r >> 2) + 4 * hi + (r & 3);
      S[kt][r] = (!fresh && on && row < Dk) ? sp[(long long)row * Dv] : 0.f;
    }
  const float skip = a.skip != nullptr ? a.skip[hd] : 0.f;

  for (int t0 = 0; t0 < len; t0 += kC) {
    const int n = min(kC, len - t0);
    const long long row0 = r0 + t0;
    __syncthreads();                                 // the previous chunk has been consumed
    // the wave's values: lane = column, register r = token 8 (r >> 2) + 4 hi + (r & 3)
    float V[16];
#pragma unroll
    for (int r = 0; r < 16; ++r) {
      const int i = 8 * (r >> 2) + 4 * hi + (r & 3);
      V[r] = (on && i < n) ? to_f32(a.v[(row0 + i) * a.ldv + (long long)hd * Dv + col]) : 0.f;
    }
    // ---- stage q and k: TPR threads per token ----
    {
      const int i = tid / TPR, p = tid % TPR;
      float ssq = 0.f, ssk = 0.f;
      const T* qr = a.q + (row0 + i) * a.ldq + qcol;
      const T* kr = a.k + (row0 + i) * a.ldk + qcol;
#pragma unroll 4
      for (int g = p; g < DKP / 4; g += TPR) {
        const int d = 4 * g;
        float qv[4] = {0.f, 0.f, 0.f, 0.f}, kv[4] = {0.f, 0.f, 0.f, 0.f};
        if (i < n && d < Dk) {
          if (a.vec) {
            load4<T>(qr + d, qv);
            load4<T>(kr + d, kv);
          } else {
#pragma unroll
            for (int e = 0; e < 4; ++e)
              if (d + e < Dk) { qv[e] = to_f32(qr[d + e]); kv[e] = to_f32(kr[d + e]); }
          }
          if (a.silu_in) {
#pragma unroll
            for (int e = 0; e < 4; ++e) { qv[e] = silu_stored<T>(qv[e]); kv[e] = silu_stored<T>(kv[e]); }
          }
          if (DELTA) {
#pragma unroll
            for (int e = 0; e < 4; ++e) { ssq += qv[e] * qv[e]; ssk += kv[e] * kv[e]; }
          }
        }
        store4<float>(&s_q[i * LK + d], qv);
        store4<float>(&s_k[i * LK + d], kv);
      }
      if (DELTA) {                                   // unit vectors: a thread rescales its own
#pragma unroll
        for (int m = 1; m < TPR; m <<= 1) {
          ssq += __shfl_xor(ssq, m, 64);
          ssk += __shfl_xor(ssk, m, 64);
        }
        const float fq = a.q_scale / sqrtf(ssq + a.key_eps), fk = 1.f / sqrtf(ssk + a.key_eps);
#pragma unroll 4
        for (int g = p; g < DKP / 4; g += TPR) {
          float4* q4 = reinterpret_cast<float4*>(&s_q[i * LK + 4 * g]);
          float4* k4 = reinterpret_cast<float4*>(&s_k[i * LK + 4 * g]);
          float4 x = *q4, y = *k4;
          x.x *= fq; x.y *= fq; x.z *= fq; x.w *= fq;
          y.x *= fk; y.y *= fk; y.z *= fk; y.w *= fk;
          *q4 = x; *k4 = y;
        }
      }
    }
    // ---- decays: wave 0, one lane per token (both halves compute the same) ----
    if (w == 0) {
      float ld = 0.f, dt = 0.f;
      if (c < n) head_decay(a, row0 + c, hd, ld, dt);
      double L = (double)ld;
#pragma unroll
      for (int m = 1; m < 32; m <<= 1) {
        const double o = __shfl_up(L, m, 32);
        if (c >= m) L += o;
      }
      const double Lc = __shfl(L, 31, 32);           // tokens past the end add nothing
      if (hi == 0) {
        s_L[c] = L;
        s_g[c] = expf((float)L);
        s_e[c] = expf((float)(Lc - L));
        s_w[c] = DELTA ? (c < n ? sigmoid_f(to_f32(a.b[(row0 + c) * a.ldb + hd])) : 0.f) : dt;
        if (c == 0) s_gc = expf((float)Lc);
      }
    }
    __syncthreads();
    // ---- the chunk matrices, 16x16 tiles on and below the diagonal dealt out to the waves ----
    {
      constexpr int NJ = DELTA ? 6 : 3;
      const int lr = lane & 15, lg = lane >> 4;
      for (int job = w; job < NJ; job += NW) {
        const int tile = job % 3, ti = tile > 0, tj = tile > 1;   // (0,0) (1,0) (1,1)
        const bool kk = job >= 3;
        const float* x = (kk ? s_k : s_q) + (16 * ti + lr) * LK + 4 * lg;
        const float* y = s_k + (16 * tj + lr) * LK + 4 * lg;
        f32x4 acc = {0.f, 0.f, 0.f, 0.f};
#pragma unroll 4
        for (int m = 0; m < DKP / 16; ++m) {
          const float4 xa = *reinterpret_cast<const float4*>(x + 16 * m);
          const float4 ya = *reinterpret_cast<const float4*>(y + 16 * m);
          acc = mma16(xa.x, ya.x, acc);
          acc = mma16(xa.y, ya.y, acc);
          acc = mma16(xa.z, ya.z, acc);
          acc = mma16(xa.w, ya.w, acc);
        }
        float* dst = kk ? s_a : s_p;
        const int j = 16 * tj + lr;
        const double Lj = s_L[j];
#pragma unroll
        for (int e = 0; e < 4; ++e) {
          const int i = 16 * ti + 4 * lg + e;
          const bool low = kk ? j < i : j <= i;
          float z = low ? acc[e] * expf((float)(s_L[i] - Lj)) : 0.f;
          if (kk) z *= s_w[i];
          dst[i * LP + j] = z;
        }
        if (tile == 0) {                             // the tile above the diagonal
#pragma unroll
          for (int e = 0; e < 4; ++e) dst[(4 * lg + e) * LP + 16 + lr] = 0.f;
        }
      }
    }
    if (DELTA) {
      __syncthreads();
      // ---- (I + A)^-1 in place: the two diagonal 16x16 blocks by substitution (a lane per
      //      column), the block below as -T11 A10 T00 ----
      if (w == 0) {
        if (lane < 32) {
          const int b0 = lane & 16, cc = lane & 15;
          float t[16];
#pragma unroll
          for (int i = 0; i < 16; ++i) {
            float acc = 0.f;
#pragma unroll
            for (int j4 = 0; j4 < 16; j4 += 4) {
              if (j4 < i) {
                const float4 x = *reinterpret_cast<const float4*>(&s_a[(b0 + i) * LP + b0 + j4]);
                acc += x.x * t[j4];
                if (j4 + 1 < i) acc += x.y * t[j4 + 1];
                if (j4 + 2 < i) acc += x.z * t[j4 + 2];
                if (j4 + 3 < i) acc += x.w * t[j4 + 3];
              }
            }
            t[i] = i == cc ? 1.f : (i > cc ? -acc : 0.f);
          }
          wave_lds_fence();
#pragma unroll
          for (int i = 0; i < 16; ++i) s_a[(b0 + i) * LP + b0 + cc] = t[i];
        }
        wave_lds_fence();
        const int lr = lane & 15, lg = lane >> 4;
        f32x4 x = {0.f, 0.f, 0.f, 0.f}, y = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int m = 0; m < 4; ++m)                  // X = A10 T00
          x = mma16(s_a[(16 + lr) * LP + 4 * m + lg], s_a[(4 * m + lg) * LP + lr], x);
#pragma unroll
        for (int e = 0; e < 4; ++e)                  // inner index 4 lg + e is X's register e
          y = mma16(s_a[(16 + lr) * LP + 16 + 4 * lg + e], x[e], y);
        wave_lds_fence();
#pragma unroll
        for (int e = 0; e < 4; ++e) s_a[(16 + 4 * lg + e) * LP + lr] = -y[e];
      }
    }
    // ---- what the old state gives: Q S_0 and (delta) K S_0 ----
    f32x16 O, U;
#pragma unroll
    for (int r = 0; r < 16; ++r) { O[r] = 0.f; U[r] = 0.f; }
    if (wave_on) {
#pragma unroll
      for (int kt = 0; kt < KT; ++kt) {
        O = mma_rows(&s_q[c * LK + 32 * kt + 4 * hi], S[kt], O);
        if (DELTA) U = mma_rows(&s_k[c * LK + 32 * kt + 4 * hi], S[kt], U);
      }
    }
    __syncthreads();                                 // chunk matrices complete
    if (!wave_on) continue;
    if (a.silu_in) {
#pragma unroll
      for (int r = 0; r < 16; ++r) V[r] = silu_f(V[r]);    // silu(0) = 0
    }
    if (DELTA) {
      f32x16 R;
#pragma unroll
      for (int r = 0; r < 16; ++r) {
        const int i = 8 * (r >> 2) + 4 * hi + (r & 3);
        R[r] = s_w[i] * (V[r] - s_g[i] * U[r]);
        U[r] = 0.f;
      }
      U = mma_rows(&s_a[c * LP + 4 * hi], R, U);
    } else {
#pragma unroll
      for (int r = 0; r < 16; ++r) U[r] = s_w[8 * (r >> 2) + 4 * hi + (r & 3)] * V[r];
    }
#pragma unroll
    for (int r = 0; r < 16; ++r) O[r] = s_g[8 * (r >> 2) + 4 * hi + (r & 3)] * O[r] + skip * V[r];
    O = mma_rows(&s_p[c * LP + 4 * hi], U, O);
    if (on) {
#pragma unroll
      for (int r = 0; r < 16; ++r) {
        const int i = 8 * (r >> 2) + 4 * hi + (r & 3);
        if (i < n) a.out[(row0 + i) * ((long long)a.H * Dv) + (long long)hd * Dv + col] = O[r];
      }
    }
    // ---- the state moves on ----
    const float gc = s_gc;
#pragma unroll
    for (int r = 0; r < 16; ++r) U[r] *= s_e[8 * (r >> 2) + 4 * hi + (r & 3)];
#pragma unroll
    for (int kt = 0; kt < KT; ++kt) {
#pragma unroll
      for (int r = 0; r < 16; ++r) S[kt][r] *= gc;
#pragma unroll
      for (int r = 0; r < 16; ++r)
        S[kt] = mma32(s_k[(8 * (r >> 2) + 4 * hi + (r & 3)) * LK + 32 * kt + c], U[r], S[kt]);
    }
  }
  if (on) {
#pragma unroll
    for (int kt = 0; kt < KT; ++kt)
#pragma unroll
      for (int r = 0; r < 16; ++r) {
        const int row = 32 * kt + 8 * (r >> 2) + 4 * hi + (r & 3);
        if (row < Dk) sp[(long long)row * Dv] = S[kt][r];
      }
  }
}

template <typename T, bool DELTA>
hipError_t launch_chunk(const HeadScanArgs<T>& a, int n_seg, hipStream_t st) {
  const int cb = (a.Dv + 31) / 32;                   // 32-column blocks
#define GO(KT, NW)                                                             \
  head_scan_chunk_kernel<T, KT, NW, DELTA>                                     \
      <<<dim3(n_seg, a.H, (cb + NW - 1) / NW), 64 * NW, 0, st>>>(a)
#define GO_K(KT)                 \
  if (cb == 1) GO(KT, 1);        \
  else if (cb == 2) GO(KT, 2);   \
  else GO(KT, 4)
  if (a.Dk <= 32) { GO_K(1); }
  else if (a.Dk <= 64) { GO_K(2); }
  else if (a.Dk <= 128) { GO_K(4); }
  else { GO_K(8); }
#undef GO_K
#undef GO
  return hipGetLastError();
}

}  // namespace

extern "C" {

hipError_t sm_head_scan_chunk(int dt, int delta, const void* q, long long ldq, const void* k,
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
  const int vec = Dk % 4 == 0 && ldq % 4 == 0 && ldk % 4 == 0 && (uintptr_t)q % 16 == 0 &&
                  (uintptr_t)k % 16 == 0;
#define ARGS(T)                                                                               \
  HeadScanArgs<T> a{(const T*)q, ldq, (const T*)k, ldk, (const T*)v, ldv, (const T*)al, lda,  \
                    (const T*)bl, ldb, A_log, dt_bias, log_decay, skip, state, out, cu, slot, \
                    start, H, rep, Dk, Dv, silu_in, vec, key_eps, q_scale}
  if (dt == kBF16) {
    ARGS(bf16);
    return head_scan_chunk16(a, delta != 0, n_seg, st);
  }
#define CALL(T)                                                                                 \
  {                                                                                             \
    ARGS(T);                                                                                    \
    return delta ? launch_chunk<T, true>(a, n_seg, st) : launch_chunk<T, false>(a, n_seg, st);  \
  }
  if (dt == kF32) CALL(float)
  if (dt == kF16) CALL(fp16)
  return hipErrorInvalidValue;
#undef CALL
#undef ARGS
}

}  // extern "C"
