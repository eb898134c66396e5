// The chunked matrix-state recurrences of head_scan_chunk.hip for bf16 models, on the bf16 matrix
// instructions (sixteen times the fp32 ones' rate) at fp32-level accuracy, with the chunk matrices
// built ahead of their use.
//
//   U   = dt * V                                                   (linear)
//   U   = (I + strict_lower(beta_i G_ij k_i.k_j))^-1 (beta (V - e^L K S_0))       (delta)
//   O   = e^L (Q S_0) + (G . Q K^T) U (+ skip V)
//   S_C = e^{L_C} S_0 + K^T (e^{L_C - L} U)
//
// Operands: the rows of q and k ARE bf16 (convolution outputs, or silu of a projection rounded
// once), so they enter exactly; the delta rule's unit lengths are fp32 factors of rows and columns
// (of Q S_0, K S_0, Q K^T, K K^T and U) instead of a rescaled copy.  Every fp32 operand -- the
// state, U, the two chunk matrices -- is split into a bf16 head and a bf16 remainder: two products
// (three where both sides are split) keep ~16 mantissa bits; sums are fp32.  The state itself
// stays fp32 in accumulator registers, a wave holding [Dk x 32 value columns].
//
// A workgroup is NW column waves and TWO producer waves, and two LDS buffers: while the column waves
// run chunk n, the producers build chunk n + 1 in two phases with a barrier after each.  First one
// stores q and the decays, the other k and k transposed, from registers they loaded one chunk
// earlier, and both start loading chunk n + 2 (meanwhile the column waves take Q S_0 and K S_0);
// then one forms G . Q K^T and the other the triangular inverse (meanwhile: U, O and the state).
//
// 32x32x16 products: accumulator register r of lane half hi is row 8 (r >> 2) + 4 hi + (r & 3); the
// registers 8s .. 8s+7 therefore hold inner indices {16s + 4hi + 0..3, 16s + 8 + 4hi + 0..3} and are
// a right operand as they are when the left operand is stored in that order: in every 16 entries of
// an LDS row the 4-entry groups 1 and 2 are swapped, and a lane reads its 8 entries as 16 bytes.
#include "head_scan.h"

#include <type_traits>

using namespace lumen;

namespace {

typedef float f32x16 __attribute__((ext_vector_type(16)));
typedef float f32x4 __attribute__((ext_vector_type(4)));
typedef __bf16 bf16x8v __attribute__((ext_vector_type(8)));

constexpr int kC = 32;             // tokens per chunk
constexpr int LT = kC + 8;         // row stride of token-inner LDS images
constexpr int LA = kC + 4;         // row stride of the fp32 scratch of the inverse

__device__ __forceinline__ f32x16 mma(uint4 a, uint4 b, f32x16 c) {
  return __builtin_amdgcn_mfma_f32_32x32x16_bf16(__builtin_bit_cast(bf16x8v, a),
                                                 __builtin_bit_cast(bf16x8v, b), c, 0, 0, 0);
}
__device__ __forceinline__ f32x4 mma16f(float a, float b, f32x4 c) {
  return __builtin_amdgcn_mfma_f32_16x16x4f32(a, b, c, 0, 0, 0);
}
__device__ __forceinline__ float lo_half(unsigned v) { return __uint_as_float(v << 16); }
__device__ __forceinline__ float hi_half(unsigned v) { return __uint_as_float(v & 0xffff0000u); }

// 8 fp32 values (registers 8s .. 8s+7 of x) -> bf16 head and remainder
__device__ __forceinline__ void split8(const f32x16& x, int s, uint4& h, uint4& l) {
  unsigned hh[4], ll[4];
#pragma unroll
  for (int e = 0; e < 4; ++e) {
    const float a = x[8 * s + 2 * e], b = x[8 * s + 2 * e + 1];
    hh[e] = pk2<bf16>(a, b);
    ll[e] = pk2<bf16>(a - lo_half(hh[e]), b - hi_half(hh[e]));
  }
  h = make_uint4(hh[0], hh[1], hh[2], hh[3]);
  l = make_uint4(ll[0], ll[1], ll[2], ll[3]);
}

// hardware exponential and reciprocal: for values that are rounded to bf16 next
__device__ __forceinline__ float silu_fast(float x) {
  return x * __builtin_amdgcn_rcpf(1.f + __expf(-x));
}
__device__ __forceinline__ unsigned silu_pair(unsigned v) {
  return pk2<bf16>(silu_fast(lo_half(v)), silu_fast(hi_half(v)));
}

__device__ __forceinline__ void wave_lds_fence() {
  __builtin_amdgcn_fence(__ATOMIC_RELEASE, "wavefront");
  __builtin_amdgcn_wave_barrier();
  __builtin_amdgcn_fence(__ATOMIC_ACQUIRE, "wavefront");
}

// place of inner index j in its LDS row
__device__ __forceinline__ int place(int j) {
  return (j & ~15) + 8 * ((j >> 2) & 1) + 4 * ((j >> 3) & 1) + (j & 3);
}

template <int DKP, bool DELTA>
struct __align__(16) ChunkBuf {
  bf16 q[kC * (DKP + 8)], k[kC * (DKP + 8)];   // [token][channel]
  bf16 kt[DKP * LT];                           // [channel][token]
  bf16 p[2][kC * LT];                          // G . Q K^T, head and remainder
  bf16 t[DELTA ? 2 : 1][DELTA ? kC * LT : 8];  // the inverse
  float gq[kC], gk[kC], w[kC], ek[kC];         // e^L |q|, e^L |k|, dt or beta, e^{L_C - L} |k|
  float gc, pad[3];                            // e^{L_C}
};

// four rows of 8 channels each of q or k
struct Item { uint4 r[4]; };

// four fp32 values -> bf16 head and remainder, 8 bytes each
__device__ __forceinline__ void put4(bf16* h, bf16* l, float a, float b, float c, float d) {
  const unsigned h0 = pk2<bf16>(a, b), h1 = pk2<bf16>(c, d);
  *reinterpret_cast<uint2*>(h) = make_uint2(h0, h1);
  *reinterpret_cast<uint2*>(l) = make_uint2(pk2<bf16>(a - lo_half(h0), b - hi_half(h0)),
                                            pk2<bf16>(c - lo_half(h1), d - hi_half(h1)));
}

// the diagonal entry of a 32x32 accumulator: lane c's column c, in either half
__device__ __forceinline__ float diagonal(const f32x16& x, int c, int hi) {
  float d = 0.f;
#pragma unroll
  for (int r = 0; r < 16; ++r) d = 8 * (r >> 2) + 4 * hi + (r & 3) == c ? x[r] : d;
  return d + __shfl_xor(d, 32, 64);
}

template <int KT, int NW, bool DELTA>
__global__ void __launch_bounds__(64 * (NW + 2))
head_scan_chunk16_kernel(const HeadScanArgs<bf16> a) {
  constexpr int DKP = 32 * KT, LK = DKP + 8, NV = DKP / 8;
  constexpr int NI = (DKP + 63) / 64;          // items per producer lane and matrix
  using Buf = ChunkBuf<DKP, DELTA>;
  __shared__ Buf s_buf[2];
  __shared__ __align__(16) double s_L[kC];     // the producers': log-decay sums, unit factors
  __shared__ __align__(16) float s_fk[2][kC];
  const int sg = blockIdx.x, hd = blockIdx.y;
  const int r0 = a.cu[sg], len = a.cu[sg + 1] - r0;
  if (len <= 0) return;
  const int tid = threadIdx.x, lane = tid & 63, w = tid >> 6, c = lane & 31, hi = lane >> 5;
  const int Dk = a.Dk, Dv = a.Dv;
  const int chunks = (len + kC - 1) / kC;
  const int qcol = (hd / a.rep) * Dk;

  // Rows past the segment's end are read as its last row: their step size (or beta) is zero, so
  // they add nothing to the state, and their read-outs are not stored.
  if (w >= NW) {
    // ---------------- the producer waves ----------------
    const bool is_k = w > NW;
    const bf16* base = is_k ? a.k : a.q;
    const long long ldr = is_k ? a.ldk : a.ldq;
    Item it[NI];
    float ra = 0.f, rb = 0.f;                  // the token's decay and write-strength logits
    auto fetch = [&](int t0) __attribute__((always_inline)) {
#pragma unroll
      for (int x = 0; x < NI; ++x) {
        const int item = lane + 64 * x, kq = (item / NV) & 7, d = 8 * (item % NV);
#pragma unroll
        for (int y = 0; y < 4; ++y) {
          const int i = min(t0 + 4 * kq + y, len - 1);
          const bf16* p = base + (long long)(r0 + i) * ldr + qcol + d;
          uint4 v = make_uint4(0, 0, 0, 0);
          if (d < Dk) {
            if (a.vec) {
              v = *reinterpret_cast<const uint4*>(p);
            } else {
              unsigned e[8];
#pragma unroll
              for (int z = 0; z < 8; ++z)
                e[z] = d + z < Dk ? (unsigned)__builtin_bit_cast(unsigned short, p[z]) : 0u;
              v = make_uint4(e[0] | e[1] << 16, e[2] | e[3] << 16, e[4] | e[5] << 16,
                             e[6] | e[7] << 16);
            }
          }
          it[x].r[y] = v;
        }
      }
      if (!is_k) {
        const long long i = r0 + min(t0 + c, len - 1);
        if (a.a != nullptr) ra = to_f32(a.a[i * a.lda + hd]);
        if (DELTA) rb = to_f32(a.b[i * a.ldb + hd]);
      }
    };
    const float dtb = a.a != nullptr ? a.dt_bias[hd] : 0.f;
    const float eA = a.a != nullptr ? expf(a.A_log[hd]) : 0.f;
    const float ldc = a.a != nullptr ? 0.f : a.log_decay[hd];

    double L = 0.0, Lc = 0.0;                  // (the q wave) the lane's log-decay sum, the chunk's

    // phase 1: rows into LDS, decays
    auto rows = [&](int t0, Buf& B) __attribute__((always_inline)) {
      bf16* dst = is_k ? B.k : B.q;
#pragma unroll
      for (int x = 0; x < NI; ++x) {
        const int item = lane + 64 * x, kq = item / NV, part = item % NV;
        if (a.silu_in) {
#pragma unroll
          for (int y = 0; y < 4; ++y) {
            uint4& v = it[x].r[y];
            v = make_uint4(silu_pair(v.x), silu_pair(v.y), silu_pair(v.z), silu_pair(v.w));
          }
        }
        if (item < DKP) {
          const int s16 = 16 * (part >> 1) + 4 * (part & 1);
#pragma unroll
          for (int y = 0; y < 4; ++y) {
            bf16* row = dst + (4 * kq + y) * LK + s16;
            *reinterpret_cast<uint2*>(row) = make_uint2(it[x].r[y].x, it[x].r[y].y);
            *reinterpret_cast<uint2*>(row + 8) = make_uint2(it[x].r[y].z, it[x].r[y].w);
          }
          if (is_k) {                          // transposed: 4 tokens of each of the 8 channels
            const unsigned e0[4] = {it[x].r[0].x, it[x].r[0].y, it[x].r[0].z, it[x].r[0].w};
            const unsigned e1[4] = {it[x].r[1].x, it[x].r[1].y, it[x].r[1].z, it[x].r[1].w};
            const unsigned e2[4] = {it[x].r[2].x, it[x].r[2].y, it[x].r[2].z, it[x].r[2].w};
            const unsigned e3[4] = {it[x].r[3].x, it[x].r[3].y, it[x].r[3].z, it[x].r[3].w};
            // 16-byte unit of the row (swapped by the channel group: lanes spread over banks)
            const int unit = (2 * (kq >> 2) + (kq & 1)) ^ (part & 3);
            bf16* t = B.kt + 8 * part * LT + 8 * unit + 4 * ((kq >> 1) & 1);
#pragma unroll
            for (int z = 0; z < 4; ++z) {
              *reinterpret_cast<uint2*>(t + 2 * z * LT) =
                  make_uint2((e0[z] & 0xffffu) | (e1[z] << 16), (e2[z] & 0xffffu) | (e3[z] << 16));
              *reinterpret_cast<uint2*>(t + (2 * z + 1) * LT) = make_uint2(
                  (e0[z] >> 16) | (e1[z] & 0xffff0000u), (e2[z] >> 16) | (e3[z] & 0xffff0000u));
            }
          }
        }
      }
      if (!is_k) {
        // lane c (both halves alike) is token c; tokens past the end add nothing
        const bool live = t0 + c < len;
        float ld = ldc, dt = 1.f;
        if (a.a != nullptr) {
          dt = softplus_f(ra + dtb);
          ld = -eA * dt;
        }
        const float wt = DELTA ? sigmoid_f(rb) : dt;
        L = live ? (double)fmaxf(ld, -1e4f) : 0.0;
#pragma unroll
        for (int m = 1; m < 32; m <<= 1) {
          const double o = __shfl_up(L, m, 32);
          if (c >= m) L += o;
        }
        Lc = __shfl(L, 31, 32);
        if (hi == 0) {
          s_L[c] = L;
          B.w[c] = live ? wt : 0.f;
        }
      }
      if (t0 + kC < len) fetch(t0 + kC);       // the next chunk's rows travel meanwhile
    };

    // phase 2: P^T = K Q^T (lane: query, registers: keys) times G, and the chunk's factors
    auto weights = [&](Buf& B) __attribute__((always_inline)) {
      f32x16 P, A, Q;
#pragma unroll
      for (int r = 0; r < 16; ++r) { P[r] = 0.f; A[r] = 0.f; Q[r] = 0.f; }
#pragma unroll 4
      for (int s = 0; s < 2 * KT; ++s) {
        const uint4 kv = *reinterpret_cast<const uint4*>(B.k + c * LK + 16 * s + 8 * hi);
        const uint4 qv = *reinterpret_cast<const uint4*>(B.q + c * LK + 16 * s + 8 * hi);
        P = mma(kv, qv, P);
        if (DELTA) {                           // unit lengths: the diagonals of K K^T and Q Q^T
          A = mma(kv, kv, A);
          Q = mma(qv, qv, Q);
        }
      }
      float fqc = 1.f, fkc = 1.f;
      if (DELTA) {
        fqc = a.q_scale / sqrtf(diagonal(Q, c, hi) + a.key_eps);
        fkc = 1.f / sqrtf(diagonal(A, c, hi) + a.key_eps);
        if (hi == 0) s_fk[0][c] = fkc;
        wave_lds_fence();
      }
      if (hi == 0) {
        const float g = expf((float)L);
        B.gq[c] = g * fqc;
        B.gk[c] = g * fkc;
        B.ek[c] = expf((float)(Lc - L)) * fkc;
        if (c == 0) B.gc = expf((float)Lc);
      }
#pragma unroll
      for (int g = 0; g < 4; ++g) {
        const int j0 = 8 * g + 4 * hi;         // registers 4g + e: token j0 + e
        const double2 La = *reinterpret_cast<const double2*>(&s_L[j0]);
        const double2 Lb = *reinterpret_cast<const double2*>(&s_L[j0 + 2]);
        const float d[4] = {(float)(L - La.x), (float)(L - La.y), (float)(L - Lb.x),
                            (float)(L - Lb.y)};
        float fk[4] = {1.f, 1.f, 1.f, 1.f}, z[4];
        if (DELTA) load4<float>(&s_fk[0][j0], fk);
#pragma unroll
        for (int e = 0; e < 4; ++e) {
          const float v = P[4 * g + e] * (fqc * fk[e]) * __expf(fminf(d[e], 0.f));
          z[e] = j0 + e <= c ? v : 0.f;
        }
        const int at = c * LT + place(j0);
        put4(&B.p[0][at], &B.p[1][at], z[0], z[1], z[2], z[3]);
      }
    };

    // phase 2, delta rule: T = (I + A)^-1
    auto inverse = [&](Buf& B) __attribute__((always_inline)) {
      f32x16 A;
#pragma unroll
      for (int r = 0; r < 16; ++r) A[r] = 0.f;
#pragma unroll
      for (int s = 0; s < 2 * KT; ++s) {
        const uint4 kv = *reinterpret_cast<const uint4*>(B.k + c * LK + 16 * s + 8 * hi);
        A = mma(kv, kv, A);
      }
      const float fkc = 1.f / sqrtf(diagonal(A, c, hi) + a.key_eps);
      if (hi == 0) s_fk[1][c] = fkc;
      wave_lds_fence();
      // scratch, transposed: row c, entry j = A[j][c] (j > c); it lies where T is written later
      float* sA = reinterpret_cast<float*>(B.t[0]);
      static_assert(!DELTA || sizeof(float) * kC * LA <= sizeof(B.t), "scratch fits");
      const double Lo = s_L[c];
#pragma unroll
      for (int g = 0; g < 4; ++g) {
        const int j0 = 8 * g + 4 * hi;
        const double2 La = *reinterpret_cast<const double2*>(&s_L[j0]);
        const double2 Lb = *reinterpret_cast<const double2*>(&s_L[j0 + 2]);
        const float d[4] = {(float)(La.x - Lo), (float)(La.y - Lo), (float)(Lb.x - Lo),
                            (float)(Lb.y - Lo)};
        float fk[4], be[4], x[4];
        load4<float>(&s_fk[1][j0], fk);
        load4<float>(&B.w[j0], be);
#pragma unroll
        for (int e = 0; e < 4; ++e)
          x[e] = j0 + e > c ? A[4 * g + e] * (fk[e] * fkc) * (be[e] * __expf(fminf(d[e], 0.f))) : 0.f;
        store4<float>(&sA[c * LA + j0], x);
      }
      wave_lds_fence();
      // the diagonal 16x16 blocks by back substitution along a row,
      // T[i][j] = [i = j] - sum_{k > j} T[i][k] A[k][j], a lane per row i ...
      const int b0 = lane & 16, ii = lane & 15, lr = lane & 15, lg = lane >> 4;
      float t[16];
#pragma unroll
      for (int j = 15; j >= 0; --j) {
        float acc = 0.f;
#pragma unroll
        for (int k4 = 0; k4 < 16; k4 += 4) {
          if (k4 + 3 > j) {
            const float4 x = *reinterpret_cast<const float4*>(&sA[(b0 + j) * LA + b0 + k4]);
            if (k4 > j) acc += x.x * t[k4];
            if (k4 + 1 > j) acc += x.y * t[k4 + 1];
            if (k4 + 2 > j) acc += x.z * t[k4 + 2];
            acc += x.w * t[k4 + 3];
          }
        }
        t[j] = j == ii ? 1.f : (j < ii ? -acc : 0.f);
      }
      wave_lds_fence();
      if (lane < 32) {
#pragma unroll
        for (int j = 0; j < 16; j += 4)
          *reinterpret_cast<float4*>(&sA[(b0 + ii) * LA + b0 + j]) =
              make_float4(t[j], t[j + 1], t[j + 2], t[j + 3]);
      }
      wave_lds_fence();
      // ... and the block below as -T11 (A10 T00); A10[r][k] lies at scratch [k][16 + r]
      f32x4 x = {0.f, 0.f, 0.f, 0.f}, y = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int m = 0; m < 4; ++m)
        x = mma16f(sA[(4 * m + lg) * LA + 16 + lr], sA[(4 * m + lg) * LA + lr], x);
#pragma unroll
      for (int e = 0; e < 4; ++e) y = mma16f(sA[(16 + lr) * LA + 16 + 4 * lg + e], x[e], y);
      wave_lds_fence();                        // scratch read: T may be written over it
      bf16 *th = B.t[0], *tl = B.t[DELTA ? 1 : 0];
      if (lane < 32) {
#pragma unroll
        for (int j = 0; j < 16; j += 4) {
          const int at = (b0 + ii) * LT + place(b0 + j);
          put4(th + at, tl + at, t[j], t[j + 1], t[j + 2], t[j + 3]);
        }
      } else if (lane < 48) {                  // the block above the diagonal
#pragma unroll
        for (int j = 16; j < 32; j += 4) {
          const int at = ii * LT + place(j);
          put4(th + at, tl + at, 0.f, 0.f, 0.f, 0.f);
        }
      }
#pragma unroll
      for (int e = 0; e < 4; ++e) {
        const int at = (16 + 4 * lg + e) * LT + place(lr);
        const bf16 h = __float2bfloat16(-y[e]);
        th[at] = h;
        tl[at] = __float2bfloat16(-y[e] - __bfloat162float(h));
      }
    };

    fetch(0);
    for (int n = 0; n <= chunks; ++n) {        // chunk n is built while the others run chunk n - 1
      Buf& B = s_buf[n & 1];
      if (n < chunks) rows(n * kC, B);
      __syncthreads();
      if (n < chunks) {
        if (!is_k) weights(B);
        else if (DELTA) inverse(B);
      }
      __syncthreads();
    }
    return;
  }

  // ---------------- the column waves ----------------
  const int col = (blockIdx.z * NW + w) * 32 + c;
  const bool on = col < Dv;
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
  const bf16* vp = a.v + (long long)r0 * a.ldv + (long long)hd * Dv + (on ? col : 0);
  float* op = a.out + (long long)r0 * ((long long)a.H * Dv) + (long long)hd * Dv + col;
  const long long ldo = (long long)a.H * Dv;
  bf16 vn[16];
  auto fetch_v = [&](int t0) __attribute__((always_inline)) {
#pragma unroll
    for (int r = 0; r < 16; ++r) {
      const int i = min(t0 + 8 * (r >> 2) + 4 * hi + (r & 3), len - 1);
      vn[r] = vp[(long long)i * a.ldv];
    }
  };
  fetch_v(0);
  __syncthreads();
  __syncthreads();
  for (int ch = 0; ch < chunks; ++ch) {
    const Buf& B = s_buf[ch & 1];
    const int t0 = ch * kC, n = min(kC, len - t0);
    float V[16];
#pragma unroll
    for (int r = 0; r < 16; ++r) {
      V[r] = to_f32(vn[r]);
      if (a.silu_in) V[r] = silu_fast(V[r]);
    }
    if (ch + 1 < chunks) fetch_v(t0 + kC);
    // what the old state gives: Q S_0 and (delta) K S_0
    f32x16 O, U;
#pragma unroll
    for (int r = 0; r < 16; ++r) { O[r] = 0.f; U[r] = 0.f; }
#pragma unroll
    for (int kt = 0; kt < KT; ++kt)
#pragma unroll
      for (int s = 0; s < 2; ++s) {
        uint4 h, l;
        split8(S[kt], s, h, l);
        const int at = c * LK + 32 * kt + 16 * s + 8 * hi;
        const uint4 qv = *reinterpret_cast<const uint4*>(B.q + at);
        O = mma(qv, h, O);
        O = mma(qv, l, O);
        if (DELTA) {
          const uint4 kv = *reinterpret_cast<const uint4*>(B.k + at);
          U = mma(kv, h, U);
          U = mma(kv, l, U);
        }
      }
    __syncthreads();
    // the chunk matrices times a split right operand
    auto apply = [&](const bf16* mh, const bf16* ml, const f32x16& x, f32x16 acc) __attribute__((always_inline)) {
#pragma unroll
      for (int s = 0; s < 2; ++s) {
        uint4 h, l;
        split8(x, s, h, l);
        const int at = c * LT + 16 * s + 8 * hi;
        const uint4 ah = *reinterpret_cast<const uint4*>(mh + at);
        const uint4 al = *reinterpret_cast<const uint4*>(ml + at);
        acc = mma(ah, h, acc);
        acc = mma(ah, l, acc);
        acc = mma(al, h, acc);
      }
      return acc;
    };
#pragma unroll
    for (int g = 0; g < 4; ++g) {
      float ww[4], gk[4];
      load4<float>(&B.w[8 * g + 4 * hi], ww);
      if (DELTA) load4<float>(&B.gk[8 * g + 4 * hi], gk);
#pragma unroll
      for (int e = 0; e < 4; ++e) {
        const int r = 4 * g + e;
        U[r] = DELTA ? ww[e] * (V[r] - gk[e] * U[r]) : ww[e] * V[r];
      }
    }
    if (DELTA) {
      f32x16 z;
#pragma unroll
      for (int r = 0; r < 16; ++r) z[r] = 0.f;
      U = apply(B.t[0], B.t[DELTA ? 1 : 0], U, z);
    }
#pragma unroll
    for (int g = 0; g < 4; ++g) {
      float gq[4];
      load4<float>(&B.gq[8 * g + 4 * hi], gq);
#pragma unroll
      for (int e = 0; e < 4; ++e) O[4 * g + e] = gq[e] * O[4 * g + e] + skip * V[4 * g + e];
    }
    O = apply(B.p[0], B.p[1], U, O);
    if (on) {
      float* orow = op + (long long)(t0 + 4 * hi) * ldo;
      if (n == kC) {
#pragma unroll
        for (int r = 0; r < 16; ++r) orow[(8 * (r >> 2) + (r & 3)) * ldo] = O[r];
      } else {
#pragma unroll
        for (int r = 0; r < 16; ++r)
          if (8 * (r >> 2) + 4 * hi + (r & 3) < n) orow[(8 * (r >> 2) + (r & 3)) * ldo] = O[r];
      }
    }
    // the state moves on
    const float gc = B.gc;
#pragma unroll
    for (int g = 0; g < 4; ++g) {
      float ek[4];
      load4<float>(&B.ek[8 * g + 4 * hi], ek);
#pragma unroll
      for (int e = 0; e < 4; ++e) U[4 * g + e] *= ek[e];
    }
    uint4 uh[2], ul[2];
    split8(U, 0, uh[0], ul[0]);
    split8(U, 1, uh[1], ul[1]);
#pragma unroll
    for (int kt = 0; kt < KT; ++kt) {
#pragma unroll
      for (int r = 0; r < 16; ++r) S[kt][r] *= gc;
#pragma unroll
      for (int s = 0; s < 2; ++s) {
        const int unit = (2 * s + hi) ^ ((c >> 3) & 3);
        const uint4 kv = *reinterpret_cast<const uint4*>(B.kt + (32 * kt + c) * LT + 8 * unit);
        S[kt] = mma(kv, uh[s], S[kt]);
        S[kt] = mma(kv, ul[s], S[kt]);
      }
    }
    __syncthreads();
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

template <bool DELTA>
hipError_t launch(const HeadScanArgs<bf16>& a, int n_seg, hipStream_t st) {
  // 32-column blocks; a grid that leaves half the CUs idle is cut finer (each column block's result
  // is the same whichever workgroup computes it)
  const int cb = (a.Dv + 31) / 32;
  const bool fine = cb > 2 && (long long)n_seg * a.H * ((cb + 3) / 4) <= 128;
#define GO(KT, NW)                                                             \
  head_scan_chunk16_kernel<KT, NW, DELTA>                                      \
      <<<dim3(n_seg, a.H, (cb + NW - 1) / NW), 64 * (NW + 2), 0, st>>>(a)
#define GO_K(KT)                                                               \
  if (cb == 1) GO(KT, 1);                                                      \
  else if (cb == 2 || fine) GO(KT, 2);                                         \
  else if (cb == 3) GO(KT, (KT == 8 ? 2 : 3));                                 \
  else GO(KT, (KT == 8 ? 2 : 4))   /* 256 state rows: two column waves' registers */
  if (a.Dk <= 32) { GO_K(1); }
  else if (a.Dk <= 64) { GO_K(2); }
  else if (a.Dk <= 128) { GO_K(4); }
  else { GO_K(8); }
#undef GO_K
#undef GO
  return hipGetLastError();
}

}  // namespace

namespace lumen {

hipError_t head_scan_chunk16(const HeadScanArgs<bf16>& args, bool delta, int n_seg,
                             hipStream_t st) {
  HeadScanArgs<bf16> a = args;
  a.vec = a.Dk % 8 == 0 && a.ldq % 8 == 0 && a.ldk % 8 == 0 && (uintptr_t)a.q % 16 == 0 &&
          (uintptr_t)a.k % 16 == 0;
  return delta ? launch<true>(a, n_seg, st) : launch<false>(a, n_seg, st);
}

}  // namespace lumen
