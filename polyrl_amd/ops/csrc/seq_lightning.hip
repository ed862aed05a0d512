// Linear attention with one fixed decay per head:
//
//   S <- d S + k v^T ,   o = S^T q ,   q, k, v = silu(projections)
//
// The state (Dk x Dv per head and sequence) is fp32 and carried in place; o
// leaves as fp32 for the norm over all heads.  Three kernels:
//
// lightning_step_kernel: single-token steps.  A block streams a 64-column
// piece of one state once (in and out, 16 bytes a lane, whole 128-byte lines a
// wave), row groups meet in LDS.  Bound: HBM.
//
// lightning_walk_kernel: any portion in either type, token by token (fp32
// activations, odd sizes).  16 columns x 4 row groups per wave, the state in
// registers, token tiles staged in LDS.
//
// lightning_chunk_kernel: bf16 portions, 64 tokens at a time on the matrix
// cores.  With a chunk's rows i, j and the state S before it,
//
//   o_i = d^(i+1) S^T q_i + sum_{j<=i} d^(i-j) (q_i . k_j) v_j
//   S   <- d^c S + sum_j d^(c-1-j) k_j v_j^T              (c rows)
//
// Powers of d, scores and the state are fp32.  An fp32 operand of a product
// (the state, a decayed key, a decayed score) enters the bf16 matrix cores as
// the sum of two bf16 numbers, which keeps 16 bits of it; q, k and v are bf16
// activations as they are.  A block holds one (sequence, head, 64 value
// columns); wave w owns rows 16w.. of the chunk for o and columns 16w.. of
// the state, which stays in its accumulators for the whole portion.
#include <torch/extension.h>
#include <ATen/hip/HIPContext.h>

#include "seq_common.h"

typedef __attribute__((ext_vector_type(8))) __bf16 bf16x8_t;
typedef __attribute__((ext_vector_type(4))) __bf16 bf16x4_t;
typedef __attribute__((ext_vector_type(4))) float f32x4_t;

// ------------------------------------------------------ single-token steps
constexpr int STEP_COLS = 64;

template <typename T, bool VEC>
__global__ __launch_bounds__(256) void lightning_step_kernel(
    float* __restrict__ out, const T* __restrict__ q, long ldq,
    const T* __restrict__ k, long ldk, const T* __restrict__ v, long ldv,
    const float* __restrict__ decay, float* __restrict__ state,
    const int* __restrict__ cu_q, const int* __restrict__ state_slot, int H,
    int Dk, int Dv) {
  constexpr int E = VEC ? 4 : 1;                 // columns of a lane
  constexpr int LPR = STEP_COLS / E;             // lanes of a state row
  constexpr int RGS = 256 / LPR;                 // row groups
  extern __shared__ float lds[];                 // [q | k | partial sums]
  float* q_s = lds;
  float* k_s = lds + Dk;
  float* o_s = lds + 2 * Dk;
  const int cblocks = (Dv + STEP_COLS - 1) / STEP_COLS;
  const int b = blockIdx.x / (H * cblocks);
  const int h = (blockIdx.x / cblocks) % H;
  const int cb = blockIdx.x % cblocks;
  const int n = cu_q[b];
  if (cu_q[b + 1] <= n) return;                  // the whole block
  for (int i = threadIdx.x; i < Dk; i += 256) {
    q_s[i] = siluf_acc(ldf(q + (long)n * ldq + h * Dk + i));
    k_s[i] = siluf_acc(ldf(k + (long)n * ldk + h * Dk + i));
  }
  const int rg = threadIdx.x / LPR;
  const int col = cb * STEP_COLS + (threadIdx.x % LPR) * E;
  const bool ok = col < Dv;
  const float dec = decay[h];
  float vv[E], o[E];
#pragma unroll
  for (int e = 0; e < E; ++e) {
    vv[e] = ok ? siluf_acc(ldf(v + (long)n * ldv + h * Dv + col + e)) : 0.f;
    o[e] = 0.f;
  }
  __syncthreads();
  float* S = state + ((long)state_slot[b] * H + h) * Dk * Dv + col;
  constexpr int U = 4;                           // rows in flight
  if (ok) {
    for (int r0 = rg; r0 < Dk; r0 += U * RGS) {
      float s[U][E];
#pragma unroll
      for (int u = 0; u < U; ++u) {
        const int r = min(r0 + u * RGS, Dk - 1);
        if (VEC) {
          const f32x4v x = *reinterpret_cast<const f32x4v*>(S + (long)r * Dv);
#pragma unroll
          for (int e = 0; e < E; ++e) s[u][e] = x.v[e];
        } else {
          s[u][0] = S[(long)r * Dv];
        }
      }
#pragma unroll
      for (int u = 0; u < U; ++u) {
        const int r = r0 + u * RGS;
        if (r < Dk) {
          const float kr = k_s[r], qr = q_s[r];
#pragma unroll
          for (int e = 0; e < E; ++e) {
            s[u][e] = dec * s[u][e] + kr * vv[e];
            o[e] += qr * s[u][e];
          }
          if (VEC) {
            f32x4v x;
#pragma unroll
            for (int e = 0; e < E; ++e) x.v[e] = s[u][e];
            *reinterpret_cast<f32x4v*>(S + (long)r * Dv) = x;
          } else {
            S[(long)r * Dv] = s[u][0];
          }
        }
      }
    }
  }
#pragma unroll
  for (int e = 0; e < E; ++e)
    o_s[rg * STEP_COLS + (threadIdx.x % LPR) * E + e] = o[e];
  __syncthreads();
  if (threadIdx.x < STEP_COLS) {
    const int c = cb * STEP_COLS + threadIdx.x;
    if (c < Dv) {
      float acc = 0.f;
#pragma unroll
      for (int g = 0; g < RGS; ++g) acc += o_s[g * STEP_COLS + threadIdx.x];
      out[((long)n * H + h) * Dv + c] = acc;
    }
  }
}

// ------------------------------------------------------------ token by token
constexpr int WALK_RG = 4;            // lanes sharing one column
constexpr int WALK_COLS = 16;         // columns per wave

// tokens per LDS tile: at most 32, and the tile within 48 KB
constexpr int walk_tile_tokens(int dkp) {
  const int fit = 48 * 1024 / (4 * (2 * dkp + 64));
  return fit < 32 ? fit : 32;
}

template <typename T, int RPL>
__global__ __launch_bounds__(256) void lightning_walk_kernel(
    float* __restrict__ out, const T* __restrict__ q, long ldq,
    const T* __restrict__ k, long ldk, const T* __restrict__ v, long ldv,
    const float* __restrict__ decay, float* __restrict__ state,
    const int* __restrict__ cu_q, const int* __restrict__ state_slot, int H,
    int Dk, int Dv) {
  constexpr int DKP = WALK_RG * RPL;
  constexpr int TT = walk_tile_tokens(DKP);
  __shared__ __attribute__((aligned(16))) float q_s[TT * DKP];
  __shared__ __attribute__((aligned(16))) float k_s[TT * DKP];
  __shared__ float v_s[TT * 64];
  const int cblocks = (Dv + 63) / 64;
  const int b = blockIdx.x / (H * cblocks);
  const int h = (blockIdx.x / cblocks) % H;
  const int cb = blockIdx.x % cblocks;
  const int lane = threadIdx.x & 63, wid = threadIdx.x >> 6;
  const int wcol = wid * WALK_COLS + lane / WALK_RG;
  const int col = cb * 64 + wcol;
  const int rg = lane % WALK_RG, row0 = rg * RPL;
  const bool colok = col < Dv;
  const int q0 = cu_q[b], q1 = cu_q[b + 1];
  if (q1 <= q0) return;                           // the whole block
  const bool wave_live = cb * 64 + wid * WALK_COLS < Dv;
  const float dec = decay[h];
  float* S = state + ((long)state_slot[b] * H + h) * Dk * Dv;
  float s[RPL];
#pragma unroll
  for (int i = 0; i < RPL; ++i) {
    const int row = row0 + i;
    s[i] = (colok && row < Dk) ? S[(long)row * Dv + col] : 0.f;
  }
  for (int n0 = q0; n0 < q1; n0 += TT) {
    const int cnt = q1 - n0 < TT ? q1 - n0 : TT;
    __syncthreads();                    // the tile before this one is used up
    for (int idx = threadIdx.x; idx < cnt * DKP; idx += 256) {
      const int t = idx / DKP, r = idx % DKP;
      const long n = n0 + t;
      q_s[idx] = r < Dk ? siluf_acc(ldf(q + n * ldq + h * Dk + r)) : 0.f;
      k_s[idx] = r < Dk ? siluf_acc(ldf(k + n * ldk + h * Dk + r)) : 0.f;
    }
    for (int idx = threadIdx.x; idx < cnt * 64; idx += 256) {
      const int t = idx >> 6, c = cb * 64 + (idx & 63);
      v_s[idx] = c < Dv
          ? siluf_acc(ldf(v + (long)(n0 + t) * ldv + h * Dv + c)) : 0.f;
    }
    __syncthreads();
    if (!wave_live) continue;
    for (int t = 0; t < cnt; ++t) {
      const float* qr = q_s + t * DKP + row0;
      const float* kr = k_s + t * DKP + row0;
      const float vv = v_s[t * 64 + wcol];
      float o = 0.f;
#pragma unroll
      for (int i = 0; i < RPL; ++i) {
        s[i] = dec * s[i] + kr[i] * vv;
        o += s[i] * qr[i];
      }
      o = quad_sum(o);
      if (colok && rg == 0) out[((long)(n0 + t) * H + h) * Dv + col] = o;
    }
  }
#pragma unroll
  for (int i = 0; i < RPL; ++i) {
    const int row = row0 + i;
    if (colok && row < Dk) S[(long)row * Dv + col] = s[i];
  }
}

// ----------------------------------------------------- chunks of 64 tokens
constexpr int CH = 64;                 // tokens of a chunk, columns of a block
constexpr int CHP = CH + 8;            // padded LDS row of tokens

// x as the sum of two bf16 numbers
DEV_INLINE void split2(float x, __bf16& hi, __bf16& lo) {
  hi = (__bf16)x;
  lo = (__bf16)(x - (float)hi);
}

template <int KS>
__global__ __launch_bounds__(256) void lightning_chunk_kernel(
    float* __restrict__ out, const bf16_t* __restrict__ q, long ldq,
    const bf16_t* __restrict__ k, long ldk, const bf16_t* __restrict__ v,
    long ldv, const float* __restrict__ decay, float* __restrict__ state,
    const int* __restrict__ cu_q, const int* __restrict__ state_slot, int H,
    int Dk, int Dv) {
  constexpr int DKP = KS * 32;
  constexpr int KROW = DKP + 8;        // padded LDS row of key channels
  constexpr int NT = KS * 2;           // 16-row tiles of the state
  constexpr int NKI = (CH / 4) * (DKP / 4);      // 4x4 pieces of a key tile
  constexpr int KI = (NKI + 255) / 256;
  __shared__ __attribute__((aligned(16))) __bf16 Ks[CH * KROW];
  __shared__ __attribute__((aligned(16))) __bf16 Kh[DKP * CHP], Kl[DKP * CHP];
  __shared__ __attribute__((aligned(16))) __bf16 Vt[CH * CHP];
  __shared__ __attribute__((aligned(16))) __bf16 Sh[CH * KROW], Sl[CH * KROW];
  __shared__ __attribute__((aligned(16))) __bf16 Ph[4][16 * CHP],
      Pl[4][16 * CHP];
  __shared__ float pw[CH + 1];         // powers of the decay
  const int cblocks = (Dv + CH - 1) / CH;
  const int b = blockIdx.x / (H * cblocks);
  const int h = (blockIdx.x / cblocks) % H;
  const int cb = blockIdx.x % cblocks;
  const int lane = threadIdx.x & 63, wid = threadIdx.x >> 6;
  const int l15 = lane & 15, lhi = lane >> 4;
  const int q0 = cu_q[b], q1 = cu_q[b + 1];
  if (q1 <= q0) return;                // the whole block
  if (threadIdx.x <= CH) {             // d^t by squaring, rounded once
    double p = 1.0, s = (double)decay[h];
    for (int t = threadIdx.x; t; t >>= 1) {
      if (t & 1) p *= s;
      s *= s;
    }
    pw[threadIdx.x] = (float)p;
  }
  // state tiles in accumulator layout: row nt*16 + lhi*4 + r, column l15
  float* S = state + ((long)state_slot[b] * H + h) * Dk * Dv;
  const int scol = cb * CH + wid * 16 + l15;
  f32x4_t sacc[NT];
#pragma unroll
  for (int nt = 0; nt < NT; ++nt)
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int d = nt * 16 + lhi * 4 + r;
      sacc[nt][r] = d < Dk && scol < Dv ? S[(long)d * Dv + scol] : 0.f;
    }

  // a chunk's words of this thread, requested one chunk ahead of their use
  uint2 rk[KI][4], rv[4], rq[KS][2];
  const uint2 z2 = make_uint2(0u, 0u);
  auto fetch = [&](int n0) {
    const int cnt = q1 - n0 < CH ? q1 - n0 : CH;
#pragma unroll
    for (int it = 0; it < KI; ++it) {
      const int idx = threadIdx.x + it * 256;
      const int t0 = idx / (DKP / 4) * 4, c = idx % (DKP / 4) * 4;
#pragma unroll
      for (int t = 0; t < 4; ++t)
        rk[it][t] = t0 + t < cnt && c < Dk
            ? *reinterpret_cast<const uint2*>(
                  k + (long)(n0 + t0 + t) * ldk + h * Dk + c) : z2;
    }
    const int t0 = threadIdx.x / 16 * 4, c = cb * CH + threadIdx.x % 16 * 4;
#pragma unroll
    for (int t = 0; t < 4; ++t)
      rv[t] = t0 + t < cnt && c < Dv
          ? *reinterpret_cast<const uint2*>(
                v + (long)(n0 + t0 + t) * ldv + h * Dv + c) : z2;
    const int i = wid * 16 + l15;
    const bf16_t* qr = q + (long)(n0 + (i < cnt ? i : 0)) * ldq + h * Dk;
#pragma unroll
    for (int ks = 0; ks < KS; ++ks)
#pragma unroll
      for (int e = 0; e < 2; ++e) {
        const int d = ks * 32 + lhi * 8 + e * 4;
        rq[ks][e] = d < Dk ? *reinterpret_cast<const uint2*>(qr + d) : z2;
      }
  };
  auto silu4 = [](const uint2& r, float (&o)[4]) {
    o[0] = __builtin_bit_cast(float, r.x << 16);
    o[1] = __builtin_bit_cast(float, r.x & 0xffff0000u);
    o[2] = __builtin_bit_cast(float, r.y << 16);
    o[3] = __builtin_bit_cast(float, r.y & 0xffff0000u);
#pragma unroll
    for (int e = 0; e < 4; ++e) o[e] *= sigmoidf_fast(o[e]);
  };
  fetch(q0);
  __syncthreads();                     // the powers are there
  const float* pwp = pw;
  for (int n0 = q0; n0 < q1; n0 += CH) {
    const int cnt = q1 - n0 < CH ? q1 - n0 : CH;
    // ---- keys (rows; columns with their decay), values, state into LDS ----
#pragma unroll
    for (int it = 0; it < KI; ++it) {
      const int idx = threadIdx.x + it * 256;
      if (NKI % 256 && idx >= NKI) break;
      const int t0 = idx / (DKP / 4) * 4, c = idx % (DKP / 4) * 4;
      bf16x4_t hi[4], lo[4];
#pragma unroll
      for (int t = 0; t < 4; ++t) {
        float x[4];
        silu4(rk[it][t], x);
        const int age = cnt - 1 - (t0 + t);
        const float w = pwp[age > 0 ? age : 0];
        bf16x4_t kr;
#pragma unroll
        for (int e = 0; e < 4; ++e) {
          kr[e] = (__bf16)x[e];
          __bf16 a, l;
          split2((float)kr[e] * w, a, l);
          hi[e][t] = a;
          lo[e][t] = l;
        }
        *reinterpret_cast<bf16x4_t*>(Ks + (t0 + t) * KROW + c) = kr;
      }
#pragma unroll
      for (int e = 0; e < 4; ++e) {
        *reinterpret_cast<bf16x4_t*>(Kh + (c + e) * CHP + t0) = hi[e];
        *reinterpret_cast<bf16x4_t*>(Kl + (c + e) * CHP + t0) = lo[e];
      }
    }
    {
      const int t0 = threadIdx.x / 16 * 4, c = threadIdx.x % 16 * 4;
      bf16x4_t vt[4];
#pragma unroll
      for (int t = 0; t < 4; ++t) {
        float x[4];
        silu4(rv[t], x);
#pragma unroll
        for (int e = 0; e < 4; ++e) vt[e][t] = (__bf16)x[e];
      }
#pragma unroll
      for (int e = 0; e < 4; ++e)
        *reinterpret_cast<bf16x4_t*>(Vt + (c + e) * CHP + t0) = vt[e];
    }
#pragma unroll
    for (int nt = 0; nt < NT; ++nt) {
      bf16x4_t hi, lo;
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        __bf16 a, l;
        split2(sacc[nt][r], a, l);
        hi[r] = a;
        lo[r] = l;
      }
      const int o = (wid * 16 + l15) * KROW + nt * 16 + lhi * 4;
      *reinterpret_cast<bf16x4_t*>(Sh + o) = hi;
      *reinterpret_cast<bf16x4_t*>(Sl + o) = lo;
    }
    bf16x8_t qf[KS];                   // A layout: row l15, k = lhi*8 ..
#pragma unroll
    for (int ks = 0; ks < KS; ++ks)
#pragma unroll
      for (int e = 0; e < 2; ++e) {
        float x[4];
        silu4(rq[ks][e], x);
#pragma unroll
        for (int c = 0; c < 4; ++c) qf[ks][e * 4 + c] = (__bf16)x[c];
      }
    __syncthreads();
    if (n0 + CH < q1) fetch(n0 + CH);

    // ---- decayed scores of this wave's rows against the keys up to them ---
    __bf16* ph = Ph[wid];
    __bf16* pl = Pl[wid];
    const int ktiles = (wid | 1) + 1;  // whole pairs of 16-key tiles
    for (int nt = 0; nt < ktiles; ++nt) {
      f32x4_t c = {0.f, 0.f, 0.f, 0.f};
      if (nt <= wid) {
#pragma unroll
        for (int ks = 0; ks < KS; ++ks) {
          const bf16x8_t kf = *reinterpret_cast<const bf16x8_t*>(
              Ks + (nt * 16 + l15) * KROW + ks * 32 + lhi * 8);
          c = __builtin_amdgcn_mfma_f32_16x16x32_bf16(qf[ks], kf, c, 0, 0, 0);
        }
      }
      const int j = nt * 16 + l15;
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int i = wid * 16 + lhi * 4 + r;
        const float x = j <= i ? c[r] * pwp[i >= j ? i - j : 0] : 0.f;
        __bf16 a, l;
        split2(x, a, l);
        ph[(lhi * 4 + r) * CHP + j] = a;
        pl[(lhi * 4 + r) * CHP + j] = l;
      }
    }
    __builtin_amdgcn_fence(__ATOMIC_ACQ_REL, "wavefront");

    // ---- o: the state's share, then the chunk's own ------------------------
    float rowpw[4];
#pragma unroll
    for (int r = 0; r < 4; ++r) rowpw[r] = pwp[wid * 16 + lhi * 4 + r + 1];
#pragma unroll
    for (int ct = 0; ct < 4; ++ct) {
      f32x4_t o = {0.f, 0.f, 0.f, 0.f};
      const int srow = (ct * 16 + l15) * KROW + lhi * 8;
#pragma unroll
      for (int ks = 0; ks < KS; ++ks) {
        const bf16x8_t sl =
            *reinterpret_cast<const bf16x8_t*>(Sl + srow + ks * 32);
        const bf16x8_t sh =
            *reinterpret_cast<const bf16x8_t*>(Sh + srow + ks * 32);
        o = __builtin_amdgcn_mfma_f32_16x16x32_bf16(qf[ks], sl, o, 0, 0, 0);
        o = __builtin_amdgcn_mfma_f32_16x16x32_bf16(qf[ks], sh, o, 0, 0, 0);
      }
#pragma unroll
      for (int r = 0; r < 4; ++r) o[r] *= rowpw[r];
      for (int kb = 0; kb <= wid / 2; ++kb) {
        const bf16x8_t vf = *reinterpret_cast<const bf16x8_t*>(
            Vt + (ct * 16 + l15) * CHP + kb * 32 + lhi * 8);
        const int po = l15 * CHP + kb * 32 + lhi * 8;
        const bf16x8_t pfl = *reinterpret_cast<const bf16x8_t*>(pl + po);
        const bf16x8_t pfh = *reinterpret_cast<const bf16x8_t*>(ph + po);
        o = __builtin_amdgcn_mfma_f32_16x16x32_bf16(pfl, vf, o, 0, 0, 0);
        o = __builtin_amdgcn_mfma_f32_16x16x32_bf16(pfh, vf, o, 0, 0, 0);
      }
      const int c = cb * CH + ct * 16 + l15;
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int i = wid * 16 + lhi * 4 + r;
        if (i < cnt && c < Dv) out[((long)(n0 + i) * H + h) * Dv + c] = o[r];
      }
    }

    // ---- the state behind the chunk ----------------------------------------
    const float dc = pwp[cnt];
#pragma unroll
    for (int nt = 0; nt < NT; ++nt)
#pragma unroll
      for (int r = 0; r < 4; ++r) sacc[nt][r] *= dc;
#pragma unroll
    for (int kb = 0; kb < 2; ++kb) {
      const bf16x8_t vf = *reinterpret_cast<const bf16x8_t*>(
          Vt + (wid * 16 + l15) * CHP + kb * 32 + lhi * 8);
#pragma unroll
      for (int nt = 0; nt < NT; ++nt) {
        const int ko = (nt * 16 + l15) * CHP + kb * 32 + lhi * 8;
        const bf16x8_t kl = *reinterpret_cast<const bf16x8_t*>(Kl + ko);
        const bf16x8_t kh = *reinterpret_cast<const bf16x8_t*>(Kh + ko);
        sacc[nt] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(kl, vf, sacc[nt],
                                                           0, 0, 0);
        sacc[nt] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(kh, vf, sacc[nt],
                                                           0, 0, 0);
      }
    }
    __syncthreads();                   // every wave is done with the tiles
  }
#pragma unroll
  for (int nt = 0; nt < NT; ++nt)
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int d = nt * 16 + lhi * 4 + r;
      if (d < Dk && scol < Dv) S[(long)d * Dv + scol] = sacc[nt][r];
    }
}

#define LIGHTNING_ARGS(TT)                                                    \
  out.data_ptr<float>(), (const TT*)q.data_ptr(), q.stride(0),                \
      (const TT*)k.data_ptr(), k.stride(0), (const TT*)v.data_ptr(),          \
      v.stride(0), decay.data_ptr<float>(), state.data_ptr<float>(),          \
      cu_q.data_ptr<int>(), state_slot.data_ptr<int>(), H, Dk, Dv
#define WALK_LAUNCH(RPLV)                                                     \
  hipLaunchKernelGGL((lightning_walk_kernel<T, RPLV>), dim3(grid), dim3(256), \
                     0, stream, LIGHTNING_ARGS(T))
#define CHUNK_LAUNCH(KSV)                                                     \
  hipLaunchKernelGGL((lightning_chunk_kernel<KSV>), dim3(grid), dim3(256), 0, \
                     stream, LIGHTNING_ARGS(bf16_t))

void seq_lightning_scan(torch::Tensor out, torch::Tensor q, torch::Tensor k,
                        torch::Tensor v, torch::Tensor decay,
                        torch::Tensor state, torch::Tensor cu_q,
                        torch::Tensor state_slot, int64_t max_rows) {
  CHECK_ROWS(q); CHECK_ROWS(k); CHECK_ROWS(v);
  CHECK_F32(decay); CHECK_F32(state); CHECK_F32(out);
  CHECK_I32(cu_q); CHECK_I32(state_slot);
  TORCH_CHECK(state.dim() == 4);
  const int H = state.size(1), Dk = state.size(2), Dv = state.size(3);
  const long N = q.size(0);
  TORCH_CHECK(q.size(1) == (long)H * Dk && k.size(1) == (long)H * Dk &&
              v.size(1) == (long)H * Dv, "linear attention operand widths");
  TORCH_CHECK(k.size(0) == N && v.size(0) == N && out.dim() == 2 &&
              out.size(0) == N && out.size(1) == (long)H * Dv);
  TORCH_CHECK(decay.numel() == H, "one decay per head");
  auto dt = q.scalar_type();
  TORCH_CHECK(k.scalar_type() == dt && v.scalar_type() == dt);
  TORCH_CHECK(Dk >= 1 && Dk <= 512,
              "linear attention: key dim above 512 not supported");
  const int B = state_slot.numel();
  TORCH_CHECK(cu_q.numel() == B + 1);
  if (N == 0 || B == 0) return;
  const int grid = B * H * ((Dv + 63) / 64);
  auto stream = at::hip::getCurrentHIPStream();
  if (max_rows == 1) {
    const bool vec = Dv % 4 == 0 && (uintptr_t)state.data_ptr() % 16 == 0;
    const int rgs = vec ? 16 : 4;
    const size_t bytes = (2 * Dk + rgs * STEP_COLS) * sizeof(float);
    SEQ_DISPATCH_T(dt, {
      if (vec)
        hipLaunchKernelGGL((lightning_step_kernel<T, true>), dim3(grid),
                           dim3(256), bytes, stream, LIGHTNING_ARGS(T));
      else
        hipLaunchKernelGGL((lightning_step_kernel<T, false>), dim3(grid),
                           dim3(256), bytes, stream, LIGHTNING_ARGS(T));
    });
    HIP_CHECK_KERNEL();
    return;
  }
  if (dt == torch::kBFloat16 && Dk <= 128 && rows_by4<bf16_t>(q, Dk) &&
      rows_by4<bf16_t>(k, Dk) && rows_by4<bf16_t>(v, Dv)) {
    switch ((Dk + 31) / 32) {
      case 1: CHUNK_LAUNCH(1); break;
      case 2: CHUNK_LAUNCH(2); break;
      case 3: CHUNK_LAUNCH(3); break;
      default: CHUNK_LAUNCH(4); break;
    }
    HIP_CHECK_KERNEL();
    return;
  }
  const int rpl = (Dk + WALK_RG - 1) / WALK_RG;
  SEQ_DISPATCH_T(dt, {
    if (rpl <= 4) WALK_LAUNCH(4);
    else if (rpl <= 8) WALK_LAUNCH(8);
    else if (rpl <= 16) WALK_LAUNCH(16);
    else if (rpl <= 32) WALK_LAUNCH(32);
    else if (rpl <= 64) WALK_LAUNCH(64);
    else WALK_LAUNCH(128);
  });
  HIP_CHECK_KERNEL();
}
