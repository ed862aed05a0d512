// Selective scan (Mamba-1 form; fp32 state, in place) with its step sizes,
// skip and output gate.
//
// Per channel c and state entry n, for a sequence's rows in order:
//   dt = softplus(dt_lin + dt_bias[c])
//   S[c,n] <- exp(-exp(a_log[c,n]) dt) S[c,n] + dt x[c] B[n]
//   y[c] = sum_n S[c,n] C[n] + d_skip[c] x[c]
//   out[c] = y[c] * silu(z[c]) * out_scale
// One launch serves prompt portions and decode tokens.
//
// A block owns 64 channels of one sequence: four lanes share a channel and
// hold RPL of its (at most 4*RPL) state entries in registers for the whole
// portion; the read-out sum is two quad permutes.  Token inputs come in tiles
// of TT rows through LDS: B and C once per token, the step size and dt*x once
// per (token, channel); the next tile's words are requested into registers
// before the current one is walked.  The walk's sums meet in LDS and leave
// with skip, gate and scale from the lanes that staged x and z.
// exp(-A dt) is taken as exp2 of the product with log2(e) folded into A.
#include <torch/extension.h>
#include <ATen/hip/HIPContext.h>

#include "seq_common.h"

constexpr int SCH = 64;                     // channels of a block

constexpr int sscan_tile(int nsp) {
  const int fit = 60 * 1024 / (4 * (2 * nsp + 3 * SCH));
  return fit < 32 ? fit : 32;
}

template <typename T, int RPL>
__global__ __launch_bounds__(256) void selective_scan_kernel(
    T* __restrict__ out, long ldo, const T* __restrict__ x, long ldx,
    const T* __restrict__ dtl, long ldd, const float* __restrict__ dt_bias,
    const T* __restrict__ Bm, long ldb, const T* __restrict__ Cm, long ldc,
    const float* __restrict__ a_log, const float* __restrict__ d_skip,
    const T* __restrict__ z, long ldz, float* __restrict__ state,
    const int* __restrict__ cu_q, const int* __restrict__ state_slot, int C,
    int Ns, float out_scale, bool vecc, bool vecn, bool veco) {
  constexpr int NSP = 4 * RPL;              // state entries incl. padding
  constexpr int TT = sscan_tile(NSP);
  constexpr int CU = TT * SCH / 4;          // four-number units of a tile
  constexpr int NU = TT * NSP / 4;
  constexpr int NCI = (CU + 255) / 256;
  constexpr int NNI = (NU + 255) / 256;
  __shared__ f32x4v b_s[NU], c_s[NU], y_s[CU];
  __shared__ float2 dx_s[TT * SCH];         // dt, dt * x

  const int cblocks = (C + SCH - 1) / SCH;
  const int b = blockIdx.x / cblocks;
  const int c0 = (blockIdx.x % cblocks) * SCH;
  const int q0 = cu_q[b], q1 = cu_q[b + 1];
  if (q1 <= q0) return;                     // the whole block
  const int tid = threadIdx.x;
  const int sg = tid & 3, ch = tid >> 2;    // state group, channel in block
  const int c = c0 + ch;
  const bool cok = c < C;

  // entry i of a lane: four consecutive entries per four-lane stripe
  auto ent = [&](int i) { return ((i >> 2) * 4 + sg) * 4 + (i & 3); };
  float* S = state + ((long)state_slot[b] * C + c) * Ns;
  float s[RPL], a2[RPL];
#pragma unroll
  for (int i = 0; i < RPL; ++i) {
    const bool ok = cok && ent(i) < Ns;
    s[i] = ok ? S[ent(i)] : 0.f;
    a2[i] = ok ? -expf(a_log[(long)c * Ns + ent(i)]) * 1.4426950408889634f
               : 0.f;
  }

  f32x4v rd[NCI], rx[NCI], rz[NCI], rB[NNI], rC[NNI];
  auto fetch = [&](int n0) {
    const int cnt = q1 - n0 < TT ? q1 - n0 : TT;
#pragma unroll
    for (int it = 0; it < NCI; ++it) {
      if (it * 1024 >= cnt * SCH) break;    // block-uniform
      const int u = tid + it * 256;
      const int t = u / (SCH / 4), cc = c0 + (u % (SCH / 4)) * 4;
      const f32x4v z4 = {{0.f, 0.f, 0.f, 0.f}};
      rd[it] = z4; rx[it] = z4; rz[it] = z4;
      if (t < cnt && cc < C) {
        const long n = n0 + t;
        rd[it] = load4(dtl + n * ldd + cc, C - cc, vecc);
        rx[it] = load4(x + n * ldx + cc, C - cc, vecc);
        rz[it] = load4(z + n * ldz + cc, C - cc, vecc);
        const f32x4v bi = load4(dt_bias + cc, C - cc, vecc);
#pragma unroll
        for (int e = 0; e < 4; ++e) rd[it].v[e] += bi.v[e];
      }
    }
#pragma unroll
    for (int it = 0; it < NNI; ++it) {
      if (it * 1024 >= cnt * NSP) break;
      const int u = tid + it * 256;
      const int t = u / (NSP / 4), e = (u % (NSP / 4)) * 4;
      const f32x4v z4 = {{0.f, 0.f, 0.f, 0.f}};
      rB[it] = z4; rC[it] = z4;
      if (t < cnt && e < Ns) {
        rB[it] = load4(Bm + (long)(n0 + t) * ldb + e, Ns - e, vecn);
        rC[it] = load4(Cm + (long)(n0 + t) * ldc + e, Ns - e, vecn);
      }
    }
  };
  fetch(q0);

  for (int n0 = q0; n0 < q1; n0 += TT) {
    const int cnt = q1 - n0 < TT ? q1 - n0 : TT;
    __syncthreads();                        // the tile before is used up
    f32x4v cx[NCI], cz[NCI];
#pragma unroll
    for (int it = 0; it < NCI; ++it) {
      cx[it] = rx[it];
      cz[it] = rz[it];
      const int u = tid + it * 256;
      if (u * 4 < cnt * SCH) {
#pragma unroll
        for (int e = 0; e < 4; ++e) {
          const float dt = softplusf_acc(rd[it].v[e]);
          dx_s[u * 4 + e] = {dt, dt * rx[it].v[e]};
        }
      }
    }
#pragma unroll
    for (int it = 0; it < NNI; ++it) {
      const int u = tid + it * 256;
      if (u * 4 < cnt * NSP) {
        b_s[u] = rB[it];
        c_s[u] = rC[it];
      }
    }
    __syncthreads();
    if (n0 + TT < q1) fetch(n0 + TT);       // in flight during the walk
    auto step = [&](int t) {
      const float2 dx = dx_s[t * SCH + ch];
      float y = 0.f;
#pragma unroll
      for (int j = 0; j < RPL / 4; ++j) {
        const f32x4v bv = b_s[t * (NSP / 4) + j * 4 + sg];
        const f32x4v cv = c_s[t * (NSP / 4) + j * 4 + sg];
#pragma unroll
        for (int e = 0; e < 4; ++e) {
          const int i = 4 * j + e;
          s[i] = __builtin_amdgcn_exp2f(dx.x * a2[i]) * s[i] + dx.y * bv.v[e];
          y += s[i] * cv.v[e];
        }
      }
      y = quad_sum(y);
      if (sg == 0) reinterpret_cast<float*>(y_s)[t * SCH + ch] = y;
    };
    int t = 0;
    for (; t + 4 <= cnt; t += 4) {          // four tokens' LDS reads in flight
#pragma unroll
      for (int u = 0; u < 4; ++u) step(t + u);
    }
    for (; t < cnt; ++t) step(t);
    __syncthreads();                        // the sums are complete
#pragma unroll
    for (int it = 0; it < NCI; ++it) {
      const int u = tid + it * 256;
      const int tt = u / (SCH / 4), cc = c0 + (u % (SCH / 4)) * 4;
      if (tt < cnt && cc < C) {
        const f32x4v dv = load4(d_skip + cc, C - cc, vecc);
        const f32x4v ys = y_s[u];
        f32x4v y;
#pragma unroll
        for (int e = 0; e < 4; ++e)
          y.v[e] = (ys.v[e] + dv.v[e] * cx[it].v[e]) *
                   siluf_acc(cz[it].v[e]) * out_scale;
        store4(out + (long)(n0 + tt) * ldo + cc, y, C - cc, veco);
      }
    }
  }
#pragma unroll
  for (int i = 0; i < RPL; ++i)
    if (cok && ent(i) < Ns) S[ent(i)] = s[i];
}

#define SSCAN(RPLV)                                                           \
  hipLaunchKernelGGL((selective_scan_kernel<T, RPLV>), dim3(grid), dim3(256), \
      0, stream, (T*)out.data_ptr(), out.stride(0), (const T*)x.data_ptr(),   \
      x.stride(0), (const T*)dt_lin.data_ptr(), dt_lin.stride(0),             \
      dt_bias.data_ptr<float>(), (const T*)Bm.data_ptr(), Bm.stride(0),       \
      (const T*)Cm.data_ptr(), Cm.stride(0), a_log.data_ptr<float>(),         \
      d_skip.data_ptr<float>(), (const T*)z.data_ptr(), z.stride(0),          \
      state.data_ptr<float>(), cu_q.data_ptr<int>(),                          \
      state_slot.data_ptr<int>(), C, Ns, (float)out_scale, vecc, vecn, veco)

void seq_selective_scan(torch::Tensor out, torch::Tensor x,
                        torch::Tensor dt_lin, torch::Tensor dt_bias,
                        torch::Tensor Bm, torch::Tensor Cm,
                        torch::Tensor a_log, torch::Tensor d_skip,
                        torch::Tensor z, torch::Tensor state,
                        torch::Tensor cu_q, torch::Tensor state_slot,
                        double out_scale) {
  CHECK_ROWS(out); CHECK_ROWS(x); CHECK_ROWS(dt_lin); CHECK_ROWS(Bm);
  CHECK_ROWS(Cm); CHECK_ROWS(z);
  CHECK_F32(dt_bias); CHECK_F32(a_log); CHECK_F32(d_skip); CHECK_F32(state);
  CHECK_I32(cu_q); CHECK_I32(state_slot);
  TORCH_CHECK(state.dim() == 3);
  const int C = state.size(1), Ns = state.size(2);
  const long N = x.size(0);
  TORCH_CHECK(C > 0 && Ns > 0 && x.size(1) == C && dt_lin.size(1) == C &&
              z.size(1) == C && out.size(1) == C && Bm.size(1) == Ns &&
              Cm.size(1) == Ns, "selective scan operand widths");
  TORCH_CHECK(dt_lin.size(0) == N && z.size(0) == N && out.size(0) == N &&
              Bm.size(0) == N && Cm.size(0) == N);
  TORCH_CHECK(dt_bias.numel() == C && d_skip.numel() == C &&
              a_log.numel() == (long)C * Ns);
  auto ty = x.scalar_type();
  for (const torch::Tensor* t : {&dt_lin, &Bm, &Cm, &z, &out})
    TORCH_CHECK(t->scalar_type() == ty, "one activation type");
  TORCH_CHECK(Ns <= 256, "state size above 256 not supported");
  const int B = state_slot.numel();
  TORCH_CHECK(cu_q.numel() == B + 1);
  if (N == 0 || B == 0) return;
  const int grid = B * ((C + SCH - 1) / SCH);
  auto stream = at::hip::getCurrentHIPStream();
  SEQ_DISPATCH_T(ty, {
    const bool vecc = rows_by4<T>(x, C) && rows_by4<T>(dt_lin, C) &&
                      rows_by4<T>(z, C) &&
                      (uintptr_t)dt_bias.data_ptr() % 16 == 0 &&
                      (uintptr_t)d_skip.data_ptr() % 16 == 0;
    const bool vecn = rows_by4<T>(Bm, Ns) && rows_by4<T>(Cm, Ns);
    const bool veco = rows_by4<T>(out, C);
    if (Ns <= 16) SSCAN(4);
    else if (Ns <= 32) SSCAN(8);
    else if (Ns <= 64) SSCAN(16);
    else if (Ns <= 128) SSCAN(32);
    else SSCAN(64);
  });
  HIP_CHECK_KERNEL();
}
