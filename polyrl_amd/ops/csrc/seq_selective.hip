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

// a token's words of one lane
template <int RPL>
struct SScanIn {
  f32x4v b[RPL / 4], c[RPL / 4];
  float2 dx;
};

// ONE: every sequence brings one row (tiles of one token, little LDS).  VEC:
// all rows allow loads of four numbers.  Addresses beyond a tile's rows, the
// channels or the state entries are clamped to the last ones and the numbers
// dropped, so that the loads of a tile are one straight run.
template <typename T, int RPL, bool ONE, bool VEC>
__global__ __launch_bounds__(256) void selective_scan_kernel(
    T* __restrict__ out, long ldo, const T* __restrict__ x, long ldx,
    const T* __restrict__ dtl, long ldd, const float* __restrict__ dt_bias,
    const T* __restrict__ Bm, long ldb, const T* __restrict__ Cm, long ldc,
    const float* __restrict__ a_log, const float* __restrict__ d_skip,
    const T* __restrict__ z, long ldz, float* __restrict__ state,
    const int* __restrict__ cu_q, const int* __restrict__ state_slot, int C,
    int Ns, float out_scale) {
  constexpr int NSP = 4 * RPL;              // state entries incl. padding
  constexpr int TT = ONE ? 1 : sscan_tile(NSP);
  constexpr int CU = TT * SCH / 4;          // four-number units of a tile
  constexpr int NU = TT * NSP / 4;
  constexpr int NCI = (CU + 255) / 256;
  constexpr int NNI = (NU + 255) / 256;
  __shared__ f32x4v b_s[NU], c_s[NU];
  __shared__ f32x4v y_s[CU + 64];           // + where the copies go
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
  const long srow = (long)state_slot[b] * C + min(c, C - 1);
  float* S = state + srow * Ns;
  const float* Ar = a_log + (long)min(c, C - 1) * Ns;
  float s[RPL], a2[RPL];
#pragma unroll
  for (int j = 0; j < RPL / 4; ++j) {
    const int at = VEC ? min(ent(4 * j), Ns - 4) : min(ent(4 * j), Ns - 1);
    Raw4<float> x, y;
    x.template load<VEC>(S + at, Ns - at);
    y.template load<VEC>(Ar + at, Ns - at);
#pragma unroll
    for (int e = 0; e < 4; ++e) {
      s[4 * j + e] = x.r.v[e];
      a2[4 * j + e] = y.r.v[e];
    }
  }

  // staging: my four channels (state entries) of every TPC-th (TPN-th) token
  constexpr int TPC = 256 / (SCH / 4), TPN = 256 / (NSP / 4);
  const int ct = tid / (SCH / 4), cc0 = c0 + (tid % (SCH / 4)) * 4;
  const int nt = tid / (NSP / 4), ne = (tid % (NSP / 4)) * 4;
  const int cca = VEC ? min(cc0, C - 4) : min(cc0, C - 1);
  const int nea = VEC ? min(ne, Ns - 4) : min(ne, Ns - 1);
  const bool neok = ne < Ns;
  Raw4<float> bias, skip;
  bias.template load<VEC>(dt_bias + cca, C - cca);
  skip.template load<VEC>(d_skip + cca, C - cca);

  Raw4<T> rd[NCI], rx[NCI], rz[NCI], rB[NNI], rC[NNI];
  auto fetch = [&](int n0) {
    const int last = min(q1 - n0, TT) - 1;
#pragma unroll
    for (int it = 0; it < NCI; ++it) {
      const long n = n0 + min(ct + it * TPC, last);
      rd[it].template load<VEC>(dtl + n * ldd + cca, C - cca);
      rx[it].template load<VEC>(x + n * ldx + cca, C - cca);
      rz[it].template load<VEC>(z + n * ldz + cca, C - cca);
    }
#pragma unroll
    for (int it = 0; it < NNI; ++it) {
      const long n = n0 + min(nt + it * TPN, last);
      rB[it].template load<VEC>(Bm + n * ldb + nea, Ns - nea);
      rC[it].template load<VEC>(Cm + n * ldc + nea, Ns - nea);
    }
  };
  fetch(q0);
  // wait for the state and the rates here, or every walk would also wait for
  // the next tile's words
  __builtin_amdgcn_sched_barrier(0);
#pragma unroll
  for (int i = 0; i < RPL; ++i) {
    const bool ok = cok && ent(i) < Ns;
    s[i] = ok ? s[i] : 0.f;
    a2[i] = ok ? -1.4426950408889634f * expf(a2[i]) : 0.f;
    if (!ONE) asm volatile("" : "+v"(s[i]), "+v"(a2[i]));
  }
  // the four lanes of a channel hold its sum: the first writes it to the
  // tile, the others to words of their own (no branch in the walk)
  float* y_at = reinterpret_cast<float*>(y_s) + (sg == 0 ? ch : TT * SCH + tid);
  const int y_step = sg == 0 ? SCH : 0;

  for (int n0 = q0; n0 < q1; n0 += TT) {
    const int cnt = q1 - n0 < TT ? q1 - n0 : TT;
    __syncthreads();                        // the tile before is used up
    f32x4v cx[NCI];
    Raw4<T> cz[NCI];
#pragma unroll
    for (int it = 0; it < NCI; ++it) {
      cx[it] = rx[it].get();
      cz[it] = rz[it];
      const int u = tid + it * 256;
      if (u * 4 < cnt * SCH) {
        const f32x4v dl = rd[it].get(), bi = bias.get();
#pragma unroll
        for (int e = 0; e < 4; ++e) {
          const float dt = softplusf_fast(dl.v[e] + bi.v[e]);
          dx_s[u * 4 + e] = {dt, dt * cx[it].v[e]};
        }
      }
    }
#pragma unroll
    for (int it = 0; it < NNI; ++it) {
      const int u = tid + it * 256;
      if (u * 4 < cnt * NSP) {
        f32x4v bv = rB[it].get(), cv = rC[it].get();
#pragma unroll
        for (int e = 0; e < 4; ++e)
          if (!neok) bv.v[e] = cv.v[e] = 0.f;
        b_s[u] = bv;
        c_s[u] = cv;
      }
    }
    __syncthreads();
    if (!ONE && n0 + TT < q1) fetch(n0 + TT);   // in flight during the walk
    auto words = [&](SScanIn<RPL>& in, int t) {
      in.dx = dx_s[t * SCH + ch];
#pragma unroll
      for (int j = 0; j < RPL / 4; ++j) {
        in.b[j] = b_s[t * (NSP / 4) + j * 4 + sg];
        in.c[j] = c_s[t * (NSP / 4) + j * 4 + sg];
      }
    };
    auto step = [&](const SScanIn<RPL>& in, int t) {
      float y = 0.f;
#pragma unroll
      for (int i = 0; i < RPL; ++i) {
        s[i] = __builtin_amdgcn_exp2f(in.dx.x * a2[i]) * s[i] +
               in.dx.y * in.b[i / 4].v[i % 4];
        y += s[i] * in.c[i / 4].v[i % 4];
      }
      y_at[t * y_step] = quad_sum(y);
    };
    if (ONE || RPL > 16) {
      for (int t = 0; t < cnt; ++t) {
        SScanIn<RPL> in;
        words(in, t);
        step(in, t);
      }
    } else {
      // the next token's words are read while this one is worked on
      SScanIn<RPL> a, d;
      words(a, 0);
      int t = 0;
      for (; t + 2 <= cnt; t += 2) {
        words(d, t + 1);
        __builtin_amdgcn_sched_barrier(0);
        step(a, t);
        words(a, t + 2 < cnt ? t + 2 : t + 1);
        __builtin_amdgcn_sched_barrier(0);
        step(d, t + 1);
      }
      if (t < cnt) step(a, t);
    }
    __syncthreads();                        // the sums are complete
#pragma unroll
    for (int it = 0; it < NCI; ++it) {
      const int u = tid + it * 256;
      const int tt = u / (SCH / 4);
      if (tt < cnt && cc0 < C) {
        const f32x4v dv = skip.get(), ys = y_s[u], zv = cz[it].get();
        f32x4v y;
#pragma unroll
        for (int e = 0; e < 4; ++e)
          y.v[e] = (ys.v[e] + dv.v[e] * cx[it].v[e]) * zv.v[e] *
                   sigmoidf_fast(zv.v[e]) * out_scale;
        store4(out + (long)(n0 + tt) * ldo + cc0, y, C - cc0, VEC);
      }
    }
  }
#pragma unroll
  for (int j = 0; j < RPL / 4; ++j) {
    f32x4v x;
#pragma unroll
    for (int e = 0; e < 4; ++e) x.v[e] = s[4 * j + e];
    if (cok && ent(4 * j) < Ns)
      store4(S + ent(4 * j), x, Ns - ent(4 * j), VEC);
  }
}

#define SSCAN_LAUNCH(RPLV, ONEV, VECV)                                        \
  hipLaunchKernelGGL((selective_scan_kernel<T, RPLV, ONEV, VECV>),            \
      dim3(grid), dim3(256), 0, stream, (T*)out.data_ptr(), out.stride(0),    \
      (const T*)x.data_ptr(), x.stride(0), (const T*)dt_lin.data_ptr(),       \
      dt_lin.stride(0), dt_bias.data_ptr<float>(), (const T*)Bm.data_ptr(),   \
      Bm.stride(0), (const T*)Cm.data_ptr(), Cm.stride(0),                    \
      a_log.data_ptr<float>(), d_skip.data_ptr<float>(),                      \
      (const T*)z.data_ptr(), z.stride(0), state.data_ptr<float>(),           \
      cu_q.data_ptr<int>(), state_slot.data_ptr<int>(), C, Ns,                \
      (float)out_scale)
#define SSCAN(RPLV)                                                           \
  do {                                                                        \
    if (!vec) SSCAN_LAUNCH(RPLV, false, false);                               \
    else if (max_rows == 1) SSCAN_LAUNCH(RPLV, true, true);                   \
    else SSCAN_LAUNCH(RPLV, false, true);                                     \
  } while (0)

void seq_selective_scan(torch::Tensor out, torch::Tensor x,
                        torch::Tensor dt_lin, torch::Tensor dt_bias,
                        torch::Tensor Bm, torch::Tensor Cm,
                        torch::Tensor a_log, torch::Tensor d_skip,
                        torch::Tensor z, torch::Tensor state,
                        torch::Tensor cu_q, torch::Tensor state_slot,
                        double out_scale, int64_t max_rows) {
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
    const bool vec = rows_by4<T>(x, C) && rows_by4<T>(dt_lin, C) &&
                     rows_by4<T>(z, C) && rows_by4<T>(out, C) &&
                     rows_by4<T>(Bm, Ns) && rows_by4<T>(Cm, Ns) &&
                     (uintptr_t)dt_bias.data_ptr() % 16 == 0 &&
                     (uintptr_t)d_skip.data_ptr() % 16 == 0 &&
                     (uintptr_t)a_log.data_ptr() % 16 == 0 &&
                     (uintptr_t)state.data_ptr() % 16 == 0;
    if (Ns <= 16) SSCAN(4);
    else if (Ns <= 32) SSCAN(8);
    else if (Ns <= 64) SSCAN(16);
    else if (Ns <= 128) SSCAN(32);
    else SSCAN(64);
  });
  HIP_CHECK_KERNEL();
}
