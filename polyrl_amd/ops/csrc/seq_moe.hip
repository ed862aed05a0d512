// Table-routed expert feed-forward for decode-sized batches (bf16, MFMA).
//
// Routing is a table over token ids, so a block finds its expert's rows by
// scanning the batch's (token, choice) slots itself: no host routing, no
// sort, no gather copy, and the launch shape depends only on the batch size
// (capturable in a graph).  Grid = (16-column tile, expert); a block whose
// expert got no row exits at once.  The op is weight-read bound at these
// batch sizes (every live expert streams its matrices once per step), so the
// four waves of a block take a quarter of the columns' K each and stream
// their 16 weight rows with 16-byte loads, several k-steps in flight,
// straight into v_mfma_f32_16x16x32_bf16 B fragments while the A fragments
// come from the activations; the partial sums (fp32) meet in LDS.  Up to 64
// token rows go along with one pass over the weights.
//
//   ACT 1 : act[slot, j] = silu(x_t . Wg[e][j]) * (x_t . Wu[e][j])   (gated)
//   ACT 2 : act[slot, j] = gelu_erf(x_t . Wu[e][j])                  (plain)
//   ACT 3 : act[slot, j] = g * sigmoid(slope g) * (u + shift) with
//           g = min(x_t . Wg, limit), u = clamp(x_t . Wu, +-limit)    (gated)
//   ACT 0 : y[slot, n]   = act[slot] . Wd[e][n]
// slot = t * top + choice, e = table[token_t][choice], or, for experts
// chosen by a router, e = slot_expert[slot] (an index >= the number of
// expert matrices names an expert without matrices: no block serves it).
//
// The router itself (softmax, selection-only correction, group-limited
// top-k) and the weighted combine of the chosen rows are here too.
#include <torch/extension.h>
#include <ATen/hip/HIPContext.h>

#include "seq_common.h"

typedef __attribute__((ext_vector_type(8))) __bf16 bf16x8_t;
typedef __attribute__((ext_vector_type(4))) float f32x4_t;
typedef __attribute__((ext_vector_type(4))) int i32x4_t;

constexpr int MOE_MAX_SLOTS = 1024;

constexpr int MOE_COLS = 16;          // output columns of a block

// RT row tiles of 16 (slots c0 .. c0 + 16*RT of this expert) against the
// block's columns; U k-steps in flight per wave
template <int ACT, int RT, int U>
DEV_INLINE void moe_tile(bf16_t* __restrict__ out, const bf16_t* __restrict__ x,
                         long ldx, const bf16_t* __restrict__ wrow,
                         const bf16_t* __restrict__ wrow2, const int* slots,
                         int cnt, int c0, int top, int K, int Nout, int n0,
                         float limit, float slope, float shift, float* red) {
  constexpr bool GATED = ACT == 1 || ACT == 3;
  constexpr bool BYTOKEN = ACT != 0;  // x rows by token, else by slot
  constexpr int NA = GATED ? 2 : 1;
  const int lane = threadIdx.x & 63, wid = threadIdx.x >> 6;
  const int l15 = lane & 15, lhi = lane >> 4;
  // this wave's k-steps: an even number, so that it reads whole 128-byte lines
  const int steps = K / 32, per = (steps + 7) / 8 * 2;
  const int s0 = wid * per, s1 = min(s0 + per, steps);
  const bf16_t* xrow[RT];
#pragma unroll
  for (int t = 0; t < RT; ++t) {      // rows past cnt: any row, dropped below
    const int slot = slots[min(c0 + t * 16 + l15, cnt - 1)];
    xrow[t] = x + (long)(BYTOKEN ? slot / top : slot) * ldx + lhi * 8;
  }
  f32x4_t acc[NA][RT];
#pragma unroll
  for (int a = 0; a < NA; ++a)
#pragma unroll
    for (int t = 0; t < RT; ++t) acc[a][t] = {0.f, 0.f, 0.f, 0.f};
  const i32x4_t zi = {0, 0, 0, 0};
#pragma unroll 1
  for (int s = s0; s < s1; s += U) {
    i32x4_t b[U], b2[U], a[RT][U];
#pragma unroll
    for (int u = 0; u < U; ++u) {     // past the end: the last step again
      const long o = (long)min(s + u, s1 - 1) * 32;
      b[u] = *reinterpret_cast<const i32x4_t*>(wrow + o);
      if (GATED) b2[u] = *reinterpret_cast<const i32x4_t*>(wrow2 + o);
#pragma unroll
      for (int t = 0; t < RT; ++t)
        a[t][u] = *reinterpret_cast<const i32x4_t*>(xrow[t] + o);
    }
#pragma unroll
    for (int u = 0; u < U; ++u) {
      const bool on = s + u < s1;     // wave-uniform
#pragma unroll
      for (int t = 0; t < RT; ++t) {
        const bf16x8_t av = __builtin_bit_cast(bf16x8_t, on ? a[t][u] : zi);
        acc[0][t] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(
            av, __builtin_bit_cast(bf16x8_t, b[u]), acc[0][t], 0, 0, 0);
        if (GATED)
          acc[NA - 1][t] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(
              av, __builtin_bit_cast(bf16x8_t, b2[u]), acc[NA - 1][t], 0, 0, 0);
      }
    }
  }
  // C layout: row = lhi*4 + r, col = l15
#pragma unroll
  for (int a = 0; a < NA; ++a)
#pragma unroll
    for (int t = 0; t < RT; ++t)
#pragma unroll
      for (int r = 0; r < 4; ++r)
        red[((wid * NA + a) * RT + t) * 256 + (lhi * 4 + r) * 16 + l15] =
            acc[a][t][r];
  __syncthreads();
  const int n = n0 + threadIdx.x % 16;
#pragma unroll
  for (int t = 0; t < RT; ++t) {
    const int ri = c0 + t * 16 + threadIdx.x / 16;
    float v[NA];
#pragma unroll
    for (int a = 0; a < NA; ++a) {
      v[a] = 0.f;
#pragma unroll
      for (int w = 0; w < 4; ++w)
        v[a] += red[((w * NA + a) * RT + t) * 256 + threadIdx.x];
    }
    float y = v[0];
    if (ACT == 1) y = siluf_acc(v[0]) * v[NA - 1];
    if (ACT == 2) y = gelu_erff_acc(v[0]);
    if (ACT == 3) {
      const float g = fminf(v[0], limit);
      const float u = fminf(fmaxf(v[NA - 1], -limit), limit);
      y = g * sigmoidf_acc(slope * g) * (u + shift);
    }
    if (ri < cnt && n < Nout) out[(long)slots[ri] * Nout + n] = f2bf(y);
  }
  __syncthreads();                    // red may be written again
}

template <int ACT>
__global__ __launch_bounds__(256) void moe_table_gemm_kernel(
    bf16_t* __restrict__ out,           // (B*top, Nout)
    const bf16_t* __restrict__ x, long ldx,   // gated: (B, K) by token; else (B*top, K) by slot
    const long* __restrict__ tokens,    // (B,)
    const int* __restrict__ table,      // (V, top)
    const int* __restrict__ slot_expert,   // (B*top,) or null (use the table)
    const bf16_t* __restrict__ w,       // (E, Nw, K): Nw = 2*Nout if gated
    int B, int top, int K, int Nout, float limit, float slope, float shift) {
  constexpr bool GATED = ACT == 1 || ACT == 3;
  __shared__ int slots[MOE_MAX_SLOTS];
  __shared__ int count;
  __shared__ float red[4 * (GATED ? 2 : 1) * 4 * 256];
  const int e = blockIdx.y;
  if (threadIdx.x == 0) count = 0;
  __syncthreads();
  const int S = B * top;
  for (int s = threadIdx.x; s < S; s += 256) {
    const int es = slot_expert ? slot_expert[s]
                               : table[tokens[s / top] * top + s % top];
    if (es == e) slots[atomicAdd(&count, 1)] = s;
  }
  __syncthreads();
  const int cnt = count;
  if (cnt == 0) return;

  const int lane = threadIdx.x & 63;
  const int n0 = blockIdx.x * MOE_COLS;
  const int n = min(n0 + (lane & 15), Nout - 1);      // this lane's B column
  const long Nw = GATED ? 2L * Nout : Nout;
  const bf16_t* wrow = w + ((long)e * Nw + n) * K + (lane >> 4) * 8;
  const bf16_t* wrow2 = wrow + (long)Nout * K;        // up rows (gated)
#define MOE_TILE(RTV, UV, C0)                                                 \
  moe_tile<ACT, RTV, UV>(out, x, ldx, wrow, wrow2, slots, cnt, C0, top, K,    \
                         Nout, n0, limit, slope, shift, red)
  if (cnt <= 16) MOE_TILE(1, 8, 0);
  else if (cnt <= 32) MOE_TILE(2, 4, 0);
  else
    for (int c0 = 0; c0 < cnt; c0 += 64) MOE_TILE(4, 4, c0);
}

// y (B*top, width) = table-routed experts on h (B, width); fills ``act``
// (B*top, ff) on the way.
void seq_moe_table_ffn(torch::Tensor y, torch::Tensor act, torch::Tensor h,
                       torch::Tensor tokens, torch::Tensor table,
                       torch::Tensor w_gu, torch::Tensor w_down) {
  CHECK_I32(table);
  TORCH_CHECK(h.is_cuda() && h.dim() == 2 && h.stride(1) == 1 &&
              h.scalar_type() == torch::kBFloat16);
  TORCH_CHECK(tokens.is_cuda() && tokens.dtype() == torch::kInt64 &&
              tokens.is_contiguous());
  TORCH_CHECK(w_gu.is_contiguous() && w_down.is_contiguous() &&
              w_gu.dim() == 3 && w_down.dim() == 3 &&
              w_gu.scalar_type() == torch::kBFloat16 &&
              w_down.scalar_type() == torch::kBFloat16);
  const int B = h.size(0), W = h.size(1), top = table.size(1);
  const int E = w_gu.size(0), ff = w_gu.size(1) / 2;
  TORCH_CHECK(tokens.numel() == B && table.dim() == 2);
  TORCH_CHECK(w_gu.size(2) == W && w_down.size(0) == E &&
              w_down.size(1) == W && w_down.size(2) == ff);
  TORCH_CHECK(W % 32 == 0 && ff % 32 == 0 && h.stride(0) % 8 == 0,
              "expert GEMM needs widths in multiples of 32");
  TORCH_CHECK(B * top <= MOE_MAX_SLOTS, "batch too large for the decode path");
  TORCH_CHECK(act.is_contiguous() && act.scalar_type() == torch::kBFloat16 &&
              act.size(0) == (long)B * top && act.size(1) == ff);
  TORCH_CHECK(y.is_contiguous() && y.scalar_type() == torch::kBFloat16 &&
              y.size(0) == (long)B * top && y.size(1) == W);
  if (B == 0) return;
  auto stream = at::hip::getCurrentHIPStream();
  hipLaunchKernelGGL((moe_table_gemm_kernel<1>), dim3((ff + MOE_COLS - 1) / MOE_COLS, E),
                     dim3(256), 0, stream, (bf16_t*)act.data_ptr(),
                     (const bf16_t*)h.data_ptr(), h.stride(0),
                     (const long*)tokens.data_ptr<int64_t>(),
                     table.data_ptr<int>(), (const int*)nullptr,
                     (const bf16_t*)w_gu.data_ptr(), B, top, W, ff, 0.f,
                     0.f, 0.f);
  hipLaunchKernelGGL((moe_table_gemm_kernel<0>), dim3((W + MOE_COLS - 1) / MOE_COLS, E),
                     dim3(256), 0, stream, (bf16_t*)y.data_ptr(),
                     (const bf16_t*)act.data_ptr(), (long)ff,
                     (const long*)tokens.data_ptr<int64_t>(),
                     table.data_ptr<int>(), (const int*)nullptr,
                     (const bf16_t*)w_down.data_ptr(), B, top, ff, W, 0.f,
                     0.f, 0.f);
  HIP_CHECK_KERNEL();
}

// y (B*top, width) = router-chosen experts on h (B, width), plain
// (gelu(W_up h), w_up (E, ff, W)) or gated (silu(W_gate h) * W_up h, w_up
// (E, 2*ff, W) with the gate rows first; limit > 0: the clamped form); fills
// ``act`` (B*top, ff) on the way.  Rows of identity experts stay unwritten.
void seq_moe_routed_ffn(torch::Tensor y, torch::Tensor act, torch::Tensor h,
                        torch::Tensor idx, torch::Tensor w_up,
                        torch::Tensor w_down, bool gated, double limit,
                        double slope, double shift) {
  CHECK_I32(idx);
  TORCH_CHECK(h.is_cuda() && h.dim() == 2 && h.stride(1) == 1 &&
              h.scalar_type() == torch::kBFloat16);
  TORCH_CHECK(w_up.is_contiguous() && w_down.is_contiguous() &&
              w_up.dim() == 3 && w_down.dim() == 3 &&
              w_up.scalar_type() == torch::kBFloat16 &&
              w_down.scalar_type() == torch::kBFloat16);
  const int B = h.size(0), W = h.size(1);
  TORCH_CHECK(idx.dim() == 2 && idx.size(0) == B);
  const int top = idx.size(1);
  const int E = w_up.size(0), ff = w_up.size(1) / (gated ? 2 : 1);
  TORCH_CHECK(!gated || w_up.size(1) % 2 == 0);
  TORCH_CHECK(limit >= 0 && (gated || limit == 0), "clamped experts are gated");
  TORCH_CHECK(w_up.size(2) == W && w_down.size(0) == E &&
              w_down.size(1) == W && w_down.size(2) == ff);
  TORCH_CHECK(W % 32 == 0 && ff % 32 == 0 && h.stride(0) % 8 == 0,
              "expert GEMM needs widths in multiples of 32");
  TORCH_CHECK(B * top <= MOE_MAX_SLOTS, "batch too large for the decode path");
  TORCH_CHECK(act.is_contiguous() && act.scalar_type() == torch::kBFloat16 &&
              act.size(0) == (long)B * top && act.size(1) == ff);
  TORCH_CHECK(y.is_contiguous() && y.scalar_type() == torch::kBFloat16 &&
              y.size(0) == (long)B * top && y.size(1) == W);
  if (B == 0 || E == 0) return;
  auto stream = at::hip::getCurrentHIPStream();
  const float lim = (float)limit, sl = (float)slope, sh = (float)shift;
#define MOE_UP(ACTV)                                                          \
  hipLaunchKernelGGL((moe_table_gemm_kernel<ACTV>),                           \
                     dim3((ff + MOE_COLS - 1) / MOE_COLS, E), dim3(256), 0, stream, (bf16_t*)act.data_ptr(),           \
                     (const bf16_t*)h.data_ptr(), h.stride(0),                \
                     (const long*)nullptr, (const int*)nullptr,               \
                     idx.data_ptr<int>(), (const bf16_t*)w_up.data_ptr(), B,  \
                     top, W, ff, lim, sl, sh)
  if (!gated) MOE_UP(2);
  else if (lim > 0.f) MOE_UP(3);
  else MOE_UP(1);
  hipLaunchKernelGGL((moe_table_gemm_kernel<0>), dim3((W + MOE_COLS - 1) / MOE_COLS, E),
                     dim3(256), 0, stream, (bf16_t*)y.data_ptr(),
                     (const bf16_t*)act.data_ptr(), (long)ff,
                     (const long*)nullptr, (const int*)nullptr,
                     idx.data_ptr<int>(), (const bf16_t*)w_down.data_ptr(), B,
                     top, ff, W, 0.f, 0.f, 0.f);
  HIP_CHECK_KERNEL();
}

// ------------------------------------------------------------------ router
// One wave per token, four tokens a block.  s = softmax(logits) over all E
// router outputs, or (act 1) the logistic function of every logit, or (act 2)
// the logit itself; choice = s + correction; experts form ``groups`` equal groups of
// neighbours, a group's score is the sum of its ``gtop`` largest choices,
// and only the ``keep`` groups with the largest score stay eligible (the
// others count as minus infinity); the ``top`` largest eligible choices
// win, ties to the lower index.  Writes the indices and the UNcorrected s
// at them, or (act 2) exp(choice - best choice).
constexpr int ROUTE_MAX_E = 512;

DEV_INLINE void wave_argmax(float& v, int& i) {
#pragma unroll
  for (int off = 32; off > 0; off >>= 1) {
    const float ov = __shfl_xor(v, off, WAVE_SIZE);
    const int oi = __shfl_xor(i, off, WAVE_SIZE);
    if (ov > v || (ov == v && oi < i)) {
      v = ov;
      i = oi;
    }
  }
}

// order of a wave's own LDS accesses (scratch that no other wave touches)
DEV_INLINE void wave_sync() {
  __builtin_amdgcn_fence(__ATOMIC_ACQ_REL, "wavefront");
  __builtin_amdgcn_wave_barrier();
}

// the choice for one token by one wave, on LDS scratch of its own; z: the
// token's E logits
DEV_INLINE void route_token(const float* z, float* s, float* c, float* gb,
                            int* __restrict__ idx, float* __restrict__ wout,
                            long n, bool live,
                            const float* __restrict__ correction, int E,
                            int top, int groups, int keep, int act, int gtop) {
  const int lane = threadIdx.x & 63;
  if (act >= 1) {
    for (int e = lane; e < E; e += 64) {
      const float p = act == 1 ? sigmoidf_acc(z[e]) : z[e];
      s[e] = p;
      c[e] = p + correction[e];
    }
  } else {
    float mx = -INFINITY;
    for (int e = lane; e < E; e += 64) mx = fmaxf(mx, z[e]);
    mx = wave_reduce_max(mx);
    float sum = 0.f;
    for (int e = lane; e < E; e += 64) {
      const float p = expf(z[e] - mx);
      s[e] = p;
      sum += p;
    }
    sum = wave_reduce_sum(sum);
    const float inv = 1.f / sum;
    for (int e = lane; e < E; e += 64) {
      const float p = s[e] * inv;
      s[e] = p;
      c[e] = p + correction[e];
    }
  }
  wave_sync();
  if (groups > 1) {
    const int per = E / groups;
    for (int g = lane; g < groups; g += 64) {
      // sum of the gtop largest choices of the group: pick them one by one,
      // each below the last pick in (value, -index) order
      float b = 0.f, lv = INFINITY;
      int li = -1;
      const int take = gtop < per ? gtop : per;
      for (int r = 0; r < take; ++r) {
        float bv = -INFINITY;
        int bi = -1;
        for (int e = g * per; e < (g + 1) * per; ++e) {
          const float v = c[e];
          const bool below = v < lv || (v == lv && e > li);
          if (below && (bi < 0 || v > bv)) {
            bv = v;
            bi = e;
          }
        }
        b += bv;
        lv = bv;
        li = bi;
      }
      gb[g] = b;
    }
    wave_sync();
    // mark the best ``keep`` groups: their best becomes +inf
    for (int r = 0; r < keep; ++r) {
      float bv = -INFINITY;
      int bi = 0x7fffffff;
      for (int g = lane; g < groups; g += 64) {
        const float v = gb[g];
        if (v != INFINITY && (v > bv || (v == bv && g < bi))) {
          bv = v;
          bi = g;
        }
      }
      wave_argmax(bv, bi);
      if (lane == 0 && bi != 0x7fffffff) gb[bi] = INFINITY;
      wave_sync();
    }
    for (int e = lane; e < E; e += 64)
      if (gb[e / per] != INFINITY) c[e] = -INFINITY;
    wave_sync();
  }
  float best = 0.f;                   // the first pick is the largest
  for (int r = 0; r < top; ++r) {
    float bv = -INFINITY;
    int bi = 0x7fffffff;
    for (int e = lane; e < E; e += 64) {
      const float v = c[e];
      if (v > bv || (v == bv && e < bi && v != -INFINITY)) {
        bv = v;
        bi = e;
      }
    }
    wave_argmax(bv, bi);
    if (bi == 0x7fffffff) bi = 0;     // fewer eligible experts than top
    if (r == 0) best = bv;
    if (lane == 0) {
      if (live) {
        idx[n * top + r] = bi;
        wout[n * top + r] = act == 2 ? expf(bv - best) : s[bi];
      }
      c[bi] = -INFINITY;
    }
    wave_sync();
  }
}

__global__ __launch_bounds__(256) void moe_route_kernel(
    int* __restrict__ idx, float* __restrict__ wout,
    const float* __restrict__ logits, long ldl,
    const float* __restrict__ correction, long N, int E, int top, int groups,
    int keep, int act, int gtop) {
  __shared__ float s_sh[4][ROUTE_MAX_E], c_sh[4][ROUTE_MAX_E];
  __shared__ float g_sh[4][ROUTE_MAX_E];
  const int wid = threadIdx.x >> 6;
  const long n0 = (long)blockIdx.x * 4 + wid;
  const bool live = n0 < N;           // idle waves shadow the last token
  const long n = live ? n0 : N - 1;
  route_token(logits + n * ldl, s_sh[wid], c_sh[wid], g_sh[wid], idx, wout, n,
              live, correction, E, top, groups, keep, act, gtop);
}

// Router product and choice in one launch, for batches of few tokens: one
// block of sixteen waves per token, a wave per router row in turn (rows from
// the XCD's L2, fp32 products and sums); the first wave makes the choice.
// Rows past the E choices (R > E) are further numbers per token: they go to
// ``extra``.
template <typename T, bool VEC>
__global__ __launch_bounds__(1024) void moe_router_kernel(
    int* __restrict__ idx, float* __restrict__ wout, float* __restrict__ extra,
    const T* __restrict__ h, long ldh, const float* __restrict__ w,
    const float* __restrict__ correction, int W, int R, int E, int top,
    int groups, int keep, int act, int gtop) {
  constexpr int C = VEC ? 4 : 1;        // columns of a lane
  __shared__ float z[ROUTE_MAX_E + 8], s_sh[ROUTE_MAX_E], c_sh[ROUTE_MAX_E];
  __shared__ float g_sh[ROUTE_MAX_E];
  const long n = blockIdx.x;
  const int wid = threadIdx.x >> 6, lane = threadIdx.x & 63;
  const T* hr = h + n * ldh;
  for (int r = wid; r < R; r += 16) {
    const float* wr = w + (long)r * W;
    float a = 0.f;
#pragma unroll 8
    for (int i = lane * C; i < W; i += 64 * C) {
      const f32x4v x = load4(hr + i, C, VEC), u = load4(wr + i, C, VEC);
#pragma unroll
      for (int c = 0; c < C; ++c) a += x.v[c] * u.v[c];
    }
    a = wave_reduce_sum(a);
    if (lane == 0) z[r] = a;
  }
  __syncthreads();
  if (wid) return;
  if (lane < R - E) extra[n * (R - E) + lane] = z[E + lane];
  route_token(z, s_sh, c_sh, g_sh, idx, wout, n, true, correction, E, top,
              groups, keep, act, gtop);
}

void seq_moe_route(torch::Tensor idx, torch::Tensor w, torch::Tensor logits,
                   torch::Tensor correction, int64_t groups, int64_t keep,
                   int64_t act, int64_t group_top) {
  CHECK_I32(idx);
  CHECK_F32(w);
  CHECK_F32(correction);
  TORCH_CHECK(logits.is_cuda() && logits.dim() == 2 &&
              logits.stride(1) == 1 && logits.dtype() == torch::kFloat32);
  const long N = logits.size(0);
  const int E = logits.size(1);
  TORCH_CHECK(idx.dim() == 2 && idx.size(0) == N && w.sizes() == idx.sizes());
  const int top = idx.size(1);
  TORCH_CHECK(E >= 1 && E <= ROUTE_MAX_E, "router outputs above 512");
  TORCH_CHECK(correction.numel() == E && top >= 1 && top <= E);
  TORCH_CHECK(groups >= 1 && E % groups == 0 && keep >= 1 && keep <= groups);
  TORCH_CHECK(act >= 0 && act <= 2 && group_top >= 1);
  if (N == 0) return;
  auto stream = at::hip::getCurrentHIPStream();
  hipLaunchKernelGGL(moe_route_kernel, dim3((N + 3) / 4), dim3(256), 0, stream,
                     idx.data_ptr<int>(), w.data_ptr<float>(),
                     logits.data_ptr<float>(), logits.stride(0),
                     correction.data_ptr<float>(), N, E, top, (int)groups,
                     (int)keep, (int)act, (int)group_top);
  HIP_CHECK_KERNEL();
}

void seq_moe_router(torch::Tensor idx, torch::Tensor w, torch::Tensor extra,
                    torch::Tensor h, torch::Tensor router,
                    torch::Tensor correction, int64_t groups, int64_t keep,
                    int64_t act, int64_t group_top) {
  CHECK_I32(idx);
  CHECK_F32(w); CHECK_F32(router); CHECK_F32(correction); CHECK_F32(extra);
  CHECK_ROWS(h);
  const long N = h.size(0), W = h.size(1);
  TORCH_CHECK(router.dim() == 2 && router.size(1) == W);
  const int R = router.size(0), E = correction.numel();
  TORCH_CHECK(idx.dim() == 2 && idx.size(0) == N && w.sizes() == idx.sizes());
  const int top = idx.size(1);
  TORCH_CHECK(E >= 1 && E <= ROUTE_MAX_E && R >= E && R - E <= 8,
              "router outputs above 512");
  TORCH_CHECK(extra.numel() == N * (R - E) && top >= 1 && top <= E);
  TORCH_CHECK(groups >= 1 && E % groups == 0 && keep >= 1 && keep <= groups);
  TORCH_CHECK(act >= 0 && act <= 2 && group_top >= 1);
  if (N == 0) return;
  auto stream = at::hip::getCurrentHIPStream();
  SEQ_DISPATCH_T(h.scalar_type(), {
    const bool vec = W % 4 == 0 && rows_by4<T>(h, W) &&
                     (uintptr_t)router.data_ptr() % 16 == 0;
#define ROUTER_LAUNCH(VECV)                                                   \
    hipLaunchKernelGGL((moe_router_kernel<T, VECV>), dim3(N), dim3(1024), 0,  \
        stream, idx.data_ptr<int>(), w.data_ptr<float>(),                     \
        extra.data_ptr<float>(), (const T*)h.data_ptr(), h.stride(0),         \
        router.data_ptr<float>(), correction.data_ptr<float>(), (int)W, R, E, \
        top, (int)groups, (int)keep, (int)act, (int)group_top)
    if (vec) ROUTER_LAUNCH(true);
    else ROUTER_LAUNCH(false); });
  HIP_CHECK_KERNEL();
}

// out[n, d] = sum_k w'[n,k] * (idx[n,k] < E ? ys[n*top+k, d] : h[n, d])
//             (+ shared[n, d] [* sigmoid(sgate[n])]),  w' = scale * w / (sum_k w + weight_eps)
// (a slot's expert row is ys[slot], or ys[place[slot]] where the rows lie in
// another order).  Four consecutive numbers per thread and step.
template <typename T>
__global__ __launch_bounds__(256) void moe_weighted_combine_kernel(
    T* __restrict__ out, const T* __restrict__ ys, const int* __restrict__ idx,
    const float* __restrict__ w, const T* __restrict__ h, long ldh,
    const T* __restrict__ shared, long lds_, int top, int E, float weight_eps,
    long rows, int D, float scale, const float* __restrict__ sgate, long ldsg,
    const int* __restrict__ place, bool vec) {
  const int dq = (D + 3) / 4;
  const long total = rows * dq;
  const long stride = (long)gridDim.x * blockDim.x;
  for (long i = (long)blockIdx.x * blockDim.x + threadIdx.x; i < total;
       i += stride) {
    const long n = i / dq;
    const int d = (int)(i - n * dq) * 4;
    float wsum = 0.f;
    for (int k = 0; k < top; ++k) wsum += w[n * top + k];
    const float inv = scale / (wsum + weight_eps);
    f32x4v acc = {{0.f, 0.f, 0.f, 0.f}};
    for (int k = 0; k < top; ++k) {
      const long slot = n * top + k;
      const T* src = idx[slot] < E
          ? ys + (place ? (long)place[slot] : slot) * D : h + n * ldh;
      const f32x4v v = load4(src + d, D - d, vec);
      const float wk = w[slot] * inv;
#pragma unroll
      for (int c = 0; c < 4; ++c) acc.v[c] += wk * v.v[c];
    }
    if (shared) {
      const f32x4v v = load4(shared + n * lds_ + d, D - d, vec);
      const float g = sgate ? sigmoidf_acc(sgate[n * ldsg]) : 1.f;
#pragma unroll
      for (int c = 0; c < 4; ++c) acc.v[c] += g * v.v[c];
    }
    store4(out + n * D + d, acc, D - d, vec);
  }
}

void seq_moe_weighted_combine(torch::Tensor out, torch::Tensor ys,
                              torch::Tensor idx, torch::Tensor w,
                              torch::Tensor h, torch::Tensor shared,
                              int64_t E, double weight_eps, double scale,
                              torch::Tensor shared_gate, torch::Tensor place) {
  CHECK_I32(idx);
  CHECK_F32(w);
  CHECK_ROWS(h);
  const long N = h.size(0);
  const int D = h.size(1);
  TORCH_CHECK(idx.dim() == 2 && idx.size(0) == N && w.sizes() == idx.sizes());
  const int top = idx.size(1);
  auto ty = h.scalar_type();
  TORCH_CHECK(ys.is_cuda() && ys.is_contiguous() && ys.dim() == 2 &&
              ys.size(0) == N * top && ys.size(1) == D &&
              ys.scalar_type() == ty);
  TORCH_CHECK(out.is_cuda() && out.is_contiguous() && out.size(0) == N &&
              out.size(1) == D && out.scalar_type() == ty);
  const bool has_shared = shared.defined() && shared.numel() > 0;
  if (has_shared) {
    CHECK_ROWS(shared);
    TORCH_CHECK(shared.size(0) == N && shared.size(1) == D &&
                shared.scalar_type() == ty);
  }
  const bool has_sg = shared_gate.defined() && shared_gate.numel() > 0;
  if (has_sg)
    TORCH_CHECK(has_shared && shared_gate.is_cuda() && shared_gate.dim() == 2 &&
                shared_gate.size(0) == N && shared_gate.size(1) == 1 &&
                shared_gate.scalar_type() == torch::kFloat32,
                "shared gate: one fp32 number per token");
  const bool has_place = place.defined() && place.numel() > 0;
  if (has_place) {
    CHECK_I32(place);
    TORCH_CHECK(place.numel() == N * top, "one row per slot");
  }
  if (N == 0) return;
  const long nblk = std::min<long>((N * ((D + 3) / 4) + 255) / 256,
                                   MAX_RESIDENT_BLOCKS * 4);
  auto stream = at::hip::getCurrentHIPStream();
  SEQ_DISPATCH_T(ty, {
      const bool vec = D % 4 == 0 && rows_by4<T>(ys, D) && rows_by4<T>(h, D) &&
                       rows_by4<T>(out, D) &&
                       (!has_shared || rows_by4<T>(shared, D));
      hipLaunchKernelGGL((moe_weighted_combine_kernel<T>), dim3(nblk), dim3(256), 0, stream,
      (T*)out.data_ptr(), (const T*)ys.data_ptr(), idx.data_ptr<int>(),
      w.data_ptr<float>(), (const T*)h.data_ptr(), h.stride(0),
      has_shared ? (const T*)shared.data_ptr() : nullptr,
      has_shared ? shared.stride(0) : 0, top, (int)E, (float)weight_eps, N,
      D, (float)scale, has_sg ? shared_gate.data_ptr<float>() : nullptr,
      has_sg ? shared_gate.stride(0) : 0,
      has_place ? place.data_ptr<int>() : nullptr, vec); });
  HIP_CHECK_KERNEL();
}
