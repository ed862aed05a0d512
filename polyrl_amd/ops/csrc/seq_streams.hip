// Row-wise kernels of stacks with several residual streams, and the tanh norm.
//
// The streams of a row lie next to each other, xs (rows, S, D) fp32.  A
// sublayer reads u = sum_s in[s] x_s through tanh(alpha * u) * w + b; behind
// it every stream becomes x_t <- sum_s mix[s, t] x_s + out[t] * y, all from
// the old streams.  The joint does both in one pass over the row: the old
// streams come in once, the new ones go out once, and the next sublayer's
// input is computed from the registers that hold them.  None of this needs a
// reduction over the row.  Only the other form of y does: two sublayer
// outputs, each (with an optional bias) divided by its root mean square and
// multiplied by a weight, added and scaled; their sums of squares are taken
// while the streams are on their way.
//
// Bound: HBM.  One block per row, four consecutive numbers per thread and
// step.  A row of up to 1024*EPT numbers of up to four streams stays in
// registers across the reduction (EPT = 0: read again behind it).
#include <torch/extension.h>
#include <ATen/hip/HIPContext.h>

#include "seq_common.h"

constexpr int MAX_STREAMS = 32;

struct StreamsArgs {
  const float* bias_a; const float* wa;      // wa null: the branch is a alone
  const float* bias_b; const float* wb;
  float scale, eps;
  const float* mix;                          // (S, S) [from, to]
  const float* wout;                         // (S)
  const float* win;                          // (S), null: write the sum
  const float* alpha;                        // (1)
  const float* nw; const float* nb;          // (D)
  int S, D;
};

DEV_INLINE f32x4v zero4() { return {{0.f, 0.f, 0.f, 0.f}}; }

template <typename T, int NS, int EPT>
__global__ __launch_bounds__(256) void streams_join_kernel(
    T* __restrict__ h_out, float* __restrict__ sum_out,
    float* __restrict__ xs, const T* __restrict__ a, long lda,
    const T* __restrict__ b, long ldb, StreamsArgs p, bool vec) {
  __shared__ float red_a[8], red_b[8];
  const long row = blockIdx.x;
  const int D = p.D, S = p.S;
  float* xr = xs + row * S * D;
  const T* ar = a + row * lda;
  const T* br = b + row * ldb;
  const bool pair = p.wa != nullptr;
  constexpr int NE = EPT > 0 ? EPT : 1;
  f32x4v av[NE], bv[NE], xv[NE][NS];
  // four numbers of a branch, its bias added
  auto branch = [&](const T* r, const float* bias, int i) {
    f32x4v v = load4(r + i, D - i, vec);
    if (bias) {
      const f32x4v c = load4(bias + i, D - i, vec);
#pragma unroll
      for (int e = 0; e < 4; ++e) v.v[e] += c.v[e];
    }
    return v;
  };
  auto streams = [&](f32x4v (&x)[NS], int i) {
#pragma unroll
    for (int s = 0; s < NS; ++s)
      x[s] = NS <= 4 || s < S
                 ? load4((const float*)xr + (long)s * D + i, D - i, vec)
                 : zero4();
  };
  float sa = 0.f, sb = 0.f;
  if (EPT > 0) {
#pragma unroll
    for (int e = 0; e < EPT; ++e) {
      const int i = (threadIdx.x + e * 256) * 4;
      av[e] = bv[e] = zero4();
      if (i < D) {
        av[e] = branch(ar, p.bias_a, i);
        if (pair) bv[e] = branch(br, p.bias_b, i);
        streams(xv[e], i);
      }
    }
  }
  float inv_a = 1.f, inv_b = 1.f;
  if (pair) {
    if (EPT > 0) {
#pragma unroll
      for (int e = 0; e < EPT; ++e)
#pragma unroll
        for (int c = 0; c < 4; ++c) {
          sa += av[e].v[c] * av[e].v[c];
          sb += bv[e].v[c] * bv[e].v[c];
        }
    } else {
      for (int i = threadIdx.x * 4; i < D; i += 1024) {
        const f32x4v u = branch(ar, p.bias_a, i), w = branch(br, p.bias_b, i);
#pragma unroll
        for (int c = 0; c < 4; ++c) {
          if (i + c < D) {
            sa += u.v[c] * u.v[c];
            sb += w.v[c] * w.v[c];
          }
        }
      }
    }
    inv_a = rsqrtf(block_reduce_sum<4>(sa, red_a) / D + p.eps) * p.scale;
    inv_b = rsqrtf(block_reduce_sum<4>(sb, red_b) / D + p.eps) * p.scale;
  }
  auto join = [&](int i, const f32x4v& ya, const f32x4v& yb,
                  const f32x4v (&x)[NS]) {
    f32x4v y = ya;
    if (pair) {
      const f32x4v wa = load4(p.wa + i, D - i, vec);
      const f32x4v wb = load4(p.wb + i, D - i, vec);
#pragma unroll
      for (int c = 0; c < 4; ++c)
        y.v[c] = ya.v[c] * inv_a * wa.v[c] + yb.v[c] * inv_b * wb.v[c];
    }
    f32x4v u = zero4();
#pragma unroll
    for (int t = 0; t < NS; ++t) {
      if (NS > 4 && t >= S) break;
      const float o = p.wout[t];
      f32x4v n;
#pragma unroll
      for (int c = 0; c < 4; ++c) n.v[c] = o * y.v[c];
#pragma unroll
      for (int s = 0; s < NS; ++s) {
        if (NS > 4 && s >= S) break;
        const float m = p.mix[s * S + t];
#pragma unroll
        for (int c = 0; c < 4; ++c) n.v[c] += m * x[s].v[c];
      }
      const float r = p.win ? p.win[t] : 1.f;
#pragma unroll
      for (int c = 0; c < 4; ++c) u.v[c] += r * n.v[c];
      if (p.win) store4(xr + (long)t * D + i, n, D - i, vec);
    }
    if (!p.win) {
      store4(sum_out + row * D + i, u, D - i, vec);
      return;
    }
    const float al = p.alpha[0];
    const f32x4v w = load4(p.nw + i, D - i, vec);
    const f32x4v bb = load4(p.nb + i, D - i, vec);
#pragma unroll
    for (int c = 0; c < 4; ++c) u.v[c] = tanhf(al * u.v[c]) * w.v[c] + bb.v[c];
    store4(h_out + row * D + i, u, D - i, vec);
  };
  if (EPT > 0) {
#pragma unroll
    for (int e = 0; e < EPT; ++e) {
      const int i = (threadIdx.x + e * 256) * 4;
      if (i < D) join(i, av[e], bv[e], xv[e]);
    }
  } else {
    for (int i = threadIdx.x * 4; i < D; i += 1024) {
      const f32x4v ya = branch(ar, p.bias_a, i);
      const f32x4v yb = pair ? branch(br, p.bias_b, i) : zero4();
      streams(xv[0], i);
      join(i, ya, yb, xv[0]);
    }
  }
}

// S copies of the token's table row and the first sublayer's input
template <typename T>
__global__ __launch_bounds__(256) void streams_open_kernel(
    float* __restrict__ xs, T* __restrict__ h_out, const T* __restrict__ table,
    const long* __restrict__ tokens, StreamsArgs p, bool vec) {
  const long row = blockIdx.x;
  const int D = p.D, S = p.S;
  const T* er = table + tokens[row] * D;
  const float al = p.alpha[0];
  for (int i = threadIdx.x * 4; i < D; i += 1024) {
    const f32x4v x = load4(er + i, D - i, vec);
    const f32x4v w = load4(p.nw + i, D - i, vec);
    const f32x4v b = load4(p.nb + i, D - i, vec);
    f32x4v u = zero4();
    for (int s = 0; s < S; ++s) {
      const float r = p.win[s];
#pragma unroll
      for (int c = 0; c < 4; ++c) u.v[c] += r * x.v[c];
      store4(xs + (row * S + s) * D + i, x, D - i, vec);
    }
#pragma unroll
    for (int c = 0; c < 4; ++c) u.v[c] = tanhf(al * u.v[c]) * w.v[c] + b.v[c];
    store4(h_out + row * D + i, u, D - i, vec);
  }
}

template <typename T>
__global__ __launch_bounds__(256) void tanh_norm_kernel(
    T* __restrict__ out, const float* __restrict__ x,
    const float* __restrict__ alpha, const float* __restrict__ w,
    const float* __restrict__ b, int D) {
  const long row = blockIdx.x;
  const float al = alpha[0];
  for (int i = threadIdx.x; i < D; i += 256)
    stf(out + row * D + i, tanhf(al * x[row * D + i]) * w[i] + b[i]);
}

static void check_read(const torch::Tensor& w_in, const torch::Tensor& alpha,
                       const torch::Tensor& w, const torch::Tensor& b, long S,
                       long D) {
  CHECK_F32(w_in); CHECK_F32(alpha); CHECK_F32(w); CHECK_F32(b);
  TORCH_CHECK(w_in.numel() == S && alpha.numel() == 1 && w.numel() == D &&
              b.numel() == D, "stream input weights");
}

static bool aligned16(const torch::Tensor& t) {
  return !t.defined() || (uintptr_t)t.data_ptr() % 16 == 0;
}

void seq_streams_open(torch::Tensor xs, torch::Tensor h, torch::Tensor table,
                      torch::Tensor tokens, torch::Tensor w_in,
                      torch::Tensor alpha, torch::Tensor w, torch::Tensor b) {
  CHECK_F32(xs);
  TORCH_CHECK(table.is_cuda() && table.is_contiguous() && table.dim() == 2);
  TORCH_CHECK(tokens.is_cuda() && tokens.dtype() == torch::kInt64 &&
              tokens.is_contiguous());
  const long N = tokens.numel(), D = table.size(1);
  TORCH_CHECK(xs.dim() == 3 && xs.size(0) == N && xs.size(2) == D);
  const long S = xs.size(1);
  TORCH_CHECK(S >= 1);
  check_read(w_in, alpha, w, b, S, D);
  TORCH_CHECK(h.is_cuda() && h.is_contiguous() && h.dim() == 2 &&
              h.size(0) == N && h.size(1) == D &&
              h.scalar_type() == table.scalar_type());
  if (N == 0) return;
  StreamsArgs p = {};
  p.win = w_in.data_ptr<float>();
  p.alpha = alpha.data_ptr<float>();
  p.nw = w.data_ptr<float>();
  p.nb = b.data_ptr<float>();
  p.S = (int)S;
  p.D = (int)D;
  auto stream = at::hip::getCurrentHIPStream();
  SEQ_DISPATCH_T(table.scalar_type(), {
    const bool vec = rows_by4<T>(table, D) && rows_by4<T>(h, D) &&
                     aligned16(xs) && aligned16(w) && aligned16(b);
    hipLaunchKernelGGL((streams_open_kernel<T>), dim3(N), dim3(256), 0, stream,
        xs.data_ptr<float>(), (T*)h.data_ptr(), (const T*)table.data_ptr(),
        (const long*)tokens.data_ptr<int64_t>(), p, vec); });
  HIP_CHECK_KERNEL();
}

#define JOIN_LAUNCH(NSV, EPTV)                                                \
  hipLaunchKernelGGL((streams_join_kernel<T, NSV, EPTV>), dim3(N), dim3(256), \
      0, stream, p.win ? (T*)out.data_ptr() : nullptr,                        \
      p.win ? nullptr : (float*)out.data_ptr(), xs.data_ptr<float>(),         \
      (const T*)a.data_ptr(), a.stride(0), pair ? (const T*)b.data_ptr()      \
      : nullptr, pair ? b.stride(0) : 0, p, vec)
#define JOIN_BY_WIDTH(NSV)                                                    \
  do {                                                                        \
    if (D <= 1024) JOIN_LAUNCH(NSV, 1);                                       \
    else if (D <= 2048) JOIN_LAUNCH(NSV, 2);                                  \
    else if (D <= 4096) JOIN_LAUNCH(NSV, 4);                                  \
    else JOIN_LAUNCH(NSV, 0);                                                 \
  } while (0)

void seq_streams_join(torch::Tensor out, torch::Tensor xs, torch::Tensor a,
                      torch::Tensor bias_a, torch::Tensor wa, torch::Tensor b,
                      torch::Tensor bias_b, torch::Tensor wb, double scale,
                      double eps, torch::Tensor w_mix, torch::Tensor w_out,
                      torch::Tensor w_in, torch::Tensor alpha,
                      torch::Tensor nw, torch::Tensor nb) {
  CHECK_F32(xs);
  CHECK_ROWS(a);
  CHECK_F32(w_mix);
  CHECK_F32(w_out);
  TORCH_CHECK(xs.dim() == 3);
  const long N = xs.size(0), S = xs.size(1), D = xs.size(2);
  TORCH_CHECK(S >= 1 && S <= MAX_STREAMS, "1 to 32 residual streams");
  TORCH_CHECK(a.size(0) == N && a.size(1) == D, "branch shape");
  TORCH_CHECK(w_mix.numel() == S * S && w_out.numel() == S, "stream weights");
  auto has = [](const torch::Tensor& t) { return t.defined() && t.numel() > 0; };
  auto vecD = [&](const torch::Tensor& t, const char* what) -> const float* {
    if (!has(t)) return nullptr;
    CHECK_F32(t);
    TORCH_CHECK(t.numel() == D, what);
    return t.data_ptr<float>();
  };
  const bool pair = has(wa);
  StreamsArgs p = {};
  p.wa = vecD(wa, "branch norm weight");
  p.wb = vecD(wb, "branch norm weight");
  p.bias_a = vecD(bias_a, "branch bias");
  p.bias_b = vecD(bias_b, "branch bias");
  TORCH_CHECK(has(b) == pair && has(wb) == pair, "a pair has two branches");
  if (pair) {
    CHECK_ROWS(b);
    TORCH_CHECK(b.sizes() == a.sizes() && b.scalar_type() == a.scalar_type());
  }
  p.scale = (float)scale;
  p.eps = (float)eps;
  p.mix = w_mix.data_ptr<float>();
  p.wout = w_out.data_ptr<float>();
  p.S = (int)S;
  p.D = (int)D;
  if (has(w_in)) {
    check_read(w_in, alpha, nw, nb, S, D);
    p.win = w_in.data_ptr<float>();
    p.alpha = alpha.data_ptr<float>();
    p.nw = nw.data_ptr<float>();
    p.nb = nb.data_ptr<float>();
  }
  TORCH_CHECK(out.is_cuda() && out.is_contiguous() && out.dim() == 2 &&
              out.size(0) == N && out.size(1) == D &&
              out.scalar_type() == (p.win ? a.scalar_type() : torch::kFloat32));
  if (N == 0) return;
  auto stream = at::hip::getCurrentHIPStream();
  SEQ_DISPATCH_T(a.scalar_type(), {
    const bool vec = D % 4 == 0 && rows_by4<T>(a, D) &&
                     (!pair || rows_by4<T>(b, D)) && aligned16(xs) &&
                     aligned16(out) && aligned16(wa) && aligned16(wb) &&
                     aligned16(bias_a) && aligned16(bias_b) && aligned16(nw) &&
                     aligned16(nb);
    switch (S) {
      case 1: JOIN_BY_WIDTH(1); break;
      case 2: JOIN_BY_WIDTH(2); break;
      case 3: JOIN_BY_WIDTH(3); break;
      case 4: JOIN_BY_WIDTH(4); break;
      default:
        if (S <= 8) JOIN_LAUNCH(8, 0);
        else JOIN_LAUNCH(32, 0);
    }
  });
  HIP_CHECK_KERNEL();
}

void seq_tanh_norm(torch::Tensor out, torch::Tensor x, torch::Tensor alpha,
                   torch::Tensor w, torch::Tensor b) {
  CHECK_F32(x); CHECK_F32(alpha); CHECK_F32(w); CHECK_F32(b);
  TORCH_CHECK(x.dim() == 2 && out.is_cuda() && out.is_contiguous() &&
              out.sizes() == x.sizes());
  const long N = x.size(0), D = x.size(1);
  TORCH_CHECK(alpha.numel() == 1 && w.numel() == D && b.numel() == D);
  if (N == 0) return;
  auto stream = at::hip::getCurrentHIPStream();
  SEQ_DISPATCH_T(out.scalar_type(), {
    hipLaunchKernelGGL((tanh_norm_kernel<T>), dim3(N), dim3(256), 0, stream,
        (T*)out.data_ptr(), x.data_ptr<float>(), alpha.data_ptr<float>(),
        w.data_ptr<float>(), b.data_ptr<float>(), (int)D); });
  HIP_CHECK_KERNEL();
}
