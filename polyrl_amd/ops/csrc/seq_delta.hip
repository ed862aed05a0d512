// Gated delta rule with per-channel decays (fp32 state, in place), with the
// unit vectors, decays, per-head norm and output gate around it.
//
// Per head, S (Dk key channels x Dv columns), for a sequence's rows in order:
//   qn = q / sqrt(|q|^2 + key_eps) * Dk^-1/2,  kn = k / sqrt(|k|^2 + key_eps)
//   g = exp(-exp(a_log) * softplus(z + dt_bias))           per key channel
//   S <- g S;  u = sigmoid(b) (v - S^T kn);  S <- S + kn u^T;  o = S^T qn
//   out = o / sqrt(mean(o^2) + eps) * norm_w * sigmoid(gate)
// Heads share q/k heads in equal groups of neighbours.  One launch serves
// prompt portions and decode tokens (a portion of one row).
//
// A block owns one (sequence, head, column block) and keeps the state in
// registers for the whole portion: a wave spans 8*CPL columns, eight lanes
// share CPL of them and hold RPL = DKP/8 rows each.  Both products with the
// state are taken from the decayed state before the write -- S^T qn of the
// new state is (g S)^T qn + (qn . kn) u -- so a token costs one reduction
// over the eight lanes (three DPP adds) instead of two in sequence.
//
// Token inputs come in tiles of TT rows through LDS: raw q and k, and the
// decays, each computed once per (token, channel).  The lengths of q and k
// and their product are taken from the tile by eight lanes per token, and
// enter the walk as three numbers per token, so the tile itself is never
// scaled.  The walk reads a row's words as b128 loads of which the eight
// row groups cover 128 consecutive bytes.  The next tile's words are
// requested into registers before the current tile is walked; head outputs
// meet in LDS and leave normed and gated, eight lanes per token.
// Columns beyond one block (Dv > COLS) leave as raw fp32 for a separate
// norm-and-gate pass.
#include <torch/extension.h>
#include <ATen/hip/HIPContext.h>

#include "seq_common.h"

// tokens per tile: at most 32, the tile within 58 KB of LDS
constexpr int cdelta_tile(int dkp, int cols) {
  const int fit = 58 * 1024 / (4 * (3 * dkp + 2 * cols + 4));
  return fit < 32 ? fit : 32;
}

// a token's words of one lane
template <int RPL, int CPL>
struct CDeltaIn {
  f32x4v k[RPL / 4], d[RPL / 4], q[RPL / 4], sc;
  float v[CPL];
};

// ONE: every sequence brings one row (tiles of one token, little LDS, so that
// many blocks share a CU; with four columns per lane a wave reads and writes
// whole 128-byte lines of the state, which is what such a step is bound by).
// VEC: all rows allow loads of four numbers.
// Addresses beyond a tile's rows or a head's channels are clamped to its last
// ones and the numbers dropped, so that the loads of a tile are one straight
// run with nothing waiting between them.
template <typename T, int RPL, int CPL, int NW, bool ONE, bool VEC>
__global__ __launch_bounds__(64 * NW, ONE && RPL <= 8 ? 4 : 1)
void channel_delta_kernel(
    T* __restrict__ out, float* __restrict__ out32, const T* __restrict__ q,
    const T* __restrict__ k, const T* __restrict__ v,
    const T* __restrict__ bl, const T* __restrict__ zl,
    const T* __restrict__ gate, long ldq, long ldk, long ldv, long ldb,
    long ldz, long ldg, const float* __restrict__ dt_bias,
    const float* __restrict__ a_log, const float* __restrict__ norm_w,
    float* __restrict__ state, const int* __restrict__ cu_q,
    const int* __restrict__ state_slot, int H, int G, int Dk, int Dv,
    float q_scale, float key_eps, float eps) {
  constexpr int DKP = 8 * RPL;              // key rows incl. padding
  constexpr int CW = 8 * CPL;               // columns of a wave
  constexpr int COLS = NW * CW;
  constexpr int THREADS = 64 * NW;
  constexpr int TT = ONE ? 1 : cdelta_tile(DKP, COLS);
  constexpr int KU = TT * DKP / 4;          // four-number units of a tile
  constexpr int VU = TT * COLS / 4;
  constexpr int NIT = (KU + THREADS - 1) / THREADS;
  constexpr int NVI = (VU + THREADS - 1) / THREADS;
  constexpr int EC = COLS / 8;              // a lane's columns in the norm pass
  static_assert(TT <= 8 * NW, "one pass of eight lanes per token");
  __shared__ f32x4v q_s[KU], k_s[KU], d_s[KU], v_s[VU];
  __shared__ f32x4v o_s[VU + NW * 16 * CPL];   // + where the copies go
  __shared__ f32x4v sc_s[TT];               // 1/|k|, scale/|q|, q.k, beta

  const int cblocks = (Dv + COLS - 1) / COLS;
  const int b = blockIdx.x / (H * cblocks);
  const int h = (blockIdx.x / cblocks) % H;
  const int cb = blockIdx.x % cblocks;
  const int q0 = cu_q[b], q1 = cu_q[b + 1];
  if (q1 <= q0) return;                     // the whole block
  const int tid = threadIdx.x;
  const int lane = tid & 63, wid = tid >> 6;
  const int rg = lane & 7, cl = lane >> 3;
  const int cb0 = cb * COLS;                // first column of the block
  const int wcol = wid * CW + cl * CPL;     // my first column in the block
  const int col = cb0 + wcol;
  const int hk = (h / (H / G)) * Dk;        // q/k columns of this head
  const bool wave_live = cb0 + wid * CW < Dv;

  // row i of a lane: four consecutive rows per eight-lane stripe
  auto row_of = [&](int i) { return ((i >> 2) * 8 + rg) * 4 + (i & 3); };
  float* S = state + ((long)state_slot[b] * H + h) * Dk * Dv;
  // VEC: a lane's columns exist together and are aligned to their number
  struct alignas(4 * CPL) Cols { float x[CPL]; };
  float s[CPL][RPL];
#pragma unroll
  for (int i = 0; i < RPL; ++i) {
    const int row = min(row_of(i), Dk - 1);
    if (VEC) {
      const Cols x = *reinterpret_cast<const Cols*>(
          S + (long)row * Dv + min(col, Dv - CPL));
#pragma unroll
      for (int c = 0; c < CPL; ++c) s[c][i] = x.x[c];
    } else {
#pragma unroll
      for (int c = 0; c < CPL; ++c)
        s[c][i] = S[(long)row * Dv + min(col + c, Dv - 1)];
    }
  }
  const float A2 = -1.4426950408889634f * expf(a_log[h]);
  const int tn = wid * 8 + cl;              // my token in the norm passes
  const int ec0 = rg * EC;                  // ... and my first column there
  auto out_col = [&](int e) {               // VEC: Dv is a multiple of four
    return min(ec0 + 4 * e, Dv - (VEC ? 4 : 1));
  };
  Raw4<float> nw[EC / 4];
#pragma unroll
  for (int e = 0; e < EC / 4; ++e)
    nw[e].template load<VEC>(norm_w + out_col(e), Dv - out_col(e));

  // staging: my four channels (columns) of every TPK-th (TPV-th) token
  constexpr int TPK = THREADS / (DKP / 4), TPV = THREADS / (COLS / 4);
  static_assert(THREADS % (DKP / 4) == 0 && THREADS % (COLS / 4) == 0, "");
  const int kt = tid / (DKP / 4), kr = (tid % (DKP / 4)) * 4;
  const int vt = tid / (COLS / 4), vc = (tid % (COLS / 4)) * 4;
  const int krl = max(min(kr, Dk - 4), 0);  // VEC: Dk and Dv are multiples
  const int kra = VEC ? krl : min(kr, Dk - 1);                   // of four
  const int vca = VEC ? min(cb0 + vc, Dv - 4) : min(cb0 + vc, Dv - 1);
  const bool kok = kr < Dk;
  Raw4<float> bias;
  bias.template load<VEC>(dt_bias + h * Dk + kra, Dk - kra);

  Raw4<T> rq[NIT], rk[NIT], rz[NIT], rv[NVI], gt[EC / 4];
  T rb;
  auto fetch = [&](int n0) {
    const int last = min(q1 - n0, TT) - 1;
#pragma unroll
    for (int it = 0; it < NIT; ++it) {
      const long n = n0 + min(kt + it * TPK, last);
      rq[it].template load<VEC>(q + n * ldq + hk + kra, Dk - kra);
      rk[it].template load<VEC>(k + n * ldk + hk + kra, Dk - kra);
      rz[it].template load<VEC>(zl + n * ldz + h * Dk + kra, Dk - kra);
    }
#pragma unroll
    for (int it = 0; it < NVI; ++it) {
      const long n = n0 + min(vt + it * TPV, last);
      rv[it].template load<VEC>(v + n * ldv + h * Dv + vca, Dv - vca);
    }
    const long n = n0 + min(tn, last);
    rb = bl[n * ldb + h];
#pragma unroll
    for (int e = 0; e < EC / 4; ++e)
      gt[e].template load<VEC>(gate + n * ldg + h * Dv + out_col(e),
                               Dv - out_col(e));
  };
  fetch(q0);
  // the state is needed in the first walk only once: wait for it here, or
  // every walk would also wait for the next tile's words
  __builtin_amdgcn_sched_barrier(0);
#pragma unroll
  for (int i = 0; i < RPL; ++i)
#pragma unroll
    for (int c = 0; c < CPL; ++c) {
      if (col + c >= Dv || row_of(i) >= Dk) s[c][i] = 0.f;
      if (!ONE) asm volatile("" : "+v"(s[c][i]));
    }
  // all eight lanes of a column hold its output: the first writes it to the
  // tile, the others to words of their own (no branch in the walk)
  float* o_at = reinterpret_cast<float*>(o_s) +
                (rg == 0 ? wcol : TT * COLS + tid * CPL);
  const int o_step = rg == 0 ? COLS : 0;

  for (int n0 = q0; n0 < q1; n0 += TT) {
    const int cnt = q1 - n0 < TT ? q1 - n0 : TT;
    __syncthreads();                        // the tile before is used up
#pragma unroll
    for (int it = 0; it < NIT; ++it) {
      const int u = tid + it * THREADS;
      if (u * 4 < cnt * DKP) {
        const f32x4v z = rz[it].get(), bi = bias.get();
        f32x4v d, qv = rq[it].get(), kv = rk[it].get();
#pragma unroll
        for (int e = 0; e < 4; ++e) {
          d.v[e] = __builtin_amdgcn_exp2f(
              A2 * softplusf_fast(z.v[e] + bi.v[e]));
          if (!kok) qv.v[e] = kv.v[e] = 0.f;
        }
        q_s[u] = qv;
        k_s[u] = kv;
        d_s[u] = d;
      }
    }
#pragma unroll
    for (int it = 0; it < NVI; ++it) {
      const int u = tid + it * THREADS;
      if (u * 4 < cnt * COLS) v_s[u] = rv[it].get();
    }
    const float bcur = ldf(&rb);
    Raw4<T> gc[EC / 4];
#pragma unroll
    for (int e = 0; e < EC / 4; ++e) gc[e] = gt[e];
    __syncthreads();
    if (!ONE && n0 + TT < q1) fetch(n0 + TT);   // in flight during the walk
    if (tn < cnt) {                         // lengths, eight lanes per token
      float sq = 0.f, sk = 0.f, qk = 0.f;
#pragma unroll
      for (int j = 0; j < RPL / 4; ++j) {
        const f32x4v a = q_s[tn * (DKP / 4) + j * 8 + rg];
        const f32x4v c = k_s[tn * (DKP / 4) + j * 8 + rg];
#pragma unroll
        for (int e = 0; e < 4; ++e) {
          sq += a.v[e] * a.v[e];
          sk += c.v[e] * c.v[e];
          qk += a.v[e] * c.v[e];
        }
      }
      sq = oct_sum(sq);
      sk = oct_sum(sk);
      qk = oct_sum(qk);
      if (rg == 0) {
        const float iq = q_scale * rsqrtf(sq + key_eps);
        const float ik = rsqrtf(sk + key_eps);
        sc_s[tn] = {{ik, iq, qk * ik * iq, sigmoidf_fast(bcur)}};
      }
    }
    __syncthreads();
    if (wave_live) {
      using In = CDeltaIn<RPL, CPL>;
      auto words = [&](In& in, int t) {
        in.sc = sc_s[t];
        const float* vr = reinterpret_cast<const float*>(v_s) + t * COLS + wcol;
#pragma unroll
        for (int c = 0; c < CPL; ++c) in.v[c] = vr[c];
#pragma unroll
        for (int j = 0; j < RPL / 4; ++j) {
          const int at = t * (DKP / 4) + j * 8 + rg;
          in.k[j] = k_s[at];
          in.d[j] = d_s[at];
          in.q[j] = q_s[at];
        }
      };
      auto step = [&](const In& in, int t) {
        float p[CPL], o[CPL];
#pragma unroll
        for (int c = 0; c < CPL; ++c) p[c] = o[c] = 0.f;
#pragma unroll
        for (int i = 0; i < RPL; ++i)
#pragma unroll
          for (int c = 0; c < CPL; ++c) {
            const float x = s[c][i] * in.d[i / 4].v[i % 4];
            s[c][i] = x;
            p[c] += x * in.k[i / 4].v[i % 4];
            o[c] += x * in.q[i / 4].v[i % 4];
          }
#pragma unroll
        for (int c = 0; c < CPL; ++c) p[c] = oct_sum(p[c]);
#pragma unroll
        for (int c = 0; c < CPL; ++c) {
          const float u = in.sc.v[3] * (in.v[c] - in.sc.v[0] * p[c]);
          const float ku = in.sc.v[0] * u;
#pragma unroll
          for (int i = 0; i < RPL; ++i) s[c][i] += in.k[i / 4].v[i % 4] * ku;
          p[c] = u;
        }
#pragma unroll
        for (int c = 0; c < CPL; ++c)
          o_at[t * o_step + c] = in.sc.v[1] * oct_sum(o[c]) + in.sc.v[2] * p[c];
      };
      if (ONE) {
        In in;
        words(in, 0);
        step(in, 0);
      } else if (RPL <= 16) {
        // the next token's words are read while this one is worked on
        In a, b;
        words(a, 0);
        int t = 0;
        for (; t + 2 <= cnt; t += 2) {
          words(b, t + 1);
          __builtin_amdgcn_sched_barrier(0);
          step(a, t);
          words(a, t + 2 < cnt ? t + 2 : t + 1);
          __builtin_amdgcn_sched_barrier(0);
          step(b, t + 1);
        }
        if (t < cnt) step(a, t);
      } else {
        for (int t = 0; t < cnt; ++t) {
          In in;
          words(in, t);
          step(in, t);
        }
      }
    }
    __syncthreads();                        // head outputs are complete
    if (tn < cnt) {
      const long n = n0 + tn;
      const float* orow = reinterpret_cast<const float*>(o_s) + tn * COLS + ec0;
      if (out) {
        float ov[EC], ss = 0.f;
#pragma unroll
        for (int e = 0; e < EC; ++e) {
          ov[e] = ec0 + e < Dv ? orow[e] : 0.f;
          ss += ov[e] * ov[e];
        }
        const float inv = rsqrtf(oct_sum(ss) / Dv + eps);
#pragma unroll
        for (int e = 0; e < EC / 4; ++e) {
          const int c = ec0 + 4 * e;
          if (c >= Dv) continue;
          f32x4v y;
          const f32x4v g4 = gc[e].get(), w4 = nw[e].get();
#pragma unroll
          for (int x = 0; x < 4; ++x)
            y.v[x] = ov[4 * e + x] * inv * w4.v[x] *
                     sigmoidf_fast(g4.v[x]);
          store4(out + (n * H + h) * Dv + c, y, Dv - c, VEC);
        }
      } else {
#pragma unroll
        for (int e = 0; e < EC; ++e)
          if (cb0 + ec0 + e < Dv)
            out32[(n * H + h) * Dv + cb0 + ec0 + e] = orow[e];
      }
    }
  }
#pragma unroll
  for (int i = 0; i < RPL; ++i) {
    if (row_of(i) >= Dk) continue;
    float* at = S + (long)row_of(i) * Dv + col;
    if (VEC) {
      Cols x;
#pragma unroll
      for (int c = 0; c < CPL; ++c) x.x[c] = s[c][i];
      if (col < Dv) *reinterpret_cast<Cols*>(at) = x;
    } else {
#pragma unroll
      for (int c = 0; c < CPL; ++c)
        if (col + c < Dv) at[c] = s[c][i];
    }
  }
}

void seq_group_rmsnorm(torch::Tensor out, torch::Tensor y,
                       torch::Tensor weight, int64_t groups, double eps,
                       torch::Tensor gate, int64_t gate_act);

template <typename T, int RPL, int CPL, int NW, bool ONE, bool VEC>
static void cdelta_launch(torch::Tensor& out, torch::Tensor& q,
                          torch::Tensor& k, torch::Tensor& v,
                          torch::Tensor& bl, torch::Tensor& zl,
                          torch::Tensor& dt_bias, torch::Tensor& a_log,
                          torch::Tensor& gate, torch::Tensor& norm_w,
                          torch::Tensor& state, torch::Tensor& cu_q,
                          torch::Tensor& slot, double key_eps, double eps) {
  const int H = state.size(1), Dk = state.size(2), Dv = state.size(3);
  const int G = q.size(1) / Dk;
  constexpr int COLS = NW * 8 * CPL;
  const int cblocks = (Dv + COLS - 1) / COLS;
  const bool fused = cblocks == 1;
  torch::Tensor raw;
  if (!fused)
    raw = torch::empty({q.size(0), (long)H * Dv},
                       q.options().dtype(torch::kFloat32));
  auto stream = at::hip::getCurrentHIPStream();
  hipLaunchKernelGGL((channel_delta_kernel<T, RPL, CPL, NW, ONE, VEC>),
      dim3((unsigned)(slot.numel() * H * cblocks)), dim3(64 * NW), 0, stream,
      fused ? (T*)out.data_ptr() : nullptr,
      fused ? nullptr : raw.data_ptr<float>(), (const T*)q.data_ptr(),
      (const T*)k.data_ptr(), (const T*)v.data_ptr(), (const T*)bl.data_ptr(),
      (const T*)zl.data_ptr(), (const T*)gate.data_ptr(), q.stride(0),
      k.stride(0), v.stride(0), bl.stride(0), zl.stride(0), gate.stride(0),
      dt_bias.data_ptr<float>(), a_log.data_ptr<float>(),
      norm_w.data_ptr<float>(), state.data_ptr<float>(),
      cu_q.data_ptr<int>(), slot.data_ptr<int>(), H, G, Dk, Dv,
      1.f / sqrtf((float)Dk), (float)key_eps, (float)eps);
  HIP_CHECK_KERNEL();
  if (!fused) seq_group_rmsnorm(out, raw, norm_w, H, eps, gate, 1);
}

void seq_channel_delta(torch::Tensor out, torch::Tensor q, torch::Tensor k,
                       torch::Tensor v, torch::Tensor b_lin,
                       torch::Tensor z_lin, torch::Tensor dt_bias,
                       torch::Tensor a_log, torch::Tensor gate,
                       torch::Tensor norm_w, torch::Tensor state,
                       torch::Tensor cu_q, torch::Tensor state_slot,
                       double key_eps, double eps, int64_t max_rows) {
  CHECK_ROWS(q); CHECK_ROWS(k); CHECK_ROWS(v); CHECK_ROWS(b_lin);
  CHECK_ROWS(z_lin); CHECK_ROWS(gate);
  CHECK_F32(dt_bias); CHECK_F32(a_log); CHECK_F32(norm_w); CHECK_F32(state);
  CHECK_I32(cu_q); CHECK_I32(state_slot);
  TORCH_CHECK(state.dim() == 4);
  const int H = state.size(1), Dk = state.size(2), Dv = state.size(3);
  const long N = q.size(0);
  TORCH_CHECK(H > 0 && Dk > 0 && Dv > 0 && q.size(1) % Dk == 0);
  const int G = q.size(1) / Dk;
  TORCH_CHECK(G > 0 && H % G == 0 && k.size(1) == (long)G * Dk &&
              v.size(1) == (long)H * Dv && b_lin.size(1) == H &&
              z_lin.size(1) == (long)H * Dk && gate.size(1) == (long)H * Dv,
              "delta rule operand widths");
  TORCH_CHECK(k.size(0) == N && v.size(0) == N && b_lin.size(0) == N &&
              z_lin.size(0) == N && gate.size(0) == N);
  TORCH_CHECK(dt_bias.numel() == (long)H * Dk && a_log.numel() == H &&
              norm_w.numel() == Dv);
  TORCH_CHECK(out.is_cuda() && out.is_contiguous() && out.dim() == 2 &&
              out.size(0) == N && out.size(1) == (long)H * Dv);
  auto dt = q.scalar_type();
  for (const torch::Tensor* t : {&k, &v, &b_lin, &z_lin, &gate, &out})
    TORCH_CHECK(t->scalar_type() == dt, "one activation type");
  TORCH_CHECK(Dk <= 512, "delta rule: key dim above 512 not supported");
  TORCH_CHECK(cu_q.numel() == state_slot.numel() + 1);
  if (N == 0 || state_slot.numel() == 0) return;
#define CDELTA_ARGS                                                           \
  (out, q, k, v, b_lin, z_lin, dt_bias, a_log, gate, norm_w, state, cu_q,     \
   state_slot, key_eps, eps)
// CPLV / NWV: columns per lane and waves of portions, CPL1 / NW1 of single
// tokens
#define CDELTA(RPLV, CPLV, NWV, CPL1, NW1)                                    \
  do {                                                                        \
    if (!vec) cdelta_launch<T, RPLV, CPLV, 8, false, false> CDELTA_ARGS;      \
    else if (max_rows == 1)                                                   \
      cdelta_launch<T, RPLV, CPL1, NW1, true, true> CDELTA_ARGS;              \
    else cdelta_launch<T, RPLV, CPLV, NWV, false, true> CDELTA_ARGS;          \
  } while (0)
#define CDELTA_W(RPLV, CPLV, CPL1)                                            \
  do {                                                                        \
    if (Dv <= 64) CDELTA(RPLV, CPLV, 8 / CPLV, CPL1, 8 / CPL1);               \
    else CDELTA(RPLV, CPLV, 8, CPL1, 16 / CPL1);                              \
  } while (0)
  SEQ_DISPATCH_T(dt, {
    const bool vec = rows_by4<T>(q, Dk) && rows_by4<T>(k, Dk) &&
                     rows_by4<T>(z_lin, Dk) && rows_by4<T>(v, Dv) &&
                     rows_by4<T>(gate, Dv) && rows_by4<T>(out, Dv) &&
                     (uintptr_t)dt_bias.data_ptr() % 16 == 0 &&
                     (uintptr_t)state.data_ptr() % 16 == 0;
    if (Dk <= 32) CDELTA_W(4, 2, 4);
    else if (Dk <= 64) CDELTA_W(8, 2, 4);
    else if (Dk <= 128) CDELTA_W(16, 2, 4);
    else if (Dk <= 256) CDELTA_W(32, 1, 1);
    else CDELTA(64, 1, 8, 1, 8);
  });
#undef CDELTA_W
#undef CDELTA
#undef CDELTA_ARGS
}
