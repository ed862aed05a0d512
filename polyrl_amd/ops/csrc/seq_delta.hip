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

// tokens per tile: at most 32, the tile within 60 KB of LDS
constexpr int cdelta_tile(int dkp, int cols) {
  const int fit = 60 * 1024 / (4 * (3 * dkp + 2 * cols + 4));
  return fit < 32 ? fit : 32;
}

template <typename T, int RPL, int CPL, int NW>
__global__ __launch_bounds__(64 * NW) void channel_delta_kernel(
    T* __restrict__ out, float* __restrict__ out32, const T* __restrict__ q,
    const T* __restrict__ k, const T* __restrict__ v,
    const T* __restrict__ bl, const T* __restrict__ zl,
    const T* __restrict__ gate, long ldq, long ldk, long ldv, long ldb,
    long ldz, long ldg, const float* __restrict__ dt_bias,
    const float* __restrict__ a_log, const float* __restrict__ norm_w,
    float* __restrict__ state, const int* __restrict__ cu_q,
    const int* __restrict__ state_slot, int H, int G, int Dk, int Dv,
    float q_scale, float key_eps, float eps, bool veck, bool vecv,
    bool vecg) {
  constexpr int DKP = 8 * RPL;              // key rows incl. padding
  constexpr int CW = 8 * CPL;               // columns of a wave
  constexpr int COLS = NW * CW;
  constexpr int THREADS = 64 * NW;
  constexpr int TT = cdelta_tile(DKP, COLS);
  constexpr int KU = TT * DKP / 4;          // four-number units of a tile
  constexpr int VU = TT * COLS / 4;
  constexpr int NIT = (KU + THREADS - 1) / THREADS;
  constexpr int NVI = (VU + THREADS - 1) / THREADS;
  constexpr int EC = COLS / 8;              // a lane's columns in the norm pass
  static_assert(TT <= 8 * NW, "one pass of eight lanes per token");
  __shared__ f32x4v q_s[KU], k_s[KU], d_s[KU], v_s[VU], o_s[VU];
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
  float s[CPL][RPL];
#pragma unroll
  for (int i = 0; i < RPL; ++i)
#pragma unroll
    for (int c = 0; c < CPL; ++c)
      s[c][i] = (col + c < Dv && row_of(i) < Dk)
                    ? S[(long)row_of(i) * Dv + col + c] : 0.f;
  const float A = expf(a_log[h]);
  const int tn = wid * 8 + cl;              // my token in the norm passes
  const int ec0 = rg * EC;                  // ... and my first column there
  float nw[EC];
#pragma unroll
  for (int e = 0; e < EC; ++e)
    nw[e] = (out && ec0 + e < Dv) ? norm_w[ec0 + e] : 0.f;

  f32x4v rq[NIT], rk[NIT], rz[NIT], rv[NVI], gt[EC / 4];
  float rb = 0.f;
  auto fetch = [&](int n0) {
    const int cnt = q1 - n0 < TT ? q1 - n0 : TT;
#pragma unroll
    for (int it = 0; it < NIT; ++it) {
      if (it * THREADS * 4 >= cnt * DKP) break;      // block-uniform
      const int u = tid + it * THREADS;
      const int t = u / (DKP / 4), r = (u % (DKP / 4)) * 4;
      const bool ok = t < cnt && r < Dk;
      const f32x4v z4 = {{0.f, 0.f, 0.f, 0.f}};
      rq[it] = z4; rk[it] = z4; rz[it] = z4;
      if (ok) {
        const long n = n0 + t;
        rq[it] = load4(q + n * ldq + hk + r, Dk - r, veck);
        rk[it] = load4(k + n * ldk + hk + r, Dk - r, veck);
        rz[it] = load4(zl + n * ldz + h * Dk + r, Dk - r, veck);
        const f32x4v bi = load4(dt_bias + h * Dk + r, Dk - r, veck);
#pragma unroll
        for (int e = 0; e < 4; ++e) rz[it].v[e] += bi.v[e];
      }
    }
#pragma unroll
    for (int it = 0; it < NVI; ++it) {
      if (it * THREADS * 4 >= cnt * COLS) break;
      const int u = tid + it * THREADS;
      const int t = u / (COLS / 4), c = cb0 + (u % (COLS / 4)) * 4;
      if (t < cnt && c < Dv)
        rv[it] = load4(v + (long)(n0 + t) * ldv + h * Dv + c, Dv - c, vecv);
      else
        rv[it] = {{0.f, 0.f, 0.f, 0.f}};
    }
    rb = tn < cnt ? ldf(bl + (long)(n0 + tn) * ldb + h) : 0.f;
  };
  fetch(q0);

  for (int n0 = q0; n0 < q1; n0 += TT) {
    const int cnt = q1 - n0 < TT ? q1 - n0 : TT;
    __syncthreads();                        // the tile before is used up
#pragma unroll
    for (int it = 0; it < NIT; ++it) {
      const int u = tid + it * THREADS;
      if (u * 4 < cnt * DKP) {
        q_s[u] = rq[it];
        k_s[u] = rk[it];
        f32x4v d;
#pragma unroll
        for (int e = 0; e < 4; ++e)
          d.v[e] = expf(-A * softplusf_acc(rz[it].v[e]));
        d_s[u] = d;
      }
    }
#pragma unroll
    for (int it = 0; it < NVI; ++it) {
      const int u = tid + it * THREADS;
      if (u * 4 < cnt * COLS) v_s[u] = rv[it];
    }
    const float bcur = rb;
    __syncthreads();
    if (out && tn < cnt) {                  // this tile's output gates
#pragma unroll
      for (int e = 0; e < EC / 4; ++e) {
        const int c = ec0 + 4 * e;
        gt[e] = c < Dv ? load4(gate + (long)(n0 + tn) * ldg + h * Dv + c,
                               Dv - c, vecg)
                       : f32x4v{{0.f, 0.f, 0.f, 0.f}};
      }
    }
    if (n0 + TT < q1) fetch(n0 + TT);       // in flight during the walk
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
        sc_s[tn] = {{ik, iq, qk * ik * iq, sigmoidf_acc(bcur)}};
      }
    }
    __syncthreads();
    if (wave_live) {
      auto step = [&](int t) {
        const f32x4v sc = sc_s[t];
        float kk[RPL], p[CPL], o[CPL], vv[CPL];
        const float* vr = reinterpret_cast<const float*>(v_s) + t * COLS + wcol;
#pragma unroll
        for (int c = 0; c < CPL; ++c) {
          p[c] = 0.f;
          o[c] = 0.f;
          vv[c] = vr[c];
        }
#pragma unroll
        for (int j = 0; j < RPL / 4; ++j) {
          const int at = t * (DKP / 4) + j * 8 + rg;
          const f32x4v kq = k_s[at], dq = d_s[at], qq = q_s[at];
#pragma unroll
          for (int e = 0; e < 4; ++e) {
            kk[4 * j + e] = kq.v[e];
#pragma unroll
            for (int c = 0; c < CPL; ++c) {
              const float x = s[c][4 * j + e] * dq.v[e];
              s[c][4 * j + e] = x;
              p[c] += x * kq.v[e];
              o[c] += x * qq.v[e];
            }
          }
        }
        float* orow = reinterpret_cast<float*>(o_s) + t * COLS + wcol;
#pragma unroll
        for (int c = 0; c < CPL; ++c) {
          p[c] = oct_sum(p[c]);
          o[c] = oct_sum(o[c]);
          const float u = sc.v[3] * (vv[c] - sc.v[0] * p[c]);
          const float ku = sc.v[0] * u;
#pragma unroll
          for (int i = 0; i < RPL; ++i) s[c][i] += kk[i] * ku;
          o[c] = sc.v[1] * o[c] + sc.v[2] * u;
          if (rg == 0) orow[c] = o[c];
        }
      };
      int t = 0;
      for (; t + 2 <= cnt; t += 2) {
        step(t);
        step(t + 1);
      }
      if (t < cnt) step(t);
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
#pragma unroll
          for (int x = 0; x < 4; ++x)
            y.v[x] = ov[4 * e + x] * inv * nw[4 * e + x] *
                     sigmoidf_acc(gt[e].v[x]);
          store4(out + (n * H + h) * Dv + c, y, Dv - c, vecv);
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
  for (int i = 0; i < RPL; ++i)
#pragma unroll
    for (int c = 0; c < CPL; ++c)
      if (col + c < Dv && row_of(i) < Dk)
        S[(long)row_of(i) * Dv + col + c] = s[c][i];
}

void seq_group_rmsnorm(torch::Tensor out, torch::Tensor y,
                       torch::Tensor weight, int64_t groups, double eps,
                       torch::Tensor gate, int64_t gate_act);

template <typename T, int RPL, int CPL, int NW>
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
  const bool veck = rows_by4<T>(q, Dk) && rows_by4<T>(k, Dk) &&
                    rows_by4<T>(zl, Dk) &&
                    (uintptr_t)dt_bias.data_ptr() % 16 == 0;
  const bool vecv = rows_by4<T>(v, Dv) && rows_by4<T>(out, Dv);
  const bool vecg = rows_by4<T>(gate, Dv);
  auto stream = at::hip::getCurrentHIPStream();
  hipLaunchKernelGGL((channel_delta_kernel<T, RPL, CPL, NW>),
      dim3((unsigned)(slot.numel() * H * cblocks)), dim3(64 * NW), 0, stream,
      fused ? (T*)out.data_ptr() : nullptr,
      fused ? nullptr : raw.data_ptr<float>(), (const T*)q.data_ptr(),
      (const T*)k.data_ptr(), (const T*)v.data_ptr(), (const T*)bl.data_ptr(),
      (const T*)zl.data_ptr(), (const T*)gate.data_ptr(), q.stride(0),
      k.stride(0), v.stride(0), bl.stride(0), zl.stride(0), gate.stride(0),
      dt_bias.data_ptr<float>(), a_log.data_ptr<float>(),
      norm_w.data_ptr<float>(), state.data_ptr<float>(),
      cu_q.data_ptr<int>(), slot.data_ptr<int>(), H, G, Dk, Dv,
      1.f / sqrtf((float)Dk), (float)key_eps, (float)eps, veck, vecv, vecg);
  HIP_CHECK_KERNEL();
  if (!fused) seq_group_rmsnorm(out, raw, norm_w, H, eps, gate, 1);
}

void seq_channel_delta(torch::Tensor out, torch::Tensor q, torch::Tensor k,
                       torch::Tensor v, torch::Tensor b_lin,
                       torch::Tensor z_lin, torch::Tensor dt_bias,
                       torch::Tensor a_log, torch::Tensor gate,
                       torch::Tensor norm_w, torch::Tensor state,
                       torch::Tensor cu_q, torch::Tensor state_slot,
                       double key_eps, double eps) {
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
#define CDELTA(RPLV, CPLV, NWV)                                               \
  cdelta_launch<T, RPLV, CPLV, NWV>(out, q, k, v, b_lin, z_lin, dt_bias,      \
      a_log, gate, norm_w, state, cu_q, state_slot, key_eps, eps)
#define CDELTA_W(RPLV, CPLV)                                                  \
  do { if (Dv <= 32 * CPLV) CDELTA(RPLV, CPLV, 4);                            \
       else CDELTA(RPLV, CPLV, 8); } while (0)
  SEQ_DISPATCH_T(dt, {
    if (Dk <= 32) CDELTA_W(4, 2);
    else if (Dk <= 64) CDELTA_W(8, 2);
    else if (Dk <= 128) CDELTA_W(16, 2);
    else if (Dk <= 256) CDELTA_W(32, 1);
    else CDELTA(64, 1, 8);
  });
#undef CDELTA_W
#undef CDELTA
}
