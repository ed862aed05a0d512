// Grouped-query window attention on the matrix cores (bf16).
//
// Same operation as gqa_attn_kernel (seq_gqa.hip), which stays the fp32 /
// odd-size / single-token path.  A block is 4 waves x 16 rows: up to 64
// consecutive tokens of one sequence for one query head.  Their
// windows overlap, so the block walks the union of the visible keys in tiles
// of GKV -- first the kept first tokens that lie before the union's window
// ([0, min(keep, kmin))), then [kmin, last position] -- and masks per
// element, in tiles that need it: key j is live for the row at position p
// when j <= p and (p - j < window or j < keep); with chunks a windowed key
// must also lie in the row's own chunk of positions.
//
// K and V tiles of the head's key/value group come from the paged cache rows
// ([G*D keys | G*Dv values]) into LDS, keys as they are (16-byte pieces
// XOR-swizzled by row), values turned to [entry][key] in 4x4 pieces on the
// way.  The wave computes the scores as K Q^T, so that a lane's accumulators
// hold many keys of ONE row: the softmax needs two lane exchanges per tile,
// and the weights, rounded to bf16, are at once the B operand of V^T P^T (the
// order of keys inside a product's K index is free: both operands use the
// order the accumulators have).  The output accumulates as [entry][row].
// Products run on v_mfma_f32_16x16x32_bf16 with fp32 accumulators; scale, the
// optional distance-bucket bias (this head's column of the table sits in
// LDS), the online softmax and the sigmoid head gate are fp32; so are the
// optional sink (the running maximum starts at the head's sink, the running
// sum at one) and the per-row query temperature folded into the score scale.
// Options: scores capped as cap * tanh(score / cap), a number per head added
// to the capped score, and weights sigmoid(score) per live key without any
// normalisation over keys (no running maximum, no rescaling); head sums as
// fp32 into a separate buffer for the pass that turns rotated values back.
// The next tile's words are fetched into registers while the current one is
// multiplied; the cache rows of the tile after that are looked up meanwhile.
// Key and value head sizes are apart (KS and KV chunks of 32), up to 256 each.
//
// Grid: one dimension.  Workgroups go to the 8 XCDs in turn (id mod 8), each
// with an L2 of its own, so the id is taken apart as XCD = id % 8 and, inside
// an XCD's sequence, the H/G query heads that share a key/value head follow
// each other for the same row tile: their K and V tiles are fetched into that
// XCD's L2 once and hit there for the other heads of the group.  With eight
// key/value heads or a multiple of that, every XCD takes whole key/value
// heads and walks their row tiles in order: successive tiles of a sequence
// read the same rows, which then stay in that one L2 (with few query heads
// per group -- one, for keys expanded per head -- a round-robin over the
// dies would make every die fetch every head's rows).
#include <torch/extension.h>
#include <ATen/hip/HIPContext.h>

#include "seq_common.h"

// tanh through the hardware exponential and reciprocal: 1 - 2 / (1 + e^2x),
// absolute error a few 1e-7, exact limits for large |x|
DEV_INLINE float tanhf_fast(float x) {
  return 1.f - 2.f * __builtin_amdgcn_rcpf(
                         1.f + __builtin_amdgcn_exp2f(2.8853900817779268f * x));
}

typedef __attribute__((ext_vector_type(8))) __bf16 bf16x8_t;
typedef __attribute__((ext_vector_type(4))) float f32x4_t;
typedef __attribute__((ext_vector_type(4))) int i32x4_t;

constexpr int GQA_MAX_REL = 256; // bias-table rows held in LDS
constexpr int GQA_XCDS = 8;      // accelerator dies, each with its own L2

template <int KS>
DEV_INLINE int gtile_off(int row, int byte_col) {
  return row * (KS * 64) + (byte_col ^ ((row & 3) << 4));
}

template <int KS, int KV, int GKV>
__global__ __launch_bounds__(256) void gqa_attn_mfma_kernel(
    bf16_t* __restrict__ out,            // (N, H*Dv), row stride ldo
    const bf16_t* __restrict__ q,        // (N, H*D)
    const bf16_t* __restrict__ cache,    // (slots, G*(D+Dv))
    const int* __restrict__ page_table, int max_pages,
    const int* __restrict__ seq_of_tok, const int* __restrict__ positions,
    const int* __restrict__ tile_n0, const int* __restrict__ tile_cnt,
    int ntiles_rows, const float* __restrict__ rel, int rel_rows,
    const int* __restrict__ dist_bucket,
    const bf16_t* __restrict__ gate, long ldg, int H, int G, int D, int Dv,
    int page_size, int window, int keep, float scale,
    const float* __restrict__ sink, float qt_coef, int qt_every, float cap,
    const float* __restrict__ hbias, bool sigm, float* __restrict__ out32,
    int chunk, long ldo, float out_scale) {
  constexpr int NVT = KV * 2;            // 16-wide output tiles
  constexpr int NKT = GKV / 16;          // 16-key score tiles
  constexpr int VROW = GKV + 8;          // padded LDS row of one value entry
  __shared__ __attribute__((aligned(16))) bf16_t Ks[GKV * KS * 32];
  __shared__ __attribute__((aligned(16))) bf16_t Vt[KV * 32 * VROW];
  __shared__ int slot_s[2][GKV];         // cache rows of a tile's keys
  __shared__ float rel_s[GQA_MAX_REL];

  const int lane = threadIdx.x & 63;
  const int wid = threadIdx.x >> 6;
  const int l15 = lane & 15, lhi = lane >> 4;
  const int per = H / G;                 // query heads per key/value head
  const int xcd = blockIdx.x % GQA_XCDS;
  const int seq_in_xcd = blockIdx.x / GQA_XCDS;
  // (tile, kv head) unit of this block
  const int unit = G % GQA_XCDS == 0
      ? xcd * (ntiles_rows * (G / GQA_XCDS)) + seq_in_xcd / per
      : (seq_in_xcd / per) * GQA_XCDS + xcd;
  if (unit >= ntiles_rows * G) return;   // padding of the last round
  // later row tiles see more keys: they start first, the short ones fill
  // the end of the launch
  const int tile = ntiles_rows - 1 - unit % ntiles_rows;
  const int g = unit / ntiles_rows;
  const int h = g * per + seq_in_xcd % per;
  const int row = G * (D + Dv);
  const int koff = g * D, voff = G * D + g * Dv;
  const int n0 = tile_n0[tile];
  const int cnt = tile_cnt[tile];
  const int b = seq_of_tok[n0];
  const int* ptab = page_table + (long)b * max_pages;
  const int pos0 = positions[n0];
  const int pmax = pos0 + cnt - 1;
  // first windowed key of the row at position p
  auto row_lo = [&](int p) {
    int lo = p - window + 1 > 0 ? p - window + 1 : 0;
    if (chunk > 0) lo = max(lo, p / chunk * chunk);
    return lo;
  };
  const int kmin = row_lo(pos0);
  const int nk = keep < kmin ? keep : kmin;      // kept keys before kmin
  const int nkt = (nk + GKV - 1) / GKV;          // their tiles
  const int nwt = (pmax - kmin) / GKV + 1;       // window tiles
  const int ntiles = nkt + nwt;
  // tile ti covers keys [t0, t0+GKV) up to jmax
  auto tile_t0 = [&](int ti) { return ti < nkt ? ti * GKV : kmin + (ti - nkt) * GKV; };
  auto tile_jmax = [&](int ti) { return ti < nkt ? nk - 1 : pmax; };
  // cache row of a tile's key i (keys past the tile's last: that one)
  auto slot_of = [&](int ti, int i) {
    const int j = min(tile_t0(ti) + i, tile_jmax(ti));
    return ptab[j / page_size] * page_size + j % page_size;
  };
  if (threadIdx.x < GKV) slot_s[0][threadIdx.x] = slot_of(0, threadIdx.x);
  else if ((int)threadIdx.x < 2 * GKV && ntiles > 1)
    slot_s[1][threadIdx.x - GKV] = slot_of(1, threadIdx.x - GKV);
  if (rel)
    for (int i = threadIdx.x; i < rel_rows; i += 256)
      rel_s[i] = rel[(long)i * H + h];

  // ---- this lane's row: Q fragments (k = ks*32 + lhi*8 ..), its state -----
  const int ri = wid * 16 + l15;
  const bool rok = ri < cnt;
  const int rpos = pos0 + ri, rlo = row_lo(rpos);
  bf16x8_t qfrag[KS];
  {
    const bf16_t* qp = q + ((long)(n0 + (rok ? ri : 0)) * H + h) * D;
    const i32x4_t zi = {0, 0, 0, 0};
#pragma unroll
    for (int ks = 0; ks < KS; ++ks) {
      const int d = ks * 32 + lhi * 8;
      qfrag[ks] = d < D ? *reinterpret_cast<const bf16x8_t*>(qp + d)
                        : __builtin_bit_cast(bf16x8_t, zi);
    }
  }
  const float hb = hbias ? hbias[h] : 0.f;
  const float inv_cap = cap > 0.f ? 1.f / cap : 0.f;
  float rscale = scale;
  if (qt_coef != 0.f)
    rscale *= 1.f + qt_coef * logf((float)((rpos + 1) / qt_every + 1));
  // running maximum of the row; each of its four lanes sums its own keys
  float m_run = sink ? sink[h] : -1e30f;
  float l_run = sink && lhi == 0 ? 1.f : 0.f;
  f32x4_t o_acc[NVT];
#pragma unroll
  for (int nt = 0; nt < NVT; ++nt) o_acc[nt] = {0.f, 0.f, 0.f, 0.f};
  // first and last position of the wave's rows (rows past cnt included: what
  // they compute is dropped)
  const int wp0 = pos0 + wid * 16, wp1 = wp0 + 15;
  const int wlo = row_lo(wp1);

  // ---- global -> registers: 16-byte key pieces, 4x4 value pieces ----------
  constexpr int NKI = GKV * KS * 4;              // key pieces of a tile
  constexpr int NK = (NKI + 255) / 256;
  constexpr int KG = GKV / 4;                    // groups of four keys
  constexpr int NVI = KG * KV * 8;               // value pieces of a tile
  constexpr int NV = (NVI + 255) / 256;
  i32x4_t prek[NK];
  uint2 prev[NV][4];
  auto fetch = [&](int ti) {
    const int last = tile_jmax(ti) - tile_t0(ti);   // last live key's place
    const int* sl = slot_s[ti & 1];
#pragma unroll
    for (int i = 0; i < NK; ++i) {
      const int v = threadIdx.x + i * 256;
      const int kr = v / (KS * 4), col = (v % (KS * 4)) * 8;
      prek[i] = {0, 0, 0, 0};
      if (v < NKI && kr <= last && col < D)
        prek[i] = *reinterpret_cast<const i32x4_t*>(
            cache + (long)sl[kr] * row + koff + col);
    }
#pragma unroll
    for (int i = 0; i < NV; ++i) {
      const int v = threadIdx.x + i * 256;
      const int kg = v % KG * 4, col = v / KG * 4;
#pragma unroll
      for (int t = 0; t < 4; ++t) {
        prev[i][t] = make_uint2(0u, 0u);
        if (v < NVI && kg + t <= last && col < Dv)
          prev[i][t] = *reinterpret_cast<const uint2*>(
              cache + (long)sl[kg + t] * row + voff + col);
      }
    }
  };
  __syncthreads();                       // the first two tiles' rows
  fetch(0);

  for (int ti = 0; ti < ntiles; ++ti) {
    const int t0 = tile_t0(ti), jmax = tile_jmax(ti);
    // ---- registers -> LDS tiles, then request the next tile ---------------
#pragma unroll
    for (int i = 0; i < NK; ++i) {
      const int v = threadIdx.x + i * 256;
      if (v < NKI)
        *reinterpret_cast<i32x4_t*>(
            reinterpret_cast<char*>(Ks) +
            gtile_off<KS>(v / (KS * 4), (v % (KS * 4)) * 16)) = prek[i];
    }
#pragma unroll
    for (int i = 0; i < NV; ++i) {
      const int v = threadIdx.x + i * 256;
      if (v < NVI) {
        bf16_t* vt = Vt + v / KG * 4 * VROW + v % KG * 4;
        const uint2* p = prev[i];
        // entry e of the four keys, two per word
        *reinterpret_cast<uint2*>(vt) = make_uint2(
            __builtin_amdgcn_perm(p[1].x, p[0].x, 0x05040100u),
            __builtin_amdgcn_perm(p[3].x, p[2].x, 0x05040100u));
        *reinterpret_cast<uint2*>(vt + VROW) = make_uint2(
            __builtin_amdgcn_perm(p[1].x, p[0].x, 0x07060302u),
            __builtin_amdgcn_perm(p[3].x, p[2].x, 0x07060302u));
        *reinterpret_cast<uint2*>(vt + 2 * VROW) = make_uint2(
            __builtin_amdgcn_perm(p[1].y, p[0].y, 0x05040100u),
            __builtin_amdgcn_perm(p[3].y, p[2].y, 0x05040100u));
        *reinterpret_cast<uint2*>(vt + 3 * VROW) = make_uint2(
            __builtin_amdgcn_perm(p[1].y, p[0].y, 0x07060302u),
            __builtin_amdgcn_perm(p[3].y, p[2].y, 0x07060302u));
      }
    }
    __syncthreads();
    if (ti + 1 < ntiles) fetch(ti + 1);
    int next_slot = 0;                   // stored before the closing barrier
    const bool look = threadIdx.x < GKV && ti + 2 < ntiles;
    if (look) next_slot = slot_of(ti + 2, threadIdx.x);

    // ---- S^T (GKV keys x 16 rows) = K Q^T; row l15, keys lhi*4 + r --------
    float p[NKT][4];
#pragma unroll
    for (int nt = 0; nt < NKT; ++nt) {
      f32x4_t c = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int ks = 0; ks < KS; ++ks) {
        const bf16x8_t kf = *reinterpret_cast<const bf16x8_t*>(
            reinterpret_cast<const char*>(Ks) +
            gtile_off<KS>(nt * 16 + l15, (ks * 32 + lhi * 8) * 2));
        c = __builtin_amdgcn_mfma_f32_16x16x32_bf16(kf, qfrag[ks], c, 0, 0, 0);
      }
#pragma unroll
      for (int r = 0; r < 4; ++r) p[nt][r] = c[r] * rscale;
    }
    // ---- bias, cap, mask ----------------------------------------------------
    // (wave-uniform) every key of the tile is live for every row
    const bool full = t0 + GKV - 1 <= min(wp0, jmax) && t0 >= wlo;
    if (rel || cap > 0.f || hbias) {
#pragma unroll
      for (int nt = 0; nt < NKT; ++nt)
#pragma unroll
        for (int r = 0; r < 4; ++r) {
          float sv = p[nt][r];
          if (rel) {
            const int dist = rpos - (t0 + nt * 16 + lhi * 4 + r);
            if (dist >= 0 && dist < window) sv += rel_s[dist_bucket[dist]];
          }
          if (cap > 0.f) sv = cap * tanhf_fast(sv * inv_cap);
          p[nt][r] = sv + hb;
        }
    }
    if (!full) {
#pragma unroll
      for (int nt = 0; nt < NKT; ++nt)
#pragma unroll
        for (int r = 0; r < 4; ++r) {
          const int j = t0 + nt * 16 + lhi * 4 + r;
          const bool live = j <= jmax && j <= rpos && (j >= rlo || j < keep);
          if (!live) p[nt][r] = -1e30f;
        }
    }
    // ---- weights --------------------------------------------------------------
    if (sigm) {
#pragma unroll
      for (int nt = 0; nt < NKT; ++nt)
#pragma unroll
        for (int r = 0; r < 4; ++r)
          p[nt][r] = p[nt][r] > -1e29f ? sigmoidf_acc(p[nt][r]) : 0.f;
    } else {
      float mx = p[0][0];
#pragma unroll
      for (int nt = 0; nt < NKT; ++nt)
#pragma unroll
        for (int r = 0; r < 4; ++r) mx = fmaxf(mx, p[nt][r]);
      mx = fmaxf(mx, __shfl_xor(mx, 16, 64));
      mx = fmaxf(mx, __shfl_xor(mx, 32, 64));
      const float mn = fmaxf(m_run, mx);
      if (__any(mn > m_run)) {           // some row's maximum moved
        const float alpha = __expf(m_run - mn);
        l_run *= alpha;
#pragma unroll
        for (int nt = 0; nt < NVT; ++nt)
#pragma unroll
          for (int r = 0; r < 4; ++r) o_acc[nt][r] *= alpha;
        m_run = mn;
      }
      float rs = 0.f;
#pragma unroll
      for (int nt = 0; nt < NKT; ++nt)
#pragma unroll
        for (int r = 0; r < 4; ++r) {
          // (a row without a live key so far has m_run = -1e30)
          const float e = __expf(p[nt][r] - m_run);
          p[nt][r] = full || p[nt][r] > -1e29f ? e : 0.f;
          rs += p[nt][r];
        }
      l_run += rs;
    }

    // ---- O^T += V^T P^T, keys in the accumulators' order ---------------------
#pragma unroll
    for (int kb = 0; kb < NKT / 2; ++kb) {
      bf16x8_t pb;
#pragma unroll
      for (int j = 0; j < 4; ++j) {
        pb[j] = (__bf16)p[2 * kb][j];
        pb[4 + j] = (__bf16)p[2 * kb + 1][j];
      }
#pragma unroll
      for (int nt = 0; nt < NVT; ++nt) {
        if (nt * 16 < Dv) {
          const bf16_t* vr = Vt + (nt * 16 + l15) * VROW + kb * 32 + lhi * 4;
          const uint2 a = *reinterpret_cast<const uint2*>(vr);
          const uint2 c = *reinterpret_cast<const uint2*>(vr + 16);
          const i32x4_t av = {(int)a.x, (int)a.y, (int)c.x, (int)c.y};
          o_acc[nt] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(
              __builtin_bit_cast(bf16x8_t, av), pb, o_acc[nt], 0, 0, 0);
        }
      }
    }
    if (look) slot_s[ti & 1][threadIdx.x] = next_slot;
    __syncthreads();   // every wave is done with the tiles before restaging
  }

  l_run += __shfl_xor(l_run, 16, 64);
  l_run += __shfl_xor(l_run, 32, 64);
  if (!rok) return;
  const long tok = n0 + ri;
  float inv = (sigm ? 1.f : 1.f / l_run) * out_scale;
  if (gate && !out32) inv *= sigmoidf_acc(bf2f(gate[tok * ldg + h]));
  bf16_t* op = out + tok * ldo + h * Dv;
  float* op32 = out32 ? out32 + (tok * H + h) * Dv : nullptr;
  const bool by8 = ((uintptr_t)op & 7) == 0;
#pragma unroll
  for (int nt = 0; nt < NVT; ++nt) {
    const int d = nt * 16 + lhi * 4;     // four entries; Dv is a multiple of 8
    if (d < Dv) {
      f32x4v o;
#pragma unroll
      for (int r = 0; r < 4; ++r) o.v[r] = o_acc[nt][r] * inv;
      if (op32) store4(op32 + d, o, 4, true);
      else store4(op + d, o, 4, by8);
    }
  }
}

void gqa_attention_check(torch::Tensor out, torch::Tensor q,
                         torch::Tensor cache, torch::Tensor page_table,
                         torch::Tensor seq_of_tok, torch::Tensor positions,
                         int64_t H, int64_t G, int64_t D, int64_t Dv,
                         int64_t window, int64_t keep_first,
                         torch::Tensor rel, torch::Tensor dist_bucket,
                         torch::Tensor gate, torch::Tensor sink,
                         int64_t q_temp_every);
void seq_gqa_window_attention(torch::Tensor out, torch::Tensor q,
                              torch::Tensor cache, torch::Tensor page_table,
                              torch::Tensor seq_of_tok,
                              torch::Tensor positions, int64_t H, int64_t G,
                              int64_t D, int64_t Dv, int64_t window,
                              int64_t keep_first, torch::Tensor rel,
                              torch::Tensor dist_bucket, torch::Tensor gate,
                              double scale, torch::Tensor sink,
                              double q_temp_coef, int64_t q_temp_every,
                              double softcap, torch::Tensor head_bias,
                              bool sigmoid_weights, torch::Tensor v_inv_freq,
                              int64_t chunk, double out_scale);
void seq_rotate_back_heads(torch::Tensor out, torch::Tensor x,
                           torch::Tensor inv_freq, torch::Tensor positions,
                           torch::Tensor gate, int64_t H);

#define GQA_MFMA_LAUNCH(KSV, KVV)                                             \
  hipLaunchKernelGGL(                                                         \
      (gqa_attn_mfma_kernel<KSV, KVV, (KVV > 4 ? 32 : 64)>), grid, dim3(256), \
      0, stream,                                                              \
      (bf16_t*)out.data_ptr(), (const bf16_t*)q.data_ptr(),                   \
      (const bf16_t*)cache.data_ptr(), page_table.data_ptr<int>(),            \
      (int)page_table.size(1), seq_of_tok.data_ptr<int>(),                    \
      positions.data_ptr<int>(), tile_n0.data_ptr<int>(),                     \
      tile_cnt.data_ptr<int>(), ntiles,                                       \
      has_rel ? rel.data_ptr<float>() : nullptr,                              \
      has_rel ? (int)rel.size(0) : 0,                                         \
      has_rel ? dist_bucket.data_ptr<int>() : nullptr,                        \
      has_gate ? (const bf16_t*)gate.data_ptr() : nullptr,                    \
      has_gate ? gate.stride(0) : 0, (int)H, (int)G, (int)D, (int)Dv,         \
      (int)cache.size(1), (int)window, (int)keep_first, (float)scale,         \
      has_sink ? sink.data_ptr<float>() : nullptr, (float)q_temp_coef,        \
      (int)q_temp_every, (float)softcap,                                      \
      has_hb ? head_bias.data_ptr<float>() : nullptr, sigmoid_weights, o32,   \
      (int)chunk, (long)out.stride(0), (float)out_scale)

void seq_gqa_window_attention_mfma(
    torch::Tensor out, torch::Tensor q, torch::Tensor tile_n0,
    torch::Tensor tile_cnt, torch::Tensor cache, torch::Tensor page_table,
    torch::Tensor seq_of_tok, torch::Tensor positions, int64_t H, int64_t G,
    int64_t D, int64_t Dv, int64_t window, int64_t keep_first,
    torch::Tensor rel, torch::Tensor dist_bucket, torch::Tensor gate,
    double scale, torch::Tensor sink, double q_temp_coef,
    int64_t q_temp_every, double softcap, torch::Tensor head_bias,
    bool sigmoid_weights, torch::Tensor v_inv_freq, int64_t chunk,
    double out_scale) {
  gqa_attention_check(out, q, cache, page_table, seq_of_tok, positions, H, G,
                      D, Dv, window, keep_first, rel, dist_bucket, gate, sink,
                      q_temp_every);
  const bool has_sink = sink.defined() && sink.numel() > 0;
  CHECK_I32(tile_n0); CHECK_I32(tile_cnt);
  TORCH_CHECK(tile_n0.numel() == tile_cnt.numel());
  const bool has_rel = rel.defined() && rel.numel() > 0;
  const bool has_gate = gate.defined() && gate.numel() > 0;
  const int ks = (int)((D + 31) / 32), kv = (int)((Dv + 31) / 32);
  if (q.scalar_type() != torch::kBFloat16 || D % 8 || Dv % 8 ||
      std::max(ks, kv) > 8 ||
      (has_rel && rel.size(0) > GQA_MAX_REL)) {
    seq_gqa_window_attention(out, q, cache, page_table, seq_of_tok, positions,
                             H, G, D, Dv, window, keep_first, rel,
                             dist_bucket, gate, scale, sink, q_temp_coef,
                             q_temp_every, softcap, head_bias,
                             sigmoid_weights, v_inv_freq, chunk, out_scale);
    return;
  }
  const int ntiles = tile_n0.numel();
  if (q.size(0) == 0 || ntiles == 0) return;
  const bool has_hb = head_bias.defined() && head_bias.numel() > 0;
  if (has_hb) {
    CHECK_F32(head_bias);
    TORCH_CHECK(head_bias.numel() == H, "one bias per query head");
  }
  TORCH_CHECK(!sigmoid_weights || !has_sink, "a sink needs softmax weights");
  const bool v_rot = v_inv_freq.defined() && v_inv_freq.numel() > 0;
  TORCH_CHECK(chunk >= 0 && (!v_rot || (out.is_contiguous() && out_scale == 1.0)),
              "rotated values are written unscaled to whole rows");
  torch::Tensor sums;
  float* o32 = nullptr;
  if (v_rot) {
    sums = torch::empty({q.size(0), H * Dv}, q.options().dtype(torch::kFloat32));
    o32 = sums.data_ptr<float>();
  }
  // (tile, kv head) units in rounds of one per XCD, H/G heads per unit
  const long units = (long)ntiles * G;
  const long rounds = (units + GQA_XCDS - 1) / GQA_XCDS;
  TORCH_CHECK(rounds * GQA_XCDS * (H / G) < (1L << 31), "grid too large");
  const dim3 grid((unsigned)(rounds * GQA_XCDS * (H / G)));
  auto stream = at::hip::getCurrentHIPStream();
  switch (std::max(ks, kv)) {
    case 1: GQA_MFMA_LAUNCH(1, 1); break;
    case 2: GQA_MFMA_LAUNCH(2, 2); break;
    case 3: GQA_MFMA_LAUNCH(3, 3); break;
    case 4: GQA_MFMA_LAUNCH(4, 4); break;
    case 5: case 6:
      if (ks <= 3) GQA_MFMA_LAUNCH(3, 6);
      else GQA_MFMA_LAUNCH(6, 6);
      break;
    default:
      if (ks <= 4) GQA_MFMA_LAUNCH(4, 8);
      else GQA_MFMA_LAUNCH(8, 8);
  }
  HIP_CHECK_KERNEL();
  if (v_rot) seq_rotate_back_heads(out, sums, v_inv_freq, positions, gate, H);
}
