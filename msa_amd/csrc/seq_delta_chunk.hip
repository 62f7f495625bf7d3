// Chunked form of the delta rule with a decay per key channel on the matrix cores (bf16 inputs, fp32 states and decays), for
// portions long enough to be cut into chunks of 64 tokens.  With G_t the sum of the chunk's log-decays up to token t (a vector
// over the key channels, in powers of two), S_0 the state in front of the chunk, and products of vectors element by element,
//   u_t = beta_t (v_t - S_0^T (2^G_t k_t) - sum_{s < t} L_ts u_s / beta_t),   L_ts = beta_t sum_d k_td k_sd 2^(G_td - G_sd)
// so that with T = (1 + L)^-1 (unit lower triangular)
//   U   = U' - W S_0,   U' = T diag(beta) V,   W = T diag(beta) (2^G K)
//   o_t = S_0^T (2^G_t q_t) + sum_{s <= t} A_ts u_s,   A_ts = sum_d q_td k_sd 2^(G_td - G_sd)
//   S   = 2^G_end S_0 + sum_s (2^(G_end - G_s) k_s) u_s^T.
//   (1) prepare_chunk  a workgroup per (chunk, head): everything that does not need S_0
//   (2) StateWalk      a workgroup per (sequence, head, 16 or 32 value columns) walks over the chunks: U, o and S
//   (3) msa_seq_head_norm_gate
// (1) is bound by memory and arithmetic, (2) by the latency of its chain, so they share launches: one launch prepares a segment of
// chunks while it walks over the segment before.  Segments also bound the workspace (two of them).
//
// Decays differ by channel, so L and A are products of operands that carry them: within blocks of 16 tokens everything is
// relative to the block's start (rows, exponents <= 0) and its end (columns, exponents <= 0), and whole blocks' decays between
// the two scale the columns.  Only inside a diagonal block the columns' exponents are positive; a block in which some channel
// falls by more than 2^-80 is taken apart once more, into four tokens a part (steep_block).
//
// Operands that carry decays or states are fp32 values: what enters the state does so as a high and a low bf16 part (three
// products, about 16 bits of mantissa).  The read-out's own operands (2^G q and A) are single bf16, like its result.
//
// The operands (2) reads lie in its own order: fragments of 16 rows and 32 summands, 16 bytes a lane.  Two accumulator tiles of 16
// rows hold, in a lane of quarter g of the wavefront, rows 4 g + 0..3 each; taken as the next product's operand that names an order
// of its 32 summands, {4 g + 0..3, 16 + 4 g + 0..3}, which the other operand follows: nothing is transposed on the way.
#include <algorithm>

#include "seq_mfma.h"

namespace {

constexpr int kC = 64;                   // tokens of a chunk
constexpr int kB = 16;                   // of a block
constexpr int kTS = kC + 8;              // LDS row stride of [.., 64] bf16 tiles
constexpr int kLS = kC + 4;              // and of fp32 ones
constexpr int kVB = 128, kVS = kVB + 8;  // value columns prepared at a time
constexpr float kMaxFall = 80.f;

// Byte offsets of a (chunk, head)'s operands.  DP: D padded to a multiple of 32.
template <int DP>
struct Layout {
  static constexpr int w = 0;                       // -W: [row tile 4][DP / 32][high, low] fragments of 1 KB
  static constexpr int q = w + DP * 256;            // 2^G q: [row tile 4][DP / 32]
  static constexpr int k = q + DP * 128;            // 2^(G_end - G) k, transposed: [DP / 16][2][high, low]
  static constexpr int a = k + DP * 256;            // A: row tiles 0 and 1: one fragment each, 2 and 3: two
  static constexpr int gamma = a + 6 * 1024;        // 2^G_end: [DP] fp32
  static constexpr int u = gamma + DP * 4;          // U': [E / 16][row tile 4] accumulators of 1 KB
  static constexpr int64_t bytes(int E) { return u + (int64_t)(E + 31) / 32 * 8192; }
};

struct ChunkArgs {
  msa_delta_args d;
  char* ws;                // [n_seq, H, seg] units of Layout::bytes
  int64_t unit;
  int32_t first, seg;      // first chunk and number of chunks of the segment
};

__device__ __forceinline__ void wave_fence() {
  __builtin_amdgcn_fence(__ATOMIC_ACQ_REL, "wavefront");
  __builtin_amdgcn_wave_barrier();
}
// log2(1 + 2^y): its series where 1 + e would round e away (above 24 it is y).
__device__ __forceinline__ float softplus2_f(float y) {
  const float yc = fminf(y, 24.f), e = __builtin_amdgcn_exp2f(yc);
  const float small = e * (1.0f + e * (-0.5f + e * (0.33333333f - 0.25f * e))) * kLog2e;
  const float big = __builtin_amdgcn_logf(1.0f + e);
  return (e < 0.015625f ? small : big) + (y - yc);
}
__device__ __forceinline__ float lane_value(float v, int lane) {
  return __uint_as_float(__builtin_amdgcn_readlane(__float_as_uint(v), lane));
}
__device__ __forceinline__ __amdgpu_buffer_rsrc_t rows_rsrc(const bf16_t* p, int rows, int64_t stride, int n) {
  return __builtin_amdgcn_make_buffer_rsrc(const_cast<bf16_t*>(p), 0, __builtin_amdgcn_readfirstlane(rows > 0 ? (int)((rows - 1) * stride + n) * 2 : 0), 0x00020000);
}
__device__ __forceinline__ u32x4_t as_u32(bf16x8_t v) { return __builtin_bit_cast(u32x4_t, v); }
__device__ __forceinline__ bf16x8_t as_bf16(u32x4_t v) { return __builtin_bit_cast(bf16x8_t, v); }
__device__ __forceinline__ floatx16_t zero16() {
  floatx16_t z;
#pragma unroll
  for (int e = 0; e < 16; ++e) z[e] = 0.f;
  return z;
}

// Sums over d of k_t k_s 2^(G_t - G_s) and q_t k_s 2^(G_t - G_s) of a 16-token block in which decays may be of any size, one
// wavefront: parts of four tokens, factored at the row part's start where row and column lie in different ones (all exponents
// <= 0), pair by pair within a part.  LDS rows of this block: g [16][DP + 4] log-decays, k and q [16][DP + 8].  Results: row
// 4 (lane / 16) + e, column lane % 16.
template <int DP>
__device__ void steep_block(const float* g, const bf16_t* k, const bf16_t* q, floatx4_t& dk, floatx4_t& dq) {
  constexpr int kKS = DP + 8, kES = DP + 4, kN = DP / 32;
  const int lane = threadIdx.x & 63, l15 = lane & 15, g4 = lane >> 4;
  // within parts: lane = (part, row, column)
  float in_k = 0.f, in_q = 0.f;
  {
    const int t = 4 * g4 + (l15 >> 2), u = 4 * g4 + (l15 & 3);
    for (int d = 0; d < DP; d += 4) {
      float gt[4], gu[4], kt[4], ku[4], qt[4];
      load_vec<float, 4>(g + t * kES + d, gt);
      load_vec<float, 4>(g + u * kES + d, gu);
      load_vec<bf16_t, 4>(k + t * kKS + d, kt);
      load_vec<bf16_t, 4>(k + u * kKS + d, ku);
      load_vec<bf16_t, 4>(q + t * kKS + d, qt);
#pragma unroll
      for (int e = 0; e < 4; ++e) {
        const float w = __builtin_amdgcn_exp2f(fminf(gt[e] - gu[e], 0.f)) * ku[e];
        in_k += w * kt[e];
        in_q += w * qt[e];
      }
    }
  }
  bf16x8_t kh[kN], kl[kN], qh[kN];                               // rows: decayed from their part's start
#pragma unroll
  for (int i = 0; i < kN; ++i) {
    const int d = 32 * i + 8 * g4, start = 4 * (l15 >> 2) - 1;
    float x[8], y[8], w[8], r[8] = {};
    load_vec<float, 8>(g + l15 * kES + d, w);
    if (start >= 0) load_vec<float, 8>(g + start * kES + d, r);
    load_vec<bf16_t, 8>(k + l15 * kKS + d, x);
    load_vec<bf16_t, 8>(q + l15 * kKS + d, y);
#pragma unroll
    for (int e = 0; e < 8; ++e) {
      const float f = __builtin_amdgcn_exp2f(w[e] - r[e]);
      x[e] *= f;
      y[e] *= f;
    }
    split8(x, kh[i], kl[i]);
    bf16x8_t rest;
    split8(y, qh[i], rest);
  }
#pragma unroll
  for (int part = 1; part < 4; ++part) {
    floatx4_t pk = {0.f, 0.f, 0.f, 0.f}, pq = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int i = 0; i < kN; ++i) {
      const int d = 32 * i + 8 * g4;
      float x[8], w[8], r[8];
      load_vec<float, 8>(g + l15 * kES + d, w);
      load_vec<float, 8>(g + (4 * part - 1) * kES + d, r);
      load_vec<bf16_t, 8>(k + l15 * kKS + d, x);
#pragma unroll
      for (int e = 0; e < 8; ++e) x[e] *= __builtin_amdgcn_exp2f(fminf(r[e] - w[e], 0.f));
      bf16x8_t hi, low;
      split8(x, hi, low);
      pk = __builtin_amdgcn_mfma_f32_16x16x32_bf16(kh[i], hi, pk, 0, 0, 0);
      pq = __builtin_amdgcn_mfma_f32_16x16x32_bf16(qh[i], hi, pq, 0, 0, 0);
      pk = __builtin_amdgcn_mfma_f32_16x16x32_bf16(kh[i], low, pk, 0, 0, 0);
      pq = __builtin_amdgcn_mfma_f32_16x16x32_bf16(qh[i], low, pq, 0, 0, 0);
      pk = __builtin_amdgcn_mfma_f32_16x16x32_bf16(kl[i], hi, pk, 0, 0, 0);
    }
    if (g4 == part) {
      dk = pk;
      dq = pq;
    }
  }
#pragma unroll
  for (int e = 0; e < 4; ++e) {
    const float vk = __shfl(in_k, 16 * g4 + 4 * e + (l15 & 3)), vq = __shfl(in_q, 16 * g4 + 4 * e + (l15 & 3));
    if ((l15 >> 2) == g4) {
      dk[e] = vk;
      dq[e] = vq;
    }
  }
}

template <int DP>
constexpr int prepare_lds() {
  const int ke = kC * (DP + 4) * 4, tv = 2 * kC * kTS * 2 + kC * kVS * 2;
  return 2 * kC * (DP + 8) * 2 + (ke > tv ? ke : tv) + 3 * 4 * DP * 4 + kC * 4;
}

template <int DP>
__device__ __forceinline__ void prepare_chunk(const ChunkArgs& c, const msa_seq_batch& b, char* lds, int head, int chunk, int s) {
  constexpr int kKS = DP + 8, kES = DP + 4, kN = DP / 32;
  constexpr int kKE = kC * kES * 4, kTV = 2 * kC * kTS * 2 + kC * kVS * 2;
  bf16_t* kph = reinterpret_cast<bf16_t*>(lds);                  // [64][kKS] 2^(G - block start) k, high
  bf16_t* kpl = kph + kC * kKS;                                  // and low parts
  char* shared = lds + 2 * kC * kKS * 2;
  float* ke = reinterpret_cast<float*>(shared);                  // [64][kES] 2^(block end - G) k; then
  float* lt = reinterpret_cast<float*>(shared);                  // [64][kLS] L, with T's diagonal blocks in place of its own; then
  bf16_t* th = reinterpret_cast<bf16_t*>(shared);                // [64][kTS] T diag(beta), high
  bf16_t* tl = th + kC * kTS;                                    // and low parts
  bf16_t* as = tl + kC * kTS;                                    // [64][kTS] A; then
  bf16_t* vs = as;                                               // [64][kVS] values
  float* e2 = reinterpret_cast<float*>(shared + (kKE > kTV ? kKE : kTV));   // [4][DP] decay over a whole block,
  float* inv2 = e2 + 4 * DP;                                     // its inverse,
  float* pre = inv2 + 4 * DP;                                    // and the decay in front of a block
  float* beta = pre + 4 * DP;                                    // [64]
  static_assert(kC * kLS * 4 <= 2 * kC * kTS * 2, "L lies in front of A");

  const msa_delta_args& a = c.d;
  const int tid = threadIdx.x, lane = tid & 63, wave = __builtin_amdgcn_readfirstlane(tid >> 6), l15 = lane & 15, g4 = lane >> 4;
  const int kvh = head / (a.H / a.G);
  const int lo = b.cu[s], t0 = (c.first + chunk) * kC, rows = min(kC, b.cu[s + 1] - lo - t0);
  if (rows <= 0) return;
  char* unit = c.ws + (((int64_t)s * a.H + head) * c.seg + chunk) * c.unit;
  const int brow = kB * wave, live = rows - brow;                // this wavefront's block and its tokens (may be none)
  const bf16_t* qkv = static_cast<const bf16_t*>(a.qkv) + (int64_t)(lo + t0) * a.qkv_stride;
  const bf16_t* kp = qkv + (int64_t)brow * a.qkv_stride + (int64_t)(a.G + kvh) * a.D;
  const __amdgpu_buffer_rsrc_t rs_q = rows_rsrc(kp - (int64_t)a.G * a.D, live, a.qkv_stride, a.D);
  const __amdgpu_buffer_rsrc_t rs_k = rows_rsrc(kp, live, a.qkv_stride, a.D);
  const __amdgpu_buffer_rsrc_t rs_a = rows_rsrc(static_cast<const bf16_t*>(a.a) + (int64_t)(lo + t0 + brow) * a.a_stride + (int64_t)head * a.D,
                                                live, a.a_stride, a.D);

  // ---- a wavefront's block: unit vectors, decays from its start and to its end.  Lane = two channels.
  const int c0 = 2 * lane, row_bytes = (int)a.qkv_stride * 2;
  const bool mine = DP == 128 || lane < DP / 2, in = c0 < a.D;
  const int c_at = in ? c0 * 2 : kOutside;
  uint32_t kw[kB], qw[kB], aw[kB];
#pragma unroll
  for (int t = 0; t < kB; ++t) {
    kw[t] = __builtin_amdgcn_raw_buffer_load_b32(rs_k, c_at + t * row_bytes, 0, 0);
    qw[t] = __builtin_amdgcn_raw_buffer_load_b32(rs_q, c_at + t * row_bytes, 0, 0);
    aw[t] = __builtin_amdgcn_raw_buffer_load_b32(rs_a, c_at + t * (int)a.a_stride * 2, 0, 0);
  }
  float kinv = 0.f, qinv = 0.f;                                  // of row lane / 4
#pragma unroll
  for (int j = 0; j < kN; ++j) {
    const int col = 32 * j + 8 * (lane & 3), at = col < a.D ? col * 2 + (lane >> 2) * row_bytes : kOutside;
    const u32x4_t kv = __builtin_amdgcn_raw_buffer_load_b128(rs_k, at, 0, 0), qv = __builtin_amdgcn_raw_buffer_load_b128(rs_q, at, 0, 0);
#pragma unroll
    for (int e = 0; e < 4; ++e) {
      kinv += bf16lo(kv[e]) * bf16lo(kv[e]) + bf16hi(kv[e]) * bf16hi(kv[e]);
      qinv += bf16lo(qv[e]) * bf16lo(qv[e]) + bf16hi(qv[e]) * bf16hi(qv[e]);
    }
  }
  kinv += __shfl_xor(kinv, 1);
  qinv += __shfl_xor(qinv, 1);
  kinv += __shfl_xor(kinv, 2);
  qinv += __shfl_xor(qinv, 2);
  kinv = 1.0f / sqrtf(kinv + 1e-6f);
  qinv = 1.0f / sqrtf((qinv + 1e-6f) * (float)a.D);
  if (lane < kB)
    beta[brow + lane] = lane < live ? sigmoid_f(bf16_to_f32(static_cast<const bf16_t*>(a.b)[(int64_t)(lo + t0 + brow + lane) * a.b_stride + head])) : 0.f;
  float gx[kB], gy[kB];                                          // log-decays from the block's start
  {
    const float rate = -expf(a.A_log[head]);
    const float2 bias = in ? *reinterpret_cast<const float2*>(a.dt_bias + (int64_t)head * a.D + c0) : make_float2(0.f, 0.f);
    float x = 0.f, y = 0.f;
#pragma unroll
    for (int t = 0; t < kB; ++t) {
      const float on = t < live ? rate : 0.f;                    // no decay behind the sequence
      x += on * softplus2_f((bf16lo(aw[t]) + bias.x) * kLog2e);
      y += on * softplus2_f((bf16hi(aw[t]) + bias.y) * kLog2e);
      gx[t] = x;
      gy[t] = y;
    }
  }
  const float totx = gx[kB - 1], toty = gy[kB - 1];
  if (mine) {
    *reinterpret_cast<float2*>(e2 + wave * DP + c0) = make_float2(__builtin_amdgcn_exp2f(totx), __builtin_amdgcn_exp2f(toty));
    *reinterpret_cast<float2*>(inv2 + wave * DP + c0) = make_float2(__builtin_amdgcn_exp2f(-totx), __builtin_amdgcn_exp2f(-toty));
  }
  float* ke_b = ke + brow * kES;                                 // this block's rows
  bf16_t* kph_b = kph + brow * kKS;
  bf16_t* kpl_b = kpl + brow * kKS;
  const bool steep = __any(in && fminf(totx, toty) < -kMaxFall);
  floatx4_t dk = {0.f, 0.f, 0.f, 0.f}, dq = {0.f, 0.f, 0.f, 0.f};    // a steep diagonal block's sums: row 4 g4 + e, column l15
  if (steep) {
#pragma unroll
    for (int t = 0; t < kB; ++t) {                               // log-decays and the plain vectors, where products with them will be
      if (!mine) continue;
      *reinterpret_cast<float2*>(ke_b + t * kES + c0) = make_float2(gx[t], gy[t]);
      *reinterpret_cast<uint32_t*>(kph_b + t * kKS + c0) = kw[t];
      *reinterpret_cast<uint32_t*>(kpl_b + t * kKS + c0) = qw[t];
    }
    wave_fence();
    steep_block<DP>(ke_b, kph_b, kpl_b, dk, dq);
    const float ks = __shfl(kinv, 4 * l15);
#pragma unroll
    for (int e = 0; e < 4; ++e) {
      dk[e] *= ks * __shfl(kinv, 4 * (4 * g4 + e));
      dq[e] *= ks * __shfl(qinv, 4 * (4 * g4 + e));
    }
    wave_fence();
  }
  bf16x8_t qf[kN];                                               // 2^(G - block start) q, row l15, channels 32 i + 8 g4 + 0..7
  {
    bf16_t* qs = reinterpret_cast<bf16_t*>(ke_b);                // through the block's rows of `ke`, before those are written
#pragma unroll
    for (int t = 0; t < kB; ++t) {
      const float qi = lane_value(qinv, 4 * t);
      const float px = __builtin_amdgcn_exp2f(gx[t]), py = __builtin_amdgcn_exp2f(gy[t]);
      if (mine) *reinterpret_cast<uint32_t*>(qs + t * kKS + c0) = pack_bf16x2(bf16lo(qw[t]) * qi * px, bf16hi(qw[t]) * qi * py);
      const float ki = lane_value(kinv, 4 * t), x = bf16lo(kw[t]) * ki, y = bf16hi(kw[t]) * ki;
      const uint32_t hi = pack_bf16x2(x * px, y * py);
      if (!mine) continue;
      *reinterpret_cast<uint32_t*>(kph_b + t * kKS + c0) = hi;
      *reinterpret_cast<uint32_t*>(kpl_b + t * kKS + c0) = pack_bf16x2(x * px - bf16lo(hi), y * py - bf16hi(hi));
    }
    wave_fence();
#pragma unroll
    for (int i = 0; i < kN; ++i) qf[i] = *reinterpret_cast<const bf16x8_t*>(qs + l15 * kKS + 32 * i + 8 * g4);
    wave_fence();
#pragma unroll
    for (int t = 0; t < kB; ++t) {
      const float ki = lane_value(kinv, 4 * t);
      if (mine)
        *reinterpret_cast<float2*>(ke_b + t * kES + c0) =
            make_float2(bf16lo(kw[t]) * ki * __builtin_amdgcn_exp2f(totx - gx[t]), bf16hi(kw[t]) * ki * __builtin_amdgcn_exp2f(toty - gy[t]));
    }
  }
  // the first values are on their way meanwhile
  const bf16_t* vp = qkv + 2LL * a.G * a.D + (int64_t)head * a.E;
  u32x4_t vw[kC * kVB / 8 / 256];
  auto fetch_v = [&](int e0) {
    const __amdgpu_buffer_rsrc_t rs_v = rows_rsrc(vp + e0, rows, a.qkv_stride, a.E - e0);
#pragma unroll
    for (int i = 0; i < kC * kVB / 8 / 256; ++i) {
      const int at = tid + 256 * i, col = at % (kVB / 8) * 8;
      vw[i] = __builtin_amdgcn_raw_buffer_load_b128(rs_v, e0 + col < a.E ? at / (kVB / 8) * row_bytes + col * 2 : kOutside, 0, 0);
    }
  };
  fetch_v(0);
  __syncthreads();

  // ---- scores of this block's rows with the columns of blocks 0 .. wave
  floatx4_t ak[4], aq[4];
  {
    bf16x8_t kh[kN], kl[kN];
    float f[kN][8];                                              // decay from the column block's end to the row block's start
#pragma unroll
    for (int i = 0; i < kN; ++i) {
      const int at = l15 * kKS + 32 * i + 8 * g4;
      kh[i] = *reinterpret_cast<const bf16x8_t*>(kph_b + at);
      kl[i] = *reinterpret_cast<const bf16x8_t*>(kpl_b + at);
#pragma unroll
      for (int e = 0; e < 8; ++e) f[i][e] = 1.f;
    }
#pragma unroll
    for (int j = 3; j >= 0; --j) {
      ak[j] = floatx4_t{0.f, 0.f, 0.f, 0.f};
      aq[j] = floatx4_t{0.f, 0.f, 0.f, 0.f};
      if (j > wave) continue;
      const bool diag = j == wave;
      if (diag && steep) {
        ak[j] = dk;
        aq[j] = dq;
        continue;
      }
#pragma unroll
      for (int i = 0; i < kN; ++i) {
        const int d = 32 * i + 8 * g4;
        float x[8], w[8];
        load_vec<float, 8>(ke + (kB * j + l15) * kES + d, x);
        if (diag) {
          load_vec<float, 8>(inv2 + j * DP + d, w);
#pragma unroll
          for (int e = 0; e < 8; ++e) x[e] *= w[e];
        } else {
          if (j + 1 < wave) {
            load_vec<float, 8>(e2 + (j + 1) * DP + d, w);
#pragma unroll
            for (int e = 0; e < 8; ++e) f[i][e] *= w[e];
          }
#pragma unroll
          for (int e = 0; e < 8; ++e) x[e] *= f[i][e];
        }
        bf16x8_t hi, low;
        split8(x, hi, low);
        ak[j] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(kh[i], hi, ak[j], 0, 0, 0);
        aq[j] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(qf[i], hi, aq[j], 0, 0, 0);
        ak[j] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(kh[i], low, ak[j], 0, 0, 0);
        aq[j] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(qf[i], low, aq[j], 0, 0, 0);
        ak[j] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(kl[i], hi, ak[j], 0, 0, 0);
      }
    }
  }
  // ---- 2^G q of this block's rows: a lane's eight channels are half a slot of two quarters
#pragma unroll
  for (int i = 0; i < kN; ++i) {
    const int d = 32 * i + 8 * g4;
    const u32x4_t qv = as_u32(qf[i]);
    float x[8] = {bf16lo(qv[0]), bf16hi(qv[0]), bf16lo(qv[1]), bf16hi(qv[1]), bf16lo(qv[2]), bf16hi(qv[2]), bf16lo(qv[3]), bf16hi(qv[3])};
    for (int j = 0; j < wave; ++j) {
      float w[8];
      load_vec<float, 8>(e2 + j * DP + d, w);
#pragma unroll
      for (int e = 0; e < 8; ++e) x[e] *= w[e];
    }
    char* dst = unit + Layout<DP>::q + (wave * kN + i) * 1024 + (l15 + 32 * (g4 & 1)) * 16 + (g4 >> 1) * 8;
    *reinterpret_cast<uint2*>(dst) = make_uint2(pack_bf16x2(x[0], x[1]), pack_bf16x2(x[2], x[3]));
    *reinterpret_cast<uint2*>(dst + 256) = make_uint2(pack_bf16x2(x[4], x[5]), pack_bf16x2(x[6], x[7]));
  }
  // ---- 2^(G_end - G) k: more of it for the wavefronts with fewer score blocks
#pragma unroll
  for (int f = 0; f < DP / 8; ++f) {
    const int share = f * 16 / (DP / 8), owner = share < 8 ? 0 : share < 13 ? 1 : 2;
    if (owner != wave) continue;
    const int kk = f % 2, d = 16 * (f / 2) + l15;               // tokens of blocks 2 kk and 2 kk + 1
    float post[2] = {1.f, 1.f};
    if (kk == 0) post[1] = e2[2 * DP + d] * e2[3 * DP + d];
    post[0] = post[1] * e2[(2 * kk + 1) * DP + d];
    float x[8];
#pragma unroll
    for (int e = 0; e < 8; ++e) x[e] = ke[(32 * kk + 4 * g4 + (e & 3) + 16 * (e >> 2)) * kES + d] * post[e >> 2];
    bf16x8_t hi, low;
    split8(x, hi, low);
    u32x4_t* dst = reinterpret_cast<u32x4_t*>(unit + Layout<DP>::k + f * 2048) + lane;
    dst[0] = as_u32(hi);
    dst[64] = as_u32(low);
  }
  if (tid < DP) {
    float p = 1.f;
#pragma unroll
    for (int j = 0; j < 4; ++j) {
      pre[j * DP + tid] = p;
      p *= e2[j * DP + tid];
    }
    reinterpret_cast<float*>(unit + Layout<DP>::gamma)[tid] = p;
  }
  __syncthreads();                                               // `ke` is free

  // ---- L and A; the inverses of L's diagonal blocks
#pragma unroll
  for (int j = 0; j < 4; ++j) {
    const bool upper = j > wave;
    if (upper && j != (wave | 1)) continue;                      // (the zero block that shares a 32-token tile with a diagonal one)
#pragma unroll
    for (int e = 0; e < 4; ++e) {
      const int t = brow + 4 * g4 + e, col = kB * j + l15;
      if (!upper) lt[t * kLS + col] = col < t ? beta[t] * ak[j][e] : 0.f;
      as[t * kTS + col] = col <= t ? f32_to_bf16(aq[j][e]) : 0;
    }
  }
  wave_fence();
  {
    float x[kB];                                                 // column l15 of the inverse, every row
    const float* lb = lt + brow * kLS + brow;
#pragma unroll
    for (int r = 0; r < kB; ++r) {
      float v = r == l15 ? 1.f : 0.f;
#pragma unroll
      for (int k = 0; k < r; k += 4) {
        const floatx4_t l = *reinterpret_cast<const floatx4_t*>(lb + r * kLS + k);
#pragma unroll
        for (int e = 0; e < 4; ++e)
          if (k + e < r) v -= l[e] * x[k + e];
      }
      x[r] = v;
    }
    wave_fence();
#pragma unroll
    for (int r = 0; r < kB; ++r)
      if (g4 == (r >> 2)) lt[(brow + r) * kLS + brow + l15] = x[r];
  }
  __syncthreads();

  // ---- T below the diagonal, a column of blocks per wavefront, in accumulators: rows 4 g4 + e of block i, column l15
  floatx4_t tj[4];
  {
    auto block = [&](int i, int k) { return *reinterpret_cast<const floatx4_t*>(lt + (kB * i + l15) * kLS + kB * k + 4 * g4); };
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      tj[i] = floatx4_t{0.f, 0.f, 0.f, 0.f};
      if (i < wave) continue;
      if (i == wave) {
#pragma unroll
        for (int e = 0; e < 4; ++e) tj[i][e] = lt[(brow + 4 * g4 + e) * kLS + brow + l15];
        continue;
      }
      floatx4_t x = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int k = 0; k < 3; ++k) {
        if (k < wave || k >= i) continue;
        const floatx4_t l = block(i, k);
#pragma unroll
        for (int e = 0; e < 4; ++e) x = __builtin_amdgcn_mfma_f32_16x16x4f32(l[e], tj[k][e], x, 0, 0, 0);
      }
      const floatx4_t d = block(i, i);
#pragma unroll
      for (int e = 0; e < 4; ++e) tj[i] = __builtin_amdgcn_mfma_f32_16x16x4f32(-d[e], x[e], tj[i], 0, 0, 0);
    }
  }
#pragma unroll
  for (int f = 0; f < 6; ++f) {                                  // A's fragments
    if ((f & 3) != wave) continue;
    const int tile = f < 2 ? f : f / 2 + 1, kk = f < 2 ? 0 : f & 1;
    const bf16_t* src = as + (16 * tile + l15) * kTS + 32 * kk + 4 * g4;
    const uint2 x = *reinterpret_cast<const uint2*>(src), y = *reinterpret_cast<const uint2*>(src + 16);
    reinterpret_cast<uint4*>(unit + Layout<DP>::a + f * 1024)[lane] = make_uint4(x.x, x.y, y.x, y.y);
  }
  __syncthreads();                                               // L and A are free
  {
    const float bt = beta[brow + l15];
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      if (i < wave && i != (wave ^ 1)) continue;                 // (of the zero blocks, the one in a diagonal block's tile)
#pragma unroll
      for (int e = 0; e < 4; ++e) {
        const float v = tj[i][e] * bt;
        const bf16_t hi = f32_to_bf16(v);
        th[(kB * i + 4 * g4 + e) * kTS + brow + l15] = hi;
        tl[(kB * i + 4 * g4 + e) * kTS + brow + l15] = f32_to_bf16(v - bf16_to_f32(hi));
      }
    }
  }
  const int half = lane >> 5, l32 = lane & 31, tr_row = 8 * half + (l15 >> 2), tr_col = (lane & 16) + (l15 & 3) * 4;
  for (int e0 = 0; e0 < a.E; e0 += kVB) {
    if (e0 > 0) __syncthreads();                                 // the last reads of the values before
#pragma unroll
    for (int i = 0; i < kC * kVB / 8 / 256; ++i) {
      const int at = tid + 256 * i;
      *reinterpret_cast<u32x4_t*>(vs + at / (kVB / 8) * kVS + at % (kVB / 8) * 8) = vw[i];
    }
    __syncthreads();
    if (e0 + kVB < a.E) fetch_v(e0 + kVB);
    // U' = T diag(beta) V: (32 columns, row tile) per turn
    const int tiles = (min(kVB, a.E - e0) + 31) / 32;
    for (int task = wave; task < 2 * tiles; task += 4) {
      const int n0 = task / 2 * 32, tile = task & 1;
      floatx16_t acc = zero16();
#pragma unroll
      for (int j = 0; j < 4; ++j) {
        if (j >= 2 + 2 * tile) continue;
        const int at = (32 * tile + l32) * kTS + 16 * j + 8 * half;
        const bf16x8_t v = read_tr8(vs + (16 * j + tr_row) * kVS + n0 + tr_col, 4 * kVS);
        acc = __builtin_amdgcn_mfma_f32_32x32x16_bf16(*reinterpret_cast<const bf16x8_t*>(th + at), v, acc, 0, 0, 0);
        acc = __builtin_amdgcn_mfma_f32_32x32x16_bf16(*reinterpret_cast<const bf16x8_t*>(tl + at), v, acc, 0, 0, 0);
      }
      // rows 8 x + 4 half + 0..3 of column l32: quarter 2 (x % 2) + half of row tile 2 tile + x / 2
      floatx4_t* dst = reinterpret_cast<floatx4_t*>(unit + Layout<DP>::u + (((e0 + n0) / 16 + (l32 >> 4)) * 4 + 2 * tile) * 1024) + l15 + 16 * half;
#pragma unroll
      for (int x = 0; x < 4; ++x) dst[64 * (x >> 1) + 32 * (x & 1)] = floatx4_t{acc[4 * x], acc[4 * x + 1], acc[4 * x + 2], acc[4 * x + 3]};
    }
  }
  // -W^T = -(2^G K)^T diag(beta) T^T, whose accumulators are -W's fragments: (32 channels, token tile) per turn
#pragma unroll 1
  for (int task = wave; task < 2 * kN; task += 4) {
    const int d0 = task / 2 * 32, tile = task & 1;
    floatx16_t acc = zero16();
#pragma unroll
    for (int j = 0; j < 4; ++j) {
      if (j >= 2 + 2 * tile) continue;
      const int at = (32 * tile + l32) * kTS + 16 * j + 8 * half, kt = (16 * j + tr_row) * kKS + d0 + tr_col;
      const bf16x8_t h = *reinterpret_cast<const bf16x8_t*>(th + at), l = *reinterpret_cast<const bf16x8_t*>(tl + at);
      const bf16x8_t xh = read_tr8(kph + kt, 4 * kKS), xl = read_tr8(kpl + kt, 4 * kKS);
      floatx16_t p = zero16();
      p = __builtin_amdgcn_mfma_f32_32x32x16_bf16(xh, h, p, 0, 0, 0);
      p = __builtin_amdgcn_mfma_f32_32x32x16_bf16(xh, l, p, 0, 0, 0);
      p = __builtin_amdgcn_mfma_f32_32x32x16_bf16(xl, h, p, 0, 0, 0);
#pragma unroll
      for (int x = 0; x < 4; ++x) {
        const float4 w = *reinterpret_cast<const float4*>(pre + j * DP + d0 + 8 * x + 4 * half);
        acc[4 * x] += w.x * p[4 * x];
        acc[4 * x + 1] += w.y * p[4 * x + 1];
        acc[4 * x + 2] += w.z * p[4 * x + 2];
        acc[4 * x + 3] += w.w * p[4 * x + 3];
      }
    }
#pragma unroll
    for (int i = 0; i < 2; ++i) {
      // channels 8 i + 4 half + 0..3 and 16 behind them: quarter 2 i + half
      const float x[8] = {-acc[4 * i], -acc[4 * i + 1], -acc[4 * i + 2], -acc[4 * i + 3], -acc[4 * i + 8], -acc[4 * i + 9], -acc[4 * i + 10], -acc[4 * i + 11]};
      bf16x8_t hi, low;
      split8(x, hi, low);
      u32x4_t* dst = reinterpret_cast<u32x4_t*>(unit + Layout<DP>::w + ((2 * tile + (l32 >> 4)) * kN + d0 / 32) * 2048) + l15 + 16 * (2 * i + half);
      dst[0] = as_u32(hi);
      dst[64] = as_u32(low);
    }
  }
}

// A workgroup takes CT tiles of 16 value columns.  Wavefronts 0 and 1 make U of 32 tokens each, wavefronts 2 and 3 the outputs, and
// wavefront w < DP / 32 owns 32 state rows, whose fragments all of them read.  Two barriers a chunk: S -> U, U -> S; the outputs'
// part with U follows beside the next chunk's first half.  A chunk's operands are requested as soon as the registers of the chunk
// before are free.  The two kinds run code of their own (with the same barriers), in which no load is conditional (what lies outside
// a buffer reads as zero), so that the waits are counted.
template <int DP, int CT>
struct StateWalk {
  static constexpr int kN = DP / 32;
  struct Shared {
    u32x4_t s[kN][CT][2][64];    // fragments of S, high and low
    u32x4_t u[2][2][CT][2][64];  // of U, for even and odd chunks
  };
  template <bool kMakesU>
  struct Ops {
    u32x4_t p[2][kN][kMakesU ? 2 : 1];  // two row tiles of -W (high, low) or of 2^G q
    u32x4_t k[2][2][2];                 // two row tiles of (2^(G_end - G) k)^T
    u32x4_t a[kMakesU ? 1 : 4];         // two row tiles of A
    floatx4_t u[kMakesU ? CT : 1][2];   // of U'
    floatx4_t gamma[2];
  };
  struct Tiles { floatx4_t t[CT][2]; };

  // accumulator tiles as a fragment per column tile
  static __device__ __forceinline__ void share(const Tiles& v, u32x4_t (*to)[2][64], int lane) {
#pragma unroll
    for (int c = 0; c < CT; ++c) {
      const float x[8] = {v.t[c][0][0], v.t[c][0][1], v.t[c][0][2], v.t[c][0][3], v.t[c][1][0], v.t[c][1][1], v.t[c][1][2], v.t[c][1][3]};
      bf16x8_t hi, low;
      split8(x, hi, low);
      to[c][0][lane] = as_u32(hi);
      to[c][1][lane] = as_u32(low);
    }
  }
  static __device__ __forceinline__ floatx4_t mul(u32x4_t a, u32x4_t b, floatx4_t c) {
    return __builtin_amdgcn_mfma_f32_16x16x32_bf16(as_bf16(a), as_bf16(b), c, 0, 0, 0);
  }
  static __device__ __forceinline__ u32x4_t load(__amdgpu_buffer_rsrc_t rs, int at) { return __builtin_amdgcn_raw_buffer_load_b128(rs, at, 0, 0); }

  template <bool kMakesU>
  static __device__ __forceinline__ void run(const ChunkArgs& c, const msa_seq_batch& b, Shared& sh, int wave, int head, int tile0, int s) {
    const msa_delta_args& a = c.d;
    const int lane = threadIdx.x & 63, l15 = lane & 15, g4 = lane >> 4, pair = wave & 1;
    const int lo = b.cu[s], n_tok = b.cu[s + 1] - lo - c.first * kC;
    const int n = min(c.seg, (n_tok + kC - 1) / kC);
    const int col = tile0 * 16 + l15, d0 = 32 * wave + 4 * g4, row_elems = a.H * a.E;
    const bool own = DP == 128 || wave < DP / 32;
    const char* units = c.ws + ((int64_t)s * a.H + head) * c.seg * c.unit;

    Tiles S;                                                     // rows d0 + 16 t + 0..3, column col + 16 i
    float* st = a.state + (((int64_t)b.slot[s] * a.H + head) * a.D + d0) * a.E + col;
#pragma unroll
    for (int i = 0; i < CT; ++i)
#pragma unroll
      for (int e = 0; e < 8; ++e) {
        const int r = 16 * (e >> 2) + (e & 3);
        S.t[i][e >> 2][e & 3] = own && col + 16 * i < a.E && d0 + r < a.D ? st[(int64_t)r * a.E + 16 * i] : 0.f;
      }
    const int p_at = (kMakesU ? Layout<DP>::w + pair * 2 * kN * 2048 : Layout<DP>::q + pair * 2 * kN * 1024) + lane * 16;
    const int u_at = Layout<DP>::u + (tile0 * 4 + 2 * pair) * 1024 + lane * 16, a_at = Layout<DP>::a + pair * 2048 + lane * 16;
    const int k_at = own ? Layout<DP>::k + wave * 8192 + lane * 16 : kOutside, g_at = own ? Layout<DP>::gamma + d0 * 4 : kOutside;
    using O = Ops<kMakesU>;
    auto chunk_rsrc = [&](int i) {
      return __builtin_amdgcn_make_buffer_rsrc(const_cast<char*>(units + (int64_t)max(0, min(i, n - 1)) * c.unit), 0, (int)c.unit, 0x00020000);
    };
    auto load_p = [&](O& o, int i) {
      const __amdgpu_buffer_rsrc_t rs = chunk_rsrc(i);
      constexpr int kParts = kMakesU ? 2 : 1;
#pragma unroll
      for (int f = 0; f < 2 * kN * kParts; ++f) o.p[f / (kN * kParts)][f / kParts % kN][f % kParts] = load(rs, p_at + 1024 * f);
      __builtin_amdgcn_sched_barrier(0);
    };
    auto load_x = [&](O& o, int i) {
      const __amdgpu_buffer_rsrc_t rs = chunk_rsrc(i);
      if constexpr (kMakesU) {
#pragma unroll
        for (int f = 0; f < 2 * CT; ++f) o.u[f / 2][f % 2] = __builtin_bit_cast(floatx4_t, load(rs, u_at + 4096 * (f / 2) + 1024 * (f % 2)));
      } else {                                                   // (of the first four two are tiles 0 and 1)
#pragma unroll
        for (int f = 0; f < 4; ++f) o.a[f] = load(rs, a_at + 1024 * f);
      }
      __builtin_amdgcn_sched_barrier(0);
    };
    auto load_k = [&](O& o, int i) {
      const __amdgpu_buffer_rsrc_t rs = chunk_rsrc(i);
#pragma unroll
      for (int f = 0; f < 8; ++f) o.k[f / 4][f / 2 % 2][f % 2] = load(rs, k_at + 1024 * f);
#pragma unroll
      for (int t = 0; t < 2; ++t) o.gamma[t] = __builtin_bit_cast(floatx4_t, load(rs, g_at + 64 * t));
      __builtin_amdgcn_sched_barrier(0);
    };
    const floatx4_t none = {0.f, 0.f, 0.f, 0.f};
    Tiles out;                                                   // 2^G q S of the chunk before
#pragma unroll
    for (int i = 0; i < CT; ++i) out.t[i][0] = out.t[i][1] = none;
    // its stores: tokens 32 pair + 16 t + 4 g4 + 0..3 (what lies outside is not written)
    auto store = [&](int i) {
      const __amdgpu_buffer_rsrc_t rs = rows_rsrc(static_cast<bf16_t*>(a.out) + ((int64_t)(lo + (c.first + i) * kC) * a.H + head) * a.E,
                                                  i < 0 ? 0 : min(kC, n_tok - i * kC), row_elems, a.E);
#pragma unroll
      for (int j = 0; j < CT; ++j) {
        const int at = col + 16 * j < a.E ? ((32 * pair + 4 * g4) * row_elems + col + 16 * j) * 2 : kOutside;
#pragma unroll
        for (int e = 0; e < 8; ++e)
          __builtin_amdgcn_raw_buffer_store_b16(f32_to_bf16(out.t[j][e >> 2][e & 3]), rs, at + (16 * (e >> 2) + (e & 3)) * row_elems * 2, 0, 0);
      }
    };
    // its part with U
    auto finish = [&](O& o, int i) {
#pragma unroll
      for (int kk = 0; kk < 2; ++kk) {
        if (kk > pair) continue;
#pragma unroll
        for (int h = 0; h < 2; ++h)
#pragma unroll
          for (int j = 0; j < CT; ++j)
#pragma unroll
            for (int t = 0; t < 2; ++t) out.t[j][t] = mul(pair ? o.a[2 * t + kk] : o.a[t], sh.u[i & 1][kk][j][h][lane], out.t[j][t]);
      }
      load_x(o, i + 1);
      store(i);
    };
    auto step = [&](O& o, int i) {
      __syncthreads();
      u32x4_t f[kN][CT][2];
#pragma unroll
      for (int kk = 0; kk < kN; ++kk)
#pragma unroll
        for (int j = 0; j < CT; ++j)
#pragma unroll
          for (int h = 0; h < 2; ++h) f[kk][j][h] = sh.s[kk][j][h][lane];
      __builtin_amdgcn_sched_barrier(0);
      if constexpr (kMakesU) {
        Tiles u;
#pragma unroll
        for (int j = 0; j < CT; ++j)
#pragma unroll
          for (int t = 0; t < 2; ++t) u.t[j][t] = o.u[j][t];
#pragma unroll
        for (int kk = 0; kk < kN; ++kk)
#pragma unroll
          for (int x = 0; x < 3; ++x)                            // high x high, high x low, low x high
#pragma unroll
            for (int j = 0; j < CT; ++j)
#pragma unroll
              for (int t = 0; t < 2; ++t) u.t[j][t] = mul(o.p[t][kk][x >> 1], f[kk][j][x & 1], u.t[j][t]);
        share(u, sh.u[i & 1][pair], lane);
        load_x(o, i + 1);
      } else {
        finish(o, i - 1);                                   // (in front of the first chunk: nothing is written)
#pragma unroll
        for (int j = 0; j < CT; ++j) out.t[j][0] = out.t[j][1] = none;
#pragma unroll
        for (int kk = 0; kk < kN; ++kk)
#pragma unroll
          for (int h = 0; h < 2; ++h)
#pragma unroll
            for (int j = 0; j < CT; ++j)
#pragma unroll
              for (int t = 0; t < 2; ++t) out.t[j][t] = mul(o.p[t][kk][0], f[kk][j][h], out.t[j][t]);
      }
      load_p(o, i + 1);
      __syncthreads();
      if (own) {
        u32x4_t g[2][CT][2];
#pragma unroll
        for (int kk = 0; kk < 2; ++kk)
#pragma unroll
          for (int j = 0; j < CT; ++j)
#pragma unroll
            for (int h = 0; h < 2; ++h) g[kk][j][h] = sh.u[i & 1][kk][j][h][lane];
#pragma unroll
        for (int j = 0; j < CT; ++j)
#pragma unroll
          for (int t = 0; t < 2; ++t) S.t[j][t] *= o.gamma[t];
        __builtin_amdgcn_sched_barrier(0);
#pragma unroll
        for (int kk = 0; kk < 2; ++kk)
#pragma unroll
          for (int x = 0; x < 3; ++x)
#pragma unroll
            for (int j = 0; j < CT; ++j)
#pragma unroll
              for (int t = 0; t < 2; ++t) S.t[j][t] = mul(o.k[t][kk][x >> 1], g[kk][j][x & 1], S.t[j][t]);
        share(S, sh.s[wave], lane);
      }
      load_k(o, i + 1);
    };
    O o;
    load_x(o, 0);                // (in the order the loop makes them, stores included, so that the first pass counts like the others)
    if constexpr (!kMakesU) store(-1);
    load_p(o, 0);
    load_k(o, 0);
    if (own) share(S, sh.s[wave], lane);
    for (int i = 0; i < n; ++i) step(o, i);
    if constexpr (!kMakesU) finish(o, n - 1);
    if (!own) return;
#pragma unroll
    for (int i = 0; i < CT; ++i)
#pragma unroll
      for (int e = 0; e < 8; ++e) {
        const int r = 16 * (e >> 2) + (e & 3);
        if (col + 16 * i < a.E && d0 + r < a.D) st[(int64_t)r * a.E + 16 * i] = S.t[i][e >> 2][e & 3];
      }
  }
};

// Workgroups 0 .. n_walk - 1 walk over the chunks of `walk`, the others prepare those of `prep`.  Either part's workgroups of a head
// follow one another at a distance of H, so that with a multiple of eight heads they share an L2.
template <int DP, int CT>
__global__ __launch_bounds__(256, 2) void delta_chunk_kernel(ChunkArgs walk, ChunkArgs prep, int32_t n_walk, int32_t n_prep, msa_seq_batch b) {
  extern __shared__ __align__(16) char lds[];
  static_assert(sizeof(typename StateWalk<DP, CT>::Shared) <= prepare_lds<DP>(), "either part's tiles");
  const int H = walk.d.H;
  if ((int)blockIdx.x < n_walk) {
    const int head = blockIdx.x % H, rest = blockIdx.x / H, tiles = ((walk.d.E + 15) / 16 + CT - 1) / CT, s = rest / tiles;
    if (b.cu[s + 1] - b.cu[s] <= walk.first * kC) return;
    auto& sh = *reinterpret_cast<typename StateWalk<DP, CT>::Shared*>(lds);
    const int wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6);
    if (wave < 2) StateWalk<DP, CT>::template run<true>(walk, b, sh, wave, head, rest % tiles * CT, s);
    else StateWalk<DP, CT>::template run<false>(walk, b, sh, wave, head, rest % tiles * CT, s);
  } else {
    const int id = blockIdx.x - n_walk, head = id % H, rest = id / H;
    prepare_chunk<DP>(prep, b, lds, head, rest % n_prep, rest / n_prep);
  }
}

constexpr int64_t kMaxSegment = (int64_t)88 << 20;        // bytes: two segments stay in the memory-side cache
constexpr int kSegments = 6, kLeastChunks = 22;           // segments of a long portion, chunks that are worth a launch

int64_t unit_bytes(int32_t D, int32_t E) {
  switch ((D + 31) / 32) {
    case 1: return Layout<32>::bytes(E);
    case 2: return Layout<64>::bytes(E);
    case 3: return Layout<96>::bytes(E);
    default: return Layout<128>::bytes(E);
  }
}
// Chunks of a segment: enough to be worth a launch, few enough to overlap, at most what the workspace holds.
int segment(const msa_delta_args& a, int32_t max_rows, int32_t n_seq) {
  const int64_t chunks = (max_rows + kC - 1) / kC, per = unit_bytes(a.D, a.E) * a.H * n_seq;
  const int64_t most = std::max<int64_t>(1, kMaxSegment / per), want = std::max<int64_t>(kLeastChunks, (chunks + kSegments - 1) / kSegments);
  const int64_t parts = (chunks + std::min(most, want) - 1) / std::min(most, want);
  return (int)((chunks + parts - 1) / parts);
}

template <int DP, int CT>
int launch_chunked(const ChunkArgs& c, const msa_seq_batch& b, hipStream_t st) {
  constexpr int lds = prepare_lds<DP>();
  static_assert(lds <= 80 * 1024, "two workgroups per compute unit");
  static std::atomic<int> raised{0};
  MSA_HIP(raise_dynamic_lds_limit(raised, reinterpret_cast<const void*>(delta_chunk_kernel<DP, CT>), lds));
  const int chunks = (b.max_rows + kC - 1) / kC, parts = (chunks + c.seg - 1) / c.seg;
  const int walks = c.d.H * (((c.d.E + 15) / 16 + CT - 1) / CT) * b.n_seq;
  const int64_t half = c.unit * c.d.H * c.seg * b.n_seq;
  for (int part = 0; part <= parts; ++part) {
    ChunkArgs walk = c, prep = c;
    walk.first = (part - 1) * c.seg;
    walk.ws = c.ws + ((part + 1) & 1) * half;
    prep.first = part * c.seg;
    prep.ws = c.ws + (part & 1) * half;
    const int n_walk = part > 0 ? walks : 0, n_prep = part < parts ? std::min(c.seg, chunks - prep.first) : 0;
    delta_chunk_kernel<DP, CT><<<n_walk + c.d.H * n_prep * b.n_seq, 256, lds, st>>>(walk, prep, n_walk, n_prep, b);
    MSA_LAUNCH_CHECK();
  }
  return MSA_OK;
}
template <int DP>
int launch_chunked(const ChunkArgs& c, const msa_seq_batch& b, hipStream_t st) {
  // narrow column tiles as long as they find compute units
  if ((int64_t)c.d.H * ((c.d.E + 15) / 16) * b.n_seq <= device_compute_units()) return launch_chunked<DP, 1>(c, b, st);
  return launch_chunked<DP, 2>(c, b, st);
}

}  // namespace

extern "C" size_t msa_seq_delta_chunked_workspace_bytes(const msa_delta_args* args, int32_t max_rows, int32_t n_seq) {
  if (!args || max_rows <= 0 || n_seq <= 0 || args->H <= 0 || args->D <= 0 || args->D > 128 || args->E <= 0) return 0;
  const int chunks = (max_rows + kC - 1) / kC, seg = segment(*args, max_rows, n_seq);
  return (size_t)unit_bytes(args->D, args->E) * args->H * n_seq * seg * (seg < chunks ? 2 : 1);
}

extern "C" int msa_seq_delta_chunked(const msa_delta_args* args, const msa_seq_batch* batch, void* workspace, size_t workspace_bytes, void* stream) {
  MSA_CHECK_BATCH(batch, "msa_seq_delta_chunked");
  MSA_REQUIRE(args && args->qkv && args->a && args->b && args->gate && args->A_log && args->dt_bias && args->norm && args->state && args->out && workspace,
              "msa_seq_delta_chunked: null pointer");
  const msa_delta_args& a = *args;
  MSA_REQUIRE(a.H > 0 && a.H <= 65535 && a.G > 0 && a.H % a.G == 0 && a.D > 0 && a.D % 8 == 0 && a.D <= 128 && a.E > 0 && a.E % 8 == 0 && batch->n_seq <= 65535,
              "msa_seq_delta_chunked: H=%d G=%d D=%d (a multiple of 8 up to 128) E=%d (a multiple of 8)", a.H, a.G, a.D, a.E);
  MSA_REQUIRE(a.qkv_stride >= 2LL * a.G * a.D + (int64_t)a.H * a.E && a.a_stride >= (int64_t)a.H * a.D && a.b_stride >= a.H &&
                  a.gate_stride >= (int64_t)a.H * a.E && a.qkv_stride % 8 == 0 && a.a_stride % 2 == 0 && a.qkv_stride < (1 << 21) && a.a_stride < (1 << 21) &&
                  (int64_t)a.H * a.E < (1 << 21) && (((uintptr_t)a.qkv | (uintptr_t)workspace) & 15) == 0 && ((uintptr_t)a.a & 3) == 0 && ((uintptr_t)a.dt_bias & 7) == 0,
              "msa_seq_delta_chunked: strides or alignment");
  if (workspace_bytes < msa_seq_delta_chunked_workspace_bytes(args, batch->max_rows, batch->n_seq)) {
    msa_set_error("msa_seq_delta_chunked: workspace of %zu bytes is too small", workspace_bytes);
    return MSA_ESIZE;
  }
  const ChunkArgs c{a, static_cast<char*>(workspace), unit_bytes(a.D, a.E), 0, segment(a, batch->max_rows, batch->n_seq)};
  MSA_REQUIRE((int64_t)a.H * batch->n_seq * std::max<int64_t>(2 * c.seg, (a.E + 15) / 8) < ((int64_t)1 << 30), "msa_seq_delta_chunked: step too large");
  hipStream_t st = as_stream(stream);
  const int tiles = (a.D + 31) / 32;
  const int rc = tiles == 1   ? launch_chunked<32>(c, *batch, st)
                 : tiles == 2 ? launch_chunked<64>(c, *batch, st)
                 : tiles == 3 ? launch_chunked<96>(c, *batch, st)
                              : launch_chunked<128>(c, *batch, st);
  if (rc != MSA_OK) return rc;
  return msa_seq_head_norm_gate(a.out, a.gate, a.gate_stride, a.norm, a.eps, MSA_BF16, batch->rows, a.H, a.E, stream);
}
