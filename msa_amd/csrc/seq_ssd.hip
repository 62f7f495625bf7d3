// Chunked form of the state-space recurrence on the matrix cores (bf16 inputs, fp32 states and decays), for portions long
// enough to be worth cutting into chunks of Q tokens (Q = 128, or 64 when the state has more than 128 rows).  With
// a_t = sum of the chunk's log-decays up to t, inside a chunk
//   y_t = exp(a_t) S_in^T C_t + sum_{s <= t} exp(a_t - a_s) dt_s (B_s . C_t) x_s,   S_out = exp(a_end) S_in + S_loc,
//   S_loc = sum_s exp(a_end - a_s) dt_s B_s x_s^T.
//   (1) ssd_decay_kernel   dt and a_t of every token and head
//   (2) ssd_local_kernel   every chunk's S_loc
//   (3) ssd_carry_kernel   the chunk-to-chunk recurrence, element by element; leaves each chunk's S_in in its place
//   (4) ssd_output_kernel  the outputs
// A workgroup of (2) and (4) takes one chunk and several heads of one group, whose B, C and B . C^T are the same: those are read /
// formed once and stay in registers; a head's x and S_in are fetched while the head before is multiplied.  (Walking over the chunks
// with the state in accumulators instead of (2) and (3) moves fewer bytes but is a chain of latencies: faster only with several
// hundred heads in the step, 1.7 times slower with 32.)
// Operands that carry decays or states are fp32 values: they enter the bf16 products as a high and a low part (two products
// with about 16 bits of mantissa), so only x, B and C, which are bf16 to begin with, set the precision.
//
// The score tile is taken transposed, G^T[s, t] = B . C^T, so that its accumulator layout (lane = column t) is the operand
// layout of the second product y^T[p, t] += x^T . M^T, and a_t is one scalar per lane; x^T and S_in^T come out of LDS through
// the transposing read.
#include <algorithm>

#include "seq_mfma.h"

namespace {

constexpr int kPB = 64;                  // state columns (p) per workgroup
constexpr int kXS = kPB + 8;             // LDS row stride of [.., p] tiles

struct ChunkArgs {
  const bf16_t* xbc;
  const bf16_t* z;
  const bf16_t* dt_raw;
  const float* dt_bias;
  const float* A_log;
  const float* D;
  float* state;
  bf16_t* v;
  uint32_t* chunk_state;   // [n_seq, n_chunks, H, N, P]: S_loc (fp32), then S_in as packed (high, low) bf16 pairs
  float* dts;              // [n_seq, n_chunks, H, Q]: dt, and
  float* acs;              // the running log-decay of the chunk (in powers of two)
  int64_t xbc_stride, z_stride, dt_stride;
  int32_t H, P, N, G, n_chunks, heads_per_wg;
};

constexpr int kMaxHeads = 8;             // heads of a group per workgroup

// A wavefront per (chunk, head).  Tokens behind the sequence have dt = 0.
template <int Q>
__global__ __launch_bounds__(256) void ssd_decay_kernel(ChunkArgs a, msa_seq_batch b) {
  const int lane = threadIdx.x & 63, head = blockIdx.x * 4 + (threadIdx.x >> 6), s = blockIdx.z;
  const int lo = b.cu[s], t0 = blockIdx.y * Q, rows = min(Q, b.cu[s + 1] - lo - t0);
  if (head >= a.H || rows <= 0) return;
  const float rate = -expf(a.A_log[head]) * kLog2e, bias = a.dt_bias[head];
  const int64_t at = (((int64_t)s * a.n_chunks + blockIdx.y) * a.H + head) * Q;
  float before = 0.f;
#pragma unroll
  for (int t = lane; t < Q; t += 64) {
    const float dt = t < rows ? softplus_f(bf16_to_f32(a.dt_raw[(int64_t)(lo + t0 + t) * a.dt_stride + head]) + bias) : 0.f;
    float ac = rate * dt;
#pragma unroll
    for (int o = 1; o < 64; o <<= 1) {
      const float up = __shfl_up(ac, o);
      if (lane >= o) ac += up;
    }
    ac += before;
    before = __shfl(ac, 63);
    a.dts[at + t] = dt;
    a.acs[at + t] = ac;
  }
}

// All global accesses inside the loops below go through buffer resources whose extent is the valid rows: what lies outside
// reads as zero and is not written, nothing is conditional, and the compiler can count the loads and stores in flight (behind a
// conditional one it would wait for every store of the step before).
__device__ __forceinline__ __amdgpu_buffer_rsrc_t rows_rsrc(const bf16_t* p, int rows, int64_t stride, int n) {
  return __builtin_amdgcn_make_buffer_rsrc(const_cast<bf16_t*>(p), 0, __builtin_amdgcn_readfirstlane((int)((rows - 1) * stride + n) * 2), 0x00020000);
}

// `n` columns of the chunk's rows on their way into an LDS tile of WIDTH columns (zeros behind n and behind the sequence): all
// loads of a tile are issued before anything waits for one, and several tiles' loads before the first is stored.
template <int Q, int WIDTH, int THREADS>
struct RowTile {
  static constexpr int kUnits = WIDTH / 8, kPieces = Q * kUnits / THREADS;
  static_assert(Q * kUnits % THREADS == 0, "whole pieces per thread");
  u32x4_t w[kPieces];
  // A thread's byte offsets in a chunk's rows, the same for every chunk and head.
  struct Offsets {
    int at[kPieces];
    __device__ __forceinline__ Offsets(int stride, int n) {
#pragma unroll
      for (int k = 0; k < kPieces; ++k) {
        const int i = threadIdx.x + k * THREADS, u = i % kUnits * 8, in = (i / kUnits * stride + u) * 2;
        at[k] = u < n ? in : kOutside;
      }
    }
  };
  __device__ __forceinline__ void load(const Offsets& off, const bf16_t* src, int stride, int rows, int n) {
    const __amdgpu_buffer_rsrc_t rs = rows_rsrc(src, rows, stride, n);
#pragma unroll
    for (int k = 0; k < kPieces; ++k) w[k] = __builtin_amdgcn_raw_buffer_load_b128(rs, off.at[k], 0, 0);
  }
  __device__ __forceinline__ void store(bf16_t* dst, int dst_stride) const {
#pragma unroll
    for (int k = 0; k < kPieces; ++k) {
      const int i = threadIdx.x + k * THREADS;
      *reinterpret_cast<u32x4_t*>(dst + i / kUnits * dst_stride + i % kUnits * 8) = w[k];
    }
  }
};

__device__ __forceinline__ uint32_t pack_split(float v) {
  const uint32_t hi = f32_to_bf16(v);
  return hi | ((uint32_t)f32_to_bf16(v - bf16_to_f32((bf16_t)hi)) << 16);
}

// What a workgroup of kernels (2) and (4) works on.
struct Unit {
  int head0, heads, grp, p0, lo, t0, rows, row0;
  int64_t chunk0;          // chunk index of head0
};
template <int Q>
__device__ __forceinline__ bool unit_of(const ChunkArgs& a, const msa_seq_batch& b, Unit& u) {
  const int per_group = a.H / a.G, sets = (per_group + a.heads_per_wg - 1) / a.heads_per_wg;
  const int set = blockIdx.x % sets, rest = blockIdx.x / sets, s = blockIdx.z;
  u.grp = rest % a.G;
  u.p0 = rest / a.G * kPB;
  u.head0 = u.grp * per_group + set * a.heads_per_wg;
  u.heads = min(a.heads_per_wg, per_group - set * a.heads_per_wg);
  u.lo = b.cu[s];
  u.t0 = blockIdx.y * Q;
  const int n_tok = b.cu[s + 1] - u.lo;
  u.rows = min(Q, n_tok - u.t0);
  u.row0 = u.lo + u.t0;
  u.chunk0 = ((int64_t)s * a.n_chunks + blockIdx.y) * a.H + u.head0;
  return u.t0 < n_tok;
}

template <int Q, int NP>
__global__ __launch_bounds__(4 * Q) void ssd_local_kernel(ChunkArgs a, msa_seq_batch b) {
  constexpr int kBS = NP + 8, kWaves = Q / 16, kTiles = (NP / 32 * 2 + kWaves - 1) / kWaves;
  constexpr int kBX = Q * kBS > 2 * Q * kXS ? Q * kBS : 2 * Q * kXS;
  extern __shared__ __align__(16) bf16_t sm[];
  bf16_t* Bs = sm;                                  // [Q][kBS], until its fragments are in registers; then
  bf16_t* xh = sm;                                  // [Q][kXS] high and
  bf16_t* xl = xh + Q * kXS;                        // [Q][kXS] low parts of the weighted x
  float* ws = reinterpret_cast<float*>(sm + kBX);   // [heads][Q]
  Unit u;
  if (!unit_of<Q>(a, b, u)) return;
  const int inner = a.H * a.P, stride = (int)a.xbc_stride;
  const bf16_t* src = a.xbc + (int64_t)u.row0 * a.xbc_stride;
  RowTile<Q, NP, 4 * Q> tb;
  RowTile<Q, kPB, 4 * Q> tx;
  const typename RowTile<Q, kPB, 4 * Q>::Offsets off_x(stride, a.P - u.p0);
  tb.load(typename RowTile<Q, NP, 4 * Q>::Offsets(stride, a.N), src + inner + u.grp * a.N, stride, u.rows, a.N);
  tx.load(off_x, src + u.head0 * a.P + u.p0, stride, u.rows, a.P - u.p0);
  for (int i = threadIdx.x; i < u.heads * Q; i += 4 * Q) {      // weights of the tokens at the chunk's end
    const float* ac = a.acs + u.chunk0 * Q;
    ws[i] = a.dts[u.chunk0 * Q + i] * __builtin_amdgcn_exp2f(ac[i / Q * Q + Q - 1] - ac[i]);
  }
  tb.store(Bs, kBS);
  __syncthreads();
  const int lane = threadIdx.x & 63, wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6), half = lane >> 5, l16 = lane & 15;
  const int r = 8 * half + (l16 >> 2), c = (lane & 16) + (l16 & 3) * 4;
  bf16x8_t bf[kTiles][Q / 16];                      // B^T operands of this wavefront's tiles, for every head
  int out_at[kTiles];
#pragma unroll
  for (int i = 0; i < kTiles; ++i) {
    const int tile = wave + kWaves * i, n0 = tile / 2 * 32, p = u.p0 + tile % 2 * 32 + (lane & 31), in = ((n0 + 4 * half) * a.P + p) * 4;
    out_at[i] = p < a.P ? in : kOutside;
    if (n0 < NP)
#pragma unroll
      for (int kk = 0; kk < Q / 16; ++kk) bf[i][kk] = read_tr8(Bs + (kk * 16 + r) * kBS + n0 + c, 4 * kBS);
  }
  for (int hh = 0; hh < u.heads; ++hh) {
    __syncthreads();                                // the last reads of B or of the head before
#pragma unroll
    for (int k = 0; k < tx.kPieces; ++k) {          // x times its token's weight, split
      const int i = threadIdx.x + k * 4 * Q, t = i / tx.kUnits, at = t * kXS + i % tx.kUnits * 8;
      const float w = ws[hh * Q + t];
      const u32x4_t xw = tx.w[k];
      const float v[8] = {bf16lo(xw.x) * w, bf16hi(xw.x) * w, bf16lo(xw.y) * w, bf16hi(xw.y) * w,
                          bf16lo(xw.z) * w, bf16hi(xw.z) * w, bf16lo(xw.w) * w, bf16hi(xw.w) * w};
      bf16x8_t hi, low;
      split8(v, hi, low);
      *reinterpret_cast<bf16x8_t*>(xh + at) = hi;
      *reinterpret_cast<bf16x8_t*>(xl + at) = low;
    }
    __syncthreads();
    tx.load(off_x, src + min(u.head0 + hh + 1, a.H - 1) * a.P + u.p0, stride, u.rows, a.P - u.p0);
    const __amdgpu_buffer_rsrc_t out = __builtin_amdgcn_make_buffer_rsrc(a.chunk_state + (u.chunk0 + hh) * a.N * a.P, 0, a.N * a.P * 4, 0x00020000);
#pragma unroll
    for (int i = 0; i < kTiles; ++i) {
      const int tile = wave + kWaves * i, pb = tile % 2 * 32;
      if (NP / 32 * 2 < kWaves && tile / 2 * 32 >= NP) continue;      // (the wavefront has no tile)
      floatx16_t acc;
#pragma unroll
      for (int e = 0; e < 16; ++e) acc[e] = 0.f;
#pragma unroll
      for (int kk = 0; kk < Q / 16; ++kk) {
        const int at = (kk * 16 + r) * kXS + pb + c;
        acc = __builtin_amdgcn_mfma_f32_32x32x16_bf16(bf[i][kk], read_tr8(xh + at, 4 * kXS), acc, 0, 0, 0);
        acc = __builtin_amdgcn_mfma_f32_32x32x16_bf16(bf[i][kk], read_tr8(xl + at, 4 * kXS), acc, 0, 0, 0);
      }
#pragma unroll
      for (int e = 0; e < 16; ++e)                  // row 8 (e / 4) + 4 half + e % 4 of the tile; rows behind N are not written
        __builtin_amdgcn_raw_buffer_store_b32(__float_as_uint(acc[e]), out, out_at[i] + (8 * (e >> 2) + (e & 3)) * a.P * 4, 0, 0);
    }
  }
}

// Four state elements per thread (N P is a multiple of 8), a batch of chunks requested at a time.
template <int Q>
__global__ __launch_bounds__(256) void ssd_carry_kernel(ChunkArgs a, msa_seq_batch b) {
  const int64_t per = (int64_t)a.N * a.P;
  const int64_t i = ((int64_t)blockIdx.x * 256 + threadIdx.x) * 4;
  const int head = blockIdx.y, s = blockIdx.z;
  if (i >= per) return;
  const int n_tok = b.cu[s + 1] - b.cu[s], chunks = (n_tok + Q - 1) / Q;
  float4* keep = reinterpret_cast<float4*>(a.state + ((int64_t)b.slot[s] * a.H + head) * per + i);
  float4 S = *keep;
  const int64_t first = (int64_t)s * a.n_chunks * a.H + head;
  constexpr int kBatch = 8;
  for (int c = 0; c < chunks; c += kBatch) {
    float4 loc[kBatch];
    float d[kBatch];
    float4* at[kBatch];
#pragma unroll
    for (int k = 0; k < kBatch; ++k) {
      const int64_t chunk = first + (int64_t)min(c + k, chunks - 1) * a.H;
      at[k] = reinterpret_cast<float4*>(a.chunk_state + chunk * per + i);
      loc[k] = *at[k];
      d[k] = a.acs[chunk * Q + Q - 1];
    }
#pragma unroll
    for (int k = 0; k < kBatch; ++k) {
      if (c + k >= chunks) break;
      *reinterpret_cast<uint4*>(at[k]) = make_uint4(pack_split(S.x), pack_split(S.y), pack_split(S.z), pack_split(S.w));
      const float f = __builtin_amdgcn_exp2f(d[k]);
      S = make_float4(f * S.x + loc[k].x, f * S.y + loc[k].y, f * S.z + loc[k].z, f * S.w + loc[k].w);
    }
  }
  *keep = S;
}

template <int Q, int NP>
__global__ __launch_bounds__(4 * Q) void ssd_output_kernel(ChunkArgs a, msa_seq_batch b) {
  constexpr int kBS = NP + 8, kBlocks = Q / 32;
  constexpr int kBSt = Q * kBS > 2 * NP * kXS ? Q * kBS : 2 * NP * kXS;
  constexpr int kBefore = kBlocks * (kBlocks - 1) / 2 * 32;         // (block, earlier token) pairs
  extern __shared__ __align__(16) bf16_t sm[];
  bf16_t* Bs = sm;                                  // [Q][kBS], until B . C^T is in registers; then
  bf16_t* Sh = sm;                                  // [NP][kXS] high and
  bf16_t* Sl = Sh + NP * kXS;                       // [NP][kXS] low parts of S_in
  bf16_t* xs = sm + kBSt;                           // [Q][kXS]
  float* dts = reinterpret_cast<float*>(xs + Q * kXS);
  float* acs = dts + kMaxHeads * Q;
  float* wbs = acs + kMaxHeads * Q;                 // [heads][kBefore] weights of earlier blocks' tokens at a block's start
  Unit u;
  if (!unit_of<Q>(a, b, u)) return;
  const int inner = a.H * a.P;
  const bf16_t* src = a.xbc + (int64_t)u.row0 * a.xbc_stride;
  const int lane = threadIdx.x & 63, wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6), half = lane >> 5, l16 = lane & 15, l32 = lane & 31;
  // a wavefront's token block and half of the columns; the two wavefronts of a SIMD get a long and a short block
  const int tb = Q == 128 ? (wave < 4 ? wave >> 1 : 3 - ((wave - 4) >> 1)) : wave >> 1, pb = wave % 2 * 32;
  const int t = tb * 32 + l32;

  const int stride = (int)a.xbc_stride;
  RowTile<Q, NP, 4 * Q> tileB;
  RowTile<Q, kPB, 4 * Q> tileX;
  const typename RowTile<Q, kPB, 4 * Q>::Offsets off_x(stride, a.P - u.p0);
  constexpr int kSPieces = NP * (kPB / 4) / (4 * Q);
  u32x4_t sw[kSPieces];
  int s_at[kSPieces];
#pragma unroll
  for (int k = 0; k < kSPieces; ++k) {
    const int i = threadIdx.x + k * 4 * Q, p = u.p0 + i % (kPB / 4) * 4, in = (i / (kPB / 4) * a.P + p) * 4;
    s_at[k] = p < a.P ? in : kOutside;
  }
  auto fetch = [&](int hh) {
    tileX.load(off_x, src + (u.head0 + hh) * a.P + u.p0, stride, u.rows, a.P - u.p0);
    const __amdgpu_buffer_rsrc_t rs = __builtin_amdgcn_make_buffer_rsrc(a.chunk_state + (u.chunk0 + hh) * a.N * a.P, 0, a.N * a.P * 4, 0x00020000);
#pragma unroll
    for (int k = 0; k < kSPieces; ++k) sw[k] = __builtin_amdgcn_raw_buffer_load_b128(rs, s_at[k], 0, 0);
  };
  tileB.load(typename RowTile<Q, NP, 4 * Q>::Offsets(stride, a.N), src + inner + u.grp * a.N, stride, u.rows, a.N);
  bf16x8_t cf[NP / 16];
#pragma unroll
  for (int kk = 0; kk < NP / 16; ++kk) {
    const int n = kk * 16 + 8 * half;
    const bool in = t < u.rows && n < a.N;
    cf[kk] = __builtin_bit_cast(bf16x8_t, in ? *reinterpret_cast<const uint4*>(src + (int64_t)t * a.xbc_stride + inner + (a.G + u.grp) * a.N + n)
                                             : make_uint4(0, 0, 0, 0));
  }
  fetch(0);
  for (int i = threadIdx.x; i < u.heads * Q; i += 4 * Q) {
    dts[i] = a.dts[u.chunk0 * Q + i];
    acs[i] = a.acs[u.chunk0 * Q + i];
  }
  tileB.store(Bs, kBS);
  __syncthreads();
  for (int i = threadIdx.x; i < u.heads * kBefore; i += 4 * Q) {
    const int hh = i / kBefore, j = i % kBefore;
    const int blk = j < 32 ? 1 : j < 96 ? 2 : 3, s = j - 16 * blk * (blk - 1);
    wbs[i] = dts[hh * Q + s] * __builtin_amdgcn_exp2f(acs[hh * Q + blk * 32 - 1] - acs[hh * Q + s]);
  }
  floatx16_t g[kBlocks];                            // (B . C^T)[s, t] of block sb, the same for every head
#pragma unroll
  for (int sb = 0; sb < kBlocks; ++sb)
    if (sb <= tb) {
#pragma unroll
      for (int e = 0; e < 16; ++e) g[sb][e] = 0.f;
#pragma unroll
      for (int kk = 0; kk < NP / 16; ++kk) {
        const bf16x8_t bf = *reinterpret_cast<const bf16x8_t*>(Bs + (sb * 32 + l32) * kBS + kk * 16 + 8 * half);
        g[sb] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(bf, cf[kk], g[sb], 0, 0, 0);
      }
    }
  const __amdgpu_buffer_rsrc_t rs_z = rows_rsrc(a.z + (int64_t)u.row0 * a.z_stride, u.rows, a.z_stride, inner);
  const __amdgpu_buffer_rsrc_t rs_v = rows_rsrc(a.v + (int64_t)u.row0 * inner, u.rows, inner, inner);
  const int r = l16 >> 2, c = (lane & 16) + (l16 & 3) * 4;
  int z_at[4], v_at[4];                             // of token t's four pieces, without the head
#pragma unroll
  for (int q = 0; q < 4; ++q) {
    const int p = u.p0 + pb + 8 * q + 4 * half, zin = (t * (int)a.z_stride + p) * 2, vin = (t * inner + p) * 2;
    z_at[q] = p < a.P ? zin : kOutside;
    v_at[q] = p < a.P ? vin : kOutside;
  }
  for (int hh = 0; hh < u.heads; ++hh) {
    const int head = u.head0 + hh;
    __syncthreads();                                // the last reads of B or of the head before, and the weights
    tileX.store(xs, kXS);
#pragma unroll
    for (int k = 0; k < kSPieces; ++k) {
      const int i = threadIdx.x + k * 4 * Q, n = i / (kPB / 4), p = i % (kPB / 4) * 4;
      const u32x4_t w = sw[k];
      *reinterpret_cast<uint2*>(Sh + n * kXS + p) = make_uint2((w.x & 0xffffu) | (w.y << 16), (w.z & 0xffffu) | (w.w << 16));
      *reinterpret_cast<uint2*>(Sl + n * kXS + p) = make_uint2((w.x >> 16) | (w.y & 0xffff0000u), (w.z >> 16) | (w.w & 0xffff0000u));
    }
    __syncthreads();
    if (hh + 1 < u.heads) fetch(hh + 1);
    u32x2_t zw[4];
#pragma unroll
    for (int q = 0; q < 4; ++q) zw[q] = __builtin_amdgcn_raw_buffer_load_b64(rs_z, z_at[q], head * a.P * 2, 0);
    const float* ac = acs + hh * Q;
    const float a_t = ac[t], a_ref = tb > 0 ? ac[tb * 32 - 1] : 0.f;
    floatx16_t acc;
#pragma unroll
    for (int e = 0; e < 16; ++e) acc[e] = 0.f;
#pragma unroll
    for (int kk = 0; kk < NP / 16; ++kk) {
      const int at = (kk * 16 + 8 * half + r) * kXS + pb + c;
      acc = __builtin_amdgcn_mfma_f32_32x32x16_bf16(read_tr8(Sh + at, 4 * kXS), cf[kk], acc, 0, 0, 0);
      acc = __builtin_amdgcn_mfma_f32_32x32x16_bf16(read_tr8(Sl + at, 4 * kXS), cf[kk], acc, 0, 0, 0);
    }
    const float in = __builtin_amdgcn_exp2f(a_ref);
#pragma unroll
    for (int e = 0; e < 16; ++e) acc[e] *= in;
    auto add_block = [&](int sb, const float (&m)[16]) {
#pragma unroll
      for (int j = 0; j < 2; ++j) {
        const float part[8] = {m[8 * j], m[8 * j + 1], m[8 * j + 2], m[8 * j + 3], m[8 * j + 4], m[8 * j + 5], m[8 * j + 6], m[8 * j + 7]};
        bf16x8_t hi, low;
        split8(part, hi, low);
        const bf16x8_t xf = read_tr8(xs + (sb * 32 + 16 * j + 4 * half + r) * kXS + pb + c, 8 * kXS);
        acc = __builtin_amdgcn_mfma_f32_32x32x16_bf16(xf, hi, acc, 0, 0, 0);
        acc = __builtin_amdgcn_mfma_f32_32x32x16_bf16(xf, low, acc, 0, 0, 0);
      }
    };
    // earlier blocks, relative to this block's start; then on to token t
    const float* wb = wbs + hh * kBefore + 16 * tb * (tb - 1);
#pragma unroll
    for (int sb = 0; sb < kBlocks - 1; ++sb)
      if (sb < tb) {
        float m[16];
#pragma unroll
        for (int q = 0; q < 4; ++q) {
          const float4 w = *reinterpret_cast<const float4*>(wb + sb * 32 + 8 * q + 4 * half);
          m[4 * q] = g[sb][4 * q] * w.x;
          m[4 * q + 1] = g[sb][4 * q + 1] * w.y;
          m[4 * q + 2] = g[sb][4 * q + 2] * w.z;
          m[4 * q + 3] = g[sb][4 * q + 3] * w.w;
        }
        add_block(sb, m);
      }
    const float on = __builtin_amdgcn_exp2f(a_t - a_ref);
#pragma unroll
    for (int e = 0; e < 16; ++e) acc[e] *= on;
#pragma unroll
    for (int sb = 0; sb < kBlocks; ++sb)
      if (sb == tb) {
        float m[16];
#pragma unroll
        for (int q = 0; q < 4; ++q) {
          const int s0 = sb * 32 + 8 * q + 4 * half;
          const float4 as = *reinterpret_cast<const float4*>(ac + s0), ds = *reinterpret_cast<const float4*>(dts + hh * Q + s0);
          const float av[4] = {as.x, as.y, as.z, as.w}, dv[4] = {ds.x, ds.y, ds.z, ds.w};
#pragma unroll
          for (int x = 0; x < 4; ++x)
            m[4 * q + x] = s0 + x <= t ? g[sb][4 * q + x] * (__builtin_amdgcn_exp2f(a_t - av[x]) * dv[x]) : 0.f;
        }
        add_block(sb, m);
      }
    // acc[e] is y of token t, column pb + 8 (e / 4) + 4 half + e % 4
    const float Dh = a.D[head];
#pragma unroll
    for (int q = 0; q < 4; ++q) {
      float xv[4], y[4];
      load_vec<bf16_t, 4>(xs + t * kXS + pb + 8 * q + 4 * half, xv);
      const float zv[4] = {bf16lo(zw[q].x), bf16hi(zw[q].x), bf16lo(zw[q].y), bf16hi(zw[q].y)};
#pragma unroll
      for (int x = 0; x < 4; ++x) y[x] = (acc[4 * q + x] + Dh * xv[x]) * silu_f(zv[x]);
      __builtin_amdgcn_raw_buffer_store_b64(u32x2_t{pack_bf16x2(y[0], y[1]), pack_bf16x2(y[2], y[3])}, rs_v, v_at[q], head * a.P * 2, 0);
    }
  }
}

int chunk_tokens(int32_t N) { return N <= 128 ? 128 : 64; }

template <int Q, int NP>
int launch_chunked(ChunkArgs a, const msa_seq_batch& b, hipStream_t st) {
  constexpr int tile = Q * (NP + 8), x = Q * kXS, state = 2 * NP * kXS;
  constexpr int lds2 = (tile > 2 * x ? tile : 2 * x) * 2 + kMaxHeads * Q * 4;
  constexpr int lds3 = ((tile > state ? tile : state) + x) * 2 + kMaxHeads * (2 * Q + (Q / 32) * (Q / 32 - 1) * 16) * 4;
  static_assert(lds2 <= 160 * 1024 && lds3 <= 160 * 1024, "tiles of a chunk must fit LDS");
  // as many heads per workgroup as leave a launch two workgroups per compute unit
  const int per_group = a.H / a.G, blocks = (a.P + kPB - 1) / kPB;
  auto sets = [&](int h) { return (per_group + h - 1) / h; };
  int heads = std::min(kMaxHeads, per_group);
  while (heads > 1 && (int64_t)a.n_chunks * b.n_seq * a.G * blocks * sets(heads) < 2 * device_compute_units()) --heads;
  a.heads_per_wg = (per_group + sets(heads) - 1) / sets(heads);
  static std::atomic<int> raised2{0}, raised3{0};
  MSA_HIP(raise_dynamic_lds_limit(raised2, reinterpret_cast<const void*>(ssd_local_kernel<Q, NP>), lds2));
  MSA_HIP(raise_dynamic_lds_limit(raised3, reinterpret_cast<const void*>(ssd_output_kernel<Q, NP>), lds3));
  ssd_decay_kernel<Q><<<dim3((a.H + 3) / 4, a.n_chunks, b.n_seq), 256, 0, st>>>(a, b);
  MSA_LAUNCH_CHECK();
  const dim3 grid((unsigned)(a.G * blocks * sets(a.heads_per_wg)), a.n_chunks, b.n_seq);
  ssd_local_kernel<Q, NP><<<grid, 4 * Q, lds2, st>>>(a, b);
  MSA_LAUNCH_CHECK();
  ssd_carry_kernel<Q><<<dim3((a.N * a.P / 4 + 255) / 256, a.H, b.n_seq), 256, 0, st>>>(a, b);
  MSA_LAUNCH_CHECK();
  ssd_output_kernel<Q, NP><<<grid, 4 * Q, lds3, st>>>(a, b);
  MSA_LAUNCH_CHECK();
  return MSA_OK;
}

}  // namespace

extern "C" size_t msa_seq_ssd_chunked_workspace_bytes(int32_t max_rows, int32_t n_seq, int32_t H, int32_t P, int32_t N) {
  if (max_rows <= 0 || n_seq <= 0 || H <= 0 || P <= 0 || N <= 0) return 0;
  const int Q = chunk_tokens(N);
  return (size_t)n_seq * ((max_rows + Q - 1) / Q) * H * ((size_t)N * P + 2 * Q) * sizeof(float);
}

extern "C" int msa_seq_ssd_chunked(const void* xbc, int64_t xbc_stride, const void* z, int64_t z_stride, const void* dt_raw,
                                   int64_t dt_stride, const float* dt_bias, const float* A_log, const float* D, int32_t dtype, int32_t H,
                                   int32_t P, int32_t N, int32_t G, float* state, void* v, const msa_seq_batch* batch, void* workspace,
                                   size_t workspace_bytes, void* stream) {
  MSA_CHECK_BATCH(batch, "msa_seq_ssd_chunked");
  MSA_REQUIRE(dtype == MSA_BF16, "msa_seq_ssd_chunked: bf16 only");
  MSA_REQUIRE(xbc && z && dt_raw && dt_bias && A_log && D && state && v && workspace, "msa_seq_ssd_chunked: null pointer");
  MSA_REQUIRE(H > 0 && P > 0 && G > 0 && H % G == 0 && H <= 65535 && P % 8 == 0 && N > 0 && N % 8 == 0 && N <= 256,
              "msa_seq_ssd_chunked: H=%d P=%d N=%d (multiples of 8, N up to 256) G=%d", H, P, N, G);
  MSA_REQUIRE(xbc_stride >= (int64_t)H * P + 2LL * G * N && z_stride >= (int64_t)H * P && dt_stride >= H && xbc_stride % 8 == 0 && xbc_stride < (1 << 21) &&
                  z_stride < (1 << 21) &&
                  z_stride % 4 == 0 && (((uintptr_t)xbc | (uintptr_t)workspace | (uintptr_t)state) & 15) == 0 &&
                  (((uintptr_t)z | (uintptr_t)v) & 7) == 0, "msa_seq_ssd_chunked: strides or alignment");
  const int Q = chunk_tokens(N), chunks = (batch->max_rows + Q - 1) / Q;
  MSA_REQUIRE(chunks <= 65535 && batch->n_seq <= 65535, "msa_seq_ssd_chunked: step too large");
  if (workspace_bytes < msa_seq_ssd_chunked_workspace_bytes(batch->max_rows, batch->n_seq, H, P, N)) {
    msa_set_error("msa_seq_ssd_chunked: workspace of %zu bytes is too small", workspace_bytes);
    return MSA_ESIZE;
  }
  uint32_t* states = static_cast<uint32_t*>(workspace);
  float* dts = reinterpret_cast<float*>(states + (int64_t)batch->n_seq * chunks * H * N * P);
  const ChunkArgs a{(const bf16_t*)xbc, (const bf16_t*)z, (const bf16_t*)dt_raw, dt_bias, A_log, D, state, (bf16_t*)v, states, dts,
                    dts + (int64_t)batch->n_seq * chunks * H * Q, xbc_stride, z_stride, dt_stride, H, P, N, G, chunks, 1};
  hipStream_t st = as_stream(stream);
  if (N <= 32) return launch_chunked<128, 32>(a, *batch, st);
  if (N <= 64) return launch_chunked<128, 64>(a, *batch, st);
  if (N <= 128) return launch_chunked<128, 128>(a, *batch, st);
  return launch_chunked<64, 256>(a, *batch, st);
}
