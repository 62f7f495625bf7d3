// Attention over latents with a learned sink in the softmax denominator, and the prefill kernel of all attention layers.
//
// Decoding works on the latents themselves: a head's query is multiplied by its key matrix beforehand, so all heads of a
// token share one pass over the cached rows (scores and values come from the same bytes).  Prefill works on keys and
// values expanded per head, which costs a fraction of the multiplications per (query, key) pair.
//   latent_attn_kernel    any rank and type: a workgroup per (row, head), fp32 arithmetic throughout
//   latent_decode_kernel  bf16: a workgroup per (row, range of keys, up to 32 heads), 16x16x32 MFMA, then a combine step
//   flash_sink_kernel     bf16 prefill: 32 query columns per wavefront, transposed score tile, 32x32x16 MFMA; query heads may share
//                         keys, positions may see their own chunk only, sinks and a gate per head are optional
#include <algorithm>

#include "seq_mfma.h"

namespace {

__device__ __forceinline__ float half_wave_max(float x) {
  const auto r = __builtin_amdgcn_permlane32_swap(__float_as_uint(x), __float_as_uint(x), false, false);
  return fmaxf(__uint_as_float(r[0]), __uint_as_float(r[1]));
}
__device__ __forceinline__ float half_wave_sum(float x) {
  const auto r = __builtin_amdgcn_permlane32_swap(__float_as_uint(x), __float_as_uint(x), false, false);
  return __uint_as_float(r[0]) + __uint_as_float(r[1]);
}

// ------------------------------------------------------------------------------------------------ any rank and type
constexpr int kMaxCols = 8;            // rank <= 256 * kMaxCols

template <typename T>
__global__ __launch_bounds__(256) void latent_attn_kernel(const T* __restrict__ q, const T* __restrict__ cache, int64_t Lcap,
                                                          const float* __restrict__ sink, float scale, int32_t H, int32_t rank,
                                                          T* __restrict__ ctx, msa_seq_batch b) {
  extern __shared__ float qs[];        // [rank], then 64 scores
  float* sc = qs + rank;
  const int row = blockIdx.x, head = blockIdx.y, tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
  const int s = b.row_seq[row];
  const int n_keys = (int)(b.pos[s] + (row - b.cu[s]) + 1);
  const T* c = cache + (int64_t)b.slot[s] * Lcap * rank;
  const int64_t qat = ((int64_t)row * H + head) * rank;
  for (int i = tid; i < rank; i += 256) qs[i] = to_f32<T>(q[qat + i]);
  float m = sink[head], l = 1.f;       // the sink is the softmax's first member
  float acc[kMaxCols] = {};
  __syncthreads();
  for (int k0 = 0; k0 < n_keys; k0 += 64) {
    const int nk = min(64, n_keys - k0);
    for (int j = wave; j < nk; j += 4) {
      float d = 0.f;
      for (int i = lane; i < rank; i += 64) d += qs[i] * to_f32<T>(c[(int64_t)(k0 + j) * rank + i]);
#pragma unroll
      for (int o = 32; o > 0; o >>= 1) d += __shfl_xor(d, o);
      if (lane == 0) sc[j] = d * scale;
    }
    __syncthreads();
    const float mine = lane < nk ? sc[lane] : -INFINITY;
    float mx = mine;
#pragma unroll
    for (int o = 32; o > 0; o >>= 1) mx = fmaxf(mx, __shfl_xor(mx, o));
    const float m_new = fmaxf(m, mx), alpha = expf(m - m_new);
    const float p = expf(mine - m_new);
    float sum = p;
#pragma unroll
    for (int o = 32; o > 0; o >>= 1) sum += __shfl_xor(sum, o);
    l = l * alpha + sum;
    m = m_new;
    __syncthreads();
    if (wave == 0) sc[lane] = p;
    __syncthreads();
#pragma unroll
    for (int u = 0; u < kMaxCols; ++u) {
      const int i = tid + 256 * u;
      if (i >= rank) break;
      float a = acc[u] * alpha;
      for (int j = 0; j < nk; ++j) a += sc[j] * to_f32<T>(c[(int64_t)(k0 + j) * rank + i]);
      acc[u] = a;
    }
    __syncthreads();
  }
#pragma unroll
  for (int u = 0; u < kMaxCols; ++u) {
    const int i = tid + 256 * u;
    if (i < rank) ctx[qat + i] = from_f32<T>(acc[u] / l);
  }
}

// ------------------------------------------------------------------------------------------------ decode
constexpr int kDecKeys = 64;           // keys per tile
constexpr int kDecMaxRank = 512;

struct DecArgs {
  const bf16_t* q;
  const bf16_t* cache;
  bf16_t* part_acc;    // [rows, n_split, H, rank]
  float* part_ml;      // [rows, n_split, H, 2]
  int64_t Lcap;
  float scale_log2e;
  int32_t H, rank, n_split;
};

// HT (1 or 2) tiles of 16 heads, RP: the rank padded to 64, 128, 256 or 512 (zeros in LDS).  Eight wavefronts: wavefront w
// scores keys 16 (w % 4) .. + 16 of a tile for head tile w / 4, whose queries it holds in registers, and owns the latent columns
// of 16-column tiles w, w + 8, ... of the product with the probabilities.
constexpr int kDecWaves = 8, kDecThreads = kDecWaves * 64;
template <int HT, int RP>
__global__ __launch_bounds__(kDecThreads) void latent_decode_kernel(DecArgs a, msa_seq_batch b) {
  constexpr int kHeads = 16 * HT, kPStride = kDecKeys + 8, kPer = kDecThreads / kHeads;   // threads per head in the softmax
  constexpr int kSStride = kDecKeys + 4, stride = RP + 8;
  constexpr int kCT = (RP / 16 + kDecWaves - 1) / kDecWaves, units = RP / 8;     // 16-byte pieces of a row, zero behind the rank
  extern __shared__ __align__(16) char lds[];
  bf16_t* cs = reinterpret_cast<bf16_t*>(lds);                   // [64][stride]
  bf16_t* ps = cs + kDecKeys * stride;                           // [kHeads][kPStride]
  float* ss = reinterpret_cast<float*>(ps + kHeads * kPStride);  // [kHeads][kSStride]
  float* al = ss + kHeads * kSStride;                            // [kHeads]
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, l16 = lane & 15, g = lane >> 4;
  const int split = blockIdx.x, h0 = blockIdx.y * kHeads, row = blockIdx.z;
  const int kt = wave & 3, ht = wave >> 2;                       // score tile of this wavefront (ht < HT)
  const int s = b.row_seq[row];
  const int n_keys = (int)(b.pos[s] + (row - b.cu[s]) + 1);
  const int tiles = (n_keys + kDecKeys - 1) / kDecKeys, per = (tiles + a.n_split - 1) / a.n_split;
  const int first = split * per * kDecKeys, last = min(n_keys, first + per * kDecKeys);
  const bf16_t* c = a.cache + (int64_t)b.slot[s] * a.Lcap * a.rank;

  // a thread's pieces: column u of rows r0, r0 + kStep, ...
  const int u = tid % units * 8, r0 = tid / units;
  constexpr int kStep = kDecThreads / units, kPieces = (kDecKeys + kStep - 1) / kStep, kQPieces = (kHeads + kStep - 1) / kStep;
  static_assert(kPieces * kStep == kDecKeys, "whole pieces per thread");
  // Two register sets: a tile is requested two tiles ahead of its use, through a buffer resource whose extent is the tile's
  // valid rows (what lies outside reads as zero), so that no load is conditional and the waits can be counted.
  struct Tile { u32x4_t w[kPieces]; } set0, set1;
  const int row_bytes = a.rank * 2;
  const int voff = u < a.rank ? r0 * row_bytes + u * 2 : 0x40000000;
  auto fetch = [&](Tile& next, int k0) {
    const int extent = __builtin_amdgcn_readfirstlane(max(0, min(kDecKeys, last - k0)) * row_bytes);
    const int at = __builtin_amdgcn_readfirstlane(k0 < last ? k0 : 0);
    const __amdgpu_buffer_rsrc_t rs = __builtin_amdgcn_make_buffer_rsrc(const_cast<bf16_t*>(c + (int64_t)at * a.rank), 0, extent, 0x00020000);
#pragma unroll
    for (int i = 0; i < kPieces; ++i) next.w[i] = __builtin_amdgcn_raw_buffer_load_b128(rs, voff + kStep * i * row_bytes, 0, 0);
  };
  fetch(set0, first);
  fetch(set1, first + kDecKeys);
  bf16x8_t qf[RP / 32];
  {
    const int h = h0 + ht * 16 + l16;
    const bf16_t* at = a.q + ((int64_t)row * a.H + h) * a.rank + 8 * g;
#pragma unroll
    for (int kk = 0; kk < RP / 32; ++kk) {
      const bool in = ht < HT && h < a.H && 32 * kk + 8 * g < a.rank;
      qf[kk] = __builtin_bit_cast(bf16x8_t, in ? *reinterpret_cast<const uint4*>(at + 32 * kk) : make_uint4(0, 0, 0, 0));
    }
  }
  floatx4_t o[HT][kCT];
#pragma unroll
  for (int h = 0; h < HT; ++h)
#pragma unroll
    for (int t = 0; t < kCT; ++t) o[h][t] = floatx4_t{0.f, 0.f, 0.f, 0.f};
  float m = -INFINITY, l = 0.f;        // of head tid / kPer, the same in its kPer threads
  auto tile_step = [&](Tile& mine, int k0) {
    __syncthreads();
#pragma unroll
    for (int i = 0; i < kPieces; ++i) *reinterpret_cast<u32x4_t*>(cs + (r0 + kStep * i) * stride + u) = mine.w[i];
    __syncthreads();
    fetch(mine, k0 + 2 * kDecKeys);
    if (ht < HT) {
      // two chains of products, keys read from LDS a few products ahead
      floatx4_t sc[2] = {floatx4_t{0.f, 0.f, 0.f, 0.f}, floatx4_t{0.f, 0.f, 0.f, 0.f}};
      constexpr int kAhead = RP / 32 < 6 ? RP / 32 : 6;
      const bf16_t* kr = cs + (kt * 16 + l16) * stride + 8 * g;
      bf16x8_t kb[kAhead];
#pragma unroll
      for (int kk = 0; kk < kAhead; ++kk) kb[kk] = *reinterpret_cast<const bf16x8_t*>(kr + 32 * kk);
      __builtin_amdgcn_sched_barrier(0);
#pragma unroll
      for (int kk = 0; kk < RP / 32; ++kk) {
        sc[kk & 1] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(qf[kk], kb[kk % kAhead], sc[kk & 1], 0, 0, 0);
        if (kk + kAhead < RP / 32) kb[kk % kAhead] = *reinterpret_cast<const bf16x8_t*>(kr + 32 * (kk + kAhead));
        __builtin_amdgcn_sched_barrier(0);
      }
#pragma unroll
      for (int e = 0; e < 4; ++e) ss[(ht * 16 + 4 * g + e) * kSStride + kt * 16 + l16] = (sc[0][e] + sc[1][e]) * a.scale_log2e;
    }
    __syncthreads();
    {
      constexpr int kEach = kDecKeys / kPer;                     // keys per thread
      const int h = tid / kPer, j0 = (tid % kPer) * kEach;
      float v[kEach], mx = m;
#pragma unroll
      for (int j = 0; j < kEach; ++j) {
        v[j] = k0 + j0 + j < last ? ss[h * kSStride + j0 + j] : -INFINITY;
        mx = fmaxf(mx, v[j]);
      }
#pragma unroll
      for (int d = 1; d < kPer; d <<= 1) mx = fmaxf(mx, __shfl_xor(mx, d));
      const float alpha = __builtin_amdgcn_exp2f(m - mx);        // a tile has at least one key: mx is finite
      float sum = 0.f;
#pragma unroll
      for (int j = 0; j < kEach; j += 2) {
        const float p0 = __builtin_amdgcn_exp2f(v[j] - mx), p1 = __builtin_amdgcn_exp2f(v[j + 1] - mx);
        sum += p0 + p1;
        *reinterpret_cast<uint32_t*>(ps + h * kPStride + j0 + j) = pack_bf16x2(p0, p1);
      }
#pragma unroll
      for (int d = 1; d < kPer; d <<= 1) sum += __shfl_xor(sum, d);
      l = l * alpha + sum;
      m = mx;
      if (tid % kPer == 0) al[h] = alpha;
    }
    __syncthreads();
#pragma unroll
    for (int h = 0; h < HT; ++h) {
      const float4 f = *reinterpret_cast<const float4*>(al + h * 16 + 4 * g);
      if (!__any(f.x * f.y * f.z * f.w != 1.0f)) continue;       // no maximum moved
#pragma unroll
      for (int t = 0; t < kCT; ++t) {
        o[h][t][0] *= f.x;
        o[h][t][1] *= f.y;
        o[h][t][2] *= f.z;
        o[h][t][3] *= f.w;
      }
    }
#pragma unroll
    for (int kk = 0; kk < kDecKeys; kk += 32) {
      bf16x8_t pa[HT];
#pragma unroll
      for (int h = 0; h < HT; ++h) pa[h] = *reinterpret_cast<const bf16x8_t*>(ps + (h * 16 + l16) * kPStride + kk + 8 * g);
#pragma unroll
      for (int t = 0; t < kCT; ++t) {
        if (wave + kDecWaves * t >= RP / 16) break;
        const bf16_t* at = cs + (kk + 8 * g + (l16 >> 2)) * stride + (wave + kDecWaves * t) * 16 + (l16 & 3) * 4;
        const bf16x8_t vb = join8(lds_read_tr16(at), lds_read_tr16(at + 4 * stride));
#pragma unroll
        for (int h = 0; h < HT; ++h) o[h][t] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(pa[h], vb, o[h][t], 0, 0, 0);
      }
    }
  };
  for (int k0 = first; k0 < last; k0 += 2 * kDecKeys) {
    tile_step(set0, k0);
    if (k0 + kDecKeys < last) tile_step(set1, k0 + kDecKeys);
  }
  // o[h][t][e] belongs to head 16 h + 4 g + e, latent column 16 (wave + 8 t) + l16.  The sums leave in bf16 (as the context that
  // is made of them will), through LDS so that a row's pieces are stored 16 bytes at a time.
  const int64_t at = ((int64_t)row * a.n_split + split) * a.H;
  __syncthreads();
  static_assert(kHeads <= kDecKeys, "the key tile's LDS holds the sums");
#pragma unroll
  for (int h = 0; h < HT; ++h)
#pragma unroll
    for (int t = 0; t < kCT; ++t) {
      const int col = (wave + kDecWaves * t) * 16 + l16;
      if (col >= RP) continue;
#pragma unroll
      for (int e = 0; e < 4; ++e) cs[(h * 16 + 4 * g + e) * stride + col] = f32_to_bf16(o[h][t][e]);
    }
  __syncthreads();
#pragma unroll
  for (int i = 0; i < kQPieces; ++i) {
    const int h = r0 + kStep * i;
    if (h < kHeads && h0 + h < a.H && u < a.rank)
      *reinterpret_cast<uint4*>(a.part_acc + (at + h0 + h) * a.rank + u) = *reinterpret_cast<const uint4*>(cs + h * stride + u);
  }
  if (tid % kPer == 0 && h0 + tid / kPer < a.H) {
    a.part_ml[(at + h0 + tid / kPer) * 2] = m;
    a.part_ml[(at + h0 + tid / kPer) * 2 + 1] = l;
  }
}

// A workgroup per (row, head): folds the key ranges and the sink.  The ranges' weights first, then their sums: four wavefronts
// take a quarter of the ranges each, eight columns a lane.
constexpr int kMaxSplits = 128;
__global__ __launch_bounds__(256) void latent_combine_kernel(const bf16_t* __restrict__ part_acc, const float* __restrict__ part_ml,
                                                             const float* __restrict__ sink, int32_t H, int32_t rank, int32_t n_split,
                                                             bf16_t* __restrict__ ctx) {
  __shared__ float ws[kMaxSplits], red[8];
  __shared__ float sums[4][64 * 8];
  const int row = blockIdx.x, head = blockIdx.y, tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
  const int64_t first = (int64_t)row * n_split * H + head;
  const float sk = sink[head] * kLog2e;
  float mi = -INFINITY, li = 0.f;
  if (tid < n_split) {
    const float2 ml = *reinterpret_cast<const float2*>(part_ml + (first + (int64_t)tid * H) * 2);
    mi = ml.x;
    li = ml.y;
  }
  float m = fmaxf(mi, sk);
#pragma unroll
  for (int o = 32; o > 0; o >>= 1) m = fmaxf(m, __shfl_xor(m, o));
  if (lane == 0) red[wave] = m;
  __syncthreads();
  m = fmaxf(fmaxf(red[0], red[1]), fmaxf(red[2], red[3]));
  const float w = __builtin_amdgcn_exp2f(mi - m);                // 0 for a range without keys
  float l = w * li;
#pragma unroll
  for (int o = 32; o > 0; o >>= 1) l += __shfl_xor(l, o);
  if (lane == 0) red[4 + wave] = l;
  if (tid < kMaxSplits) ws[tid] = w;
  __syncthreads();
  const float inv = 1.0f / (red[4] + red[5] + red[6] + red[7] + __builtin_amdgcn_exp2f(sk - m));
  float v[8] = {};
  const int c = lane * 8;                                        // rank <= 512
  if (c < rank) {
    const bf16_t* src = part_acc + first * rank + c;
#pragma unroll 4
    for (int i = wave; i < n_split; i += 4) {
      float p[8];
      load_vec<bf16_t, 8>(src + (int64_t)i * H * rank, p);
      const float f = ws[i];
#pragma unroll
      for (int e = 0; e < 8; ++e) v[e] += f * p[e];
    }
  }
#pragma unroll
  for (int e = 0; e < 8; ++e) sums[wave][e * 64 + lane] = v[e];
  __syncthreads();
  if (wave != 0 || c >= rank) return;
#pragma unroll
  for (int e = 0; e < 8; ++e) v[e] = (sums[0][e * 64 + lane] + sums[1][e * 64 + lane] + sums[2][e * 64 + lane] + sums[3][e * 64 + lane]) * inv;
  store_vec<bf16_t, 8>(ctx + ((int64_t)row * H + head) * rank + c, v);
}

int latent_splits(int32_t rows, int32_t H, int64_t max_keys) {
  const int64_t tiles = std::max<int64_t>(1, (max_keys + kDecKeys - 1) / kDecKeys);
  const int64_t blocks = (int64_t)rows * ((H + 31) / 32);
  return (int)std::min<int64_t>(std::min<int64_t>(tiles, kMaxSplits), std::max<int64_t>(1, (device_compute_units() + blocks - 1) / blocks));
}

// ------------------------------------------------------------------------------------------------ prefill
struct FlashArgs {
  const bf16_t* q;
  const bf16_t* k;
  const bf16_t* v;
  const int64_t* kv_off;
  const float* sink;         // or null
  const bf16_t* gate;        // [rows, H] or null: outputs times sigmoid(gate)
  bf16_t* out;
  int64_t q_stride, k_stride, v_stride, gate_stride;
  float scale_log2e;
  int32_t H, D, E, group;    // `group` query heads share a key head
  int32_t chunk;             // positions see keys from their last multiple of this on (0: all)
};
constexpr float kNoScore = -1e30f;       // below every score, and finite
constexpr int kFlashKeys = 64, kFlashRows = 128;

// DP / EP: D and E padded to a multiple of 32 (zeros in LDS).  Two stages of K and V tiles in LDS; the next tile is
// fetched into registers while this one is multiplied.
template <int DP, int EP>
__global__ __launch_bounds__(256, (DP + EP <= 256) ? 2 : 1) void flash_sink_kernel(FlashArgs a, msa_seq_batch b) {
  constexpr int kKS = DP + 8, kVS = EP + 8;
  constexpr int kKP = kFlashKeys * DP / 8 / 256, kVP = kFlashKeys * EP / 8 / 256;   // 16-byte pieces per thread
  extern __shared__ __align__(16) bf16_t fl[];
  bf16_t* kt = fl;                                   // [2][64][kKS]
  bf16_t* vt = fl + 2 * kFlashKeys * kKS;            // [2][64][kVS]
  const int head = blockIdx.x, s = blockIdx.z;
  const int lo = b.cu[s], n_tok = b.cu[s + 1] - lo;
  const int blk = (n_tok + kFlashRows - 1) / kFlashRows - 1 - (int)blockIdx.y;   // long ones first
  if (blk < 0) return;
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, col = lane & 31, half = lane >> 5;
  const int tok = blk * kFlashRows + wave * 32 + col;
  const bool ok = tok < n_tok;
  const int base = (int)b.pos[s];
  const int limit = ok ? base + tok + 1 : 0;
  const int kmax = base + min(n_tok, (blk + 1) * kFlashRows);
  auto floor_of = [&](int pos) { return a.chunk ? pos / a.chunk * a.chunk : 0; };   // first key that position sees
  const int kmin = floor_of(base + blk * kFlashRows), lowest = floor_of(base + tok);
  // the wavefront's first column sees keys wave_lo .. wave_min - 1, its last one keys wave_hi_lo .. wave_max - 1
  const int wave_first = __builtin_amdgcn_readfirstlane(blk * kFlashRows + wave * 32), wave_last = min(n_tok, wave_first + 32) - 1;
  const int wave_min = base + wave_first + 1, wave_max = wave_first < n_tok ? base + wave_last + 1 : 0;
  const int wave_lo = floor_of(base + wave_first), wave_hi_lo = floor_of(base + max(wave_last, 0));
  const bf16_t* kg = a.k + a.kv_off[s] * a.k_stride + (int64_t)(head / a.group) * a.D;
  const bf16_t* vg = a.v + a.kv_off[s] * a.v_stride + (int64_t)(head / a.group) * a.E;

  bf16x8_t qf[DP / 16];
  {
    const bf16_t* qr = a.q + (int64_t)(lo + (ok ? tok : 0)) * a.q_stride + (int64_t)head * a.D;
#pragma unroll
    for (int i = 0; i < DP / 16; ++i) {
      const int d = 16 * i + 8 * half;
      const uint4 w = ok && d < a.D ? *reinterpret_cast<const uint4*>(qr + d) : make_uint4(0, 0, 0, 0);
      qf[i] = __builtin_bit_cast(bf16x8_t, w);
    }
  }
  // tile loads through buffer resources whose extent is the tile's valid rows: rows and dims outside read as zero
  u32x4_t kn[kKP], vn[kVP];
  int kv_off[kKP], vv_off[kVP];
#pragma unroll
  for (int i = 0; i < kKP; ++i) {
    const int idx = tid + 256 * i, key = idx / (DP / 8), d = idx % (DP / 8) * 8;
    kv_off[i] = d < a.D ? (int)(key * a.k_stride + d) * 2 : 0x7ffffff0;
  }
#pragma unroll
  for (int i = 0; i < kVP; ++i) {
    const int idx = tid + 256 * i, key = idx / (EP / 8), d = idx % (EP / 8) * 8;
    vv_off[i] = d < a.E ? (int)(key * a.v_stride + d) * 2 : 0x7ffffff0;
  }
  auto fetch = [&](int k0) {
    const int rows = min(kFlashKeys, kmax - k0);
    const __amdgpu_buffer_rsrc_t rk = __builtin_amdgcn_make_buffer_rsrc(
        const_cast<bf16_t*>(kg + (int64_t)k0 * a.k_stride), 0, (int)((rows - 1) * a.k_stride + a.D) * 2, 0x00020000);
    const __amdgpu_buffer_rsrc_t rv = __builtin_amdgcn_make_buffer_rsrc(
        const_cast<bf16_t*>(vg + (int64_t)k0 * a.v_stride), 0, (int)((rows - 1) * a.v_stride + a.E) * 2, 0x00020000);
#pragma unroll
    for (int i = 0; i < kKP; ++i) kn[i] = __builtin_amdgcn_raw_buffer_load_b128(rk, kv_off[i], 0, 0);
#pragma unroll
    for (int i = 0; i < kVP; ++i) vn[i] = __builtin_amdgcn_raw_buffer_load_b128(rv, vv_off[i], 0, 0);
  };
  auto stash = [&](int stage) {
#pragma unroll
    for (int i = 0; i < kKP; ++i) {
      const int idx = tid + 256 * i;
      *reinterpret_cast<u32x4_t*>(kt + (stage * kFlashKeys + idx / (DP / 8)) * kKS + idx % (DP / 8) * 8) = kn[i];
    }
#pragma unroll
    for (int i = 0; i < kVP; ++i) {
      const int idx = tid + 256 * i;
      *reinterpret_cast<u32x4_t*>(vt + (stage * kFlashKeys + idx / (EP / 8)) * kVS + idx % (EP / 8) * 8) = vn[i];
    }
  };
  floatx16_t o[EP / 32];
#pragma unroll
  for (int d = 0; d < EP / 32; ++d)
#pragma unroll
    for (int e = 0; e < 16; ++e) o[d][e] = 0.f;
  // a sink is the first member of every column's softmax
  float m = a.sink ? a.sink[head] * kLog2e : kNoScore, l = a.sink && half == 0 ? 1.f : 0.f;
  fetch(kmin);
  stash(0);
  __syncthreads();
  int stage = 0;
  auto multiply = [&](int k0) {
    const bf16_t* kb = kt + stage * kFlashKeys * kKS;
    const bf16_t* vb = vt + stage * kFlashKeys * kVS;
    floatx16_t sc[2];
#pragma unroll
    for (int rb = 0; rb < 2; ++rb)
#pragma unroll
      for (int e = 0; e < 16; ++e) sc[rb][e] = 0.f;
#pragma unroll
    for (int i = 0; i < DP / 16; ++i)
#pragma unroll
      for (int rb = 0; rb < 2; ++rb) {
        const bf16x8_t kf = *reinterpret_cast<const bf16x8_t*>(kb + (rb * 32 + col) * kKS + 16 * i + 8 * half);
        sc[rb] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(kf, qf[i], sc[rb], 0, 0, 0);
      }
    float mx = -INFINITY;
    if (k0 + kFlashKeys > wave_min || k0 < wave_hi_lo) {
#pragma unroll
      for (int rb = 0; rb < 2; ++rb)
#pragma unroll
        for (int e = 0; e < 16; ++e) {
          const int key = k0 + 32 * rb + 8 * (e >> 2) + 4 * half + (e & 3);
          sc[rb][e] = key < limit && key >= lowest ? sc[rb][e] : -INFINITY;
        }
    }
#pragma unroll
    for (int rb = 0; rb < 2; ++rb)
#pragma unroll
      for (int e = 0; e < 16; ++e) mx = fmaxf(mx, sc[rb][e]);
    mx = half_wave_max(mx * a.scale_log2e);
    // the reference value only follows the maximum when it is well behind it: the probabilities stay below 2^6
    if (__any(mx > m + 6.0f)) {
      const float m_new = fmaxf(m, mx), alpha = __builtin_amdgcn_exp2f(m - m_new);
      l *= alpha;
#pragma unroll
      for (int d = 0; d < EP / 32; ++d)
#pragma unroll
        for (int e = 0; e < 16; ++e) o[d][e] *= alpha;
      m = m_new;
    }
#pragma unroll
    for (int rb = 0; rb < 2; ++rb)
#pragma unroll
      for (int j = 0; j < 2; ++j) {
        uint32_t pw[4];
#pragma unroll
        for (int x = 0; x < 4; ++x) {
          const float p0 = __builtin_amdgcn_exp2f(fmaf(sc[rb][8 * j + 2 * x], a.scale_log2e, -m));
          const float p1 = __builtin_amdgcn_exp2f(fmaf(sc[rb][8 * j + 2 * x + 1], a.scale_log2e, -m));
          l += p0 + p1;
          pw[x] = pack_bf16x2(p0, p1);
        }
        const bf16x8_t pb = __builtin_bit_cast(bf16x8_t, make_uint4(pw[0], pw[1], pw[2], pw[3]));
        // keys 32 rb + 16 j + {4 half .. + 3, 8 + 4 half .. + 3}, in the order the score tile's rows hold them
        const bf16_t* vrow = vb + (rb * 32 + j * 16 + 4 * half + ((lane & 15) >> 2)) * kVS + (lane & 16) + (lane & 3) * 4;
#pragma unroll
        for (int d = 0; d < EP / 32; ++d) {
          const bf16x8_t vf = join8(lds_read_tr16(vrow + d * 32), lds_read_tr16(vrow + 8 * kVS + d * 32));
          o[d] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(vf, pb, o[d], 0, 0, 0);
        }
      }
  };
  for (int k0 = kmin; k0 < kmax; k0 += kFlashKeys, stage ^= 1) {
    const bool more = k0 + kFlashKeys < kmax;
    if (more) fetch(k0 + kFlashKeys);
    if (k0 < wave_max && k0 + kFlashKeys > wave_lo) multiply(k0);      // (the wavefront's columns see some of the tile)
    if (more) stash(stage ^ 1);
    __syncthreads();
  }
  l = half_wave_sum(l);
  if (!ok) return;
  float inv = 1.0f / l;
  if (a.gate) inv *= sigmoid_f(bf16_to_f32(a.gate[(int64_t)(lo + tok) * a.gate_stride + head]));
  bf16_t* dst = a.out + ((int64_t)(lo + tok) * a.H + head) * a.E;
#pragma unroll
  for (int d = 0; d < EP / 32; ++d)
#pragma unroll
    for (int x = 0; x < 4; ++x) {
      const int at = d * 32 + 8 * x + 4 * half;
      if (at < a.E)
        *reinterpret_cast<uint2*>(dst + at) = make_uint2(pack_bf16x2(o[d][4 * x] * inv, o[d][4 * x + 1] * inv),
                                                         pack_bf16x2(o[d][4 * x + 2] * inv, o[d][4 * x + 3] * inv));
    }
}

template <int DP, int EP>
int launch_flash(const FlashArgs& a, const msa_seq_batch& b, hipStream_t st) {
  constexpr int lds = 2 * kFlashKeys * (DP + 8 + EP + 8) * 2;
  static std::atomic<int> raised{0};
  MSA_HIP(raise_dynamic_lds_limit(raised, reinterpret_cast<const void*>(flash_sink_kernel<DP, EP>), lds));
  flash_sink_kernel<DP, EP><<<dim3(a.H, (b.max_rows + kFlashRows - 1) / kFlashRows, b.n_seq), 256, lds, st>>>(a, b);
  MSA_LAUNCH_CHECK();
  return MSA_OK;
}

template <int HT, int RP>
int launch_decode(const DecArgs& a, const msa_seq_batch& b, hipStream_t st) {
  constexpr int stride = RP + 8, heads = 16 * HT;
  constexpr int lds = kDecKeys * stride * 2 + heads * (kDecKeys + 8) * 2 + heads * (kDecKeys + 4) * 4 + heads * 4;
  static_assert(lds <= 160 * 1024, "tiles must fit LDS");
  static std::atomic<int> raised{0};
  MSA_HIP(raise_dynamic_lds_limit(raised, reinterpret_cast<const void*>(latent_decode_kernel<HT, RP>), lds));
  latent_decode_kernel<HT, RP><<<dim3(a.n_split, (a.H + heads - 1) / heads, b.rows), kDecThreads, lds, st>>>(a, b);
  MSA_LAUNCH_CHECK();
  return MSA_OK;
}
template <int HT>
int launch_decode(const DecArgs& a, const msa_seq_batch& b, hipStream_t st) {
  if (a.rank <= 64) return launch_decode<HT, 64>(a, b, st);
  if (a.rank <= 128) return launch_decode<HT, 128>(a, b, st);
  if (a.rank <= 256) return launch_decode<HT, 256>(a, b, st);
  return launch_decode<HT, 512>(a, b, st);
}

}  // namespace

extern "C" int msa_seq_latent_attn(const void* q, const void* cache, int64_t Lcap, const float* sink, float scale, int32_t dtype,
                                   int32_t H, int32_t rank, void* ctx, const msa_seq_batch* batch, void* stream) {
  MSA_CHECK_BATCH(batch, "msa_seq_latent_attn");
  MSA_CHECK_DTYPE(dtype, "msa_seq_latent_attn");
  MSA_REQUIRE(q && cache && sink && ctx && Lcap > 0 && H > 0 && H <= 65535 && rank > 0 && rank <= 256 * kMaxCols,
              "msa_seq_latent_attn: H=%d rank=%d (up to %d)", H, rank, 256 * kMaxCols);
  const dim3 grid(batch->rows, H);
  const size_t lds = (rank + 64) * sizeof(float);
  if (dtype == MSA_BF16)
    latent_attn_kernel<bf16_t><<<grid, 256, lds, as_stream(stream)>>>((const bf16_t*)q, (const bf16_t*)cache, Lcap, sink, scale, H, rank,
                                                                      (bf16_t*)ctx, *batch);
  else
    latent_attn_kernel<float><<<grid, 256, lds, as_stream(stream)>>>((const float*)q, (const float*)cache, Lcap, sink, scale, H, rank,
                                                                     (float*)ctx, *batch);
  MSA_LAUNCH_CHECK();
  return MSA_OK;
}

extern "C" size_t msa_seq_latent_decode_workspace_bytes(int32_t rows, int32_t H, int32_t rank, int64_t max_keys) {
  if (rows <= 0 || H <= 0 || rank <= 0 || max_keys <= 0) return 0;
  return (size_t)rows * latent_splits(rows, H, max_keys) * H * (2 * sizeof(float) + (size_t)rank * sizeof(bf16_t));
}

extern "C" int msa_seq_latent_decode(const void* q, const void* cache, int64_t Lcap, const float* sink, float scale, int32_t dtype,
                                     int32_t H, int32_t rank, int64_t max_keys, void* ctx, const msa_seq_batch* batch, void* workspace,
                                     size_t workspace_bytes, void* stream) {
  MSA_CHECK_BATCH(batch, "msa_seq_latent_decode");
  MSA_REQUIRE(dtype == MSA_BF16, "msa_seq_latent_decode: bf16 only");
  MSA_REQUIRE(q && cache && sink && ctx && workspace, "msa_seq_latent_decode: null pointer");
  MSA_REQUIRE(H > 0 && H <= 4096 && rank > 0 && rank % 8 == 0 && rank <= kDecMaxRank, "msa_seq_latent_decode: H=%d rank=%d (a multiple of 8 up to %d)",
              H, rank, kDecMaxRank);
  MSA_REQUIRE(batch->rows <= 65535 && max_keys > 0 && max_keys <= Lcap && Lcap < ((int64_t)1 << 31), "msa_seq_latent_decode: %d rows, %lld keys",
              batch->rows, (long long)max_keys);
  MSA_REQUIRE((((uintptr_t)q | (uintptr_t)cache | (uintptr_t)ctx | (uintptr_t)workspace) & 15) == 0, "msa_seq_latent_decode: q, cache, ctx and workspace must be 16-byte aligned");
  const int splits = latent_splits(batch->rows, H, max_keys);
  if (workspace_bytes < msa_seq_latent_decode_workspace_bytes(batch->rows, H, rank, max_keys)) {
    msa_set_error("msa_seq_latent_decode: workspace of %zu bytes is too small", workspace_bytes);
    return MSA_ESIZE;
  }
  bf16_t* acc = static_cast<bf16_t*>(workspace);                 // (rank is a multiple of 8: the pairs behind stay aligned)
  float* ml = reinterpret_cast<float*>(acc + (int64_t)batch->rows * splits * H * rank);
  const DecArgs a{(const bf16_t*)q, (const bf16_t*)cache, acc, ml, Lcap, scale * kLog2e, H, rank, splits};
  hipStream_t st = as_stream(stream);
  const int rc = H <= 16 ? launch_decode<1>(a, *batch, st) : launch_decode<2>(a, *batch, st);
  if (rc != MSA_OK) return rc;
  latent_combine_kernel<<<dim3(batch->rows, H), 256, 0, st>>>(acc, ml, sink, H, rank, splits, (bf16_t*)ctx);
  MSA_LAUNCH_CHECK();
  return MSA_OK;
}

extern "C" int msa_seq_flash(const void* q, int64_t q_stride, const void* k, int64_t k_stride, const void* v, int64_t v_stride,
                             const int64_t* kv_off, const float* sink, float scale, int32_t dtype, int32_t H, int32_t G, int32_t D, int32_t E,
                             int32_t chunk, const void* gate, int64_t gate_stride, void* out, const msa_seq_batch* batch, void* stream) {
  MSA_CHECK_BATCH(batch, "msa_seq_flash");
  MSA_REQUIRE(dtype == MSA_BF16, "msa_seq_flash: bf16 only");
  MSA_REQUIRE(q && k && v && kv_off && out && scale > 0.f && chunk >= 0, "msa_seq_flash: null pointer, scale <= 0 or chunk < 0");
  MSA_REQUIRE(H > 0 && G > 0 && H % G == 0 && (!gate || gate_stride >= H), "msa_seq_flash: %d heads over %d, or the gate's stride", H, G);
  MSA_REQUIRE(D > 0 && E > 0 && D % 8 == 0 && E % 8 == 0 && D <= 256 && E <= 256, "msa_seq_flash: D=%d E=%d (multiples of 8 up to 256)", D, E);
  MSA_REQUIRE(q_stride >= (int64_t)H * D && k_stride >= (int64_t)G * D && v_stride >= (int64_t)G * E && q_stride % 8 == 0 &&
                  k_stride % 8 == 0 && v_stride % 8 == 0 && k_stride <= (1 << 22) && v_stride <= (1 << 22) && (((uintptr_t)q | (uintptr_t)k | (uintptr_t)v | (uintptr_t)out) & 15) == 0,
              "msa_seq_flash: strides or alignment");
  MSA_REQUIRE(batch->n_seq <= 65535 && (batch->max_rows + kFlashRows - 1) / kFlashRows <= 65535, "msa_seq_flash: step too large");
  const FlashArgs a{(const bf16_t*)q, (const bf16_t*)k, (const bf16_t*)v, kv_off, sink, (const bf16_t*)gate, (bf16_t*)out, q_stride, k_stride,
                    v_stride, gate_stride, scale * kLog2e, H, D, E, H / G, chunk};
  hipStream_t st = as_stream(stream);
  if (D <= 64 && E <= 64) return launch_flash<64, 64>(a, *batch, st);
  if (D <= 128 && E <= 64) return launch_flash<128, 64>(a, *batch, st);
  if (D <= 128 && E <= 128) return launch_flash<128, 128>(a, *batch, st);
  if (D <= 192 && E <= 128) return launch_flash<192, 128>(a, *batch, st);
  return launch_flash<256, 256>(a, *batch, st);
}
