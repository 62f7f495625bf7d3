// Chunked form of the state-space recurrence on the matrix cores (bf16 inputs, fp32 states and decays), for portions long
// enough to be worth cutting into chunks of Q tokens (Q = 128, or 64 when the state has more than 128 rows).  With
// a_t = sum of the chunk's log-decays up to t, inside a chunk
//   y_t = exp(a_t) S_in^T C_t + sum_{s <= t} exp(a_t - a_s) dt_s (B_s . C_t) x_s,   S_out = exp(a_end) S_in + S_loc,
//   S_loc = sum_s exp(a_end - a_s) dt_s B_s x_s^T.
//   (1) ssd_local_kernel   every chunk's S_loc
//   (2) ssd_carry_kernel   the chunk-to-chunk recurrence, element by element; leaves each chunk's S_in in its place
//   (3) ssd_output_kernel  the outputs
// Operands that carry decays or states are fp32 values: they enter the bf16 products as a high and a low part (two products
// with about 16 bits of mantissa), so only x, B and C, which are bf16 to begin with, set the precision.
//
// The score tile is taken transposed, G^T[s, t] = B . C^T, so that its accumulator layout (lane = column t) is the operand
// layout of the second product y^T[p, t] += x^T . M^T, and a_t is one scalar per lane; x^T and S_in^T come out of LDS through
// the transposing read.
#include <algorithm>

#include "seq_common.h"

namespace {

typedef __attribute__((__vector_size__(8 * sizeof(__bf16)))) __bf16 bf16x8_t;
typedef __attribute__((__vector_size__(16 * sizeof(float)))) float floatx16_t;
typedef short shortx4_t __attribute__((ext_vector_type(4)));
typedef __attribute__((address_space(3))) shortx4_t lds_shortx4_t;

constexpr float kLog2e = 1.4426950408889634f;
constexpr int kPB = 64;                  // state columns (p) per workgroup
constexpr int kXS = kPB + 8;             // LDS row stride of [.., p] tiles

// Eight rows (two reads of four, `gap` rows apart in LDS elements) of a 16-bit tile, transposed: see flash_attn.hip.
__device__ __forceinline__ bf16x8_t read_tr8(const bf16_t* p, int gap) {
  const shortx4_t lo = __builtin_amdgcn_ds_read_tr16_b64_v4i16((lds_shortx4_t*)(p));
  const shortx4_t hi = __builtin_amdgcn_ds_read_tr16_b64_v4i16((lds_shortx4_t*)(p + gap));
  return __builtin_bit_cast(bf16x8_t, __builtin_shufflevector(lo, hi, 0, 1, 2, 3, 4, 5, 6, 7));
}
// fp32 values as bf16 operands: high part and what it leaves over.
__device__ __forceinline__ void split8(const float (&v)[8], bf16x8_t& hi, bf16x8_t& lo) {
  uint32_t h[4], l[4];
#pragma unroll
  for (int i = 0; i < 4; ++i) {
    h[i] = pack_bf16x2(v[2 * i], v[2 * i + 1]);
    l[i] = pack_bf16x2(v[2 * i] - bf16lo(h[i]), v[2 * i + 1] - bf16hi(h[i]));
  }
  hi = __builtin_bit_cast(bf16x8_t, make_uint4(h[0], h[1], h[2], h[3]));
  lo = __builtin_bit_cast(bf16x8_t, make_uint4(l[0], l[1], l[2], l[3]));
}

struct ChunkArgs {
  const bf16_t* xbc;
  const bf16_t* z;
  const bf16_t* dt_raw;
  const float* dt_bias;
  const float* A_log;
  const float* D;
  float* state;
  bf16_t* v;
  float* chunk_state;      // [n_seq, n_chunks, H, N, P]: S_loc (fp32), then S_in as packed (high, low) bf16 pairs
  float* chunk_decay;      // [n_seq, n_chunks, H]: a_end in powers of two
  int64_t xbc_stride, z_stride, dt_stride;
  int32_t H, P, N, G, n_chunks;
};

// dt and the running log-decay (base 2) of the chunk's tokens into LDS; tokens behind the sequence have dt = 0.
template <int Q>
__device__ __forceinline__ void chunk_decays(const ChunkArgs& a, int row0, int rows, int head, float* dts, float* acs) {
  const int tid = threadIdx.x;
  float dt = 0.f, ac = 0.f;
  if (tid < Q) {
    if (tid < rows) dt = softplus_f(bf16_to_f32(a.dt_raw[(int64_t)(row0 + tid) * a.dt_stride + head]) + a.dt_bias[head]);
    ac = -expf(a.A_log[head]) * dt * kLog2e;
#pragma unroll
    for (int o = 1; o < 64; o <<= 1) {
      const float up = __shfl_up(ac, o);
      if ((tid & 63) >= o) ac += up;
    }
    dts[tid] = dt;
    acs[tid] = ac;
  }
  __syncthreads();
  if (Q == 128) {
    const float first = acs[63];
    __syncthreads();
    if (tid >= 64 && tid < 128) acs[tid] = ac + first;
    __syncthreads();
  }
}

// `n` columns of the chunk's rows on their way into an LDS tile of WIDTH columns (zeros behind n and behind the sequence): all
// loads of a tile are issued before anything waits for one, and several tiles' loads before the first is stored.
template <int Q, int WIDTH, int THREADS>
struct RowTile {
  static constexpr int kUnits = WIDTH / 8, kPieces = Q * kUnits / THREADS;
  static_assert(Q * kUnits % THREADS == 0, "whole pieces per thread");
  uint4 w[kPieces];
  __device__ __forceinline__ void load(const bf16_t* src, int64_t stride, int rows, int n) {
#pragma unroll
    for (int k = 0; k < kPieces; ++k) {
      const int i = threadIdx.x + k * THREADS, r = i / kUnits, u = i % kUnits * 8;
      w[k] = make_uint4(0, 0, 0, 0);
      if (r < rows && u < n) w[k] = *reinterpret_cast<const uint4*>(src + (int64_t)r * stride + u);
    }
  }
  __device__ __forceinline__ void store(bf16_t* dst, int dst_stride) const {
#pragma unroll
    for (int k = 0; k < kPieces; ++k) {
      const int i = threadIdx.x + k * THREADS;
      *reinterpret_cast<uint4*>(dst + i / kUnits * dst_stride + i % kUnits * 8) = w[k];
    }
  }
};

template <int Q, int NP>
__global__ __launch_bounds__(4 * Q) void ssd_local_kernel(ChunkArgs a, msa_seq_batch b) {
  constexpr int kBS = NP + 8, kWaves = Q / 16;
  extern __shared__ __align__(16) bf16_t sm[];
  bf16_t* Bs = sm;                                  // [Q][kBS]
  bf16_t* xs = Bs + Q * kBS;                        // [Q][kXS]
  float* ws = reinterpret_cast<float*>(xs + Q * kXS);
  float* acs = ws + Q;
  const int head = blockIdx.x % a.H, p0 = blockIdx.x / a.H * kPB, s = blockIdx.z;
  const int lo = b.cu[s], n_tok = b.cu[s + 1] - lo, t0 = blockIdx.y * Q;
  if (t0 >= n_tok) return;
  const int rows = min(Q, n_tok - t0), row0 = lo + t0;
  const int grp = head / (a.H / a.G), inner = a.H * a.P;
  const bf16_t* src = a.xbc + (int64_t)row0 * a.xbc_stride;
  RowTile<Q, NP, 4 * Q> tb;
  RowTile<Q, kPB, 4 * Q> tx;
  tb.load(src + inner + grp * a.N, a.xbc_stride, rows, a.N);
  tx.load(src + head * a.P + p0, a.xbc_stride, rows, a.P - p0);
  chunk_decays<Q>(a, row0, rows, head, ws, acs);
  tb.store(Bs, kBS);
  tx.store(xs, kXS);
  const float a_end = acs[Q - 1];
  if (threadIdx.x < Q) ws[threadIdx.x] *= __builtin_amdgcn_exp2f(a_end - acs[threadIdx.x]);
  __syncthreads();
  const int64_t chunk = ((int64_t)s * a.n_chunks + blockIdx.y) * a.H + head;
  if (threadIdx.x == 0 && p0 == 0) a.chunk_decay[chunk] = a_end;
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6, half = lane >> 5, l16 = lane & 15;
  float* out = a.chunk_state + chunk * a.N * a.P;
  for (int tile = wave; tile < NP / 32 * 2; tile += kWaves) {
    const int n0 = tile / 2 * 32, pb = tile % 2 * 32;
    if (n0 >= a.N || p0 + pb >= a.P) continue;
    floatx16_t acc;
#pragma unroll
    for (int e = 0; e < 16; ++e) acc[e] = 0.f;
    const int r = 8 * half + (l16 >> 2), c = (lane & 16) + (l16 & 3) * 4;
#pragma unroll
    for (int kk = 0; kk < Q; kk += 16) {
      const bf16x8_t bf = read_tr8(Bs + (kk + r) * kBS + n0 + c, 4 * kBS);
      const bf16x8_t xf = read_tr8(xs + (kk + r) * kXS + pb + c, 4 * kXS);
      const uint4 xw = __builtin_bit_cast(uint4, xf);
      const float4 w0 = *reinterpret_cast<const float4*>(ws + kk + 8 * half), w1 = *reinterpret_cast<const float4*>(ws + kk + 8 * half + 4);
      const float sx[8] = {bf16lo(xw.x) * w0.x, bf16hi(xw.x) * w0.y, bf16lo(xw.y) * w0.z, bf16hi(xw.y) * w0.w,
                           bf16lo(xw.z) * w1.x, bf16hi(xw.z) * w1.y, bf16lo(xw.w) * w1.z, bf16hi(xw.w) * w1.w};
      bf16x8_t hi, low;
      split8(sx, hi, low);
      acc = __builtin_amdgcn_mfma_f32_32x32x16_bf16(bf, hi, acc, 0, 0, 0);
      acc = __builtin_amdgcn_mfma_f32_32x32x16_bf16(bf, low, acc, 0, 0, 0);
    }
    const int p = p0 + pb + (lane & 31);
    if (p < a.P)
#pragma unroll
      for (int e = 0; e < 16; ++e) {
        const int n = n0 + 8 * (e >> 2) + 4 * half + (e & 3);
        if (n < a.N) out[(int64_t)n * a.P + p] = acc[e];
      }
  }
}

__device__ __forceinline__ float pack_split(float v) {
  const uint32_t hi = f32_to_bf16(v);
  const uint32_t low = f32_to_bf16(v - bf16_to_f32((bf16_t)hi));
  return __uint_as_float(hi | (low << 16));
}

// Four state elements per thread (N P is a multiple of 8).
__global__ __launch_bounds__(256) void ssd_carry_kernel(ChunkArgs a, msa_seq_batch b, int32_t Q) {
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
      d[k] = a.chunk_decay[chunk];
    }
#pragma unroll
    for (int k = 0; k < kBatch; ++k) {
      if (c + k >= chunks) break;
      *at[k] = make_float4(pack_split(S.x), pack_split(S.y), pack_split(S.z), pack_split(S.w));
      const float f = __builtin_amdgcn_exp2f(d[k]);
      S = make_float4(f * S.x + loc[k].x, f * S.y + loc[k].y, f * S.z + loc[k].z, f * S.w + loc[k].w);
    }
  }
  *keep = S;
}

template <int Q, int NP>
__global__ __launch_bounds__(4 * Q) void ssd_output_kernel(ChunkArgs a, msa_seq_batch b) {
  constexpr int kBS = NP + 8;
  extern __shared__ __align__(16) bf16_t sm[];
  bf16_t* Bs = sm;                                  // [Q][kBS]
  bf16_t* Cs = Bs + Q * kBS;                        // [Q][kBS]
  bf16_t* xs = Cs + Q * kBS;                        // [Q][kXS]
  bf16_t* Sh = xs + Q * kXS;                        // [NP][kXS] high parts of S_in
  bf16_t* Sl = Sh + NP * kXS;                       // [NP][kXS] low parts
  float* dts = reinterpret_cast<float*>(Sl + NP * kXS);
  float* acs = dts + Q;
  const int head = blockIdx.x % a.H, p0 = blockIdx.x / a.H * kPB, s = blockIdx.z;
  const int lo = b.cu[s], n_tok = b.cu[s + 1] - lo, t0 = blockIdx.y * Q;
  if (t0 >= n_tok) return;
  const int rows = min(Q, n_tok - t0), row0 = lo + t0;
  const int grp = head / (a.H / a.G), inner = a.H * a.P;
  const bf16_t* src = a.xbc + (int64_t)row0 * a.xbc_stride;
  RowTile<Q, NP, 4 * Q> tileB, tileC;
  RowTile<Q, kPB, 4 * Q> tileX;
  tileB.load(src + inner + grp * a.N, a.xbc_stride, rows, a.N);
  tileC.load(src + inner + (a.G + grp) * a.N, a.xbc_stride, rows, a.N);
  tileX.load(src + head * a.P + p0, a.xbc_stride, rows, a.P - p0);
  const int64_t chunk = ((int64_t)s * a.n_chunks + blockIdx.y) * a.H + head;
  constexpr int kSPieces = NP * (kPB / 4) / (4 * Q);
  uint4 sw[kSPieces];
  {
    const uint32_t* packed = reinterpret_cast<const uint32_t*>(a.chunk_state + chunk * a.N * a.P) + p0;
#pragma unroll
    for (int k = 0; k < kSPieces; ++k) {
      const int i = threadIdx.x + k * 4 * Q, n = i / (kPB / 4), p = i % (kPB / 4) * 4;
      sw[k] = make_uint4(0, 0, 0, 0);
      if (n < a.N && p0 + p < a.P) sw[k] = *reinterpret_cast<const uint4*>(packed + (int64_t)n * a.P + p);
    }
  }
  chunk_decays<Q>(a, row0, rows, head, dts, acs);
  tileB.store(Bs, kBS);
  tileC.store(Cs, kBS);
  tileX.store(xs, kXS);
#pragma unroll
  for (int k = 0; k < kSPieces; ++k) {
    const int i = threadIdx.x + k * 4 * Q, n = i / (kPB / 4), p = i % (kPB / 4) * 4;
    const uint4 w = sw[k];
    *reinterpret_cast<uint2*>(Sh + n * kXS + p) = make_uint2((w.x & 0xffffu) | (w.y << 16), (w.z & 0xffffu) | (w.w << 16));
    *reinterpret_cast<uint2*>(Sl + n * kXS + p) = make_uint2((w.x >> 16) | (w.y & 0xffff0000u), (w.z >> 16) | (w.w & 0xffff0000u));
  }
  __syncthreads();
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6, half = lane >> 5, l16 = lane & 15, l32 = lane & 31;
  const int tb = wave >> 1, pb = wave % 2 * 32;
  if (p0 + pb >= a.P || tb * 32 >= rows) return;
  const int t = tb * 32 + l32;
  const float a_t = acs[t];
  const int r = l16 >> 2, c = (lane & 16) + (l16 & 3) * 4;
  floatx16_t acc;
#pragma unroll
  for (int e = 0; e < 16; ++e) acc[e] = 0.f;
  bf16x8_t cf[NP / 16];
#pragma unroll
  for (int kk = 0; kk < NP / 16; ++kk) {
    cf[kk] = *reinterpret_cast<const bf16x8_t*>(Cs + t * kBS + kk * 16 + 8 * half);
    const int at = (kk * 16 + 8 * half + r) * kXS + pb + c;
    acc = __builtin_amdgcn_mfma_f32_32x32x16_bf16(read_tr8(Sh + at, 4 * kXS), cf[kk], acc, 0, 0, 0);
    acc = __builtin_amdgcn_mfma_f32_32x32x16_bf16(read_tr8(Sl + at, 4 * kXS), cf[kk], acc, 0, 0, 0);
  }
  const float in = __builtin_amdgcn_exp2f(a_t);
#pragma unroll
  for (int e = 0; e < 16; ++e) acc[e] *= in;
  for (int sb = 0; sb <= tb; ++sb) {
    floatx16_t g;
#pragma unroll
    for (int e = 0; e < 16; ++e) g[e] = 0.f;
#pragma unroll
    for (int kk = 0; kk < NP / 16; ++kk) {
      const bf16x8_t bf = *reinterpret_cast<const bf16x8_t*>(Bs + (sb * 32 + l32) * kBS + kk * 16 + 8 * half);
      g = __builtin_amdgcn_mfma_f32_32x32x16_bf16(bf, cf[kk], g, 0, 0, 0);
    }
#pragma unroll
    for (int j = 0; j < 2; ++j) {
      float m[8];
#pragma unroll
      for (int q = 0; q < 2; ++q) {
        const int s0 = sb * 32 + 16 * j + 8 * q + 4 * half;
        const float4 as = *reinterpret_cast<const float4*>(acs + s0), ds = *reinterpret_cast<const float4*>(dts + s0);
        const float av[4] = {as.x, as.y, as.z, as.w}, dv[4] = {ds.x, ds.y, ds.z, ds.w};
#pragma unroll
        for (int x = 0; x < 4; ++x) m[4 * q + x] = s0 + x <= t ? g[8 * j + 4 * q + x] * (__builtin_amdgcn_exp2f(a_t - av[x]) * dv[x]) : 0.f;
      }
      bf16x8_t hi, low;
      split8(m, hi, low);
      const bf16x8_t xf = read_tr8(xs + (sb * 32 + 16 * j + 4 * half + r) * kXS + pb + c, 8 * kXS);
      acc = __builtin_amdgcn_mfma_f32_32x32x16_bf16(xf, hi, acc, 0, 0, 0);
      acc = __builtin_amdgcn_mfma_f32_32x32x16_bf16(xf, low, acc, 0, 0, 0);
    }
  }
  // acc[e] is y of token t, column pb + 8 (e / 4) + 4 half + e % 4
  if (t >= rows) return;
  const float Dh = a.D[head];
  const int64_t row = row0 + t;
#pragma unroll
  for (int q = 0; q < 4; ++q) {
    const int p = pb + 8 * q + 4 * half;
    if (p0 + p >= a.P) continue;
    float xv[4], zv[4], y[4];
    load_vec<bf16_t, 4>(xs + t * kXS + p, xv);
    load_vec<bf16_t, 4>(a.z + row * a.z_stride + head * a.P + p0 + p, zv);
#pragma unroll
    for (int x = 0; x < 4; ++x) y[x] = (acc[4 * q + x] + Dh * xv[x]) * silu_f(zv[x]);
    store_vec<bf16_t, 4>(a.v + row * inner + head * a.P + p0 + p, y);
  }
}

int chunk_tokens(int32_t N) { return N <= 128 ? 128 : 64; }

template <int Q, int NP>
int launch_chunked(const ChunkArgs& a, const msa_seq_batch& b, hipStream_t st) {
  constexpr int lds1 = Q * (NP + 8 + kXS) * 2 + 2 * Q * 4;
  constexpr int lds3 = (2 * Q * (NP + 8) + (Q + 2 * NP) * kXS) * 2 + 2 * Q * 4;
  static_assert(lds3 <= 160 * 1024, "tiles of a chunk must fit LDS");
  static std::atomic<int> raised1{0}, raised3{0};
  MSA_HIP(raise_dynamic_lds_limit(raised1, reinterpret_cast<const void*>(ssd_local_kernel<Q, NP>), lds1));
  MSA_HIP(raise_dynamic_lds_limit(raised3, reinterpret_cast<const void*>(ssd_output_kernel<Q, NP>), lds3));
  const dim3 grid((unsigned)(a.H * ((a.P + kPB - 1) / kPB)), a.n_chunks, b.n_seq);
  ssd_local_kernel<Q, NP><<<grid, 4 * Q, lds1, st>>>(a, b);
  MSA_LAUNCH_CHECK();
  ssd_carry_kernel<<<dim3((a.N * a.P / 4 + 255) / 256, a.H, b.n_seq), 256, 0, st>>>(a, b, Q);
  MSA_LAUNCH_CHECK();
  ssd_output_kernel<Q, NP><<<grid, 4 * Q, lds3, st>>>(a, b);
  MSA_LAUNCH_CHECK();
  return MSA_OK;
}

}  // namespace

extern "C" size_t msa_seq_ssd_chunked_workspace_bytes(int32_t max_rows, int32_t n_seq, int32_t H, int32_t P, int32_t N) {
  if (max_rows <= 0 || n_seq <= 0 || H <= 0 || P <= 0 || N <= 0) return 0;
  const int Q = chunk_tokens(N);
  return (size_t)n_seq * ((max_rows + Q - 1) / Q) * H * ((size_t)N * P + 1) * sizeof(float);
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
  MSA_REQUIRE(xbc_stride >= (int64_t)H * P + 2LL * G * N && z_stride >= (int64_t)H * P && dt_stride >= H && xbc_stride % 8 == 0 &&
                  z_stride % 4 == 0 && (((uintptr_t)xbc | (uintptr_t)workspace | (uintptr_t)state) & 15) == 0 &&
                  (((uintptr_t)z | (uintptr_t)v) & 7) == 0, "msa_seq_ssd_chunked: strides or alignment");
  const int Q = chunk_tokens(N), chunks = (batch->max_rows + Q - 1) / Q;
  MSA_REQUIRE(chunks <= 65535 && batch->n_seq <= 65535, "msa_seq_ssd_chunked: step too large");
  if (workspace_bytes < msa_seq_ssd_chunked_workspace_bytes(batch->max_rows, batch->n_seq, H, P, N)) {
    msa_set_error("msa_seq_ssd_chunked: workspace of %zu bytes is too small", workspace_bytes);
    return MSA_ESIZE;
  }
  float* states = static_cast<float*>(workspace);
  const ChunkArgs a{(const bf16_t*)xbc, (const bf16_t*)z, (const bf16_t*)dt_raw, dt_bias, A_log, D, state, (bf16_t*)v, states,
                    states + (int64_t)batch->n_seq * chunks * H * N * P, xbc_stride, z_stride, dt_stride, H, P, N, G, chunks};
  hipStream_t st = as_stream(stream);
  if (N <= 32) return launch_chunked<128, 32>(a, *batch, st);
  if (N <= 64) return launch_chunked<128, 64>(a, *batch, st);
  if (N <= 128) return launch_chunked<128, 128>(a, *batch, st);
  return launch_chunked<64, 256>(a, *batch, st);
}
