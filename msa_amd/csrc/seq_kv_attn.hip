// Grouped-query attention over cached keys and values: what prepares queries, keys and values (norms, rotation, cache rows), and
// the forms for decoding and short portions.  (Long bf16 portions go through flash_sink_kernel of seq_attn.hip, straight over
// the caches.)
//   qk_rope_append_kernel  a workgroup per row; L lanes per head, eight dimensions a lane (or a wavefront per head, any sizes)
//   kv_attn_kernel         any sizes and type: a workgroup per (row, head), fp32 arithmetic throughout
//   kv_split_kernel        bf16: a workgroup per (row, key head, range of keys).  Its wavefronts take key ranges of their own and
//                          work without a barrier: scores S^T = K Q^T straight from the rows in registers, whose accumulator
//                          layout is the operand layout of O^T = V^T P^T; only V passes LDS, to be transposed.
#include <algorithm>

#include "seq_mfma.h"

namespace {

constexpr float kNoScore = -1e30f;       // below every score, and finite

// First key position `pos` sees.
__device__ __forceinline__ int64_t first_key(int64_t pos, int32_t chunk) { return chunk ? pos / chunk * chunk : 0; }

// ------------------------------------------------------------------------------------------------ preparation
constexpr int kMaxPairs = 256;

// cos and sin of position * freq for every pair.  The angle is reduced to an eighth of a turn in fp64, so that its error does not
// grow with the position; there the Taylor series are exact to fp32.
__device__ __forceinline__ float2 cos_sin(double angle) {
  const double t = angle * 0.63661977236758134308, n = rint(t);          // quarter turns
  const float x = (float)((t - n) * 1.57079632679489661923), s = x * x;
  const float sn = x * (1.f + s * (-1.6666667e-1f + s * (8.3333333e-3f + s * (-1.9841270e-4f + s * 2.7557319e-6f))));
  const float cn = 1.f + s * (-0.5f + s * (4.1666667e-2f + s * (-1.3888889e-3f + s * (2.4801587e-5f - s * 2.7557319e-7f))));
  const int quarter = (int)(n - 4.0 * floor(n * 0.25));
  const float c = quarter & 1 ? sn : cn, v = quarter & 1 ? cn : sn;
  return make_float2(quarter == 1 || quarter == 2 ? -c : c, quarter >= 2 ? -v : v);
}
__device__ __forceinline__ void rotation_table(float2* cs, const double* freqs, int32_t n_pairs, int64_t pos) {
  for (int i = threadIdx.x; i < n_pairs; i += 256) cs[i] = cos_sin((double)pos * freqs[i]);
  __syncthreads();
}

template <typename T, int LANES>
__global__ __launch_bounds__(256) void qk_rope_append_vec_kernel(msa_qk_rope_args a, msa_seq_batch b) {
  __shared__ float2 cs[kMaxPairs];
  constexpr int kHeads = 256 / LANES;
  const int row = blockIdx.x, s = b.row_seq[row];
  const int64_t pos = b.pos[s] + (row - b.cu[s]);
  const int lane = threadIdx.x % LANES, d = lane * 8, half = a.n_pairs / 8;
  const int heads = a.H + (a.k ? a.G : 0);
  const int64_t cache_row = (int64_t)b.slot[s] * a.Lcap + pos;
  const int h_first = blockIdx.y * kHeads, h_step = gridDim.y * kHeads;
  float x[8], w[8];
  auto fetch = [&](int h0) {
    // (lanes without a head or dimensions read some other's and count nothing)
    const int h = min(h0 + (int)threadIdx.x / LANES, heads - 1), at = d < a.D ? d : 0;
    const bool query = h < a.H;
    const T* src = query ? static_cast<const T*>(a.q) + row * a.q_stride + (int64_t)h * a.D
                         : static_cast<const T*>(a.k) + row * a.k_stride + (int64_t)(h - a.H) * a.D;
    load_vec<T, 8>(src + at, x);
    load_vec<float, 8>((query ? a.q_norm : a.k_norm) + at, w);
  };
  fetch(h_first);                        // (on its way while the table is made)
  rotation_table(cs, a.freqs, a.n_pairs, pos);
  for (int h0 = h_first; h0 < heads; h0 += h_step) {
    const int h = h0 + threadIdx.x / LANES;
    const bool query = h < a.H, in = h < heads && d < a.D;
    if (h0 != h_first) fetch(h0);
    float ssq = 0.f;
#pragma unroll
    for (int e = 0; e < 8; ++e) ssq += in ? x[e] * x[e] : 0.f;
#pragma unroll
    for (int o = LANES / 2; o > 0; o >>= 1) ssq += __shfl_xor(ssq, o);
    const float inv = 1.0f / sqrtf(ssq / (float)a.D + a.eps);
#pragma unroll
    for (int e = 0; e < 8; ++e) x[e] *= inv * w[e];
    if (a.n_pairs > 0) {
      // lanes 0 .. half - 1 hold the first members of the pairs, the next `half` lanes the second ones
      const int base = (threadIdx.x & 63) - lane, partner = lane < half ? lane + half : lane < 2 * half ? lane - half : lane;
      const float sign = lane < half ? -1.f : 1.f;
      const bool turned = lane < 2 * half;
#pragma unroll
      for (int e = 0; e < 8; ++e) {
        const float y = __shfl(x[e], base + partner);
        const float2 c = turned ? cs[(lane < half ? lane : lane - half) * 8 + e] : make_float2(1.f, 0.f);
        x[e] = x[e] * c.x + sign * y * c.y;
      }
    }
    if (!in) continue;
    T* dst = query ? static_cast<T*>(a.q_out) + ((int64_t)row * a.H + h) * a.D
                   : static_cast<T*>(a.k_cache) + (cache_row * a.G + (h - a.H)) * a.D;
    if (query || pos < a.Lcap) store_vec<T, 8>(dst + d, x);
  }
  if (a.k && pos < a.Lcap)
    for (int i = (blockIdx.y * 256 + threadIdx.x) * 8; i < a.G * a.E; i += gridDim.y * 256 * 8) {
      float v[8];
      load_vec<T, 8>(static_cast<const T*>(a.v) + row * a.v_stride + i, v);
      store_vec<T, 8>(static_cast<T*>(a.v_cache) + cache_row * a.G * a.E + i, v);
    }
}

template <typename T>
__global__ __launch_bounds__(256) void qk_rope_append_kernel(msa_qk_rope_args a, msa_seq_batch b) {
  __shared__ float2 cs[kMaxPairs];
  __shared__ float normed[4][512];
  const int row = blockIdx.x, s = b.row_seq[row];
  const int64_t pos = b.pos[s] + (row - b.cu[s]);
  rotation_table(cs, a.freqs, a.n_pairs, pos);
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
  const int heads = a.H + (a.k ? a.G : 0);
  const int64_t cache_row = (int64_t)b.slot[s] * a.Lcap + pos;
  float* n = normed[wave];
  for (int h0 = 0; h0 < heads; h0 += 4) {
    const int h = h0 + wave;
    const bool live = h < heads, query = h < a.H;
    if (live) {
      const T* src = query ? static_cast<const T*>(a.q) + row * a.q_stride + (int64_t)h * a.D
                           : static_cast<const T*>(a.k) + row * a.k_stride + (int64_t)(h - a.H) * a.D;
      const float* w = query ? a.q_norm : a.k_norm;
      float ssq = 0.f;
      for (int i = lane; i < a.D; i += 64) {
        const float x = to_f32<T>(src[i]);
        ssq += x * x;
      }
#pragma unroll
      for (int o = 32; o > 0; o >>= 1) ssq += __shfl_xor(ssq, o);
      const float inv = 1.0f / sqrtf(ssq / (float)a.D + a.eps);
      for (int i = lane; i < a.D; i += 64) n[i] = to_f32<T>(src[i]) * inv * w[i];
    }
    __syncthreads();
    if (live && (query || pos < a.Lcap)) {
      T* dst = query ? static_cast<T*>(a.q_out) + ((int64_t)row * a.H + h) * a.D
                     : static_cast<T*>(a.k_cache) + (cache_row * a.G + (h - a.H)) * a.D;
      for (int i = lane; i < a.D; i += 64) {
        float x = n[i];
        if (i < a.n_pairs) x = x * cs[i].x - n[i + a.n_pairs] * cs[i].y;
        else if (i < 2 * a.n_pairs) x = x * cs[i - a.n_pairs].x + n[i - a.n_pairs] * cs[i - a.n_pairs].y;
        dst[i] = from_f32<T>(x);
      }
    }
    __syncthreads();
  }
  if (a.k && pos < a.Lcap)
    for (int i = threadIdx.x; i < a.G * a.E; i += 256)
      static_cast<T*>(a.v_cache)[cache_row * a.G * a.E + i] = static_cast<const T*>(a.v)[row * a.v_stride + i];
}

template <typename T>
int launch_prepare(const msa_qk_rope_args& a, const msa_seq_batch& b, hipStream_t st) {
  const bool vec = vec_ok(8, {a.q, a.k, a.v, a.q_norm, a.k_norm, a.q_out, a.k_cache, a.v_cache},
                          {a.q_stride, a.k ? a.k_stride : 0, a.k ? a.v_stride : 0, a.D, a.E, a.n_pairs});
  // few rows: a workgroup per set of heads
  auto grid = [&](int lanes) {
    const int heads = a.H + (a.k ? a.G : 0), per = 256 / lanes;
    return dim3(b.rows, b.rows <= device_compute_units() ? (heads + per - 1) / per : 1);
  };
  if (!vec) qk_rope_append_kernel<T><<<b.rows, 256, 0, st>>>(a, b);
  else if (a.D <= 64) qk_rope_append_vec_kernel<T, 8><<<grid(8), 256, 0, st>>>(a, b);
  else if (a.D <= 128) qk_rope_append_vec_kernel<T, 16><<<grid(16), 256, 0, st>>>(a, b);
  else qk_rope_append_vec_kernel<T, 64><<<grid(64), 256, 0, st>>>(a, b);
  MSA_LAUNCH_CHECK();
  return MSA_OK;
}

// ------------------------------------------------------------------------------------------------ any sizes and type
constexpr int kMaxCols = 4;              // values up to 256 * kMaxCols dimensions

template <typename T>
__global__ __launch_bounds__(256) void kv_attn_kernel(msa_kv_attn_args a, msa_seq_batch b) {
  extern __shared__ float qs[];          // [D], then 64 scores
  float* sc = qs + a.D;
  const int row = blockIdx.x, head = blockIdx.y, tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
  const int s = b.row_seq[row], kvh = head / (a.H / a.G);
  const int64_t pos = b.pos[s] + (row - b.cu[s]), lo = first_key(pos, a.chunk);
  const T* kc = static_cast<const T*>(a.k_cache) + ((int64_t)b.slot[s] * a.Lcap * a.G + kvh) * a.D;
  const T* vc = static_cast<const T*>(a.v_cache) + ((int64_t)b.slot[s] * a.Lcap * a.G + kvh) * a.E;
  const int64_t ks = (int64_t)a.G * a.D, vs = (int64_t)a.G * a.E;
  const T* q = static_cast<const T*>(a.q) + ((int64_t)row * a.H + head) * a.D;
  for (int i = tid; i < a.D; i += 256) qs[i] = to_f32<T>(q[i]);
  float m = kNoScore, l = 0.f, acc[kMaxCols] = {};
  __syncthreads();
  for (int64_t k0 = lo; k0 <= pos; k0 += 64) {
    const int nk = (int)min((int64_t)64, pos + 1 - k0);
    for (int j = wave; j < nk; j += 4) {
      float d = 0.f;
      for (int i = lane; i < a.D; i += 64) d += qs[i] * to_f32<T>(kc[(k0 + j) * ks + i]);
#pragma unroll
      for (int o = 32; o > 0; o >>= 1) d += __shfl_xor(d, o);
      if (lane == 0) sc[j] = d * a.scale;
    }
    __syncthreads();
    const float mine = lane < nk ? sc[lane] : -INFINITY;
    float mx = mine;
#pragma unroll
    for (int o = 32; o > 0; o >>= 1) mx = fmaxf(mx, __shfl_xor(mx, o));
    const float m_new = fmaxf(m, mx), alpha = expf(m - m_new), p = expf(mine - m_new);
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
      if (i >= a.E) break;
      float v = acc[u] * alpha;
      for (int j = 0; j < nk; ++j) v += sc[j] * to_f32<T>(vc[(k0 + j) * vs + i]);
      acc[u] = v;
    }
    __syncthreads();
  }
  float f = 1.0f / l;
  if (a.gate) f *= sigmoid_f(to_f32<T>(static_cast<const T*>(a.gate)[row * a.gate_stride + head]));
#pragma unroll
  for (int u = 0; u < kMaxCols; ++u) {
    const int i = tid + 256 * u;
    if (i < a.E) static_cast<T*>(a.out)[((int64_t)row * a.H + head) * a.E + i] = from_f32<T>(acc[u] * f);
  }
}

// ------------------------------------------------------------------------------------------------ decode
constexpr int kStepKeys = 32;            // keys of a wavefront's step
constexpr int kHeadTile = 16;            // query heads of a workgroup (of one key head)
constexpr int kMaxSplits = 64;

struct SplitArgs {
  msa_kv_attn_args a;
  float* part_o;                         // [rows, n_split, H, E]
  float* part_ml;                        // [rows, n_split, H, 2]
  float scale_log2e;
  int32_t n_split;
};

// DP / EP: D and E padded to 64, 128 or 256.
template <int DP, int EP>
__global__ __launch_bounds__(256) void kv_split_kernel(SplitArgs p, msa_seq_batch b) {
  constexpr int kVS = EP + 8, kUnits = EP / 8, kVP = kStepKeys * kUnits / 64, kK = DP / 32, kC = EP / 16;
  constexpr int kOS = EP + 4;                                    // row stride of the sums at the end
  constexpr int kBytes = kStepKeys * kVS * 2 > kHeadTile * kOS * 4 ? kStepKeys * kVS * 2 : kHeadTile * kOS * 4;
  __shared__ __align__(16) char lds[4][kBytes];
  __shared__ float ml[4][kHeadTile][2];
  const msa_kv_attn_args& a = p.a;
  const int tid = threadIdx.x, lane = tid & 63, wave = __builtin_amdgcn_readfirstlane(tid >> 6), l16 = lane & 15, g = lane >> 4;
  const int group = a.H / a.G, tiles = (group + kHeadTile - 1) / kHeadTile;
  const int split = blockIdx.x, kvh = blockIdx.y / tiles, h0 = kvh * group + blockIdx.y % tiles * kHeadTile, row = blockIdx.z;
  const int heads = min(kHeadTile, (kvh + 1) * group - h0);
  const int s = b.row_seq[row];
  const int64_t pos = b.pos[s] + (row - b.cu[s]), lo = first_key(pos, a.chunk);
  const int n_keys = (int)(pos + 1 - lo), steps = (n_keys + kStepKeys - 1) / kStepKeys;
  const int parts = p.n_split * 4, per = (steps + parts - 1) / parts, part = split * 4 + wave;
  const int first = min(steps, part * per), last = min(steps, first + per);
  const int64_t cache_row = (int64_t)b.slot[s] * a.Lcap + lo;
  const int krow = a.G * a.D * 2, vrow = a.G * a.E * 2;          // bytes between keys
  const char* kc = static_cast<const char*>(a.k_cache) + cache_row * krow + kvh * a.D * 2;
  const char* vc = static_cast<const char*>(a.v_cache) + cache_row * vrow + kvh * a.E * 2;
  bf16_t* vt = reinterpret_cast<bf16_t*>(lds[wave]);             // [32][kVS]

  // a step's rows, through buffer resources whose extent is the valid rows: rows and dimensions outside read as zero
  struct Rows { u32x4_t k[2][kK], v[kVP]; } cur, next;
  int k_at[kK], v_at[kVP];
#pragma unroll
  for (int kk = 0; kk < kK; ++kk) k_at[kk] = 32 * kk + 8 * g < a.D ? l16 * krow + (32 * kk + 8 * g) * 2 : kOutside;
#pragma unroll
  for (int i = 0; i < kVP; ++i) {
    const int at = lane + 64 * i, u = at % kUnits * 8;
    v_at[i] = u < a.E ? at / kUnits * vrow + u * 2 : kOutside;
  }
  auto fetch = [&](Rows& r, int step) {
    const int rows = step < last ? min(kStepKeys, n_keys - step * kStepKeys) : 0;
    const int64_t at = step < last ? (int64_t)step * kStepKeys : 0;
    const __amdgpu_buffer_rsrc_t rk = __builtin_amdgcn_make_buffer_rsrc(const_cast<char*>(kc + at * krow), 0, rows > 0 ? (rows - 1) * krow + a.D * 2 : 0, 0x00020000);
    const __amdgpu_buffer_rsrc_t rv = __builtin_amdgcn_make_buffer_rsrc(const_cast<char*>(vc + at * vrow), 0, rows > 0 ? (rows - 1) * vrow + a.E * 2 : 0, 0x00020000);
#pragma unroll
    for (int t = 0; t < 2; ++t)
#pragma unroll
      for (int kk = 0; kk < kK; ++kk) r.k[t][kk] = __builtin_amdgcn_raw_buffer_load_b128(rk, k_at[kk] == kOutside ? kOutside : k_at[kk] + 16 * t * krow, 0, 0);
#pragma unroll
    for (int i = 0; i < kVP; ++i) r.v[i] = __builtin_amdgcn_raw_buffer_load_b128(rv, v_at[i], 0, 0);
  };
  fetch(cur, first);
  bf16x8_t qf[kK];
  {
    const bf16_t* q = static_cast<const bf16_t*>(a.q) + ((int64_t)row * a.H + h0 + l16) * a.D + 8 * g;
#pragma unroll
    for (int kk = 0; kk < kK; ++kk) {
      const bool in = l16 < heads && 32 * kk + 8 * g < a.D;
      qf[kk] = __builtin_bit_cast(bf16x8_t, in ? *reinterpret_cast<const uint4*>(q + 32 * kk) : make_uint4(0, 0, 0, 0));
    }
  }
  floatx4_t o[kC];
#pragma unroll
  for (int c = 0; c < kC; ++c) o[c] = floatx4_t{0.f, 0.f, 0.f, 0.f};
  float m = kNoScore, l = 0.f;           // of head l16: m the same in its four lanes, l each lane's own keys
  for (int step = first; step < last; ++step) {
    fetch(next, step + 1);
    floatx4_t sc[2] = {floatx4_t{0.f, 0.f, 0.f, 0.f}, floatx4_t{0.f, 0.f, 0.f, 0.f}};
#pragma unroll
    for (int kk = 0; kk < kK; ++kk)
#pragma unroll
      for (int t = 0; t < 2; ++t)
        sc[t] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(__builtin_bit_cast(bf16x8_t, cur.k[t][kk]), qf[kk], sc[t], 0, 0, 0);
#pragma unroll
    for (int i = 0; i < kVP; ++i) {
      const int at = lane + 64 * i;
      *reinterpret_cast<u32x4_t*>(vt + at / kUnits * kVS + at % kUnits * 8) = cur.v[i];
    }
    // sc[t][e] is head l16's score of key 16 t + 4 g + e
    const int valid = n_keys - step * kStepKeys;
    float v[2][4], mx = m;
#pragma unroll
    for (int t = 0; t < 2; ++t)
#pragma unroll
      for (int e = 0; e < 4; ++e) {
        v[t][e] = 16 * t + 4 * g + e < valid ? sc[t][e] * p.scale_log2e : -INFINITY;
        mx = fmaxf(mx, v[t][e]);
      }
    mx = fmaxf(mx, __shfl_xor(mx, 16));
    mx = fmaxf(mx, __shfl_xor(mx, 32));
    if (__any(mx > m)) {
      const float alpha = __builtin_amdgcn_exp2f(m - mx);
      l *= alpha;
#pragma unroll
      for (int c = 0; c < kC; ++c)
#pragma unroll
        for (int e = 0; e < 4; ++e) o[c][e] *= alpha;
      m = mx;
    }
    uint32_t pw[4];
#pragma unroll
    for (int t = 0; t < 2; ++t)
#pragma unroll
      for (int e = 0; e < 4; e += 2) {
        const float p0 = __builtin_amdgcn_exp2f(v[t][e] - m), p1 = __builtin_amdgcn_exp2f(v[t][e + 1] - m);
        l += p0 + p1;
        pw[2 * t + e / 2] = pack_bf16x2(p0, p1);
      }
    const bf16x8_t pb = __builtin_bit_cast(bf16x8_t, make_uint4(pw[0], pw[1], pw[2], pw[3]));
    __builtin_amdgcn_fence(__ATOMIC_ACQ_REL, "wavefront");       // the rows above are in LDS before they are read back
    const bf16_t* at = vt + (4 * g + (l16 >> 2)) * kVS + (l16 & 3) * 4;
#pragma unroll
    for (int c = 0; c < kC; ++c)
      o[c] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(read_tr8(at + 16 * c, 16 * kVS), pb, o[c], 0, 0, 0);
    __builtin_amdgcn_fence(__ATOMIC_ACQ_REL, "wavefront");
    cur = next;
  }
  // o[c][e] belongs to head l16, column 16 c + 4 g + e.  The four wavefronts' sums meet in LDS.
  l += __shfl_xor(l, 16);
  l += __shfl_xor(l, 32);
  __syncthreads();
  float* os = reinterpret_cast<float*>(lds[wave]);               // [16][kOS]
#pragma unroll
  for (int c = 0; c < kC; ++c) *reinterpret_cast<floatx4_t*>(os + l16 * kOS + 16 * c + 4 * g) = o[c];
  if (g == 0) {
    ml[wave][l16][0] = m;
    ml[wave][l16][1] = l;
  }
  __syncthreads();
  const bool whole = p.n_split == 1;
  for (int i = tid; i < heads * (EP / 4); i += 256) {
    const int h = i / (EP / 4), c = i % (EP / 4) * 4;
    if (c >= a.E) continue;
    float mm = kNoScore, ll = 0.f, w[4];
#pragma unroll
    for (int k = 0; k < 4; ++k) mm = fmaxf(mm, ml[k][h][0]);
#pragma unroll
    for (int k = 0; k < 4; ++k) {
      w[k] = __builtin_amdgcn_exp2f(ml[k][h][0] - mm);
      ll += w[k] * ml[k][h][1];
    }
    float r[4] = {};
#pragma unroll
    for (int k = 0; k < 4; ++k) {
      const float4 x = *reinterpret_cast<const float4*>(reinterpret_cast<const float*>(lds[k]) + h * kOS + c);
      r[0] += w[k] * x.x;
      r[1] += w[k] * x.y;
      r[2] += w[k] * x.z;
      r[3] += w[k] * x.w;
    }
    if (whole) {
      float f = 1.0f / ll;
      if (a.gate) f *= sigmoid_f(bf16_to_f32(static_cast<const bf16_t*>(a.gate)[row * a.gate_stride + h0 + h]));
#pragma unroll
      for (int e = 0; e < 4; ++e) r[e] *= f;
      store_vec<bf16_t, 4>(static_cast<bf16_t*>(a.out) + ((int64_t)row * a.H + h0 + h) * a.E + c, r);
    } else {
      const int64_t at = ((int64_t)row * p.n_split + split) * a.H + h0 + h;
      store_vec<float, 4>(p.part_o + at * a.E + c, r);
      if (c == 0) {
        p.part_ml[at * 2] = mm;
        p.part_ml[at * 2 + 1] = ll;
      }
    }
  }
}

// A wavefront per (row, head): folds the key ranges and applies the gate.
__global__ __launch_bounds__(256) void kv_combine_kernel(SplitArgs p, int64_t items) {
  const msa_kv_attn_args& a = p.a;
  const int64_t item = (int64_t)blockIdx.x * 4 + (threadIdx.x >> 6);
  if (item >= items) return;
  const int lane = threadIdx.x & 63, head = (int)(item % a.H);
  const int64_t row = item / a.H, first = row * p.n_split * a.H + head;
  float m = kNoScore, l = 0.f;
  if (lane < p.n_split) {
    const float2 ml = *reinterpret_cast<const float2*>(p.part_ml + (first + (int64_t)lane * a.H) * 2);
    m = ml.x;
    l = ml.y;
  }
  float mm = m;
#pragma unroll
  for (int o = 32; o > 0; o >>= 1) mm = fmaxf(mm, __shfl_xor(mm, o));
  const float w = __builtin_amdgcn_exp2f(m - mm);                // (a range without keys: its sums are zero)
  l *= w;
#pragma unroll
  for (int o = 32; o > 0; o >>= 1) l += __shfl_xor(l, o);
  float f = 1.0f / l;
  if (a.gate) f *= sigmoid_f(bf16_to_f32(static_cast<const bf16_t*>(a.gate)[row * a.gate_stride + head]));
  for (int c = lane * 4; c < a.E; c += 256) {
    float r[4] = {};
    constexpr int kBatch = 8;                                    // ranges requested at a time
    for (int i0 = 0; i0 < p.n_split; i0 += kBatch) {
      float x[kBatch][4];
#pragma unroll
      for (int i = 0; i < kBatch; ++i) load_vec<float, 4>(p.part_o + (first + (int64_t)min(i0 + i, p.n_split - 1) * a.H) * a.E + c, x[i]);
#pragma unroll
      for (int i = 0; i < kBatch; ++i) {                         // (lanes without columns hold weights too, 0 behind the last range)
        const float wi = __uint_as_float(__builtin_amdgcn_readlane(__float_as_uint(w), min(i0 + i, 63)));
#pragma unroll
        for (int e = 0; e < 4; ++e) r[e] += i0 + i < p.n_split ? wi * x[i][e] : 0.f;
      }
    }
#pragma unroll
    for (int e = 0; e < 4; ++e) r[e] *= f;
    store_vec<bf16_t, 4>(static_cast<bf16_t*>(a.out) + item * a.E + c, r);
  }
}

// Ranges per row: two workgroups per compute unit, at least two steps per wavefront.
int kv_splits(const msa_kv_attn_args& a, int32_t rows) {
  const int64_t span = std::max<int64_t>(1, a.chunk > 0 ? std::min<int64_t>(a.chunk, a.max_keys) : a.max_keys);
  const int64_t steps = (span + kStepKeys - 1) / kStepKeys;
  const int64_t blocks = (int64_t)rows * a.G * ((a.H / a.G + kHeadTile - 1) / kHeadTile);
  return (int)std::min<int64_t>(std::min<int64_t>(kMaxSplits, (steps + 7) / 8), std::max<int64_t>(1, (2 * device_compute_units() + blocks - 1) / blocks));
}

template <int DP, int EP>
int launch_split(const SplitArgs& p, const msa_seq_batch& b, hipStream_t st) {
  const msa_kv_attn_args& a = p.a;
  const int tiles = (a.H / a.G + kHeadTile - 1) / kHeadTile;
  kv_split_kernel<DP, EP><<<dim3(p.n_split, a.G * tiles, b.rows), 256, 0, st>>>(p, b);
  MSA_LAUNCH_CHECK();
  if (p.n_split > 1) {
    const int64_t items = (int64_t)b.rows * a.H;
    kv_combine_kernel<<<(unsigned)((items + 3) / 4), 256, 0, st>>>(p, items);
    MSA_LAUNCH_CHECK();
  }
  return MSA_OK;
}

int check_kv(const msa_kv_attn_args* a, const char* who) {
  MSA_REQUIRE(a && a->q && a->k_cache && a->v_cache && a->out && a->Lcap > 0 && a->chunk >= 0, "%s: null pointer or chunk < 0", who);
  MSA_REQUIRE(a->H > 0 && a->G > 0 && a->H % a->G == 0 && a->H <= 65535 && a->D > 0 && a->E > 0 && (!a->gate || a->gate_stride >= a->H),
              "%s: H=%d G=%d D=%d E=%d", who, a->H, a->G, a->D, a->E);
  return MSA_OK;
}

}  // namespace

extern "C" int msa_seq_qk_rope_append(const msa_qk_rope_args* args, int32_t dtype, const msa_seq_batch* batch, void* stream) {
  MSA_CHECK_BATCH(batch, "msa_seq_qk_rope_append");
  MSA_CHECK_DTYPE(dtype, "msa_seq_qk_rope_append");
  MSA_REQUIRE(args && args->q && args->q_norm && args->q_out, "msa_seq_qk_rope_append: null pointer");
  const msa_qk_rope_args& a = *args;
  MSA_REQUIRE(a.H > 0 && a.G > 0 && a.D > 0 && a.D <= 512 && a.E > 0 && a.n_pairs >= 0 && 2 * a.n_pairs <= a.D && a.n_pairs <= kMaxPairs && (!a.n_pairs || a.freqs),
              "msa_seq_qk_rope_append: H=%d G=%d D=%d (up to 512) E=%d, %d pairs", a.H, a.G, a.D, a.E, a.n_pairs);
  MSA_REQUIRE(a.q_stride >= (int64_t)a.H * a.D, "msa_seq_qk_rope_append: query stride");
  MSA_REQUIRE(!a.k || (a.v && a.k_norm && a.k_cache && a.v_cache && a.Lcap > 0 && a.k_stride >= (int64_t)a.G * a.D && a.v_stride >= (int64_t)a.G * a.E),
              "msa_seq_qk_rope_append: key and value arguments");
  return dtype == MSA_BF16 ? launch_prepare<bf16_t>(a, *batch, as_stream(stream)) : launch_prepare<float>(a, *batch, as_stream(stream));
}

extern "C" int msa_seq_kv_attn(const msa_kv_attn_args* args, int32_t dtype, const msa_seq_batch* batch, void* stream) {
  MSA_CHECK_BATCH(batch, "msa_seq_kv_attn");
  MSA_CHECK_DTYPE(dtype, "msa_seq_kv_attn");
  const int rc = check_kv(args, "msa_seq_kv_attn");
  if (rc != MSA_OK) return rc;
  MSA_REQUIRE(args->E <= 256 * kMaxCols && args->D <= 8192, "msa_seq_kv_attn: D=%d E=%d (up to %d)", args->D, args->E, 256 * kMaxCols);
  const dim3 grid(batch->rows, args->H);
  const size_t lds = (args->D + 64) * sizeof(float);
  if (dtype == MSA_BF16) kv_attn_kernel<bf16_t><<<grid, 256, lds, as_stream(stream)>>>(*args, *batch);
  else kv_attn_kernel<float><<<grid, 256, lds, as_stream(stream)>>>(*args, *batch);
  MSA_LAUNCH_CHECK();
  return MSA_OK;
}

extern "C" size_t msa_seq_kv_decode_workspace_bytes(const msa_kv_attn_args* args, int32_t rows) {
  if (!args || rows <= 0 || args->H <= 0 || args->G <= 0 || args->E <= 0) return 0;
  const int splits = kv_splits(*args, rows);
  return splits == 1 ? 0 : (size_t)rows * splits * args->H * (args->E + 2) * sizeof(float);
}

extern "C" int msa_seq_kv_decode(const msa_kv_attn_args* args, const msa_seq_batch* batch, void* workspace, size_t workspace_bytes, void* stream) {
  MSA_CHECK_BATCH(batch, "msa_seq_kv_decode");
  const int rc = check_kv(args, "msa_seq_kv_decode");
  if (rc != MSA_OK) return rc;
  const msa_kv_attn_args& a = *args;
  MSA_REQUIRE(a.D % 8 == 0 && a.E % 8 == 0 && a.D <= 256 && a.E <= 256 && a.scale > 0.f, "msa_seq_kv_decode: D=%d E=%d (multiples of 8 up to 256), scale > 0", a.D, a.E);
  MSA_REQUIRE(batch->rows <= 65535 && a.max_keys > 0 && a.max_keys <= a.Lcap && a.Lcap < ((int64_t)1 << 31) && (int64_t)a.G * std::max(a.D, a.E) < (1 << 22),
              "msa_seq_kv_decode: %d rows, %lld keys", batch->rows, (long long)a.max_keys);
  MSA_REQUIRE((((uintptr_t)a.q | (uintptr_t)a.k_cache | (uintptr_t)a.v_cache | (uintptr_t)a.out | (uintptr_t)workspace) & 15) == 0, "msa_seq_kv_decode: alignment");
  const int64_t tiles = (a.H / a.G + kHeadTile - 1) / kHeadTile;
  MSA_REQUIRE(a.G * tiles <= 65535, "msa_seq_kv_decode: %d heads", a.H);
  const size_t need = msa_seq_kv_decode_workspace_bytes(args, batch->rows);
  if (need > workspace_bytes || (need && !workspace)) {
    msa_set_error("msa_seq_kv_decode: workspace of %zu bytes, need %zu", workspace_bytes, need);
    return MSA_ESIZE;
  }
  const int splits = kv_splits(a, batch->rows);
  float* part_o = static_cast<float*>(workspace);
  const SplitArgs p{a, part_o, splits == 1 ? nullptr : part_o + (int64_t)batch->rows * splits * a.H * a.E, a.scale * kLog2e, splits};
  hipStream_t st = as_stream(stream);
  const int big = std::max(a.D, a.E);
  if (big <= 64) return launch_split<64, 64>(p, *batch, st);
  if (big <= 128) return launch_split<128, 128>(p, *batch, st);
  return launch_split<256, 256>(p, *batch, st);
}
