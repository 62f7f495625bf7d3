// Recurrences over time: the causal convolution in front of the state-space layer, the state-space recurrence itself
// (token by token; the chunked matrix-core form is in seq_ssd.hip) and the minimal gated recurrence.
//
// A sequence's kept values (convolution inputs, states) are read and written by one thread each: the one that owns the
// channel in the workgroup of the sequence's first rows (convolution) or of the whole sequence (recurrences).
#include <algorithm>
#include <initializer_list>

#include "seq_common.h"

namespace {

// ------------------------------------------------------------------------------------------------ convolution
constexpr int kConvRows = 16;

template <typename T>
__global__ __launch_bounds__(256) void conv_silu_kernel(const T* __restrict__ in, int64_t in_stride, const float* __restrict__ taps,
                                                        const float* __restrict__ bias, int32_t C, int32_t K, float* __restrict__ state,
                                                        T* __restrict__ out, int64_t out_stride, msa_seq_batch b) {
  const int c = blockIdx.x * 256 + threadIdx.x;
  const int s = blockIdx.z;
  const int lo = b.cu[s], n = b.cu[s + 1] - lo;
  const int t0 = blockIdx.y * kConvRows;
  if (c >= C || t0 >= n) return;
  const int t1 = min(n, t0 + kConvRows);
  float* keep = state + (int64_t)b.slot[s] * (K - 1) * C + c;
  const T* src = in + (int64_t)lo * in_stride + c;
  const float* tp = taps + (int64_t)c * K;
  const float bs = bias ? bias[c] : 0.f;
  // Only the workgroup of the first rows reads the kept inputs, and only it replaces them; portions shorter than the
  // taps push them along.  (Rows t < K - 1 are in that workgroup as long as K - 1 <= kConvRows, which the host checks.)
  for (int t = t0; t < t1; ++t) {
    float acc = bs;
    for (int j = 0; j < K; ++j) {
      const int u = t - (K - 1) + j;
      acc += tp[j] * (u >= 0 ? to_f32<T>(src[u * in_stride]) : keep[(int64_t)(K - 1 + u) * C]);
    }
    out[(int64_t)(lo + t) * out_stride + c] = from_f32<T>(silu_f(acc));
  }
  if (blockIdx.y == 0)
    for (int i = 0; i < K - 1; ++i) {                      // oldest first; entry i becomes input n - (K - 1) + i
      const int u = n - (K - 1) + i;
      keep[(int64_t)i * C] = u >= 0 ? to_f32<T>(src[u * in_stride]) : keep[(int64_t)(K - 1 + u) * C];
    }
}

// The same for 2 <= K <= 5 and aligned rows: a thread owns eight channels and slides its window of K - 1 inputs along.
template <typename T, int K>
__global__ __launch_bounds__(256) void conv_silu_vec_kernel(const T* __restrict__ in, int64_t in_stride, const float* __restrict__ taps,
                                                            const float* __restrict__ bias, int32_t C, float* __restrict__ state,
                                                            T* __restrict__ out, int64_t out_stride, msa_seq_batch b) {
  const int c = (blockIdx.x * 256 + threadIdx.x) * 8;
  const int s = blockIdx.z;
  const int lo = b.cu[s], n = b.cu[s + 1] - lo;
  const int t0 = blockIdx.y * kConvRows;
  if (c >= C || t0 >= n) return;
  const int t1 = min(n, t0 + kConvRows);
  float* keep = state + (int64_t)b.slot[s] * (K - 1) * C + c;
  const T* src = in + (int64_t)lo * in_stride + c;
  float tp[K][8], bs[8] = {}, win[K - 1][8];
#pragma unroll
  for (int e = 0; e < 8; ++e)
#pragma unroll
    for (int j = 0; j < K; ++j) tp[j][e] = taps[(int64_t)(c + e) * K + j];
  if (bias) load_vec<float, 8>(bias + c, bs);
  auto input = [&](int u, float (&x)[8]) {                   // input u of the sequence's new tokens, or a kept one (u < 0)
    if (u >= 0) load_vec<T, 8>(src + u * in_stride, x);
    else load_vec<float, 8>(keep + (int64_t)(K - 1 + u) * C, x);
  };
#pragma unroll
  for (int j = 0; j < K - 1; ++j) input(t0 - (K - 1) + j, win[j]);
#pragma unroll 4
  for (int t = t0; t < t1; ++t) {
    float x[8], y[8];
    load_vec<T, 8>(src + t * in_stride, x);
#pragma unroll
    for (int e = 0; e < 8; ++e) {
      float acc = bs[e] + tp[K - 1][e] * x[e];
#pragma unroll
      for (int j = 0; j < K - 1; ++j) acc += tp[j][e] * win[j][e];
      y[e] = silu_f(acc);
#pragma unroll
      for (int j = 0; j + 1 < K - 1; ++j) win[j][e] = win[j + 1][e];
      win[K - 2][e] = x[e];
    }
    store_vec<T, 8>(out + (int64_t)(lo + t) * out_stride + c, y);
  }
  if (blockIdx.y == 0) {
    float last[K - 1][8];
#pragma unroll
    for (int i = 0; i < K - 1; ++i) input(n - (K - 1) + i, last[i]);
#pragma unroll
    for (int i = 0; i < K - 1; ++i) store_vec<float, 8>(keep + (int64_t)i * C, last[i]);
  }
}

template <typename T>
int launch_conv(const T* in, int64_t in_stride, const float* taps, const float* bias, int32_t C, int32_t K, float* state, T* out,
                int64_t out_stride, const msa_seq_batch& b, hipStream_t st) {
  const int row_blocks = (b.max_rows + kConvRows - 1) / kConvRows;
  if (K >= 2 && K <= 5 && vec_ok(8, {in, bias, state, out}, {in_stride, out_stride, C})) {
    const dim3 grid((C / 8 + 255) / 256, row_blocks, b.n_seq);
    if (K == 2) conv_silu_vec_kernel<T, 2><<<grid, 256, 0, st>>>(in, in_stride, taps, bias, C, state, out, out_stride, b);
    else if (K == 3) conv_silu_vec_kernel<T, 3><<<grid, 256, 0, st>>>(in, in_stride, taps, bias, C, state, out, out_stride, b);
    else if (K == 4) conv_silu_vec_kernel<T, 4><<<grid, 256, 0, st>>>(in, in_stride, taps, bias, C, state, out, out_stride, b);
    else conv_silu_vec_kernel<T, 5><<<grid, 256, 0, st>>>(in, in_stride, taps, bias, C, state, out, out_stride, b);
  } else {
    conv_silu_kernel<T><<<dim3((C + 255) / 256, row_blocks, b.n_seq), 256, 0, st>>>(in, in_stride, taps, bias, C, K, state, out, out_stride, b);
  }
  MSA_LAUNCH_CHECK();
  return MSA_OK;
}

// ------------------------------------------------------------------------------------------------ state-space recurrence
// A workgroup owns (sequence, head, 64 state columns): lane = column p, wavefront w holds state rows w NI .. + NI in
// registers.  A few tokens are staged at a time (B and C in LDS as fp32, read back four to an instruction): every wavefront
// adds its share of S^T C into LDS, one barrier, and all threads finish the outputs.

struct SsdArgs {
  const void* xbc;
  const void* z;
  const void* dt_raw;
  const float* dt_bias;
  const float* A_log;
  const float* D;
  float* state;
  void* v;
  int64_t xbc_stride, z_stride, dt_stride;
  int32_t H, P, N, G;
};

template <typename T, int NI, int WAVES>
__global__ __launch_bounds__(WAVES * 64) void ssd_scan_kernel(SsdArgs a, msa_seq_batch b) {
  constexpr int kRows = WAVES > 4 ? 2 : 8, kN = NI * WAVES;        // tokens per stage, state rows padded
  __shared__ float part[WAVES][kRows][64];
  __shared__ __align__(16) float bc[kRows][2][kN];
  __shared__ float dts[kRows], decays[kRows];
  const int s = blockIdx.z, head = blockIdx.y, lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
  const int p = blockIdx.x * 64 + lane;
  const bool live = p < a.P;
  const int lo = b.cu[s], n_tok = b.cu[s + 1] - lo;
  const int grp = head / (a.H / a.G), inner = a.H * a.P;
  float* st = a.state + (((int64_t)b.slot[s] * a.H + head) * a.N + wave * NI) * a.P + p;
  float S[NI];
#pragma unroll
  for (int i = 0; i < NI; ++i) S[i] = live && wave * NI + i < a.N ? st[(int64_t)i * a.P] : 0.f;
  const float rate = -expf(a.A_log[head]), bias = a.dt_bias[head], Dh = a.D[head];
  const T* xbc = static_cast<const T*>(a.xbc) + (int64_t)lo * a.xbc_stride;
  const T* dtp = static_cast<const T*>(a.dt_raw) + (int64_t)lo * a.dt_stride + head;
  for (int t0 = 0; t0 < n_tok; t0 += kRows) {
    const int rows = min(kRows, n_tok - t0);
    for (int i = threadIdx.x; i < rows * 2 * kN; i += WAVES * 64) {
      const int r = i / (2 * kN), which = i / kN & 1, n = i % kN;
      bc[r][which][n] = n < a.N ? to_f32<T>(xbc[(int64_t)(t0 + r) * a.xbc_stride + inner + (which * a.G + grp) * a.N + n]) : 0.f;
    }
    if (threadIdx.x < rows) {
      const float dt = softplus_f(to_f32<T>(dtp[(int64_t)(t0 + threadIdx.x) * a.dt_stride]) + bias);
      dts[threadIdx.x] = dt;
      decays[threadIdx.x] = expf(rate * dt);
    }
    __syncthreads();
    for (int r = 0; r < rows; ++r) {
      const float decay = decays[r];
      const float x = live ? dts[r] * to_f32<T>(xbc[(int64_t)(t0 + r) * a.xbc_stride + head * a.P + p]) : 0.f;
      float y = 0.f;
#pragma unroll
      for (int i = 0; i < NI; i += 4) {
        const float4 Bv = *reinterpret_cast<const float4*>(&bc[r][0][wave * NI + i]);
        const float4 Cv = *reinterpret_cast<const float4*>(&bc[r][1][wave * NI + i]);
        S[i] = decay * S[i] + Bv.x * x; y += S[i] * Cv.x;
        S[i + 1] = decay * S[i + 1] + Bv.y * x; y += S[i + 1] * Cv.y;
        S[i + 2] = decay * S[i + 2] + Bv.z * x; y += S[i + 2] * Cv.z;
        S[i + 3] = decay * S[i + 3] + Bv.w * x; y += S[i + 3] * Cv.w;
      }
      part[wave][r][lane] = y;
    }
    __syncthreads();
    for (int r = wave; r < rows; r += WAVES) {
      float y = 0.f;
#pragma unroll
      for (int w = 0; w < WAVES; ++w) y += part[w][r][lane];
      if (live) {
        const int64_t row = lo + t0 + r;
        y += Dh * to_f32<T>(xbc[(int64_t)(t0 + r) * a.xbc_stride + head * a.P + p]);
        y *= silu_f(to_f32<T>(static_cast<const T*>(a.z)[row * a.z_stride + head * a.P + p]));
        static_cast<T*>(a.v)[row * inner + head * a.P + p] = from_f32<T>(y);
      }
    }
  }
#pragma unroll
  for (int i = 0; i < NI; ++i)
    if (live && wave * NI + i < a.N) st[(int64_t)i * a.P] = S[i];
}

// ------------------------------------------------------------------------------------------------ minimal gated recurrence
// S_t = a_t S_(t-1) + b_t per channel.  Long portions run in chunks of kGruRows tokens: (1) every chunk's (product of a,
// last b-part), (2) the chunk-to-chunk recurrence, which leaves each chunk's incoming state, (3) the chunks again from
// their incoming states.  A portion of one chunk is phase (3) alone.
constexpr int kGruRows = 32;
constexpr int kGruGroup = 16;       // channels per group of the [16 z | 16 u | 16 g] row layout
__device__ __forceinline__ int gru_column(int c) { return (c / kGruGroup) * 3 * kGruGroup + c % kGruGroup; }

struct GruArgs {
  const void* zug;
  const float* z_bias;
  const float* u_bias;
  float* state;
  void* out;
  float2* chunk;        // [n_seq, n_chunks, n]: (product of a, b-part), then x = incoming state
  int64_t stride;
  int32_t n, n_chunks;
};

// The raw columns of a few rows of a portion, through a buffer resource whose extent is the portion's rows: nothing is
// conditional, so the compiler can count the loads in flight, and a batch is requested while the one before is worked on.
constexpr int kGruBatch = 8;
template <typename T, int VEC, int COLS>
struct GruRows {
  static constexpr int kBytes = VEC * sizeof(T);
  uint32_t v[kGruBatch][COLS][kBytes <= 4 ? 1 : kBytes / 4];
  __device__ __forceinline__ void load(__amdgpu_buffer_rsrc_t rs, int at, int stride) {
#pragma unroll
    for (int r = 0; r < kGruBatch; ++r)
#pragma unroll
      for (int k = 0; k < COLS; ++k) {
        const int off = at + r * stride + k * kGruGroup * (int)sizeof(T);
        if constexpr (kBytes == 2) v[r][k][0] = __builtin_amdgcn_raw_buffer_load_b16(rs, off, 0, 0);
        else if constexpr (kBytes == 4) v[r][k][0] = __builtin_amdgcn_raw_buffer_load_b32(rs, off, 0, 0);
        else {
          const auto w = __builtin_amdgcn_raw_buffer_load_b64(rs, off, 0, 0);
          v[r][k][0] = w[0];
          v[r][k][1] = w[1];
        }
      }
  }
  __device__ __forceinline__ float get(int r, int k, int e) const {
    if constexpr (sizeof(T) == 4) return __uint_as_float(v[r][k][e]);
    else return e == 0 ? bf16lo(v[r][k][0]) : bf16hi(v[r][k][0]);
  }
};
// keep = 1 - z and add = z * candidate, from the raw columns and the biases times -log2(e).  With ez = exp(-z_raw - z_bias) and
// eu = exp(-u) one reciprocal r = 1 / ((1 + ez) (1 + eu)) gives both: z = r (1 + eu), and z sigmoid(u) = r.  (The kernel is bound by
// instructions, the transcendental ones above all; exponents stop at 60, where a sigmoid is 1e-18.)
__device__ __forceinline__ void gru_terms(float z_raw, float u_raw, float zb, float ub, float& keep, float& add) {
  constexpr float kNegLog2e = -1.4426950408889634f, kHalfLog2e = 0.7213475204444817f, kLn2 = -0.6931471805599453f;
  const float un = fmaf(u_raw, kNegLog2e, ub);                       // -u log2(e)
  const float ez = __builtin_amdgcn_exp2f(fminf(fmaf(z_raw, kNegLog2e, zb), 60.f));
  const float q = 1.0f + __builtin_amdgcn_exp2f(fminf(un, 60.f));
  const float r = __builtin_amdgcn_rcpf((1.0f + ez) * q), z = r * q;
  keep = ez * z;
  add = un <= 0.f ? z * ((un - kHalfLog2e) * kLn2) : r;              // u + 1/2 = (un - log2(e) / 2) * -ln 2
}

template <typename T, int VEC>
__global__ __launch_bounds__(256) void gru_chunk_kernel(GruArgs a, msa_seq_batch b) {
  const int c = (blockIdx.x * 256 + threadIdx.x) * VEC, s = blockIdx.z;
  const int lo = b.cu[s], n_tok = b.cu[s + 1] - lo, t0 = blockIdx.y * kGruRows;
  if (c >= a.n || t0 >= n_tok) return;
  const int n = min(n_tok - t0, kGruRows);
  float zb[VEC], ub[VEC], A[VEC], S[VEC];
  load_vec<float, VEC>(a.z_bias + c, zb);
  load_vec<float, VEC>(a.u_bias + c, ub);
#pragma unroll
  for (int e = 0; e < VEC; ++e) zb[e] *= -1.4426950408889634f, ub[e] *= -1.4426950408889634f;
#pragma unroll
  for (int e = 0; e < VEC; ++e) A[e]  = 1.f, S[e] = 0.f;
  const int row_bytes = (int)a.stride * (int)sizeof(T);
  const __amdgpu_buffer_rsrc_t rs = __builtin_amdgcn_make_buffer_rsrc(
      const_cast<T*>(static_cast<const T*>(a.zug) + (int64_t)(lo + t0) * a.stride), 0, n * row_bytes, 0x00020000);
  int at = gru_column(c) * (int)sizeof(T);
  GruRows<T, VEC, 2> cur, next;
  cur.load(rs, at, row_bytes);
  for (int t = 0; t < n; t += kGruBatch) {
    at += kGruBatch * row_bytes;
    next.load(rs, at, row_bytes);
    const int live = n - t;
#pragma unroll
    for (int r = 0; r < kGruBatch; ++r) {
      if (r >= live) break;
#pragma unroll
      for (int e = 0; e < VEC; ++e) {
        float k, d;
        gru_terms(cur.get(r, 0, e), cur.get(r, 1, e), zb[e], ub[e], k, d);
        A[e] *= k;
        S[e] = k * S[e] + d;
      }
    }
    cur = next;
  }
  float2* dst = a.chunk + ((int64_t)s * a.n_chunks + blockIdx.y) * a.n + c;
#pragma unroll
  for (int e = 0; e < VEC; ++e) dst[e] = make_float2(A[e], S[e]);
}

__global__ __launch_bounds__(64) void gru_carry_kernel(GruArgs a, msa_seq_batch b) {
  const int c = blockIdx.x * 64 + threadIdx.x, s = blockIdx.y;
  if (c >= a.n) return;
  const int n_tok = b.cu[s + 1] - b.cu[s], chunks = (n_tok + kGruRows - 1) / kGruRows;
  float S = a.state[(int64_t)b.slot[s] * a.n + c];
  float2* ch = a.chunk + (int64_t)s * a.n_chunks * a.n + c;
  constexpr int kBatch = 32;
  for (int i = 0; i < chunks; i += kBatch) {
    float2 t[kBatch];
#pragma unroll
    for (int k = 0; k < kBatch; ++k) t[k] = ch[(int64_t)min(i + k, chunks - 1) * a.n];
#pragma unroll
    for (int k = 0; k < kBatch; ++k) {
      if (i + k >= chunks) break;
      ch[(int64_t)(i + k) * a.n].x = S;
      S = t[k].x * S + t[k].y;
    }
  }
  a.state[(int64_t)b.slot[s] * a.n + c] = S;
}

template <typename T, int VEC, bool kCarried>
__global__ __launch_bounds__(256) void gru_out_kernel(GruArgs a, msa_seq_batch b) {
  const int c = (blockIdx.x * 256 + threadIdx.x) * VEC, s = blockIdx.z;
  const int lo = b.cu[s], n_tok = b.cu[s + 1] - lo, t0 = blockIdx.y * kGruRows;
  if (c >= a.n || t0 >= n_tok) return;
  const int n = min(n_tok - t0, kGruRows);
  float zb[VEC], ub[VEC], S[VEC];
  load_vec<float, VEC>(a.z_bias + c, zb);
  load_vec<float, VEC>(a.u_bias + c, ub);
#pragma unroll
  for (int e = 0; e < VEC; ++e) zb[e] *= -1.4426950408889634f, ub[e] *= -1.4426950408889634f;
  float* st = a.state + (int64_t)b.slot[s] * a.n + c;
#pragma unroll
  for (int e = 0; e < VEC; ++e) S[e] = kCarried ? a.chunk[((int64_t)s * a.n_chunks + blockIdx.y) * a.n + c + e].x : st[e];
  const int row_bytes = (int)a.stride * (int)sizeof(T), out_bytes = a.n * (int)sizeof(T);
  const __amdgpu_buffer_rsrc_t rs = __builtin_amdgcn_make_buffer_rsrc(
      const_cast<T*>(static_cast<const T*>(a.zug) + (int64_t)(lo + t0) * a.stride), 0, n * row_bytes, 0x00020000);
  const __amdgpu_buffer_rsrc_t ro = __builtin_amdgcn_make_buffer_rsrc(static_cast<T*>(a.out) + (int64_t)(lo + t0) * a.n, 0, n * out_bytes, 0x00020000);
  int at = gru_column(c) * (int)sizeof(T), to = c * (int)sizeof(T);
  GruRows<T, VEC, 3> cur, next;
  cur.load(rs, at, row_bytes);
  for (int t = 0; t < n; t += kGruBatch, to += kGruBatch * out_bytes) {
    at += kGruBatch * row_bytes;
    next.load(rs, at, row_bytes);
    const int live = n - t;
    float ys[kGruBatch][VEC];
#pragma unroll
    for (int r = 0; r < kGruBatch; ++r) {
      if (r >= live) break;
#pragma unroll
      for (int e = 0; e < VEC; ++e) {
        float k, d;
        gru_terms(cur.get(r, 0, e), cur.get(r, 1, e), zb[e], ub[e], k, d);
        S[e] = k * S[e] + d;
        ys[r][e] = S[e] * silu_f(cur.get(r, 2, e));
      }
    }
#pragma unroll
    for (int r = 0; r < kGruBatch; ++r) {
      const float(&y)[VEC] = ys[r];
      const int off = to + r * out_bytes;                   // rows behind the portion are not written
      if constexpr (VEC == 1 && sizeof(T) == 2) __builtin_amdgcn_raw_buffer_store_b16(f32_to_bf16(y[0]), ro, off, 0, 0);
      else if constexpr (VEC == 1) __builtin_amdgcn_raw_buffer_store_b32(__float_as_uint(y[0]), ro, off, 0, 0);
      else if constexpr (sizeof(T) == 2) __builtin_amdgcn_raw_buffer_store_b32(pack_bf16x2(y[0], y[1]), ro, off, 0, 0);
      else {
        typedef unsigned int u32x2_t __attribute__((ext_vector_type(2)));
        __builtin_amdgcn_raw_buffer_store_b64(u32x2_t{__float_as_uint(y[0]), __float_as_uint(y[1])}, ro, off, 0, 0);
      }
    }
    cur = next;
  }
  if (!kCarried)
#pragma unroll
    for (int e = 0; e < VEC; ++e) st[e] = S[e];
}

template <typename T, int VEC>
int launch_gru(const GruArgs& a, const msa_seq_batch& b, hipStream_t st) {
  const dim3 grid((a.n / VEC + 255) / 256, a.n_chunks, b.n_seq);
  if (a.n_chunks > 1) {
    gru_chunk_kernel<T, VEC><<<grid, 256, 0, st>>>(a, b);
    MSA_LAUNCH_CHECK();
    gru_carry_kernel<<<dim3((a.n + 63) / 64, b.n_seq), 64, 0, st>>>(a, b);
    MSA_LAUNCH_CHECK();
    gru_out_kernel<T, VEC, true><<<grid, 256, 0, st>>>(a, b);
  } else {
    gru_out_kernel<T, VEC, false><<<grid, 256, 0, st>>>(a, b);
  }
  MSA_LAUNCH_CHECK();
  return MSA_OK;
}

template <typename T>
int launch_ssd(const SsdArgs& a, const msa_seq_batch& b, hipStream_t st) {
  const dim3 grid((a.P + 63) / 64, a.H, b.n_seq);
  if (a.N <= 16) ssd_scan_kernel<T, 4, 4><<<grid, 256, 0, st>>>(a, b);
  else if (a.N <= 32) ssd_scan_kernel<T, 8, 4><<<grid, 256, 0, st>>>(a, b);
  else if (a.N <= 64) ssd_scan_kernel<T, 16, 4><<<grid, 256, 0, st>>>(a, b);
  else if (a.N <= 128) ssd_scan_kernel<T, 32, 4><<<grid, 256, 0, st>>>(a, b);
  else if (a.N <= 256) ssd_scan_kernel<T, 64, 4><<<grid, 256, 0, st>>>(a, b);
  else ssd_scan_kernel<T, 64, 16><<<grid, 1024, 0, st>>>(a, b);
  MSA_LAUNCH_CHECK();
  return MSA_OK;
}

}  // namespace

extern "C" int msa_seq_conv_silu(const void* in, int64_t in_stride, const float* taps, const float* bias, int32_t dtype, int32_t C,
                                 int32_t K, float* state, void* out, int64_t out_stride, const msa_seq_batch* batch, void* stream) {
  MSA_CHECK_BATCH(batch, "msa_seq_conv_silu");
  MSA_CHECK_DTYPE(dtype, "msa_seq_conv_silu");
  MSA_REQUIRE(in && taps && out && C > 0 && in_stride >= C && out_stride >= C, "msa_seq_conv_silu: bad arguments");
  MSA_REQUIRE(K >= 1 && K - 1 <= kConvRows && (K == 1 || state), "msa_seq_conv_silu: K=%d (1..%d taps)", K, kConvRows + 1);
  MSA_REQUIRE(batch->n_seq <= 65535 && (batch->max_rows + kConvRows - 1) / kConvRows <= 65535, "msa_seq_conv_silu: step too large");
  if (dtype == MSA_BF16)
    return launch_conv<bf16_t>((const bf16_t*)in, in_stride, taps, bias, C, K, state, (bf16_t*)out, out_stride, *batch, as_stream(stream));
  return launch_conv<float>((const float*)in, in_stride, taps, bias, C, K, state, (float*)out, out_stride, *batch, as_stream(stream));
}

extern "C" int msa_seq_ssd_scan(const void* xbc, int64_t xbc_stride, const void* z, int64_t z_stride, const void* dt_raw,
                                int64_t dt_stride, const float* dt_bias, const float* A_log, const float* D, int32_t dtype, int32_t H,
                                int32_t P, int32_t N, int32_t G, float* state, void* v, const msa_seq_batch* batch, void* stream) {
  MSA_CHECK_BATCH(batch, "msa_seq_ssd_scan");
  MSA_CHECK_DTYPE(dtype, "msa_seq_ssd_scan");
  MSA_REQUIRE(xbc && z && dt_raw && dt_bias && A_log && D && state && v, "msa_seq_ssd_scan: null pointer");
  MSA_REQUIRE(H > 0 && H <= 65535 && P > 0 && G > 0 && H % G == 0 && N > 0 && N <= 1024 && batch->n_seq <= 65535,
              "msa_seq_ssd_scan: H=%d P=%d N=%d (up to 1024) G=%d", H, P, N, G);
  MSA_REQUIRE(xbc_stride >= (int64_t)H * P + 2LL * G * N && z_stride >= (int64_t)H * P && dt_stride >= H, "msa_seq_ssd_scan: strides");
  const SsdArgs a{xbc, z, dt_raw, dt_bias, A_log, D, state, v, xbc_stride, z_stride, dt_stride, H, P, N, G};
  return dtype == MSA_BF16 ? launch_ssd<bf16_t>(a, *batch, as_stream(stream)) : launch_ssd<float>(a, *batch, as_stream(stream));
}

extern "C" size_t msa_seq_min_gru_workspace_bytes(int32_t rows, int32_t n_seq, int32_t max_rows, int32_t n) {
  if (rows <= 0 || n_seq <= 0 || max_rows <= kGruRows || n <= 0) return 0;
  return (size_t)n_seq * ((max_rows + kGruRows - 1) / kGruRows) * n * sizeof(float2);
}

extern "C" int msa_seq_min_gru(const void* zug, int64_t zug_stride, const float* z_bias, const float* u_bias, int32_t dtype, int32_t n,
                               float* state, void* out, const msa_seq_batch* batch, void* workspace, size_t workspace_bytes,
                               void* stream) {
  MSA_CHECK_BATCH(batch, "msa_seq_min_gru");
  MSA_CHECK_DTYPE(dtype, "msa_seq_min_gru");
  MSA_REQUIRE(zug && z_bias && u_bias && state && out && n > 0 && zug_stride >= 48LL * ((n + 15) / 16) && zug_stride < (1 << 22), "msa_seq_min_gru: bad arguments");
  const size_t need = msa_seq_min_gru_workspace_bytes(batch->rows, batch->n_seq, batch->max_rows, n);
  if (need > workspace_bytes || (need && !workspace)) {
    msa_set_error("msa_seq_min_gru: workspace of %zu bytes, need %zu", workspace_bytes, need);
    return MSA_ESIZE;
  }
  const int chunks = (batch->max_rows + kGruRows - 1) / kGruRows;
  MSA_REQUIRE(chunks <= 65535 && batch->n_seq <= 65535, "msa_seq_min_gru: step too large");
  const GruArgs a{zug, z_bias, u_bias, state, out, static_cast<float2*>(workspace), zug_stride, n, chunks};
  hipStream_t st = as_stream(stream);
  const bool vec = vec_ok(2, {zug, z_bias, u_bias, out}, {zug_stride, n});
  if (dtype == MSA_BF16) return vec ? launch_gru<bf16_t, 2>(a, *batch, st) : launch_gru<bf16_t, 1>(a, *batch, st);
  return vec ? launch_gru<float, 2>(a, *batch, st) : launch_gru<float, 1>(a, *batch, st);
}
