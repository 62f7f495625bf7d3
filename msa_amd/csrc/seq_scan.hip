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
  const float bs = bias[c];
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

// ------------------------------------------------------------------------------------------------ state-space recurrence
// A workgroup owns (sequence, head, 64 state columns): lane = column p, wavefront w holds the state rows n = w + waves i in
// registers.  kScanRows tokens are staged at a time: every wavefront adds its share of S^T C into LDS, one barrier, and all
// threads finish the outputs.
constexpr int kScanRows = 8;

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
  __shared__ float part[WAVES][kScanRows][64];
  const int s = blockIdx.z, head = blockIdx.y, lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
  const int p = blockIdx.x * 64 + lane;
  const bool live = p < a.P;
  const int lo = b.cu[s], n_tok = b.cu[s + 1] - lo;
  const int grp = head / (a.H / a.G), inner = a.H * a.P;
  float* st = a.state + (((int64_t)b.slot[s] * a.H + head) * a.N) * a.P + p;
  float S[NI];
#pragma unroll
  for (int i = 0; i < NI; ++i) {
    const int n = wave + WAVES * i;
    S[i] = live && n < a.N ? st[(int64_t)n * a.P] : 0.f;
  }
  const float rate = -expf(a.A_log[head]), bias = a.dt_bias[head], Dh = a.D[head];
  const T* xbc = static_cast<const T*>(a.xbc) + (int64_t)lo * a.xbc_stride;
  const T* dtp = static_cast<const T*>(a.dt_raw) + (int64_t)lo * a.dt_stride + head;
  for (int t0 = 0; t0 < n_tok; t0 += kScanRows) {
    const int rows = min(kScanRows, n_tok - t0);
    for (int r = 0; r < rows; ++r) {
      const T* row = xbc + (int64_t)(t0 + r) * a.xbc_stride;
      const float dt = softplus_f(to_f32<T>(dtp[(int64_t)(t0 + r) * a.dt_stride]) + bias);
      const float decay = expf(rate * dt);
      const float x = live ? dt * to_f32<T>(row[head * a.P + p]) : 0.f;
      const T* Bt = row + inner + grp * a.N;
      const T* Ct = Bt + a.G * a.N;
      float y = 0.f;
#pragma unroll
      for (int i = 0; i < NI; ++i) {
        const int n = wave + WAVES * i;
        if (n < a.N) {
          S[i] = decay * S[i] + to_f32<T>(Bt[n]) * x;
          y += S[i] * to_f32<T>(Ct[n]);
        }
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
    __syncthreads();
  }
#pragma unroll
  for (int i = 0; i < NI; ++i) {
    const int n = wave + WAVES * i;
    if (live && n < a.N) st[(int64_t)n * a.P] = S[i];
  }
}

// ------------------------------------------------------------------------------------------------ minimal gated recurrence
// S_t = a_t S_(t-1) + b_t per channel.  Long portions run in chunks of kGruRows tokens: (1) every chunk's (product of a,
// last b-part), (2) the chunk-to-chunk recurrence, which leaves each chunk's incoming state, (3) the chunks again from
// their incoming states.  A portion of one chunk is phase (3) alone.
constexpr int kGruRows = 64;
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

template <typename T>
__device__ __forceinline__ void gru_terms(const T* row, int c, float zb, float ub, float& keep, float& add) {
  const float z = sigmoid_f(to_f32<T>(row[c]) + zb);
  const float u = to_f32<T>(row[c + kGruGroup]) + ub;
  keep = 1.0f - z;
  add = z * (u >= 0.f ? u + 0.5f : sigmoid_f(u));
}

template <typename T>
__global__ __launch_bounds__(256) void gru_chunk_kernel(GruArgs a, msa_seq_batch b) {
  const int c = blockIdx.x * 256 + threadIdx.x, s = blockIdx.z;
  const int lo = b.cu[s], n_tok = b.cu[s + 1] - lo, t0 = blockIdx.y * kGruRows;
  if (c >= a.n || t0 >= n_tok) return;
  const int t1 = min(n_tok, t0 + kGruRows);
  const float zb = a.z_bias[c], ub = a.u_bias[c];
  const int at = gru_column(c);
  float A = 1.f, S = 0.f;
  const T* row = static_cast<const T*>(a.zug) + (int64_t)(lo + t0) * a.stride;
#pragma unroll 4
  for (int t = t0; t < t1; ++t, row += a.stride) {
    float k, d;
    gru_terms<T>(row, at, zb, ub, k, d);
    A *= k;
    S = k * S + d;
  }
  a.chunk[((int64_t)s * a.n_chunks + blockIdx.y) * a.n + c] = make_float2(A, S);
}

__global__ __launch_bounds__(64) void gru_carry_kernel(GruArgs a, msa_seq_batch b) {
  const int c = blockIdx.x * 64 + threadIdx.x, s = blockIdx.y;
  if (c >= a.n) return;
  const int n_tok = b.cu[s + 1] - b.cu[s], chunks = (n_tok + kGruRows - 1) / kGruRows;
  float S = a.state[(int64_t)b.slot[s] * a.n + c];
  float2* ch = a.chunk + (int64_t)s * a.n_chunks * a.n + c;
#pragma unroll 8
  for (int i = 0; i < chunks; ++i) {
    const float2 t = ch[(int64_t)i * a.n];
    ch[(int64_t)i * a.n].x = S;
    S = t.x * S + t.y;
  }
  a.state[(int64_t)b.slot[s] * a.n + c] = S;
}

template <typename T, bool kCarried>
__global__ __launch_bounds__(256) void gru_out_kernel(GruArgs a, msa_seq_batch b) {
  const int c = blockIdx.x * 256 + threadIdx.x, s = blockIdx.z;
  const int lo = b.cu[s], n_tok = b.cu[s + 1] - lo, t0 = blockIdx.y * kGruRows;
  if (c >= a.n || t0 >= n_tok) return;
  const int t1 = min(n_tok, t0 + kGruRows);
  const float zb = a.z_bias[c], ub = a.u_bias[c];
  const int at = gru_column(c);
  float* st = a.state + (int64_t)b.slot[s] * a.n + c;
  float S = kCarried ? a.chunk[((int64_t)s * a.n_chunks + blockIdx.y) * a.n + c].x : *st;
  const T* row = static_cast<const T*>(a.zug) + (int64_t)(lo + t0) * a.stride;
  T* out = static_cast<T*>(a.out) + (int64_t)(lo + t0) * a.n + c;
#pragma unroll 4
  for (int t = t0; t < t1; ++t, row += a.stride, out += a.n) {
    float k, d;
    gru_terms<T>(row, at, zb, ub, k, d);
    S = k * S + d;
    *out = from_f32<T>(S * silu_f(to_f32<T>(row[at + 2 * kGruGroup])));
  }
  if (!kCarried) *st = S;
}

template <typename T>
int launch_gru(const GruArgs& a, const msa_seq_batch& b, hipStream_t st) {
  const dim3 grid((a.n + 255) / 256, a.n_chunks, b.n_seq);
  if (a.n_chunks > 1) {
    gru_chunk_kernel<T><<<grid, 256, 0, st>>>(a, b);
    MSA_LAUNCH_CHECK();
    gru_carry_kernel<<<dim3((a.n + 63) / 64, b.n_seq), 64, 0, st>>>(a, b);
    MSA_LAUNCH_CHECK();
    gru_out_kernel<T, true><<<grid, 256, 0, st>>>(a, b);
  } else {
    gru_out_kernel<T, false><<<grid, 256, 0, st>>>(a, b);
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
  MSA_REQUIRE(in && taps && bias && out && C > 0 && in_stride >= C && out_stride >= C, "msa_seq_conv_silu: bad arguments");
  MSA_REQUIRE(K >= 1 && K - 1 <= kConvRows && (K == 1 || state), "msa_seq_conv_silu: K=%d (1..%d taps)", K, kConvRows + 1);
  MSA_REQUIRE(batch->n_seq <= 65535 && (batch->max_rows + kConvRows - 1) / kConvRows <= 65535, "msa_seq_conv_silu: step too large");
  const dim3 grid((C + 255) / 256, (batch->max_rows + kConvRows - 1) / kConvRows, batch->n_seq);
  if (dtype == MSA_BF16)
    conv_silu_kernel<bf16_t><<<grid, 256, 0, as_stream(stream)>>>((const bf16_t*)in, in_stride, taps, bias, C, K, state, (bf16_t*)out, out_stride, *batch);
  else
    conv_silu_kernel<float><<<grid, 256, 0, as_stream(stream)>>>((const float*)in, in_stride, taps, bias, C, K, state, (float*)out, out_stride, *batch);
  MSA_LAUNCH_CHECK();
  return MSA_OK;
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
  MSA_REQUIRE(zug && z_bias && u_bias && state && out && n > 0 && zug_stride >= 48LL * ((n + 15) / 16), "msa_seq_min_gru: bad arguments");
  const size_t need = msa_seq_min_gru_workspace_bytes(batch->rows, batch->n_seq, batch->max_rows, n);
  if (need > workspace_bytes || (need && !workspace)) {
    msa_set_error("msa_seq_min_gru: workspace of %zu bytes, need %zu", workspace_bytes, need);
    return MSA_ESIZE;
  }
  const int chunks = (batch->max_rows + kGruRows - 1) / kGruRows;
  MSA_REQUIRE(chunks <= 65535 && batch->n_seq <= 65535, "msa_seq_min_gru: step too large");
  const GruArgs a{zug, z_bias, u_bias, state, out, static_cast<float2*>(workspace), zug_stride, n, chunks};
  return dtype == MSA_BF16 ? launch_gru<bf16_t>(a, *batch, as_stream(stream)) : launch_gru<float>(a, *batch, as_stream(stream));
}
