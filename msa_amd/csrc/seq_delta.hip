// Delta rule with a decay per key channel, token by token: the form for decoding, short portions and fp32 (the chunked
// matrix-core form is in seq_delta_chunk.hip).
//
// A workgroup owns (sequence, head, up to 128 value columns): lane = column, and the wavefronts of a column group share the
// state's rows, which they keep in registers.  A few tokens are staged at a time (unit vectors, decays, step sizes in LDS).  Both
// sums over the rows are taken from the decayed state in one pass, since
//   o = (S + k u^T)^T q = S^T q + (k . q) u,
// so a token costs one exchange and one barrier.  When the workgroup has all of a head's columns it also finishes the output
// (norm and gate); otherwise head_norm_gate_kernel does.
#include <algorithm>

#include "seq_common.h"

namespace {

constexpr int kTok = 8;                  // tokens per stage

template <typename T, int NI, int RW, int CW>
__global__ __launch_bounds__(RW * CW * 64) void delta_scan_kernel(msa_delta_args a, msa_seq_batch b) {
  constexpr int kD = NI * RW, kCols = CW * 64, kWaves = RW * CW;
  __shared__ __align__(16) float ks[kTok][kD], qs[kTok][kD], gs[kTok][kD];
  __shared__ float beta[kTok], kq[kTok];
  __shared__ float2 part[2][RW][kCols];
  __shared__ float os[kTok][kCols];
  const int s = blockIdx.z, head = blockIdx.y, tid = threadIdx.x, lane = tid & 63;
  const int wave = __builtin_amdgcn_readfirstlane(tid >> 6), cw = wave % CW, rw = wave / CW;
  const int col0 = blockIdx.x * kCols, cl = cw * 64 + lane, col = col0 + cl;
  const bool live = col < a.E, whole = gridDim.x == 1;
  const int lo = b.cu[s], n_tok = b.cu[s + 1] - lo, kvh = head / (a.H / a.G);
  float* st = a.state + (((int64_t)b.slot[s] * a.H + head) * a.D + rw * NI) * a.E + col;
  const float rate = -expf(a.A_log[head]), q_scale = 1.0f / sqrtf((float)a.D);
  const float* bias = a.dt_bias + (int64_t)head * a.D;
  const T* qkv = static_cast<const T*>(a.qkv) + (int64_t)lo * a.qkv_stride;
  const T* qp = qkv + (int64_t)kvh * a.D;
  const T* kp = qp + (int64_t)a.G * a.D;
  const T* vp = qkv + 2LL * a.G * a.D + (int64_t)head * a.E;
  const T* ap = static_cast<const T*>(a.a) + (int64_t)lo * a.a_stride + (int64_t)head * a.D;
  const T* bp = static_cast<const T*>(a.b) + (int64_t)lo * a.b_stride + head;
  const T* gp = static_cast<const T*>(a.gate) + (int64_t)lo * a.gate_stride + (int64_t)head * a.E;
  constexpr int kEach = (kD + 63) / 64, kMine = (kTok + kWaves - 1) / kWaves;    // values of a lane, tokens of a wavefront in a stage
  // What a stage reads is requested together, and the first one's in front of the state: loads arrive in the order they are made,
  // and the vectors are ready by the time the state is there.
  float k[kMine][kEach], q[kMine][kEach], x[kMine][kEach], bv[kMine], v[kTok], db[kEach];
#pragma unroll
  for (int j = 0; j < kEach; ++j) db[j] = lane + 64 * j < a.D ? bias[lane + 64 * j] : 0.f;
  auto fetch = [&](int t0) {
    const int rows = min(kTok, n_tok - t0);
#pragma unroll
    for (int m = 0; m < kMine; ++m) {
      const int r = wave + m * kWaves;
      const int64_t t = t0 + min(r, rows - 1);
#pragma unroll
      for (int j = 0; j < kEach; ++j) {
        const int i = lane + 64 * j;
        const bool in = i < a.D;
        k[m][j] = in ? to_f32<T>(kp[t * a.qkv_stride + i]) : 0.f;
        q[m][j] = in ? to_f32<T>(qp[t * a.qkv_stride + i]) : 0.f;
        x[m][j] = in ? to_f32<T>(ap[t * a.a_stride + i]) : 0.f;
      }
      bv[m] = to_f32<T>(bp[t * a.b_stride]);
    }
#pragma unroll
    for (int r = 0; r < kTok; ++r) v[r] = live && r < rows ? to_f32<T>(vp[(t0 + r) * a.qkv_stride + col]) : 0.f;
  };
  fetch(0);
  const float out_w = live && whole ? a.norm[col] : 0.f;
  const float gate0 = live && whole ? to_f32<T>(gp[col]) : 0.f;   // of the first token, all there is when decoding
  float S[NI];
#pragma unroll
  for (int i = 0; i < NI; ++i) S[i] = live && rw * NI + i < a.D ? st[(int64_t)i * a.E] : 0.f;
  for (int t0 = 0; t0 < n_tok; t0 += kTok) {
    const int rows = min(kTok, n_tok - t0);
    if (t0 > 0) fetch(t0);
#pragma unroll
    for (int m = 0; m < kMine; ++m) {                    // a wavefront per token
      const int r = wave + m * kWaves;
      if (r >= rows) break;
      float kk = 0.f, qq = 0.f, dot = 0.f;
#pragma unroll
      for (int j = 0; j < kEach; ++j) {
        const int i = lane + 64 * j;
        if (i < kD) gs[r][i] = i < a.D ? expf(rate * softplus_f(x[m][j] + db[j])) : 0.f;
        kk += k[m][j] * k[m][j];
        qq += q[m][j] * q[m][j];
        dot += k[m][j] * q[m][j];
      }
#pragma unroll
      for (int o = 32; o > 0; o >>= 1) {
        kk += __shfl_xor(kk, o);
        qq += __shfl_xor(qq, o);
        dot += __shfl_xor(dot, o);
      }
      const float ki = 1.0f / sqrtf(kk + 1e-6f), qi = q_scale / sqrtf(qq + 1e-6f);
#pragma unroll
      for (int j = 0; j < kEach; ++j) {
        const int i = lane + 64 * j;
        if (i < kD) {
          ks[r][i] = k[m][j] * ki;
          qs[r][i] = q[m][j] * qi;
        }
      }
      if (lane == 0) {
        kq[r] = dot * ki * qi;
        beta[r] = sigmoid_f(bv[m]);
      }
    }
    __syncthreads();
#pragma unroll
    for (int r = 0; r < kTok; ++r) {
      if (r >= rows) break;
      float rec = 0.f, read = 0.f;
#pragma unroll
      for (int i = 0; i < NI; i += 4) {
        const float4 g4 = *reinterpret_cast<const float4*>(&gs[r][rw * NI + i]);
        const float4 k4 = *reinterpret_cast<const float4*>(&ks[r][rw * NI + i]);
        const float4 q4 = *reinterpret_cast<const float4*>(&qs[r][rw * NI + i]);
        S[i] *= g4.x; rec += S[i] * k4.x; read += S[i] * q4.x;
        S[i + 1] *= g4.y; rec += S[i + 1] * k4.y; read += S[i + 1] * q4.y;
        S[i + 2] *= g4.z; rec += S[i + 2] * k4.z; read += S[i + 2] * q4.z;
        S[i + 3] *= g4.w; rec += S[i + 3] * k4.w; read += S[i + 3] * q4.w;
      }
      if constexpr (RW > 1) {
        part[r & 1][rw][cl] = make_float2(rec, read);
        __syncthreads();
        rec = read = 0.f;
#pragma unroll
        for (int w = 0; w < RW; ++w) {
          const float2 x = part[r & 1][w][cl];
          rec += x.x;
          read += x.y;
        }
      }
      const float u = beta[r] * (v[r] - rec);
      if (rw == 0) os[r][cl] = read + kq[r] * u;
#pragma unroll
      for (int i = 0; i < NI; i += 4) {
        const float4 k4 = *reinterpret_cast<const float4*>(&ks[r][rw * NI + i]);
        S[i] += k4.x * u;
        S[i + 1] += k4.y * u;
        S[i + 2] += k4.z * u;
        S[i + 3] += k4.w * u;
      }
    }
    __syncthreads();
    if (whole && n_tok == 1) {                           // decoding: every thread of the first row share finishes its column
      float ssq = 0.f;
#pragma unroll
      for (int c = lane; c < kCols; c += 64) ssq += c < a.E ? os[0][c] * os[0][c] : 0.f;
#pragma unroll
      for (int o = 32; o > 0; o >>= 1) ssq += __shfl_xor(ssq, o);
      if (rw == 0 && live)
        static_cast<T*>(a.out)[((int64_t)lo * a.H + head) * a.E + col] =
            from_f32<T>(os[0][cl] * (1.0f / sqrtf(ssq / (float)a.E + a.eps)) * out_w * sigmoid_f(gate0));
    } else {
      for (int r = wave; r < rows; r += kWaves) {        // outputs, a wavefront per token
        const int64_t row = lo + t0 + r;
        T* dst = static_cast<T*>(a.out) + (row * a.H + head) * a.E + col0;
        float inv = 1.f;
        if (whole) {
          float ssq = 0.f;
#pragma unroll
          for (int c = lane; c < kCols; c += 64) ssq += c < a.E ? os[r][c] * os[r][c] : 0.f;
#pragma unroll
          for (int o = 32; o > 0; o >>= 1) ssq += __shfl_xor(ssq, o);
          inv = 1.0f / sqrtf(ssq / (float)a.E + a.eps);
        }
        const T* gate = gp + (int64_t)(t0 + r) * a.gate_stride;
#pragma unroll
        for (int c = lane; c < kCols; c += 64) {
          if (col0 + c >= a.E) break;
          float y = os[r][c];
          if (whole) y *= inv * a.norm[c] * sigmoid_f(to_f32<T>(gate[c]));
          dst[c] = from_f32<T>(y);
        }
      }
    }
    // (the next stage's first barrier stands between these reads of `os` and its being written again)
  }
#pragma unroll
  for (int i = 0; i < NI; ++i)
    if (live && rw * NI + i < a.D) st[(int64_t)i * a.E] = S[i];
}

// Value columns of a workgroup.
int column_block(int32_t D, int32_t E) { return E <= 64 || D > 256 ? 64 : 128; }

template <typename T, int NI, int RW>
void launch_scan(const msa_delta_args& a, const msa_seq_batch& b, hipStream_t st) {
  const int cols = column_block(a.D, a.E);
  const dim3 grid((a.E + cols - 1) / cols, a.H, b.n_seq);
  if (cols == 64) delta_scan_kernel<T, NI, RW, 1><<<grid, RW * 64, 0, st>>>(a, b);
  else if constexpr (NI * RW <= 256) delta_scan_kernel<T, NI, RW, 2><<<grid, RW * 128, 0, st>>>(a, b);
}

template <typename T>
int launch_scan(const msa_delta_args& a, const msa_seq_batch& b, hipStream_t st) {
  if (a.D <= 16) launch_scan<T, 4, 4>(a, b, st);
  else if (a.D <= 32) launch_scan<T, 8, 4>(a, b, st);
  else if (a.D <= 64) launch_scan<T, 16, 4>(a, b, st);
  else if (a.D <= 128 && (int64_t)a.H * b.n_seq <= device_compute_units() / 2) launch_scan<T, 16, 8>(a, b, st);    // (twice the wavefronts when compute units are free)
  else if (a.D <= 128) launch_scan<T, 32, 4>(a, b, st);
  else if (a.D <= 256) launch_scan<T, 32, 8>(a, b, st);
  else launch_scan<T, 64, 8>(a, b, st);
  MSA_LAUNCH_CHECK();
  return MSA_OK;
}

}  // namespace

extern "C" int msa_seq_delta_scan(const msa_delta_args* args, int32_t dtype, const msa_seq_batch* batch, void* stream) {
  MSA_CHECK_BATCH(batch, "msa_seq_delta_scan");
  MSA_CHECK_DTYPE(dtype, "msa_seq_delta_scan");
  MSA_REQUIRE(args && args->qkv && args->a && args->b && args->gate && args->A_log && args->dt_bias && args->norm && args->state && args->out,
              "msa_seq_delta_scan: null pointer");
  const msa_delta_args& a = *args;
  MSA_REQUIRE(a.H > 0 && a.H <= 65535 && a.G > 0 && a.H % a.G == 0 && a.D > 0 && a.D <= 512 && a.E > 0 && batch->n_seq <= 65535,
              "msa_seq_delta_scan: H=%d G=%d D=%d (up to 512) E=%d", a.H, a.G, a.D, a.E);
  MSA_REQUIRE(a.qkv_stride >= 2LL * a.G * a.D + (int64_t)a.H * a.E && a.a_stride >= (int64_t)a.H * a.D && a.b_stride >= a.H &&
                  a.gate_stride >= (int64_t)a.H * a.E, "msa_seq_delta_scan: strides");
  hipStream_t st = as_stream(stream);
  const int rc = dtype == MSA_BF16 ? launch_scan<bf16_t>(a, *batch, st) : launch_scan<float>(a, *batch, st);
  if (rc != MSA_OK || a.E <= column_block(a.D, a.E)) return rc;
  return msa_seq_head_norm_gate(a.out, a.gate, a.gate_stride, a.norm, a.eps, dtype, batch->rows, a.H, a.E, stream);
}
