// Element-wise and row-wise steps of the recurrent / latent-attention decoder: gated residual + dynamic-tanh norm + token
// shift in one pass, residual + RMS norm, gelu, clamped gated units, logit softcap, grouped RMS norm, head norm + gate, latent
// norm + cache append.  All are bound by the bytes they
// move: the residual step reads the stream, one sublayer output and one gate and writes the stream and the next
// sublayer's operands, with no intermediate tensor (dynamic tanh needs no row statistics, so a thread owns columns and
// walks over tokens; the token before is the value it had in registers one step earlier).
#include <algorithm>
#include <initializer_list>

#include "seq_common.h"

namespace {

struct ResNorm {
  const float* x_in;
  const void* y;
  const void* gate;
  const float* gate_bias;
  float* x_out;
  msa_dyn_tanh norm;
  void* h;
  const float* shift;
  float* prev;
  void* h_shift;
  int64_t y_stride, gate_stride;
  int32_t W, rows_per_wg;
};

template <typename T, int VEC>
__global__ __launch_bounds__(256) void residual_norm_kernel(ResNorm a, msa_seq_batch b) {
  const int col = (blockIdx.y * 256 + threadIdx.x) * VEC;
  if (col >= a.W) return;
  const int t0 = blockIdx.x * a.rows_per_wg, t1 = min(b.rows, t0 + a.rows_per_wg);
  float gb[VEC] = {}, nw[VEC] = {}, nb[VEC] = {}, sh[VEC] = {};
  if (a.y) load_vec<float, VEC>(a.gate_bias + col, gb);
  const bool norm = a.norm.w != nullptr;
  if (norm) {
    load_vec<float, VEC>(a.norm.w + col, nw);
    load_vec<float, VEC>(a.norm.b + col, nb);
  }
  if (a.shift) load_vec<float, VEC>(a.shift + col, sh);
  struct Raw { float x[VEC], y[VEC], g[VEC]; };
  auto fetch = [&](int t, Raw& r) {
    load_vec<float, VEC>(a.x_in + (int64_t)t * a.W + col, r.x);
    if (!a.y) return;
    load_vec<T, VEC>(static_cast<const T*>(a.y) + t * a.y_stride + col, r.y);
    load_vec<T, VEC>(static_cast<const T*>(a.gate) + t * a.gate_stride + col, r.g);
  };
  auto combine = [&](const Raw& r, float (&v)[VEC]) {
#pragma unroll
    for (int i = 0; i < VEC; ++i) v[i] = a.y ? r.x[i] + sigmoid_f(r.g[i] + gb[i]) * r.y[i] : r.x[i];
  };
  auto value = [&](int t, float (&v)[VEC]) {
    Raw r;
    fetch(t, r);
    combine(r, v);
  };
  auto normed = [&](const float (&v)[VEC], float (&h)[VEC]) {
#pragma unroll
    for (int i = 0; i < VEC; ++i) h[i] = tanh_f(a.norm.alpha * v[i]) * nw[i] + nb[i];
  };
  float before[VEC] = {};
  Raw next;                             // the row ahead is on its way while this one is finished
  fetch(t0, next);
  for (int t = t0; t < t1; ++t) {
    float v[VEC], h[VEC];
    combine(next, v);
    if (t + 1 < t1) fetch(t + 1, next);
    if (a.x_out) store_vec<float, VEC>(a.x_out + (int64_t)t * a.W + col, v);
    if (!norm) continue;
    normed(v, h);
    if (a.h) store_vec<T, VEC>(static_cast<T*>(a.h) + (int64_t)t * a.W + col, h);
    if (!a.shift) continue;
    const int s = b.row_seq[t];
    if (t == b.cu[s]) {
      // the sequence's first row: its predecessor is the kept token.  The same thread replaces it (by the last row's h,
      // recomputed from the inputs), so nothing else touches it in this launch.
      float* keep = a.prev + (int64_t)b.slot[s] * a.W + col;
      load_vec<float, VEC>(keep, before);
      const int last = b.cu[s + 1] - 1;
      float hl[VEC];
      if (last == t) {
#pragma unroll
        for (int i = 0; i < VEC; ++i) hl[i] = h[i];
      } else {
        float vl[VEC];
        value(last, vl);
        normed(vl, hl);
      }
      store_vec<float, VEC>(keep, hl);
    } else if (t == t0) {
      float vp[VEC];
      value(t - 1, vp);
      normed(vp, before);
    }
    float m[VEC];
#pragma unroll
    for (int i = 0; i < VEC; ++i) {
      m[i] = h[i] + (before[i] - h[i]) * sh[i];
      before[i] = h[i];
    }
    store_vec<T, VEC>(static_cast<T*>(a.h_shift) + (int64_t)t * a.W + col, m);
  }
}

template <typename T, int VEC>
__global__ __launch_bounds__(256) void gelu_kernel(T* __restrict__ y, int64_t stride, int64_t rows, int32_t n) {
  const int64_t per_row = n / VEC, total = rows * per_row;
  for (int64_t i = (int64_t)blockIdx.x * 256 + threadIdx.x; i < total; i += (int64_t)gridDim.x * 256) {
    T* p = y + (i / per_row) * stride + (i % per_row) * VEC;
    float v[VEC];
    load_vec<T, VEC>(p, v);
#pragma unroll
    for (int e = 0; e < VEC; ++e) v[e] = gelu_tanh_f(v[e]);
    store_vec<T, VEC>(p, v);
  }
}

template <typename T>
__global__ __launch_bounds__(256) void softcap_kernel(const T* __restrict__ in, int64_t n, float cap, float* __restrict__ out) {
  for (int64_t i = (int64_t)blockIdx.x * 256 + threadIdx.x; i < n; i += (int64_t)gridDim.x * 256) {
    const float v = to_f32<T>(in[i]);
    out[i] = cap > 0.f ? cap * tanh_f(v / cap) : v;
  }
}

template <typename T>
__global__ __launch_bounds__(256) void join_kernel(const float* __restrict__ x, const float* __restrict__ x0, int64_t rows,
                                                   int32_t W, T* __restrict__ out) {
  constexpr int parts = sizeof(T) == 2 ? 3 : 2;
  const int64_t total = rows * W;
  for (int64_t i = (int64_t)blockIdx.x * 256 + threadIdx.x; i < total; i += (int64_t)gridDim.x * 256) {
    T* row = out + (i / W) * W * parts + i % W;
    const float v = x[i];
    const T hi = from_f32<T>(v);
    row[0] = hi;
    if constexpr (parts == 3) row[W] = from_f32<T>(v - to_f32<T>(hi));
    row[(parts - 1) * (int64_t)W] = from_f32<T>(x0[i]);
  }
}

// A wavefront per (row, part): the part stays in registers between the sum of squares and the output when it fits
// (VEC = 8: 16-byte accesses).
template <typename T, int VEC>
__global__ __launch_bounds__(256) void group_rmsnorm_kernel(const T* __restrict__ v, int64_t items, int32_t n, int32_t parts,
                                                            const float* __restrict__ w, float eps, T* __restrict__ out) {
  constexpr int kKeep = 4;
  const int64_t item = (int64_t)blockIdx.x * 4 + (threadIdx.x >> 6);
  if (item >= items) return;
  const int lane = threadIdx.x & 63, len = n / parts;
  const int64_t at = item * len;
  const float* wg = w + item % parts * len;
  float keep[kKeep][VEC], ssq = 0.f;
#pragma unroll
  for (int k = 0; k < kKeep; ++k) {
    const int i = (k * 64 + lane) * VEC;
    if (i < len) {
      load_vec<T, VEC>(v + at + i, keep[k]);
#pragma unroll
      for (int e = 0; e < VEC; ++e) ssq += keep[k][e] * keep[k][e];
    }
  }
  for (int i = (kKeep * 64 + lane) * VEC; i < len; i += 64 * VEC) {
    float x[VEC];
    load_vec<T, VEC>(v + at + i, x);
#pragma unroll
    for (int e = 0; e < VEC; ++e) ssq += x[e] * x[e];
  }
#pragma unroll
  for (int o = 32; o > 0; o >>= 1) ssq += __shfl_xor(ssq, o);
  const float inv = 1.0f / sqrtf(ssq / (float)len + eps);
  auto finish = [&](int i, float (&x)[VEC]) {
    float g[VEC];
    load_vec<float, VEC>(wg + i, g);
#pragma unroll
    for (int e = 0; e < VEC; ++e) x[e] *= inv * g[e];
    store_vec<T, VEC>(out + at + i, x);
  };
#pragma unroll
  for (int k = 0; k < kKeep; ++k) {
    const int i = (k * 64 + lane) * VEC;
    if (i < len) finish(i, keep[k]);
  }
  for (int i = (kKeep * 64 + lane) * VEC; i < len; i += 64 * VEC) {
    float x[VEC];
    load_vec<T, VEC>(v + at + i, x);
    finish(i, x);
  }
}

// One wavefront per row.
template <typename T, int VEC>
__global__ __launch_bounds__(256) void latent_append_kernel(const T* __restrict__ in, int64_t stride, const float* __restrict__ w,
                                                            float eps, int32_t rank, T* __restrict__ cache, int64_t Lcap,
                                                            msa_seq_batch b) {
  const int row = blockIdx.x * 4 + (threadIdx.x >> 6), lane = threadIdx.x & 63;
  if (row >= b.rows) return;
  const int s = b.row_seq[row];
  const int64_t p = b.pos[s] + (row - b.cu[s]);
  const T* src = in + row * stride;
  T* dst = cache + ((int64_t)b.slot[s] * Lcap + p) * rank;
  float ssq = 0.f;
  for (int i = lane * VEC; i < rank; i += 64 * VEC) {
    float x[VEC];
    load_vec<T, VEC>(src + i, x);
#pragma unroll
    for (int e = 0; e < VEC; ++e) ssq += x[e] * x[e];
  }
#pragma unroll
  for (int o = 32; o > 0; o >>= 1) ssq += __shfl_xor(ssq, o);
  if (p >= Lcap) return;
  const float inv = 1.0f / sqrtf(ssq / (float)rank + eps);
  for (int i = lane * VEC; i < rank; i += 64 * VEC) {
    float x[VEC], g[VEC];
    load_vec<T, VEC>(src + i, x);
    load_vec<float, VEC>(w + i, g);
#pragma unroll
    for (int e = 0; e < VEC; ++e) x[e] *= inv * g[e];
    store_vec<T, VEC>(dst + i, x);
  }
}

// A workgroup per row: x' = x + rms_norm(y) w, and the next sublayer's operand.  A row of up to 256 * kKeep vectors stays in
// registers between its sums and the outputs; what lies behind is read again (by the thread that owns it).
struct RmsResidual {
  const float* x_in;
  const void* y;
  const float* w;
  float* x_out;
  const float* next_w;
  void* h;
  int64_t y_stride;
  float eps;
  int32_t W;
};
template <typename T, int VEC>
__global__ __launch_bounds__(256) void rms_residual_kernel(RmsResidual a) {
  constexpr int kKeep = 4;
  __shared__ float red[2][4];
  const int64_t row = blockIdx.x;
  const int tid = threadIdx.x, wave = tid >> 6, lane = tid & 63;
  const float* xr = a.x_in + row * a.W;
  const T* yr = a.y ? static_cast<const T*>(a.y) + row * a.y_stride : nullptr;
  float* xo = a.y ? a.x_out + row * a.W : nullptr;
  float x[kKeep][VEC], y[kKeep][VEC], w[kKeep][VEC];             // (everything is requested before the first sum)
  auto sum_of = [&](float v, int which) {
#pragma unroll
    for (int o = 32; o > 0; o >>= 1) v += __shfl_xor(v, o);
    if (lane == 0) red[which][wave] = v;
    __syncthreads();
    return red[which][0] + red[which][1] + red[which][2] + red[which][3];
  };
  float ssq = 0.f;
#pragma unroll
  for (int k = 0; k < kKeep; ++k) {
    const int i = (k * 256 + tid) * VEC;
    if (i >= a.W) break;
    load_vec<float, VEC>(xr + i, x[k]);
    if (!a.y) continue;
    load_vec<T, VEC>(yr + i, y[k]);
    load_vec<float, VEC>(a.w + i, w[k]);
  }
  if (a.y) {
#pragma unroll
    for (int k = 0; k < kKeep; ++k)
      if ((k * 256 + tid) * VEC < a.W)
#pragma unroll
        for (int e = 0; e < VEC; ++e) ssq += y[k][e] * y[k][e];
    for (int i = (kKeep * 256 + tid) * VEC; i < a.W; i += 256 * VEC) {
      float v[VEC];
      load_vec<T, VEC>(yr + i, v);
#pragma unroll
      for (int e = 0; e < VEC; ++e) ssq += v[e] * v[e];
    }
    ssq = sum_of(ssq, 0);
  }
  const float inv = a.y ? 1.0f / sqrtf(ssq / (float)a.W + a.eps) : 0.f;
  const bool norm = a.next_w != nullptr;
  float next_ssq = 0.f;
  auto combine = [&](int i, float (&xv)[VEC], const float (&yv)[VEC], const float (&wv)[VEC]) {
#pragma unroll
    for (int e = 0; e < VEC; ++e) xv[e] += yv[e] * inv * wv[e];
    store_vec<float, VEC>(xo + i, xv);
  };
#pragma unroll
  for (int k = 0; k < kKeep; ++k) {
    const int i = (k * 256 + tid) * VEC;
    if (i >= a.W) break;
    if (a.y) combine(i, x[k], y[k], w[k]);
    if (norm)
#pragma unroll
      for (int e = 0; e < VEC; ++e) next_ssq += x[k][e] * x[k][e];
    else if (a.h) store_vec<T, VEC>(static_cast<T*>(a.h) + row * a.W + i, x[k]);
  }
  for (int i = (kKeep * 256 + tid) * VEC; i < a.W; i += 256 * VEC) {
    float xv[VEC], yv[VEC], wv[VEC];
    load_vec<float, VEC>(xr + i, xv);
    if (a.y) {
      load_vec<T, VEC>(yr + i, yv);
      load_vec<float, VEC>(a.w + i, wv);
      combine(i, xv, yv, wv);
    }
    if (norm)
#pragma unroll
      for (int e = 0; e < VEC; ++e) next_ssq += xv[e] * xv[e];
    else if (a.h) store_vec<T, VEC>(static_cast<T*>(a.h) + row * a.W + i, xv);
  }
  if (!norm) return;
  const float next_inv = 1.0f / sqrtf(sum_of(next_ssq, 1) / (float)a.W + a.eps);
  auto finish = [&](int i, float (&v)[VEC]) {
    float w[VEC];
    load_vec<float, VEC>(a.next_w + i, w);
#pragma unroll
    for (int e = 0; e < VEC; ++e) v[e] *= next_inv * w[e];
    store_vec<T, VEC>(static_cast<T*>(a.h) + row * a.W + i, v);
  };
#pragma unroll
  for (int k = 0; k < kKeep; ++k) {
    const int i = (k * 256 + tid) * VEC;
    if (i < a.W) finish(i, x[k]);
  }
  for (int i = (kKeep * 256 + tid) * VEC; i < a.W; i += 256 * VEC) {
    float v[VEC];
    load_vec<float, VEC>((xo ? xo : xr) + i, v);
    finish(i, v);
  }
}

// VEC pairs per thread and turn.
template <typename T, int VEC>
__global__ __launch_bounds__(256) void clamped_glu_kernel(const T* __restrict__ in, int64_t stride, int64_t rows, int32_t n, float limit,
                                                          float alpha, float shift, T* __restrict__ out) {
  const int64_t per_row = n / VEC, total = rows * per_row;
  for (int64_t i = (int64_t)blockIdx.x * 256 + threadIdx.x; i < total; i += (int64_t)gridDim.x * 256) {
    const int64_t row = i / per_row, c = i % per_row * VEC;
    const T* p = in + row * stride + 2 * c;
    float y[VEC];
    if constexpr (VEC == 4) {
      float v[8];
      load_vec<T, 8>(p, v);
#pragma unroll
      for (int e = 0; e < 4; ++e) y[e] = clamped_glu_f(v[2 * e], v[2 * e + 1], limit, alpha, shift);
    } else {
      y[0] = clamped_glu_f(to_f32<T>(p[0]), to_f32<T>(p[1]), limit, alpha, shift);
    }
    store_vec<T, VEC>(out + row * n + c, y);
  }
}

// LANES lanes per (row, head), a head's columns VEC at a time.
template <typename T, int VEC, int LANES>
__global__ __launch_bounds__(256) void head_norm_gate_kernel(T* o, const T* __restrict__ gate, int64_t gate_stride, const float* __restrict__ w,
                                                             float eps, int64_t items, int32_t H, int32_t E) {
  constexpr int kKeep = VEC == 8 ? 2 : 4;
  const int64_t item = ((int64_t)blockIdx.x * 256 + threadIdx.x) / LANES;
  const int lane = threadIdx.x % LANES;
  const bool live = item < items;
  T* at = o + item * E;
  const T* gt = gate + item / H * gate_stride + item % H * E;
  float keep[kKeep][VEC], ssq = 0.f;
  if (live) {
#pragma unroll
    for (int k = 0; k < kKeep; ++k) {
      const int i = (k * LANES + lane) * VEC;
      if (i < E) {
        load_vec<T, VEC>(at + i, keep[k]);
#pragma unroll
        for (int e = 0; e < VEC; ++e) ssq += keep[k][e] * keep[k][e];
      }
    }
    for (int i = (kKeep * LANES + lane) * VEC; i < E; i += LANES * VEC) {
      float x[VEC];
      load_vec<T, VEC>(at + i, x);
#pragma unroll
      for (int e = 0; e < VEC; ++e) ssq += x[e] * x[e];
    }
  }
#pragma unroll
  for (int d = LANES / 2; d > 0; d >>= 1) ssq += __shfl_xor(ssq, d);
  if (!live) return;
  const float inv = 1.0f / sqrtf(ssq / (float)E + eps);
  auto finish = [&](int i, float (&x)[VEC]) {
    float g[VEC], n[VEC];
    load_vec<T, VEC>(gt + i, g);
    load_vec<float, VEC>(w + i, n);
#pragma unroll
    for (int e = 0; e < VEC; ++e) x[e] *= inv * n[e] * sigmoid_f(g[e]);
    store_vec<T, VEC>(at + i, x);
  };
#pragma unroll
  for (int k = 0; k < kKeep; ++k) {
    const int i = (k * LANES + lane) * VEC;
    if (i < E) finish(i, keep[k]);
  }
  for (int i = (kKeep * LANES + lane) * VEC; i < E; i += LANES * VEC) {
    float x[VEC];
    load_vec<T, VEC>(at + i, x);
    finish(i, x);
  }
}

template <typename T, int VEC>
void launch_head_norm(T* o, const T* gate, int64_t gate_stride, const float* w, float eps, int64_t items, int32_t H, int32_t E, hipStream_t st) {
  const int units = (E + VEC - 1) / VEC;
  auto grid = [&](int lanes) { return (unsigned)((items * lanes + 255) / 256); };
  if (units <= 8) head_norm_gate_kernel<T, VEC, 8><<<grid(8), 256, 0, st>>>(o, gate, gate_stride, w, eps, items, H, E);
  else if (units <= 16) head_norm_gate_kernel<T, VEC, 16><<<grid(16), 256, 0, st>>>(o, gate, gate_stride, w, eps, items, H, E);
  else head_norm_gate_kernel<T, VEC, 64><<<grid(64), 256, 0, st>>>(o, gate, gate_stride, w, eps, items, H, E);
}

int grid_for(int64_t items) { return (int)std::min<int64_t>(std::max<int64_t>(1, (items + 255) / 256), 8192); }

}  // namespace

extern "C" int msa_seq_residual_norm(const float* x_in, const void* y, int64_t y_stride, const void* gate, int64_t gate_stride,
                                     const float* gate_bias, float* x_out, int32_t dtype, int32_t W, const msa_dyn_tanh* norm,
                                     void* h, const float* shift, float* prev, void* h_shift, const msa_seq_batch* batch,
                                     void* stream) {
  MSA_CHECK_BATCH(batch, "msa_seq_residual_norm");
  MSA_CHECK_DTYPE(dtype, "msa_seq_residual_norm");
  MSA_REQUIRE(x_in && W > 0, "msa_seq_residual_norm: null stream or W=%d", W);
  MSA_REQUIRE(!y || (gate && gate_bias && x_out && x_out != x_in && y_stride >= W && gate_stride >= W),
              "msa_seq_residual_norm: a sublayer output needs its gate, strides of at least W and an x_out that is not x_in");
  const bool with_norm = norm && norm->w;
  MSA_REQUIRE(!with_norm || norm->b, "msa_seq_residual_norm: norm without b");
  MSA_REQUIRE(!with_norm || h || shift, "msa_seq_residual_norm: norm without an output");
  MSA_REQUIRE(!shift || (with_norm && prev && h_shift), "msa_seq_residual_norm: shift needs norm, prev and h_shift");
  ResNorm a{x_in, y, gate, gate_bias, y ? x_out : nullptr, with_norm ? *norm : msa_dyn_tanh{}, with_norm ? h : nullptr,
            shift, prev, h_shift, y_stride, gate_stride, W, 1};
  a.rows_per_wg = batch->rows <= 256 ? 1 : 8;
  const bool vec = vec_ok(4, {x_in, y, gate, gate_bias, x_out, a.norm.w, a.norm.b, h, shift, prev, h_shift}, {W, y_stride, gate_stride});
  const int V = vec ? 4 : 1;
  const dim3 grid((batch->rows + a.rows_per_wg - 1) / a.rows_per_wg, (W + 256 * V - 1) / (256 * V));
  hipStream_t st = as_stream(stream);
  if (dtype == MSA_BF16) {
    if (vec) residual_norm_kernel<bf16_t, 4><<<grid, 256, 0, st>>>(a, *batch);
    else residual_norm_kernel<bf16_t, 1><<<grid, 256, 0, st>>>(a, *batch);
  } else {
    if (vec) residual_norm_kernel<float, 4><<<grid, 256, 0, st>>>(a, *batch);
    else residual_norm_kernel<float, 1><<<grid, 256, 0, st>>>(a, *batch);
  }
  MSA_LAUNCH_CHECK();
  return MSA_OK;
}

extern "C" int msa_seq_gelu(void* y, int64_t y_stride, int32_t dtype, int32_t rows, int32_t n, void* stream) {
  MSA_REQUIRE(y && rows > 0 && n > 0 && y_stride >= n, "msa_seq_gelu: bad arguments");
  MSA_CHECK_DTYPE(dtype, "msa_seq_gelu");
  const bool vec = vec_ok(4, {y}, {y_stride, n});
  const int grid = grid_for((int64_t)rows * n / (vec ? 4 : 1));
  hipStream_t st = as_stream(stream);
  if (dtype == MSA_BF16) {
    if (vec) gelu_kernel<bf16_t, 4><<<grid, 256, 0, st>>>((bf16_t*)y, y_stride, rows, n);
    else gelu_kernel<bf16_t, 1><<<grid, 256, 0, st>>>((bf16_t*)y, y_stride, rows, n);
  } else {
    if (vec) gelu_kernel<float, 4><<<grid, 256, 0, st>>>((float*)y, y_stride, rows, n);
    else gelu_kernel<float, 1><<<grid, 256, 0, st>>>((float*)y, y_stride, rows, n);
  }
  MSA_LAUNCH_CHECK();
  return MSA_OK;
}

extern "C" int msa_seq_softcap(const void* in, int32_t dtype, int64_t n_elems, float cap, float* out, void* stream) {
  MSA_REQUIRE(in && out && n_elems > 0 && cap >= 0.f, "msa_seq_softcap: bad arguments");
  MSA_CHECK_DTYPE(dtype, "msa_seq_softcap");
  if (dtype == MSA_BF16) softcap_kernel<bf16_t><<<grid_for(n_elems), 256, 0, as_stream(stream)>>>((const bf16_t*)in, n_elems, cap, out);
  else softcap_kernel<float><<<grid_for(n_elems), 256, 0, as_stream(stream)>>>((const float*)in, n_elems, cap, out);
  MSA_LAUNCH_CHECK();
  return MSA_OK;
}

extern "C" int msa_seq_join(const float* x, const float* x0, int32_t dtype, int32_t rows, int32_t W, void* out, void* stream) {
  MSA_REQUIRE(x && x0 && out && rows > 0 && W > 0, "msa_seq_join: bad arguments");
  MSA_CHECK_DTYPE(dtype, "msa_seq_join");
  const int grid = grid_for((int64_t)rows * W);
  if (dtype == MSA_BF16) join_kernel<bf16_t><<<grid, 256, 0, as_stream(stream)>>>(x, x0, rows, W, (bf16_t*)out);
  else join_kernel<float><<<grid, 256, 0, as_stream(stream)>>>(x, x0, rows, W, (float*)out);
  MSA_LAUNCH_CHECK();
  return MSA_OK;
}

extern "C" int msa_seq_group_rmsnorm(const void* v, int32_t dtype, int32_t rows, int32_t n, int32_t parts, const float* w, float eps,
                                     void* out, void* stream) {
  MSA_REQUIRE(v && w && out && rows > 0 && n > 0 && parts > 0 && n % parts == 0 && parts <= 65535,
              "msa_seq_group_rmsnorm: n=%d in %d parts", n, parts);
  MSA_CHECK_DTYPE(dtype, "msa_seq_group_rmsnorm");
  const int64_t items = (int64_t)rows * parts;
  const unsigned grid = (unsigned)((items + 3) / 4);
  const bool vec = vec_ok(8, {v, w, out}, {n / parts});
  hipStream_t st = as_stream(stream);
  if (dtype == MSA_BF16) {
    if (vec) group_rmsnorm_kernel<bf16_t, 8><<<grid, 256, 0, st>>>((const bf16_t*)v, items, n, parts, w, eps, (bf16_t*)out);
    else group_rmsnorm_kernel<bf16_t, 1><<<grid, 256, 0, st>>>((const bf16_t*)v, items, n, parts, w, eps, (bf16_t*)out);
  } else {
    if (vec) group_rmsnorm_kernel<float, 8><<<grid, 256, 0, st>>>((const float*)v, items, n, parts, w, eps, (float*)out);
    else group_rmsnorm_kernel<float, 1><<<grid, 256, 0, st>>>((const float*)v, items, n, parts, w, eps, (float*)out);
  }
  MSA_LAUNCH_CHECK();
  return MSA_OK;
}

extern "C" int msa_seq_latent_append(const void* in, int64_t in_stride, const float* w, float eps, int32_t dtype, int32_t rank,
                                     void* cache, int64_t Lcap, const msa_seq_batch* batch, void* stream) {
  MSA_CHECK_BATCH(batch, "msa_seq_latent_append");
  MSA_CHECK_DTYPE(dtype, "msa_seq_latent_append");
  MSA_REQUIRE(in && w && cache && rank > 0 && in_stride >= rank && Lcap > 0, "msa_seq_latent_append: bad arguments");
  const int grid = (batch->rows + 3) / 4;
  const bool vec = vec_ok(8, {in, w, cache}, {in_stride, rank});
  hipStream_t st = as_stream(stream);
  if (dtype == MSA_BF16) {
    if (vec) latent_append_kernel<bf16_t, 8><<<grid, 256, 0, st>>>((const bf16_t*)in, in_stride, w, eps, rank, (bf16_t*)cache, Lcap, *batch);
    else latent_append_kernel<bf16_t, 1><<<grid, 256, 0, st>>>((const bf16_t*)in, in_stride, w, eps, rank, (bf16_t*)cache, Lcap, *batch);
  } else {
    if (vec) latent_append_kernel<float, 8><<<grid, 256, 0, st>>>((const float*)in, in_stride, w, eps, rank, (float*)cache, Lcap, *batch);
    else latent_append_kernel<float, 1><<<grid, 256, 0, st>>>((const float*)in, in_stride, w, eps, rank, (float*)cache, Lcap, *batch);
  }
  MSA_LAUNCH_CHECK();
  return MSA_OK;
}

extern "C" int msa_seq_rms_residual(const float* x_in, const void* y, int64_t y_stride, const float* w, float eps, float* x_out,
                                    const float* next_w, void* h, int32_t dtype, int32_t rows, int32_t W, void* stream) {
  MSA_REQUIRE(x_in && rows > 0 && W > 0 && (y || h), "msa_seq_rms_residual: null stream, rows=%d or W=%d", rows, W);
  MSA_REQUIRE(!y || (w && x_out && y_stride >= W), "msa_seq_rms_residual: a sublayer output needs its norm, a stride of at least W and x_out");
  MSA_REQUIRE(!next_w || h, "msa_seq_rms_residual: norm without an output");
  MSA_CHECK_DTYPE(dtype, "msa_seq_rms_residual");
  const RmsResidual a{x_in, y, w, x_out, next_w, h, y_stride, eps, W};
  const bool vec = vec_ok(4, {x_in, y, w, x_out, next_w, h}, {W, y_stride});
  hipStream_t st = as_stream(stream);
  if (dtype == MSA_BF16) {
    if (vec) rms_residual_kernel<bf16_t, 4><<<rows, 256, 0, st>>>(a);
    else rms_residual_kernel<bf16_t, 1><<<rows, 256, 0, st>>>(a);
  } else {
    if (vec) rms_residual_kernel<float, 4><<<rows, 256, 0, st>>>(a);
    else rms_residual_kernel<float, 1><<<rows, 256, 0, st>>>(a);
  }
  MSA_LAUNCH_CHECK();
  return MSA_OK;
}

extern "C" int msa_seq_clamped_glu(const void* in, int64_t in_stride, int32_t dtype, int32_t rows, int32_t n, float limit, float alpha,
                                   float shift, void* out, void* stream) {
  MSA_REQUIRE(in && out && rows > 0 && n > 0 && in_stride >= 2LL * n && limit >= 0.f, "msa_seq_clamped_glu: bad arguments");
  MSA_CHECK_DTYPE(dtype, "msa_seq_clamped_glu");
  const bool vec = vec_ok(8, {in, out}, {in_stride}) && n % 4 == 0;
  const int grid = grid_for((int64_t)rows * n / (vec ? 4 : 1));
  hipStream_t st = as_stream(stream);
  if (dtype == MSA_BF16) {
    if (vec) clamped_glu_kernel<bf16_t, 4><<<grid, 256, 0, st>>>((const bf16_t*)in, in_stride, rows, n, limit, alpha, shift, (bf16_t*)out);
    else clamped_glu_kernel<bf16_t, 1><<<grid, 256, 0, st>>>((const bf16_t*)in, in_stride, rows, n, limit, alpha, shift, (bf16_t*)out);
  } else {
    if (vec) clamped_glu_kernel<float, 4><<<grid, 256, 0, st>>>((const float*)in, in_stride, rows, n, limit, alpha, shift, (float*)out);
    else clamped_glu_kernel<float, 1><<<grid, 256, 0, st>>>((const float*)in, in_stride, rows, n, limit, alpha, shift, (float*)out);
  }
  MSA_LAUNCH_CHECK();
  return MSA_OK;
}

extern "C" int msa_seq_head_norm_gate(void* o, const void* gate, int64_t gate_stride, const float* norm, float eps, int32_t dtype, int32_t rows,
                                      int32_t H, int32_t E, void* stream) {
  MSA_REQUIRE(o && gate && norm && rows > 0 && H > 0 && E > 0 && gate_stride >= (int64_t)H * E, "msa_seq_head_norm_gate: bad arguments");
  MSA_CHECK_DTYPE(dtype, "msa_seq_head_norm_gate");
  const bool vec = vec_ok(8, {o, gate, norm}, {gate_stride, E});
  const int64_t items = (int64_t)rows * H;
  hipStream_t st = as_stream(stream);
  if (dtype == MSA_BF16) {
    if (vec) launch_head_norm<bf16_t, 8>((bf16_t*)o, (const bf16_t*)gate, gate_stride, norm, eps, items, H, E, st);
    else launch_head_norm<bf16_t, 1>((bf16_t*)o, (const bf16_t*)gate, gate_stride, norm, eps, items, H, E, st);
  } else {
    if (vec) launch_head_norm<float, 8>((float*)o, (const float*)gate, gate_stride, norm, eps, items, H, E, st);
    else launch_head_norm<float, 1>((float*)o, (const float*)gate, gate_stride, norm, eps, items, H, E, st);
  }
  MSA_LAUNCH_CHECK();
  return MSA_OK;
}
