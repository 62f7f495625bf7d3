// Element-wise and row-wise steps of the recurrent / latent-attention decoder: gated residual + dynamic-tanh norm + token
// shift in one pass, gelu, logit softcap, grouped RMS norm, latent norm + cache append.  All are bound by the bytes they
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
