// Weight-streaming linear for the rows of a decode step (M <= 16, bf16), with the recurrent decoder's element-wise work in
// the epilogue: gelu, clamped gated units, softcap, the gated residual with the next norm and token shift, the causal convolution, the minimal
// gated recurrence.  Like the skinny linear of the attention model a workgroup owns a few 16-row groups of the weights and
// splits K over its wavefronts (16x16x32 MFMA: the 16 activation rows are exactly one operand); partial sums meet in LDS
// and are added in wavefront order.  Everything behind the sums is element-wise in this model (dynamic tanh has no row
// statistics), so a layer's chain of launches is one per weight matrix plus the state-space / attention step.
#include <algorithm>
#include <type_traits>

#include "seq_mfma.h"

namespace {

constexpr int kMaxWaves = 16;
constexpr int kGruGroup = 16;

// Units of 32 J elements of K (J 16-byte vectors per lane): shorter when three row groups share the registers.
template <int R>
constexpr int kVectors = R == 3 ? 2 : 4;

// The element-wise end of product (m, n), `col` its column in the output.  What it reads besides the product is fetched by
// `load`, which the kernels call before they multiply, so that it arrives with the weights instead of behind the sums.
template <int EPI>
struct Finish {
  __device__ __forceinline__ void load(const msa_rows_args& a, int m, int n) {}
  __device__ __forceinline__ void apply(const msa_rows_args& a, int m, int n, int64_t col, float v) const {
    if constexpr (EPI == MSA_ROWS_F32) {
      if (a.cap > 0.f) v = a.cap * tanh_f(v / a.cap);
      if (a.add) v += a.add[col];
      static_cast<float*>(a.out)[m * a.out_stride + col] = v;
    } else {
      if (EPI == MSA_ROWS_PLAIN && n < a.gelu_n) v = gelu_tanh_f(v);
      static_cast<bf16_t*>(a.out)[m * a.out_stride + col] = f32_to_bf16(v);
    }
  }
};

template <>
struct Finish<MSA_ROWS_MAMBA> {
  static constexpr int kTaps = 4;            // more taps than this are read when they are needed
  float keep[kTaps - 1], tap[kTaps], bias;
  __device__ __forceinline__ void load(const msa_rows_args& a, int m, int n) {
    const int c = n - a.conv_lo;
    if (c < 0 || c >= a.conv_n) return;
    const float* kp = a.conv_state + (int64_t)a.slot[m] * (a.conv_k - 1) * a.conv_n + c;
    const float* tp = a.taps + (int64_t)c * a.conv_k;
    bias = a.conv_bias ? a.conv_bias[c] : 0.f;
#pragma unroll
    for (int j = 0; j < kTaps; ++j) {
      if (j + 1 < a.conv_k && j < kTaps - 1) keep[j] = kp[(int64_t)j * a.conv_n];
      if (j < a.conv_k) tap[j] = tp[j];
    }
  }
  __device__ __forceinline__ void apply(const msa_rows_args& a, int m, int n, int64_t col, float v) const {
    const int c = n - a.conv_lo;
    if (c >= 0 && c < a.conv_n) {
      float* kp = a.conv_state + (int64_t)a.slot[m] * (a.conv_k - 1) * a.conv_n + c;
      float y = bias;
      if (a.conv_k <= kTaps) {
#pragma unroll
        for (int j = 0; j < kTaps; ++j) {
          if (j + 1 < a.conv_k && j < kTaps - 1) {
            y += tap[j] * keep[j];
            if (j > 0) kp[(int64_t)(j - 1) * a.conv_n] = keep[j];
          }
          if (j + 1 == a.conv_k) y += tap[j] * v;
        }
      } else {
        const float* tp = a.taps + (int64_t)c * a.conv_k;
        for (int j = 0; j + 1 < a.conv_k; ++j) {
          const float old = kp[(int64_t)j * a.conv_n];
          y += tp[j] * old;
          if (j > 0) kp[(int64_t)(j - 1) * a.conv_n] = old;
        }
        y += tp[a.conv_k - 1] * v;
      }
      if (a.conv_k > 1) kp[(int64_t)(a.conv_k - 2) * a.conv_n] = v;
      v = silu_f(y);
    }
    static_cast<bf16_t*>(a.out)[m * a.out_stride + col] = f32_to_bf16(v);
  }
};

template <>
struct Finish<MSA_ROWS_RESIDUAL> {
  float x, gate, w, b, mix, before;
  __device__ __forceinline__ void load(const msa_rows_args& a, int m, int n) {
    x = a.x_in[(int64_t)m * a.N + n];
    gate = bf16_to_f32(static_cast<const bf16_t*>(a.gate)[m * a.gate_stride + n]) + a.gate_bias[n];
    if (!a.norm.w) return;
    w = a.norm.w[n];
    b = a.norm.b[n];
    if (!a.shift) return;
    mix = a.shift[n];
    before = a.prev[(int64_t)a.slot[m] * a.N + n];
  }
  __device__ __forceinline__ void apply(const msa_rows_args& a, int m, int n, int64_t, float v) const {
    const int64_t at = (int64_t)m * a.N + n;
    const float y = x + sigmoid_f(gate) * v;
    a.x_out[at] = y;
    if (!a.norm.w) return;
    const float h = tanh_f(a.norm.alpha * y) * w + b;
    if (a.h) static_cast<bf16_t*>(a.h)[at] = f32_to_bf16(h);
    if (!a.shift) return;
    a.prev[(int64_t)a.slot[m] * a.N + n] = h;
    static_cast<bf16_t*>(a.h_shift)[at] = f32_to_bf16(h + (before - h) * mix);
  }
};

// A (gate, up) pair of neighbouring columns, in the lane of the even one.
template <>
struct Finish<MSA_ROWS_GLU> {
  __device__ __forceinline__ void load(const msa_rows_args& a, int m, int n) {}
  __device__ __forceinline__ void apply(const msa_rows_args& a, int m, int n, float gate, float up) const {
    if (n & 1) return;
    static_cast<bf16_t*>(a.out)[m * a.out_stride + (n >> 1)] = f32_to_bf16(clamped_glu_f(gate, up, a.glu_limit, a.glu_alpha, a.glu_shift));
  }
};

template <int EPI, int R>
__global__ __launch_bounds__(kMaxWaves * 64) void rows_linear_kernel(msa_rows_args a, int32_t rows_per_wg) {
  constexpr int J = kVectors<R>, kUnit = 32 * J;
  extern __shared__ __align__(16) float part[];   // [waves][R][64][4]
  const int tid = threadIdx.x, lane = tid & 63, waves = blockDim.x >> 6;
  const int wave = __builtin_amdgcn_readfirstlane(tid >> 6);
  const int n_l = lane & 15, g = lane >> 4;
  const int n_base = blockIdx.x * rows_per_wg, grp = blockIdx.y;
  const int row_bytes = a.K * 2;
  const int rows_w = min(rows_per_wg, a.N - n_base);
  const bool second = n_base >= a.n_b;
  const int64_t xs = second ? a.x_b_stride : a.x_stride;
  const char* xbase = static_cast<const char*>(second ? a.x_b : a.x) + (int64_t)grp * row_bytes;
  const __amdgpu_buffer_rsrc_t rs_w = __builtin_amdgcn_make_buffer_rsrc(
      const_cast<char*>(static_cast<const char*>(a.w)) + ((int64_t)grp * a.N + n_base) * row_bytes, 0, rows_w * row_bytes, 0x00020000);
  const __amdgpu_buffer_rsrc_t rs_x = __builtin_amdgcn_make_buffer_rsrc(
      const_cast<char*>(xbase), 0, (int)((a.M - 1) * xs * 2 + row_bytes), 0x00020000);
  const int voff_w = n_l * row_bytes + g * 16, voff_x = n_l * (int)(xs * 2) + g * 16;
  constexpr int kFar = 0x7ff00000;          // past every extent, whatever is added: reads zeros
  const int units = (a.K + kUnit - 1) / kUnit;
  const int u0 = units * wave / waves, u1 = units * (wave + 1) / waves;

  // output i of a row group: lane i / 4, element i % 4 of its accumulator
  auto row_of = [](int i) { return 4 * (i >> 6) + (i & 3); };
  auto col_of = [](int i) { return (i >> 2) & 15; };
  Finish<EPI> fin;                          // of this thread's first output
  {
    const int m = row_of(tid & 255), nr = 16 * (tid >> 8) + col_of(tid & 255);
    if (tid < R * 256 && m < a.M && nr < rows_w) fin.load(a, m, n_base + nr);
  }

  floatx4_t acc[R];
#pragma unroll
  for (int r = 0; r < R; ++r) acc[r] = floatx4_t{0.f, 0.f, 0.f, 0.f};
  u32x4_t fw[2][R][J], fx[2][J];
  auto load_unit = [&](int slot, int u) {
    const int k_off = u * kUnit * 2;
#pragma unroll
    for (int j = 0; j < J; ++j) {
      const bool in = k_off + j * 64 + g * 16 < row_bytes;        // pieces behind K read as zero
      fx[slot][j] = __builtin_amdgcn_raw_buffer_load_b128(rs_x, in ? voff_x : kFar, k_off + j * 64, 0);
#pragma unroll
      for (int r = 0; r < R; ++r)
        fw[slot][r][j] = __builtin_amdgcn_raw_buffer_load_b128(rs_w, in ? voff_w + r * 16 * row_bytes : kFar, k_off + j * 64, 0);
    }
  };
  auto mul_unit = [&](int slot) {
#pragma unroll
    for (int j = 0; j < J; ++j)
#pragma unroll
      for (int r = 0; r < R; ++r)
        acc[r] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(__builtin_bit_cast(bf16x8_t, fx[slot][j]),
                                                         __builtin_bit_cast(bf16x8_t, fw[slot][r][j]), acc[r], 0, 0, 0);
  };
  if (u0 < u1) load_unit(0, u0);
  int u = u0;
  for (; u + 2 <= u1; u += 2) {
    load_unit(1, u + 1);
    mul_unit(0);
    if (u + 2 < u1) load_unit(0, u + 2);
    mul_unit(1);
  }
  if (u < u1) mul_unit(0);

#pragma unroll
  for (int r = 0; r < R; ++r) *reinterpret_cast<floatx4_t*>(&part[((wave * R + r) * 64 + lane) * 4]) = acc[r];
  __syncthreads();

  auto total = [&](int r, int i) {
    float v = 0.f;
    for (int w = 0; w < waves; ++w) v += part[(w * R + r) * 256 + i];
    return v;
  };
  if constexpr (EPI == MSA_ROWS_GRU) {
    if (!second) {
      for (int i = tid; i < 256; i += blockDim.x) {
        const int m = row_of(i), c = n_base / (3 * kGruGroup) * kGruGroup + col_of(i);
        if (m >= a.M || c >= a.gru_n) continue;
        float* st = a.gru_state + (int64_t)a.slot[m] * a.gru_n + c;
        const float before = *st, zb = a.z_bias[c], ub = a.u_bias[c];
        const float z = sigmoid_f(total(0, i) + zb), uu = total(1, i) + ub, gt = total(2, i);
        const float S = (1.0f - z) * before + z * (uu >= 0.f ? uu + 0.5f : sigmoid_f(uu));
        *st = S;
        static_cast<bf16_t*>(a.out2)[(int64_t)m * a.gru_n + c] = f32_to_bf16(S * silu_f(gt));
      }
      return;
    }
  }
  for (int o = tid; o < R * 256; o += blockDim.x) {
    const int r = o >> 8, i = o & 255;
    const int m = row_of(i), nr = 16 * r + col_of(i), n = n_base + nr;
    if (m >= a.M || nr >= rows_w) continue;
    if constexpr (EPI == MSA_ROWS_GLU) {    // (rows come in pairs: the neighbouring column is in this wavefront, four lanes on)
      const float v = total(r, i), up = __shfl_xor(v, 4);
      fin.apply(a, m, n, v, up);
    } else {
      if (o != tid) fin.load(a, m, n);
      fin.apply(a, m, n, (int64_t)grp * a.N + n, total(r, i));
    }
  }
}

// Streaming form for matrices with many rows per compute unit (input projections, up, the head): a workgroup stays for the
// whole launch.  Wavefront w owns the K slice [32 F w, 32 F (w + 1)) for every item the workgroup visits and keeps its
// activations of that slice in registers, so they are read once per workgroup.  An item is up to 16 weight rows (as many as
// make every workgroup's share equal), its F vectors per lane requested kStages - 1 items ahead; partial sums meet in two LDS
// buffers behind one barrier per item, four threads add up an output.  A workgroup's items are contiguous, so it changes from
// the first operand's rows to the second's at most once.
constexpr int kPartStride = 260;            // floats per wavefront's partial block: the four adders of an output hit distinct banks

template <int EPI, int F>
__global__ __launch_bounds__(kMaxWaves * 64) void rows_stream_kernel(msa_rows_args a, int32_t rows_per_item, int32_t items_a,
                                                                     int32_t items, int32_t per_wg) {
  constexpr int kStages = F <= 5 ? 3 : 2;
  __shared__ __align__(16) float part[2][kMaxWaves][kPartStride];
  const int tid = threadIdx.x, lane = tid & 63;
  const int wave = __builtin_amdgcn_readfirstlane(tid >> 6);
  const int n_l = lane & 15, g = lane >> 4;
  const int row_bytes = a.K * 2, slice = wave * (F * 64);
  constexpr int kFar = 0x7ff00000;
  const int i0 = blockIdx.x * per_wg, i1 = min(items, i0 + per_wg);
  int at[F];                                // this lane's byte offsets in a row, or past every extent
#pragma unroll
  for (int f = 0; f < F; ++f) at[f] = slice + f * 64 + g * 16 < row_bytes ? slice + f * 64 + g * 16 : kFar;
  auto base_of = [&](int item) { return item < items_a ? item * rows_per_item : a.n_b + (item - items_a) * rows_per_item; };
  auto rows_of = [&](int item) {
    if (item >= i1) return 0;
    return min(rows_per_item, (item < items_a ? min(a.n_b, a.N) : a.N) - base_of(item));
  };
  u32x4_t xf[F];
  auto load_x = [&](bool second) {
    const int64_t xs = second ? a.x_b_stride : a.x_stride;
    const __amdgpu_buffer_rsrc_t rs_x = __builtin_amdgcn_make_buffer_rsrc(
        const_cast<char*>(static_cast<const char*>(second ? a.x_b : a.x)), 0, (int)((a.M - 1) * xs * 2 + row_bytes), 0x00020000);
#pragma unroll
    for (int f = 0; f < F; ++f) xf[f] = __builtin_amdgcn_raw_buffer_load_b128(rs_x, at[f] == kFar ? kFar : n_l * (int)(xs * 2) + at[f], 0, 0);
  };
  u32x4_t fw[kStages][F];
  auto load_w = [&](auto slot_tag, int item) {
    constexpr int slot = decltype(slot_tag)::value;
    // an empty extent (behind the last item) reads zeros and touches no memory
    const int extent = __builtin_amdgcn_readfirstlane(max(0, rows_of(item)) * row_bytes);
    const int base = __builtin_amdgcn_readfirstlane(item < i1 ? base_of(item) : 0);
    const __amdgpu_buffer_rsrc_t rs_w = __builtin_amdgcn_make_buffer_rsrc(
        const_cast<char*>(static_cast<const char*>(a.w)) + (int64_t)base * row_bytes, 0, extent, 0x00020000);
#pragma unroll
    for (int f = 0; f < F; ++f)
      fw[slot][f] = __builtin_amdgcn_raw_buffer_load_b128(rs_w, at[f] == kFar ? kFar : n_l * row_bytes + at[f], 0, 0);
  };
  bool second = i0 >= items_a;
  load_x(second);
  load_w(std::integral_constant<int, 0>{}, i0);
  if constexpr (kStages == 3) load_w(std::integral_constant<int, 1>{}, i0 + 1);
  const int o = tid >> 2, quarter = tid & 3;
  const int m = 4 * (o >> 6) + (o & 3), nr = (o >> 2) & 15;
  auto step = [&](int item, auto slot_tag) {
    constexpr int slot = decltype(slot_tag)::value;
    load_w(std::integral_constant<int, (slot + kStages - 1) % kStages>{}, item + kStages - 1);
    if (!second && item >= items_a && item < i1) {
      second = true;
      load_x(true);
    }
    const bool mine = quarter == 0 && m < a.M && nr < rows_of(item);
    const int n = base_of(item) + nr;
    Finish<EPI> fin;
    if (mine) fin.load(a, m, n);
    floatx4_t acc = floatx4_t{0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int f = 0; f < F; ++f)
      acc = __builtin_amdgcn_mfma_f32_16x16x32_bf16(__builtin_bit_cast(bf16x8_t, xf[f]), __builtin_bit_cast(bf16x8_t, fw[slot][f]), acc, 0, 0, 0);
    float(*buf)[kPartStride] = part[item & 1];
    *reinterpret_cast<floatx4_t*>(&buf[wave][lane * 4]) = acc;
    __syncthreads();
    float v = (buf[4 * quarter][o] + buf[4 * quarter + 1][o]) + (buf[4 * quarter + 2][o] + buf[4 * quarter + 3][o]);
    v += __shfl_xor(v, 1);
    v += __shfl_xor(v, 2);
    if constexpr (EPI == MSA_ROWS_GLU) {
      const float up = __shfl_xor(v, 16);
      if (mine) fin.apply(a, m, n, v, up);
    } else if (mine) {
      fin.apply(a, m, n, n, v);
    }
  };
  for (int item = i0; item < i1; item += kStages) {       // whole rounds: items behind the last read zeros and store nothing
    step(item, std::integral_constant<int, 0>{});
    step(item + 1, std::integral_constant<int, 1>{});
    if constexpr (kStages == 3) step(item + 2, std::integral_constant<int, 2>{});
  }
}

template <int EPI, int F>
int launch_stream(const msa_rows_args& a, hipStream_t st) {
  const int cus = device_compute_units();
  const int n_a = std::min(a.n_b, a.N), n_b = a.N - n_a;
  const int iters = (a.N + 16 * cus - 1) / (16 * cus);
  int rpi = std::min(16, std::max(1, (a.N + iters * cus - 1) / (iters * cus)));
  if (EPI == MSA_ROWS_GLU) rpi = (rpi + 1) & ~1;                      // pairs stay together
  auto split = [&] { return (n_a + rpi - 1) / rpi + (n_b + rpi - 1) / rpi; };   // the second operand's rows start an item of their own
  while (rpi < 16 && split() > iters * cus) ++rpi;
  const int items_a = (n_a + rpi - 1) / rpi, items = split();
  const int per_wg = (items + cus - 1) / cus;
  rows_stream_kernel<EPI, F><<<(items + per_wg - 1) / per_wg, kMaxWaves * 64, 0, st>>>(a, rpi, items_a, items, per_wg);
  MSA_LAUNCH_CHECK();
  return MSA_OK;
}
template <int EPI>
int launch_stream(const msa_rows_args& a, hipStream_t st) {
  const int f = (a.K + 511) / 512;
  if (f <= 2) return launch_stream<EPI, 2>(a, st);
  if (f <= 3) return launch_stream<EPI, 3>(a, st);
  if (f <= 4) return launch_stream<EPI, 4>(a, st);
  if constexpr (EPI == MSA_ROWS_MAMBA) return launch_stream<EPI, 5>(a, st);    // (its operands would not fit beside eight vectors)
  else return f <= 5 ? launch_stream<EPI, 5>(a, st) : launch_stream<EPI, 8>(a, st);
}

template <int EPI, int R>
int launch_rows(const msa_rows_args& a, int waves, int rows_per_wg, hipStream_t st) {
  const size_t lds = (size_t)waves * R * 256 * sizeof(float);       // at most 48 KB
  rows_linear_kernel<EPI, R><<<dim3((a.N + rows_per_wg - 1) / rows_per_wg, a.groups), waves * 64, lds, st>>>(a, rows_per_wg);
  MSA_LAUNCH_CHECK();
  return MSA_OK;
}

}  // namespace

extern "C" int msa_rows_linear(const msa_rows_args* args, int32_t epilogue, void* stream) {
  MSA_REQUIRE(args != nullptr, "msa_rows_linear: null arguments");
  msa_rows_args a = *args;
  MSA_REQUIRE(a.x && a.w && a.M > 0 && a.M <= 16 && a.N > 0 && a.K > 0 && a.K % 8 == 0 && a.groups > 0 && a.groups <= 65535,
              "msa_rows_linear: M=%d (1..16) N=%d K=%d (a multiple of 8) groups=%d", a.M, a.N, a.K, a.groups);
  MSA_REQUIRE(a.x_stride >= (int64_t)a.K * a.groups && a.x_stride % 8 == 0 && a.x_stride * 32 < ((int64_t)1 << 30) &&
                  (int64_t)64 * a.K * 2 < ((int64_t)1 << 30), "msa_rows_linear: x_stride=%lld K=%d", (long long)a.x_stride, a.K);
  const bool two = a.n_b < a.N;
  MSA_REQUIRE(a.n_b > 0 && (!two || (a.x_b && a.groups == 1 && a.x_b_stride >= a.K && a.x_b_stride % 8 == 0 &&
                                     a.x_b_stride * 32 < ((int64_t)1 << 30))), "msa_rows_linear: second operand");
  MSA_REQUIRE((((uintptr_t)a.x | (uintptr_t)a.x_b | (uintptr_t)a.w) & 15) == 0, "msa_rows_linear: x / x_b / w must be 16-byte aligned");
  switch (epilogue) {
    case MSA_ROWS_PLAIN:
    case MSA_ROWS_F32:
      MSA_REQUIRE(a.out && a.out_stride >= (int64_t)a.N * a.groups, "msa_rows_linear: output");
      break;
    case MSA_ROWS_RESIDUAL:
      MSA_REQUIRE(a.x_in && a.x_out && a.gate && a.gate_bias && a.gate_stride >= a.N && a.groups == 1 && !two, "msa_rows_linear: residual arguments");
      MSA_REQUIRE(!a.norm.w || (a.norm.b && (a.h || a.shift)), "msa_rows_linear: norm arguments");
      MSA_REQUIRE(!a.shift || (a.norm.w && a.prev && a.h_shift && a.slot), "msa_rows_linear: shift arguments");
      break;
    case MSA_ROWS_MAMBA:
      MSA_REQUIRE(a.out && a.out_stride >= a.N && a.groups == 1 && a.taps && a.slot && a.conv_k >= 1 && a.conv_lo >= 0 &&
                      a.conv_n > 0 && a.conv_lo + a.conv_n <= a.n_b && (a.conv_k == 1 || a.conv_state), "msa_rows_linear: convolution arguments");
      break;
    case MSA_ROWS_GLU:
      MSA_REQUIRE(a.out && a.N % 2 == 0 && a.out_stride >= a.N / 2 && a.groups == 1 && !two, "msa_rows_linear: gated unit arguments");
      break;
    case MSA_ROWS_GRU:
      MSA_REQUIRE(a.out2 && a.z_bias && a.u_bias && a.gru_state && a.slot && a.groups == 1 && a.gru_n > 0 &&
                      a.n_b == (a.gru_n + kGruGroup - 1) / kGruGroup * 3 * kGruGroup && (!two || (a.out && a.out_stride >= a.N)),
                  "msa_rows_linear: recurrence arguments");
      break;
    default:
      msa_set_error("msa_rows_linear: epilogue %d", epilogue);
      return MSA_EINVAL;
  }
  // Row groups per workgroup: two when N alone fills the chip (the activations are then read half as often); fewer than 16
  // rows when that leaves compute units without a workgroup.  Wavefronts: a few thousand in the launch, and a share of K each.
  const bool gru = epilogue == MSA_ROWS_GRU;
  int R = gru ? 3 : ((int64_t)a.N * a.groups >= 6144 && (!two || a.n_b % 32 == 0) && a.N >= 32) ? 2 : 1;
  int rows_per_wg = 16 * R;
  MSA_REQUIRE(!two || a.n_b % rows_per_wg == 0, "msa_rows_linear: n_b=%d must be a multiple of %d", a.n_b, rows_per_wg);
  if (R == 1 && !two && a.groups == 1 && (a.N + 15) / 16 < device_compute_units())
    rows_per_wg = std::min(16, std::max(8, (a.N + device_compute_units() - 1) / device_compute_units()));
  if (epilogue == MSA_ROWS_GLU) rows_per_wg = (rows_per_wg + 1) & ~1;
  const int64_t wgs = (int64_t)((a.N + rows_per_wg - 1) / rows_per_wg) * a.groups;
  const int kUnit = 32 * (R == 3 ? kVectors<3> : kVectors<1>);
  const int units = (a.K + kUnit - 1) / kUnit;
  int waves = (int)std::min<int64_t>(kMaxWaves, std::max<int64_t>(1, (4096 + wgs - 1) / wgs));
  waves = std::max(1, std::min(waves, units));
  for (int cand = waves; cand >= std::max(1, waves / 2); --cand)
    if (units % cand == 0) { waves = cand; break; }
  hipStream_t st = as_stream(stream);
  // Many rows per compute unit: the streaming form.
  if (a.groups == 1 && a.K > 512 && a.K <= 4096 && a.N >= 2 * 16 * device_compute_units()) {
    if (epilogue == MSA_ROWS_PLAIN) return launch_stream<MSA_ROWS_PLAIN>(a, st);
    if (epilogue == MSA_ROWS_F32) return launch_stream<MSA_ROWS_F32>(a, st);
    if (epilogue == MSA_ROWS_GLU) return launch_stream<MSA_ROWS_GLU>(a, st);
    if (epilogue == MSA_ROWS_MAMBA && a.K <= 2560) return launch_stream<MSA_ROWS_MAMBA>(a, st);
  }
  switch (epilogue * 4 + R) {
    case MSA_ROWS_PLAIN * 4 + 1: return launch_rows<MSA_ROWS_PLAIN, 1>(a, waves, rows_per_wg, st);
    case MSA_ROWS_PLAIN * 4 + 2: return launch_rows<MSA_ROWS_PLAIN, 2>(a, waves, rows_per_wg, st);
    case MSA_ROWS_F32 * 4 + 1: return launch_rows<MSA_ROWS_F32, 1>(a, waves, rows_per_wg, st);
    case MSA_ROWS_F32 * 4 + 2: return launch_rows<MSA_ROWS_F32, 2>(a, waves, rows_per_wg, st);
    case MSA_ROWS_RESIDUAL * 4 + 1: return launch_rows<MSA_ROWS_RESIDUAL, 1>(a, waves, rows_per_wg, st);
    case MSA_ROWS_RESIDUAL * 4 + 2: return launch_rows<MSA_ROWS_RESIDUAL, 2>(a, waves, rows_per_wg, st);
    case MSA_ROWS_MAMBA * 4 + 1: return launch_rows<MSA_ROWS_MAMBA, 1>(a, waves, rows_per_wg, st);
    case MSA_ROWS_MAMBA * 4 + 2: return launch_rows<MSA_ROWS_MAMBA, 2>(a, waves, rows_per_wg, st);
    case MSA_ROWS_GLU * 4 + 1: return launch_rows<MSA_ROWS_GLU, 1>(a, waves, rows_per_wg, st);
    case MSA_ROWS_GLU * 4 + 2: return launch_rows<MSA_ROWS_GLU, 2>(a, waves, rows_per_wg, st);
    case MSA_ROWS_GRU * 4 + 3: return launch_rows<MSA_ROWS_GRU, 3>(a, waves, rows_per_wg, st);
  }
  msa_set_error("msa_rows_linear: no kernel for epilogue %d with %d row groups", epilogue, R);
  return MSA_EINVAL;
}
