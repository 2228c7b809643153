// A residual stream that is normed behind every sum: the step of a layer whose sublayers read the stream itself and whose results enter
// it as x <- N(alpha x + f(x)).
//
// One kernel does, per row of D float32 numbers, whichever of these it is given, in this order:
//   write:  x <- N1(alpha x + y),  y the sublayer's result: the sum of whatever is there of
//             y                                            a finished result [T][D]
//             part[0] + .. + part[S-1] + part_bias         a product that has left its K ranges [S][T][D] unsummed
//             sum_c weights[t][c] expert_out[pos_of[t * top + c]]    routed experts' outputs [pairs][D] that nobody has summed, c in order
//   read:   h = x as it is, rounded to h's type, or h = N2(x)  (the norm ahead of the head), into h_out
//   rows != null: only these rows (output row r is row rows[r]); x is not stored then: a selection may name a row twice, and the rows
//                 left out stay behind anyway.
// N is a layer norm, (v - mean) / sqrt(mean squared deviation + eps) * w (+ b), or (rms) v / sqrt(mean(v^2) + eps) * w (+ b). All sums and
// statistics are 32-bit, the squared deviations from the rounded mean (two passes over registers). One workgroup of 256 threads per
// row; the row lives in registers, VEC neighbouring numbers at a time.
#include "common.h"

#define SN_NT 256
#define SN_MAX_TOP 64

struct SumNormArgs {
  float* x;
  float alpha;
  const float* y;
  const float* ranges;
  int n_ranges;
  size_t range_stride;
  const float* range_bias;
  const float* expert_out;
  const int* pos_of;
  const float* weights;
  int top;
  const float *w1, *b1;
  float eps1;
  int rms1;
  const float *w2, *b2;
  float eps2;
  int rms2;
  void* h_out;
  const int* rows;
  int D;
};

template <int VEC>
__device__ __forceinline__ void sn_load(const float* p, float (&v)[VEC]) {
  if (VEC == 4) {
    const float4 q = *reinterpret_cast<const float4*>(p);
    v[0] = q.x, v[1 % VEC] = q.y, v[2 % VEC] = q.z, v[3 % VEC] = q.w;
  } else {
    v[0] = *p;
  }
}
template <int VEC>
__device__ __forceinline__ void sn_store(float* p, const float (&v)[VEC]) {
  if (VEC == 4) *reinterpret_cast<float4*>(p) = make_float4(v[0], v[1 % VEC], v[2 % VEC], v[3 % VEC]);
  else *p = v[0];
}
template <int VEC>
__device__ __forceinline__ void sn_store(bf16_t* p, const float (&v)[VEC]) {
  if (VEC == 4) *reinterpret_cast<uint2*>(p) = make_uint2(float2_to_bf16x2(v[0], v[1 % VEC]), float2_to_bf16x2(v[2 % VEC], v[3 % VEC]));
  else *p = float_to_bf16(v[0]);
}

// the norm of the row in v, in place; w and b are in registers already
template <int VEC, int PER>
__device__ __forceinline__ void sn_norm(float (&v)[PER][VEC], const float (&w)[PER][VEC], const float (&b)[PER][VEC], int D, float eps, int rms,
                                        float* red) {
  const int e0 = threadIdx.x * VEC;
  const float inv_n = 1.0f / (float)D;
  float mean = 0.f;
  if (!rms) {
    float s = 0.f;
#pragma unroll
    for (int i = 0; i < PER; ++i)
#pragma unroll
      for (int e = 0; e < VEC; ++e) s += v[i][e];  // numbers beyond the row are zeros
    mean = block_sum<SN_NT>(s, red) * inv_n;
  }
  float ss = 0.f;
#pragma unroll
  for (int i = 0; i < PER; ++i)
    if (e0 + SN_NT * VEC * i < D)
#pragma unroll
      for (int e = 0; e < VEC; ++e) {
        v[i][e] -= mean;
        ss = fmaf(v[i][e], v[i][e], ss);
      }
  const float r = 1.0f / sqrtf(block_sum<SN_NT>(ss, red + SN_NT / 64) * inv_n + eps);
#pragma unroll
  for (int i = 0; i < PER; ++i)
    if (e0 + SN_NT * VEC * i < D)
#pragma unroll
      for (int e = 0; e < VEC; ++e) v[i][e] = v[i][e] * r * w[i][e] + b[i][e];
}

template <typename TO, int VEC, int PER>
__global__ void __launch_bounds__(SN_NT)
sum_norm_kernel(const SumNormArgs a) {
  __shared__ float red[2 * (SN_NT / 64)];
  __shared__ int pos_s[SN_MAX_TOP];
  __shared__ float wt_s[SN_MAX_TOP];
  const int tid = threadIdx.x, D = a.D;
  const int r = blockIdx.x, row = a.rows ? a.rows[r] : r;
  const size_t base = (size_t)row * D;
  const bool write = a.w1 != nullptr;
  float v[PER][VEC], w[PER][VEC], b[PER][VEC];
  int at[PER];
  if (a.top > 0) {
    if (tid < a.top) {
      pos_s[tid] = a.pos_of[(size_t)row * a.top + tid];
      wt_s[tid] = a.weights[(size_t)row * a.top + tid];
    }
    __syncthreads();
  }
  // loads stand under no condition (clamped into the row): all of them are in flight before the first is used
#pragma unroll
  for (int i = 0; i < PER; ++i) {
    at[i] = min((tid + SN_NT * i) * VEC, D - VEC);
    sn_load<VEC>(a.x + base + at[i], v[i]);
    if (write) sn_load<VEC>(a.w1 + at[i], w[i]);
  }
  if (write) {
    if (a.y != nullptr) {
      float y[PER][VEC];
#pragma unroll
      for (int i = 0; i < PER; ++i) sn_load<VEC>(a.y + base + at[i], y[i]);
#pragma unroll
      for (int i = 0; i < PER; ++i)
#pragma unroll
        for (int e = 0; e < VEC; ++e) v[i][e] = fmaf(a.alpha, v[i][e], y[i][e]);
    } else {
#pragma unroll
      for (int i = 0; i < PER; ++i)
#pragma unroll
        for (int e = 0; e < VEC; ++e) v[i][e] *= a.alpha;
    }
    if (a.n_ranges > 0) {
#pragma unroll
      for (int i = 0; i < PER; ++i) {
        float sum[VEC] = {};
#pragma unroll 8
        for (int s = 0; s < a.n_ranges; ++s) {
          float p[VEC];
          sn_load<VEC>(a.ranges + (size_t)s * a.range_stride + base + at[i], p);
#pragma unroll
          for (int e = 0; e < VEC; ++e) sum[e] += p[e];
        }
        if (a.range_bias != nullptr) {
          float p[VEC];
          sn_load<VEC>(a.range_bias + at[i], p);
#pragma unroll
          for (int e = 0; e < VEC; ++e) sum[e] += p[e];
        }
#pragma unroll
        for (int e = 0; e < VEC; ++e) v[i][e] += sum[e];
      }
    }
    if (a.top > 0) {
#pragma unroll
      for (int i = 0; i < PER; ++i) {
        float sum[VEC] = {};
#pragma unroll 4
        for (int c = 0; c < a.top; ++c) {
          float p[VEC];
          sn_load<VEC>(a.expert_out + (size_t)pos_s[c] * D + at[i], p);
          const float wt = wt_s[c];
#pragma unroll
          for (int e = 0; e < VEC; ++e) sum[e] = fmaf(wt, p[e], sum[e]);
        }
#pragma unroll
        for (int e = 0; e < VEC; ++e) v[i][e] += sum[e];
      }
    }
  }
#pragma unroll
  for (int i = 0; i < PER; ++i)
    if ((tid + SN_NT * i) * VEC >= D)
#pragma unroll
      for (int e = 0; e < VEC; ++e) v[i][e] = 0.f;
  auto load_bias = [&](const float* bias) {
#pragma unroll
    for (int i = 0; i < PER; ++i) {
      if (bias != nullptr) sn_load<VEC>(bias + at[i], b[i]);
      else
#pragma unroll
        for (int e = 0; e < VEC; ++e) b[i][e] = 0.f;
    }
  };
  if (write) {
    load_bias(a.b1);
    sn_norm<VEC, PER>(v, w, b, D, a.eps1, a.rms1, red);
    if (a.rows == nullptr)
#pragma unroll
      for (int i = 0; i < PER; ++i)
        if ((tid + SN_NT * i) * VEC < D) sn_store<VEC>(a.x + base + at[i], v[i]);
  }
  if (a.h_out == nullptr) return;
  if (a.w2 != nullptr) {
#pragma unroll
    for (int i = 0; i < PER; ++i) sn_load<VEC>(a.w2 + at[i], w[i]);
    load_bias(a.b2);
    sn_norm<VEC, PER>(v, w, b, D, a.eps2, a.rms2, red);
  }
  TO* h = (TO*)a.h_out + (size_t)r * D;
#pragma unroll
  for (int i = 0; i < PER; ++i)
    if ((tid + SN_NT * i) * VEC < D) sn_store<VEC>(h + at[i], v[i]);
}

template <typename TO>
static bool sum_norm_launch(const SumNormArgs& a, int n, bool vec, hipStream_t stream) {
#define SN_CASE(V, P)                                                        \
  if (a.D <= SN_NT * (V) * (P)) {                                            \
    sum_norm_kernel<TO, V, P><<<n, SN_NT, 0, stream>>>(a);                   \
    return true;                                                             \
  }
  if (vec) {
    SN_CASE(4, 1) SN_CASE(4, 2) SN_CASE(4, 4) SN_CASE(4, 8) SN_CASE(4, 16)
  } else {
    SN_CASE(1, 1) SN_CASE(1, 4) SN_CASE(1, 16) SN_CASE(1, 64)
  }
#undef SN_CASE
  return false;
}

extern "C" int lev_sum_norm(float* x, float alpha, const float* y, const float* ranges, int n_ranges, int T, const float* range_bias,
                            const float* expert_out, const int* pos_of, const float* weights, int top, const float* w1, const float* b1, float eps1,
                            int rms1, const float* w2, const float* b2, float eps2, int rms2, void* h_out, int out_dtype, const int* rows, int n, int D,
                            hipStream_t stream) {
  LEV_REQUIRE(x != nullptr && n >= 0 && D > 0 && T >= 0, "sum_norm: a tensor is missing or bad sizes n=%d D=%d", n, D);
  LEV_REQUIRE(D <= SN_NT * 64, "sum_norm: a row of %d numbers (at most %d)", D, SN_NT * 64);
  LEV_REQUIRE(w1 != nullptr || h_out != nullptr, "sum_norm: nothing to do");
  LEV_REQUIRE(w1 != nullptr || (y == nullptr && n_ranges == 0 && top == 0), "sum_norm: a result to add needs the norm behind the sum");
  LEV_REQUIRE(n_ranges >= 0 && (n_ranges == 0 || ranges != nullptr), "sum_norm: an unfinished product needs its ranges");
  LEV_REQUIRE(top >= 0 && top <= SN_MAX_TOP && (top == 0 || (expert_out && pos_of && weights)), "sum_norm: %d experts a token (at most %d) need outputs, places and weights", top, SN_MAX_TOP);
  LEV_REQUIRE(w2 == nullptr || h_out != nullptr, "sum_norm: the second norm needs an output");
  LEV_REQUIRE(rows == nullptr || h_out != nullptr, "sum_norm: a selection of rows needs an output");
  LEV_REQUIRE((void*)h_out != (void*)x, "sum_norm: the output must not be the stream");
  LEV_REQUIRE(out_dtype == LEV_F32 || out_dtype == LEV_BF16, "sum_norm: unknown dtype %d", out_dtype);
  if (n == 0) return 0;
  SumNormArgs a{x, alpha, y, ranges, n_ranges, (size_t)T * D, range_bias, expert_out, pos_of, weights, top, w1, b1, eps1, rms1, w2, b2, eps2, rms2, h_out, rows, D};
  const uintptr_t all = (uintptr_t)x | (uintptr_t)y | (uintptr_t)ranges | (uintptr_t)range_bias | (uintptr_t)expert_out | (uintptr_t)w1 | (uintptr_t)b1 |
                        (uintptr_t)w2 | (uintptr_t)b2 | (uintptr_t)h_out;
  const bool vec = D % 4 == 0 && (all & 15) == 0;
  const bool ok = out_dtype == LEV_F32 ? sum_norm_launch<float>(a, n, vec, stream) : sum_norm_launch<bf16_t>(a, n, vec, stream);
  LEV_REQUIRE(ok, "sum_norm: no kernel for a row of %d numbers", D);
  return lev_check_launch("sum_norm");
}
