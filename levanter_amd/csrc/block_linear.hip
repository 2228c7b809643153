// A block-diagonal linear map: the input row is B parts of n_in columns, part b goes through its own matrix
// w[b] ([n_out][n_in], each output's inputs contiguous) and gives part b of the output row:
//     out[t][b * n_out + o] = sum_i w[b][o][i] * a[t][b * n_in + i] + bias[b * n_out + o]
// times sigmoid(gate[t][b * n_out + o]) where there is a gate (of the weights' type; an output gate per element).
// (per-head projections of an attention with a latent, the gates of a recurrence that are square matrices per block).
// Plain 32-bit FMA for the few rows of a decoding step; the launcher sends prompt-sized row counts to the matrix
// products, block by block. One wave per output column and tile of TT rows: the lanes share the inputs of the column
// (coalesced over the weights' row), the sums of the lanes are added across the wave.
// a may be float32 while the weights are bfloat16 (the 32-bit result of an attention kernel goes in unrounded).
#include "common.h"

#define BL_TT 8

template <typename TA, typename TW, typename TO>
__global__ void __launch_bounds__(256)
block_linear_kernel(const TA* __restrict__ a, long a_stride, const TW* __restrict__ w, const float* __restrict__ bias, TO* __restrict__ out,
                    long o_stride, const TW* __restrict__ gate, long g_stride, int T, int B, int n_in, int n_out) {
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
  const long col = (long)blockIdx.x * 4 + wave;  // over B * n_out
  if (col >= (long)B * n_out) return;
  const int b = (int)(col / n_out);
  const int t0 = blockIdx.y * BL_TT;
  const TW* wr = w + (size_t)col * n_in;
  const TA* ar[BL_TT];
#pragma unroll
  for (int tt = 0; tt < BL_TT; ++tt) ar[tt] = a + (size_t)min(t0 + tt, T - 1) * a_stride + (size_t)b * n_in;  // rows beyond T: read, never stored
  float acc[BL_TT];
#pragma unroll
  for (int tt = 0; tt < BL_TT; ++tt) acc[tt] = 0.f;
  for (int i = lane; i < n_in; i += 64) {
    const float wv = to_float<TW>(wr[i]);
#pragma unroll
    for (int tt = 0; tt < BL_TT; ++tt) acc[tt] = fmaf(wv, to_float<TA>(ar[tt][i]), acc[tt]);
  }
  const float bv = bias ? bias[col] : 0.f;
#pragma unroll
  for (int tt = 0; tt < BL_TT; ++tt) {
    const float s = wave_sum(acc[tt]);
    if (lane == 0 && t0 + tt < T) {
      const float gv = gate ? 1.0f / (1.0f + expf(-to_float<TW>(gate[(size_t)(t0 + tt) * g_stride + col]))) : 1.0f;
      out[(size_t)(t0 + tt) * o_stride + col] = from_float<TO>((s + bv) * gv);
    }
  }
}

template <typename TA, typename TW, typename TO>
static void block_linear_launch(const void* a, long a_stride, const void* w, const float* bias, void* out, long o_stride,
                                const void* gate, long g_stride, int T, int B, int n_in, int n_out, hipStream_t stream) {
  dim3 grid((unsigned)(((long)B * n_out + 3) / 4), (T + BL_TT - 1) / BL_TT);
  block_linear_kernel<TA, TW, TO><<<grid, 256, 0, stream>>>((const TA*)a, a_stride, (const TW*)w, bias, (TO*)out, o_stride, (const TW*)gate, g_stride, T, B,
                                                         n_in, n_out);
}

extern "C" int lev_block_linear(const void* a, long a_stride, const void* w, const float* bias, void* out, long o_stride, const void* gate,
                                long g_stride, int T, int B, int n_in, int n_out, int a_dtype, int w_dtype, int out_dtype, hipStream_t stream) {
  LEV_REQUIRE(T >= 0 && B > 0 && n_in > 0 && n_out > 0, "block_linear: bad sizes T=%d blocks=%d in=%d out=%d", T, B, n_in, n_out);
  LEV_REQUIRE(a && w && out, "block_linear: a tensor is missing");
  LEV_REQUIRE(a_stride >= (long)B * n_in && o_stride >= (long)B * n_out && (!gate || g_stride >= (long)B * n_out), "block_linear: row strides are smaller than the rows");
  LEV_REQUIRE((T + BL_TT - 1) / BL_TT <= 65535, "block_linear: too many rows (%d) for this kernel", T);
  if (T == 0) return 0;
#define BL_CASE(A, W, O, TA, TW, TO)                                                                                   \
  if (a_dtype == A && w_dtype == W && out_dtype == O) {                                                                \
    block_linear_launch<TA, TW, TO>(a, a_stride, w, bias, out, o_stride, gate, g_stride, T, B, n_in, n_out, stream); \
    return lev_check_launch("block_linear");                                                                          \
  }
  BL_CASE(LEV_F32, LEV_F32, LEV_F32, float, float, float)
  BL_CASE(LEV_BF16, LEV_BF16, LEV_BF16, bf16_t, bf16_t, bf16_t)
  BL_CASE(LEV_BF16, LEV_BF16, LEV_F32, bf16_t, bf16_t, float)
  BL_CASE(LEV_F32, LEV_BF16, LEV_BF16, float, bf16_t, bf16_t)
  BL_CASE(LEV_F32, LEV_BF16, LEV_F32, float, bf16_t, float)
#undef BL_CASE
  return lev_fail("block_linear: no kernel for the dtypes a=%d w=%d out=%d", a_dtype, w_dtype, out_dtype);
}

// ------------------------------------------------------------------------------------------
// The same product on the matrix cores, for bfloat16 weights and any number of rows (prompts as well as decoding steps):
// one launch for all blocks, where a launch per block leaves the chip waiting on matrices of a few dozen KB. A wave owns
// 16 rows and NT tiles of 16 output columns of one block (4 where there are many rows, so that a fragment of inputs feeds four
// products; 1 for the few rows of a decoding step, so that the step has four times the waves); both operands go straight from global memory into
// 16x16x32 MFMA fragments (a block's weights and the rows' inputs stay in the caches between the waves that share them).
// The transposed product out^T = w a^T leaves each lane with four neighbouring outputs of one row. float32 inputs are
// rounded to bfloat16 on their way into the fragment. n_in must be a multiple of 8 (16-byte loads).
typedef __attribute__((ext_vector_type(8))) __bf16 blm_bf16x8;
typedef __attribute__((ext_vector_type(4))) float blm_f32x4;
typedef __attribute__((ext_vector_type(4))) uint32_t blm_u32x4;

__device__ __forceinline__ blm_bf16x8 blm_as_bf16x8(blm_u32x4 v) {
  union { blm_u32x4 u; blm_bf16x8 b; } c;
  c.u = v;
  return c.b;
}
__device__ __forceinline__ blm_u32x4 blm_load8(const bf16_t* p) { return *reinterpret_cast<const blm_u32x4*>(p); }
__device__ __forceinline__ blm_u32x4 blm_load8(const float* p) {
  const float4 lo = *reinterpret_cast<const float4*>(p), hi = *reinterpret_cast<const float4*>(p + 4);
  return blm_u32x4{float2_to_bf16x2(lo.x, lo.y), float2_to_bf16x2(lo.z, lo.w), float2_to_bf16x2(hi.x, hi.y), float2_to_bf16x2(hi.z, hi.w)};
}

__device__ __forceinline__ void blm_store4(float* p, const float (&v)[4]) { *reinterpret_cast<float4*>(p) = make_float4(v[0], v[1], v[2], v[3]); }
__device__ __forceinline__ void blm_store4(bf16_t* p, const float (&v)[4]) {
  *reinterpret_cast<uint2*>(p) = make_uint2(float2_to_bf16x2(v[0], v[1]), float2_to_bf16x2(v[2], v[3]));
}

template <typename TA, typename TO, int BLM_NT>
__global__ void __launch_bounds__(256)
block_linear_mfma_kernel(const TA* __restrict__ a, long a_stride, const bf16_t* __restrict__ w, const float* __restrict__ bias,
                         TO* __restrict__ out, long o_stride, const bf16_t* __restrict__ gate, long g_stride, int T, int n_in, int n_out, int col_sets,
                         int vec, int vec_gate) {
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6, col = lane & 15, g = lane >> 4;
  const int t0 = (blockIdx.x * 4 + wave) * 16;
  if (t0 >= T) return;  // the whole wave
  const int b = blockIdx.y / col_sets, o0 = (blockIdx.y % col_sets) * (16 * BLM_NT);
  const TA* arow = a + (size_t)min(t0 + col, T - 1) * a_stride + (size_t)b * n_in;  // rows beyond T: read again, never stored
  const bf16_t* wb = w + (size_t)b * n_out * n_in;
  const bf16_t* wrow[BLM_NT];
#pragma unroll
  for (int nt = 0; nt < BLM_NT; ++nt) wrow[nt] = wb + (size_t)min(o0 + 16 * nt + col, n_out - 1) * n_in;
  blm_f32x4 acc[BLM_NT];
#pragma unroll
  for (int nt = 0; nt < BLM_NT; ++nt) acc[nt] = blm_f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll 4
  for (int k0 = 0; k0 < n_in; k0 += 32) {
    const int kk = k0 + 8 * g, kc = min(kk, n_in - 8);  // loads stand under no condition; a chunk beyond the row counts as zeros
    blm_u32x4 av = blm_load8(arow + kc);
    const uint32_t keep = kk < n_in ? 0xffffffffu : 0u;
    av = blm_u32x4{av[0] & keep, av[1] & keep, av[2] & keep, av[3] & keep};
    blm_u32x4 wv[BLM_NT];
#pragma unroll
    for (int nt = 0; nt < BLM_NT; ++nt) wv[nt] = blm_load8(wrow[nt] + kc);
#pragma unroll
    for (int nt = 0; nt < BLM_NT; ++nt)
      acc[nt] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(blm_as_bf16x8(wv[nt]), blm_as_bf16x8(av), acc[nt], 0, 0, 0);
  }
  const int t = t0 + col;
  if (t >= T) return;
#pragma unroll
  for (int nt = 0; nt < BLM_NT; ++nt) {
    const int o = o0 + 16 * nt + 4 * g;
    if (o >= n_out) continue;
    const size_t c = (size_t)b * n_out + o;
    const int n = min(4, n_out - o);
    float v[4], gv[4] = {0.f, 0.f, 0.f, 0.f};
    if (gate != nullptr) {
      const bf16_t* gp = gate + (size_t)t * g_stride + c;
      if (vec_gate) {
        const uint2 x = *reinterpret_cast<const uint2*>(gp);
        gv[0] = __uint_as_float(x.x << 16), gv[1] = __uint_as_float(x.x & 0xffff0000u);
        gv[2] = __uint_as_float(x.y << 16), gv[3] = __uint_as_float(x.y & 0xffff0000u);
      } else {
#pragma unroll
        for (int r = 0; r < 4; ++r)
          if (r < n) gv[r] = bf16_to_float(gp[r]);
      }
    }
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      v[r] = acc[nt][r] + (bias && r < n ? bias[c + r] : 0.f);
      if (gate != nullptr) v[r] *= 1.0f / (1.0f + expf(-gv[r]));
    }
    TO* op = out + (size_t)t * o_stride + c;
    if (vec) {  // blocks, rows and the tensor at multiples of four numbers
      blm_store4(op, v);
    } else {
#pragma unroll
      for (int r = 0; r < 4; ++r)
        if (r < n) op[r] = from_float<TO>(v[r]);
    }
  }
}

extern "C" int lev_block_linear_mfma(const void* a, long a_stride, const void* w, const float* bias, void* out, long o_stride, const void* gate,
                                     long g_stride, int T, int B, int n_in, int n_out, int a_dtype, int out_dtype, hipStream_t stream) {
  LEV_REQUIRE(T >= 0 && B > 0 && n_in > 0 && n_out > 0, "block_linear: bad sizes T=%d blocks=%d in=%d out=%d", T, B, n_in, n_out);
  LEV_REQUIRE(a && w && out, "block_linear: a tensor is missing");
  LEV_REQUIRE(n_in % 8 == 0 && a_stride % 8 == 0 && ((uintptr_t)a & 15) == 0 && ((uintptr_t)w & 15) == 0,
              "block_linear (matrix cores): inputs of %d a block and a row stride of %ld must be multiples of 8, operands 16-byte aligned", n_in, a_stride);
  LEV_REQUIRE(a_stride >= (long)B * n_in && o_stride >= (long)B * n_out && (!gate || g_stride >= (long)B * n_out), "block_linear: row strides are smaller than the rows");
  if (T == 0) return 0;
  const int nt = T <= 32 ? 1 : 4;
  const int col_sets = (n_out + 16 * nt - 1) / (16 * nt);
  LEV_REQUIRE((long)B * col_sets <= 65535, "block_linear: too many column tiles (%ld)", (long)B * col_sets);
  dim3 grid((T + 63) / 64, B * col_sets);
  const int vec = n_out % 4 == 0 && o_stride % 4 == 0 && ((uintptr_t)out & (out_dtype == LEV_F32 ? 15 : 7)) == 0;
  const int vec_gate = n_out % 4 == 0 && g_stride % 4 == 0 && ((uintptr_t)gate & 7) == 0;
#define BLM_CASE(A, O, TA, TO)                                                                                                     \
  if (a_dtype == A && out_dtype == O) {                                                                                            \
    if (nt == 1)                                                                                                                   \
      block_linear_mfma_kernel<TA, TO, 1><<<grid, 256, 0, stream>>>((const TA*)a, a_stride, (const bf16_t*)w, bias, (TO*)out, o_stride, (const bf16_t*)gate, g_stride, T, n_in, \
                                                                   n_out, col_sets, vec, vec_gate);                                               \
    else                                                                                                                           \
      block_linear_mfma_kernel<TA, TO, 4><<<grid, 256, 0, stream>>>((const TA*)a, a_stride, (const bf16_t*)w, bias, (TO*)out, o_stride, (const bf16_t*)gate, g_stride, T, n_in, \
                                                                   n_out, col_sets, vec, vec_gate);                                               \
    return lev_check_launch("block_linear (matrix cores)");                                                                       \
  }
  BLM_CASE(LEV_BF16, LEV_BF16, bf16_t, bf16_t)
  BLM_CASE(LEV_BF16, LEV_F32, bf16_t, float)
  BLM_CASE(LEV_F32, LEV_BF16, float, bf16_t)
  BLM_CASE(LEV_F32, LEV_F32, float, float)
#undef BLM_CASE
  return lev_fail("block_linear: no kernel for the dtypes a=%d out=%d", a_dtype, out_dtype);
}
