// The recurrences of state_recurrence.hip on runs of many tokens, in chunks of 64 tokens on the matrix cores. With cs_i the running sum of a
// chunk's log decays and S0 the state that enters it:
//   SSD:    o_i = exp(cs_i) S0^T q_i + sum_{j <= i} exp(cs_i - cs_j) w_j (q_i . k_j) v_j
//           S   = exp(cs_end) S0 + sum_j exp(cs_end - cs_j) w_j k_j v_j^T
//   DELTA:  (1 + A) U = R,   A_ij = w_i exp(cs_i - cs_j) (k_i . k_j) for j < i,   R_i = w_i (v_i - exp(cs_i) S0^T k_i)
//           o_i = exp(cs_i) S0^T q_i + sum_{j <= i} exp(cs_i - cs_j) (q_i . k_j) u_j
//           S   = exp(cs_end) S0 + sum_j exp(cs_end - cs_j) k_j u_j^T
// (the second by block forward substitution over four tiles of 16 tokens, whose diagonal blocks are inverted row by row).
//
// Exactness. q, k and v are bfloat16 numbers (their unit norms are a float32 factor a row, applied behind the product), so q . k is a
// bfloat16 product with exact terms and a 32-bit sum. Every other product has one exact bfloat16 side; the 32-bit side (state, weights) is
// split into three bfloat16 numbers that hold all its 24 bits, three products for one. Products with two 32-bit sides (DELTA's A U and
// (q k) U) run on the 32-bit matrix instruction. Differences of running sums are taken in 64-bit: one fast decay must not cost the digits
// of the slow ones behind it.
//
// One workgroup of four waves per (run, head, 16 value columns) goes along the run; wave w has the 16 tokens 16 w .. of the chunk as rows of
// the result and a quarter of the state's key channels, in accumulator registers. The matrix instruction leaves rows 4 (lane / 16) + r and
// column lane % 16 in register r of a lane; as the K order of a product is free as long as both sides agree, such registers feed the next
// product directly (k slot of lane group g, register r: row 4 g + r), also two tiles side by side for an instruction with K = 32.
#include "state_recurrence.h"

typedef __attribute__((ext_vector_type(8))) __bf16 sc_bf16x8;
typedef __attribute__((ext_vector_type(4))) float sc_f32x4;
typedef __attribute__((ext_vector_type(4))) uint32_t sc_u32x4;
typedef __attribute__((ext_vector_type(2))) uint32_t sc_u32x2;

#define SC_Q 64   // tokens of a chunk
#define SC_VB 16  // value columns of a workgroup
#define SC_LDT (SC_Q + 8)

__device__ __forceinline__ sc_f32x4 sc_mfma(sc_u32x4 a, sc_u32x4 b, sc_f32x4 c) {
  union { sc_u32x4 u; sc_bf16x8 v; } x, y;
  x.u = a, y.u = b;
  return __builtin_amdgcn_mfma_f32_16x16x32_bf16(x.v, y.v, c, 0, 0, 0);
}
__device__ __forceinline__ sc_f32x4 sc_mfma32(sc_f32x4 a, sc_f32x4 b, sc_f32x4 c) {  // 16 of the K dimension: register r is k slot (lane / 16, r)
#pragma unroll
  for (int r = 0; r < 4; ++r) c = __builtin_amdgcn_mfma_f32_16x16x4f32(a[r], b[r], c, 0, 0, 0);
  return c;
}
// eight 32-bit numbers as three times eight bfloat16 numbers whose sum they are
__device__ __forceinline__ void sc_split(const float (&v)[8], sc_u32x4 (&out)[3]) {
  float rest[8];
#pragma unroll
  for (int i = 0; i < 8; ++i) rest[i] = v[i];
#pragma unroll
  for (int p = 0; p < 3; ++p)
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const uint32_t w = float2_to_bf16x2(rest[2 * i], rest[2 * i + 1]);
      out[p][i] = w;
      rest[2 * i] -= __uint_as_float(w << 16);
      rest[2 * i + 1] -= __uint_as_float(w & 0xffff0000u);
    }
}
// the decays from tokens 4 grp + r of a tile to the token whose running sum is cs_i, zero for the tokens behind it in its own tile
// (`diagonal`; the condition goes into the exponent: around the exponential it would become a branch per element)
__device__ __forceinline__ sc_f32x4 sc_decays(double cs_i, const double* cs, bool diagonal, int grp, int col) {
  typedef __attribute__((ext_vector_type(2))) double sc_f64x2;
  const sc_f64x2 a = *reinterpret_cast<const sc_f64x2*>(cs), b = *reinterpret_cast<const sc_f64x2*>(cs + 2);
  sc_f32x4 x = {(float)(cs_i - a[0]), (float)(cs_i - a[1]), (float)(cs_i - b[0]), (float)(cs_i - b[1])};
#pragma unroll
  for (int r = 0; r < 4; ++r) {
    x[r] = diagonal && 4 * grp + r > col ? -INFINITY : fminf(x[r], 0.f);
    x[r] = expf(x[r]);
  }
  return x;
}
__device__ __forceinline__ sc_u32x4 sc_read16(const bf16_t* p) { return *reinterpret_cast<const sc_u32x4*>(p); }
__device__ __forceinline__ sc_u32x4 sc_read8x2(const bf16_t* p, const bf16_t* q) {
  const sc_u32x2 a = *reinterpret_cast<const sc_u32x2*>(p), b = *reinterpret_cast<const sc_u32x2*>(q);
  return sc_u32x4{a[0], a[1], b[0], b[1]};
}
// eight channels from i0 on of a row of dk. VEC (rows are multiples of 8 channels at 16-byte boundaries): what lies beyond the row is some
// other of its channels and the load stands under no condition (nothing waits for it before it is used); sc_mask8 puts zeros there.
template <bool VEC>
__device__ __forceinline__ sc_u32x4 sc_load8(const bf16_t* row, int i0, int dk) {
  sc_u32x4 v = {0, 0, 0, 0};
  if (VEC) {
    v = *reinterpret_cast<const sc_u32x4*>(row + min(i0, dk - 8));
  } else {
#pragma unroll
    for (int e = 0; e < 8; ++e)
      if (i0 + e < dk) v[e >> 1] |= (uint32_t)row[i0 + e] << (16 * (e & 1));
  }
  return v;
}
__device__ __forceinline__ sc_u32x4 sc_mask8(sc_u32x4 v, int i0, int dk) {
  const uint32_t keep = i0 < dk ? 0xffffffffu : 0u;
  return sc_u32x4{v[0] & keep, v[1] & keep, v[2] & keep, v[3] & keep};
}

template <int DKM, int RULE, bool VEC>
__global__ void __launch_bounds__(256)
sc_chunk_kernel(const bf16_t* __restrict__ u, const float* __restrict__ scal, float* __restrict__ state, const int* __restrict__ token_slots,
                float* __restrict__ o, SrShape s) {
  constexpr int LDK = DKM + 8, KS = DKM / 32, NTW = DKM / 64, KI = DKM / 64, QI = DKM / 32;
  constexpr bool DELTA = RULE == SR_DELTA;
  __shared__ __attribute__((aligned(16))) bf16_t s_q[SC_Q][LDK], s_k[SC_Q][LDK], s_kt[DKM][SC_LDT], s_S[3][SC_VB][LDK];
  __shared__ __attribute__((aligned(16))) bf16_t s_x[DELTA ? 1 : SC_VB][SC_LDT];
  __shared__ __attribute__((aligned(16))) double s_cs[SC_Q];
  __shared__ __attribute__((aligned(16))) float s_ecs[SC_Q], s_wend[SC_Q], s_w[SC_Q], s_rk[SC_Q], s_rq[SC_Q];
  __shared__ float s_end;
  __shared__ __attribute__((aligned(16))) sc_f32x4 s_A[DELTA ? 6 : 1][64], s_R[DELTA ? 4 : 1][64], s_T[DELTA ? 4 : 1][64];
  __shared__ __attribute__((aligned(16))) float s_At[DELTA ? 4 : 1][16][16];
  __shared__ int tmp[256 + 2];
  // Workgroups go to the 8 chiplets in turn: the runs a step may have and does not must not be every second or fourth of them, so the run is
  // the slowest index; and the heads of a chiplet are neighbours, which read the same keys and queries through its cache.
  const int n_items = gridDim.x, per_xcd = n_items / 8;
  const int item = n_items % 8 == 0 ? (blockIdx.x % 8) * per_xcd + blockIdx.x / 8 : blockIdx.x;
  const int n_blocks = (s.dv + SC_VB - 1) / SC_VB, h = item / n_blocks;
  const int tid = threadIdx.x, lane = tid & 63, wave = __builtin_amdgcn_readfirstlane(tid >> 6), col = lane & 15, grp = lane >> 4;
  const int g = h / (s.H / s.G), n_scal = 2 * s.H + 2 * s.G, dk = s.dk, dv = s.dv;
  const int j = (item - h * n_blocks) * SC_VB + col;  // this lane's value column
  const bool live = j < dv;
  int t0, t_end, slot;
  if (!sr_find_run<256>(blockIdx.y, token_slots, s.Tn, tmp, t0, t_end, slot)) return;
  const bf16_t* uk = u + s.k_off + (size_t)g * dk;
  const bf16_t* uq = u + s.q_off + (size_t)g * dk;
  const bf16_t* uv = u + s.v_off + (size_t)h * dv;
  float* sp = state + (size_t)slot * s.slot_stride + (size_t)s.K * s.C + (size_t)h * dk * dv + (live ? j : 0);

  // the state: key channels 16 (wave * NTW + n) + 4 grp + r of column j
  sc_f32x4 S[NTW];
#pragma unroll
  for (int n = 0; n < NTW; ++n)
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int i = 16 * (wave * NTW + n) + 4 * grp + r;
      S[n][r] = live && i < dk ? sp[(size_t)i * dv] : 0.f;
    }

  // what of the next chunk is on its way: keys (two neighbouring tokens, eight channels), queries, values, scalars
  sc_u32x4 nk[KI][2], nq[QI];
  bf16_t nv[4];
  float n_ld = 0.f, n_w = 0.f, n_rk = 0.f, n_rq = 0.f;
  int n_tokens = 0;
  // raw loads only: whatever is computed from them here would wait for their way through the memory
  const int jc = live ? j : 0;
  auto fetch = [&](int tb) {
#pragma unroll
    for (int n = 0; n < KI; ++n) {
      const int idx = tid + 256 * n, pair = idx & 31, i0 = (idx >> 5) * 8;
#pragma unroll
      for (int e = 0; e < 2; ++e) nk[n][e] = sc_load8<VEC>(uk + (size_t)min(tb + 2 * pair + e, t_end - 1) * s.C, i0, dk);
    }
#pragma unroll
    for (int n = 0; n < QI; ++n) {
      const int idx = tid + 256 * n, row = idx / (DKM / 8), i0 = (idx % (DKM / 8)) * 8;
      nq[n] = sc_load8<VEC>(uq + (size_t)min(tb + row, t_end - 1) * s.C, i0, dk);
    }
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      // DELTA: the rows and the column of this lane's part of R; SSD: 16 columns of four tokens per thread, for the transposed copy
      const int t = DELTA ? tb + 16 * wave + 4 * grp + r : tb + (tid >> 4) + 16 * r;
      nv[r] = uv[(size_t)min(t, t_end - 1) * s.C + jc];
    }
    if (wave == 0) {
      const float* sc = scal + (size_t)min(tb + lane, t_end - 1) * n_scal;
      n_ld = sc[h], n_w = sc[s.H + h];
      if (DELTA) n_rk = sc[2 * s.H + g], n_rq = sc[2 * s.H + s.G + g];
    }
    n_tokens = t_end - tb;
  };
  auto stage = [&]() {
#pragma unroll
    for (int n = 0; n < KI; ++n) {
      const int idx = tid + 256 * n, pair = idx & 31, i0 = (idx >> 5) * 8;
#pragma unroll
      for (int e = 0; e < 2; ++e) {
        if (VEC) nk[n][e] = sc_mask8(nk[n][e], i0, dk);
        *reinterpret_cast<sc_u32x4*>(&s_k[2 * pair + e][i0]) = nk[n][e];
      }
#pragma unroll
      for (int c = 0; c < 4; ++c) {  // channels i0 + 2 c and i0 + 2 c + 1 of both tokens, transposed
        const uint32_t a = nk[n][0][c], b = nk[n][1][c];
        *reinterpret_cast<uint32_t*>(&s_kt[i0 + 2 * c][2 * pair]) = (a & 0xffffu) | (b << 16);
        *reinterpret_cast<uint32_t*>(&s_kt[i0 + 2 * c + 1][2 * pair]) = (a >> 16) | (b & 0xffff0000u);
      }
    }
#pragma unroll
    for (int n = 0; n < QI; ++n) {
      const int idx = tid + 256 * n, row = idx / (DKM / 8), i0 = (idx % (DKM / 8)) * 8;
      *reinterpret_cast<sc_u32x4*>(&s_q[row][i0]) = VEC ? sc_mask8(nq[n], i0, dk) : nq[n];
    }
    if (!DELTA)
#pragma unroll
      for (int r = 0; r < 4; ++r) s_x[col][(tid >> 4) + 16 * r] = live ? nv[r] : (bf16_t)0;
#pragma unroll
    for (int n = 0; n < NTW; ++n) {
      float rest[4];
#pragma unroll
      for (int r = 0; r < 4; ++r) rest[r] = S[n][r];
#pragma unroll
      for (int p = 0; p < 3; ++p) {
        const uint32_t lo = float2_to_bf16x2(rest[0], rest[1]), hi = float2_to_bf16x2(rest[2], rest[3]);
        *reinterpret_cast<sc_u32x2*>(&s_S[p][col][16 * (wave * NTW + n) + 4 * grp]) = sc_u32x2{lo, hi};
        rest[0] -= __uint_as_float(lo << 16), rest[1] -= __uint_as_float(lo & 0xffff0000u);
        rest[2] -= __uint_as_float(hi << 16), rest[3] -= __uint_as_float(hi & 0xffff0000u);
      }
    }
    if (wave == 0) {
      const float in = lane < n_tokens ? 1.f : 0.f;  // tokens behind the run's end: no decay, no weight
      n_ld *= in, n_w *= in, n_rk *= in, n_rq *= in;
      double cs = (double)n_ld;
#pragma unroll
      for (int d = 1; d < 64; d <<= 1) {
        const double up = __shfl_up(cs, d, 64);
        if (lane >= d) cs += up;
      }
      const double end = __shfl(cs, 63, 64);
      s_cs[lane] = cs;
      s_ecs[lane] = expf((float)cs);
      s_wend[lane] = expf((float)(end - cs)) * (DELTA ? n_rk : n_w);
      s_w[lane] = n_w, s_rk[lane] = n_rk, s_rq[lane] = n_rq;
      if (lane == 0) s_end = expf((float)end);
    }
  };

  fetch(t0);
  for (int tb = t0; tb < t_end; tb += SC_Q) {
    float v_now[4];
    stage();
#pragma unroll
    for (int r = 0; r < 4; ++r) v_now[r] = live ? to_float<bf16_t>(nv[r]) : 0.f;
    lds_barrier();  // the loads and stores in flight are the thread's own and are not waited for
    if (tb + SC_Q < t_end) fetch(tb + SC_Q);

    // rows of the result: tokens 16 wave + .. ; S0^T q and (DELTA) S0^T k
    sc_f32x4 oq = {0.f, 0.f, 0.f, 0.f}, ok = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int ks = 0; ks < KS; ++ks) {
      const sc_u32x4 aq = sc_read16(&s_q[16 * wave + col][32 * ks + 8 * grp]);
      sc_u32x4 ak;
      if (DELTA) ak = sc_read16(&s_k[16 * wave + col][32 * ks + 8 * grp]);
#pragma unroll
      for (int p = 2; p >= 0; --p) {
        const sc_u32x4 b = sc_read16(&s_S[p][col][32 * ks + 8 * grp]);
        oq = sc_mfma(aq, b, oq);
        if (DELTA) ok = sc_mfma(ak, b, ok);
      }
    }
    const sc_f32x4 ecs_rows = *reinterpret_cast<const sc_f32x4*>(&s_ecs[16 * wave + 4 * grp]);
    const double cs_i = s_cs[16 * wave + col];  // of the token that is this lane's column in the tiles below
    sc_f32x4 pq[4];
#pragma unroll
    for (int jt = 0; jt < 4; ++jt) pq[jt] = sc_f32x4{0.f, 0.f, 0.f, 0.f};
    if (DELTA) {
      const sc_f32x4 w_rows = *reinterpret_cast<const sc_f32x4*>(&s_w[16 * wave + 4 * grp]), rk_rows = *reinterpret_cast<const sc_f32x4*>(&s_rk[16 * wave + 4 * grp]);
      const sc_f32x4 rq_rows = *reinterpret_cast<const sc_f32x4*>(&s_rq[16 * wave + 4 * grp]);
      sc_f32x4 R;
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        R[r] = w_rows[r] * (v_now[r] - ecs_rows[r] * rk_rows[r] * ok[r]);
        oq[r] *= ecs_rows[r] * rq_rows[r];
      }
      s_R[wave][lane] = R;
      const float wk_i = s_w[16 * wave + col] * s_rk[16 * wave + col], rq_i = s_rq[16 * wave + col];
#pragma unroll
      for (int jt = 0; jt < 4; ++jt) {
        if (jt > wave) break;
        sc_f32x4 kk = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int ks = 0; ks < KS; ++ks) {
          const sc_u32x4 a = sc_read16(&s_k[16 * jt + col][32 * ks + 8 * grp]);
          kk = sc_mfma(a, sc_read16(&s_k[16 * wave + col][32 * ks + 8 * grp]), kk);
          pq[jt] = sc_mfma(a, sc_read16(&s_q[16 * wave + col][32 * ks + 8 * grp]), pq[jt]);
        }
        const sc_f32x4 dec = sc_decays(cs_i, &s_cs[16 * jt + 4 * grp], jt == wave, grp, col) * *reinterpret_cast<const sc_f32x4*>(&s_rk[16 * jt + 4 * grp]);
        kk *= dec * wk_i;
        pq[jt] *= dec * rq_i;
        if (jt == wave) {
#pragma unroll
          for (int r = 0; r < 4; ++r) kk[r] = 4 * grp + r == col ? 0.f : kk[r];  // A has nothing on the diagonal
        }
        if (jt < wave) {
          s_A[wave * (wave - 1) / 2 + jt][lane] = sc_f32x4{-kk[0], -kk[1], -kk[2], -kk[3]};
        } else {
#pragma unroll
          for (int r = 0; r < 4; ++r) s_At[wave][4 * grp + r][col] = kk[r];  // column 4 grp + r of the diagonal block, by rows
          __builtin_amdgcn_wave_barrier();
          // row `col` of its inverse: y (1 + A) = e_col, from the last column back
          float y[16];
#pragma unroll
          for (int c = 15; c >= 0; --c) {
            float acc = c == col ? 1.f : 0.f;
#pragma unroll
            for (int q4 = 0; q4 < 4; ++q4) {
              if (4 * q4 + 3 <= c) continue;
              const sc_f32x4 a4 = *reinterpret_cast<const sc_f32x4*>(&s_At[wave][c][4 * q4]);
#pragma unroll
              for (int e = 0; e < 4; ++e)
                if (4 * q4 + e > c) acc = fmaf(-a4[e], y[4 * q4 + e], acc);
            }
            y[c] = acc;
          }
          sc_f32x4 T;
#pragma unroll
          for (int r = 0; r < 4; ++r) T[r] = grp == 0 ? y[r] : grp == 1 ? y[4 + r] : grp == 2 ? y[8 + r] : y[12 + r];
          s_T[wave][lane] = T;
        }
      }
      lds_barrier();
      // every wave solves the whole system for the workgroup's columns: U stays in its registers
      sc_f32x4 U[4];
#pragma unroll
      for (int it = 0; it < 4; ++it) {
        sc_f32x4 acc = s_R[it][lane];
#pragma unroll
        for (int jt = 0; jt < it; ++jt) acc = sc_mfma32(s_A[it * (it - 1) / 2 + jt][lane], U[jt], acc);
        U[it] = sc_mfma32(s_T[it][lane], acc, sc_f32x4{0.f, 0.f, 0.f, 0.f});
      }
#pragma unroll
      for (int jt = 0; jt < 4; ++jt) {
        if (jt > wave) break;
        oq = sc_mfma32(pq[jt], U[jt], oq);
      }
      const float dend = s_end;
#pragma unroll
      for (int n = 0; n < NTW; ++n) S[n] = S[n] * dend;
#pragma unroll
      for (int half = 0; half < 2; ++half) {
        float w8[8];
#pragma unroll
        for (int e = 0; e < 8; ++e) w8[e] = U[2 * half + (e >> 2)][e & 3] * s_wend[32 * half + 16 * (e >> 2) + 4 * grp + (e & 3)];
        sc_u32x4 b[3];
        sc_split(w8, b);
#pragma unroll
        for (int n = 0; n < NTW; ++n) {
          const bf16_t* row = s_kt[16 * (wave * NTW + n) + col];
          const sc_u32x4 a = sc_read8x2(row + 32 * half + 4 * grp, row + 32 * half + 16 + 4 * grp);
#pragma unroll
          for (int p = 2; p >= 0; --p) S[n] = sc_mfma(a, b[p], S[n]);
        }
      }
    } else {
#pragma unroll
      for (int jt = 0; jt < 4; ++jt) {
        if (jt > wave) break;
#pragma unroll
        for (int ks = 0; ks < KS; ++ks)
          pq[jt] = sc_mfma(sc_read16(&s_k[16 * jt + col][32 * ks + 8 * grp]), sc_read16(&s_q[16 * wave + col][32 * ks + 8 * grp]), pq[jt]);
        pq[jt] *= sc_decays(cs_i, &s_cs[16 * jt + 4 * grp], jt == wave, grp, col) * *reinterpret_cast<const sc_f32x4*>(&s_w[16 * jt + 4 * grp]);
      }
      oq = oq * ecs_rows;
      const float dend = s_end;
#pragma unroll
      for (int n = 0; n < NTW; ++n) S[n] = S[n] * dend;
#pragma unroll
      for (int half = 0; half < 2; ++half) {
        const sc_u32x4 x8 = sc_read8x2(&s_x[col][32 * half + 4 * grp], &s_x[col][32 * half + 16 + 4 * grp]);
        float v8[8];
        sc_u32x4 b[3];
        if (2 * half <= wave) {
#pragma unroll
          for (int e = 0; e < 8; ++e) v8[e] = pq[2 * half + (e >> 2)][e & 3];
          sc_split(v8, b);
#pragma unroll
          for (int p = 2; p >= 0; --p) oq = sc_mfma(b[p], x8, oq);
        }
#pragma unroll
        for (int e = 0; e < 8; ++e) {
          const float xv = __uint_as_float((e & 1) ? x8[e >> 1] & 0xffff0000u : x8[e >> 1] << 16);
          v8[e] = xv * s_wend[32 * half + 16 * (e >> 2) + 4 * grp + (e & 3)];
        }
        sc_split(v8, b);
#pragma unroll
        for (int n = 0; n < NTW; ++n) {
          const bf16_t* row = s_kt[16 * (wave * NTW + n) + col];
          const sc_u32x4 a = sc_read8x2(row + 32 * half + 4 * grp, row + 32 * half + 16 + 4 * grp);
#pragma unroll
          for (int p = 2; p >= 0; --p) S[n] = sc_mfma(a, b[p], S[n]);
        }
      }
    }
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int t = tb + 16 * wave + 4 * grp + r;
      if (live && t < t_end) o[((size_t)t * s.H + h) * dv + j] = oq[r];
    }
    lds_barrier();  // the chunk's tiles have been read by every wave
  }
  if (live) {
#pragma unroll
    for (int n = 0; n < NTW; ++n)
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int i = 16 * (wave * NTW + n) + 4 * grp + r;
        if (i < dk) sp[(size_t)i * dv] = S[n][r];
      }
  }
}

int sr_chunks_launch(int rule, const bf16_t* u, const float* scal, float* state, const int* token_slots, float* o, int max_runs, const SrShape& s,
                     hipStream_t stream) {
  const int vec = s.C % 8 == 0 && s.dk % 8 == 0 && s.k_off % 8 == 0 && s.q_off % 8 == 0 && ((uintptr_t)u & 15) == 0;
  const dim3 grid(s.H * ((s.dv + SC_VB - 1) / SC_VB), max_runs);
  LEV_REQUIRE(max_runs <= 65535, "state recurrence: too many runs (%d)", max_runs);
#define SC_GO(DKM)                                                                                                                   \
  do {                                                                                                                               \
    if (rule == SR_DELTA && vec) sc_chunk_kernel<DKM, SR_DELTA, true><<<grid, 256, 0, stream>>>(u, scal, state, token_slots, o, s);     \
    else if (rule == SR_DELTA) sc_chunk_kernel<DKM, SR_DELTA, false><<<grid, 256, 0, stream>>>(u, scal, state, token_slots, o, s);      \
    else if (vec) sc_chunk_kernel<DKM, SR_SSD, true><<<grid, 256, 0, stream>>>(u, scal, state, token_slots, o, s);                      \
    else sc_chunk_kernel<DKM, SR_SSD, false><<<grid, 256, 0, stream>>>(u, scal, state, token_slots, o, s);                              \
  } while (0)
  if (s.dk <= 64) SC_GO(64);
  else if (s.dk <= 128) SC_GO(128);
  else SC_GO(256);
#undef SC_GO
  return lev_check_launch("state recurrence (chunks)");
}
