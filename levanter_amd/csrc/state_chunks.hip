// The recurrences of state_recurrence.hip on runs of many tokens, in chunks on the matrix cores. The step's tokens are cut into blocks of 64;
// a chunk is what of one run lies in one block. With cs_i the running sum of the chunk's log decays and S0 the state that enters it:
//   SSD:    P_ij = exp(cs_i - cs_j) w_j (q_i . k_j), j <= i;     o_i = exp(cs_i) S0^T q_i + sum_j P_ij v_j
//           S    = exp(cs_end) S0 + sum_j exp(cs_end - cs_j) w_j k_j v_j^T
//   DELTA:  P_ij = exp(cs_i - cs_j) (q_i . k_j), j <= i;         A_ij = w_i exp(cs_i - cs_j) (k_i . k_j), j < i;     T = (1 + A)^-1
//           R_i  = w_i (v_i - exp(cs_i) S0^T k_i);               U = T R;     o_i = exp(cs_i) S0^T q_i + sum_j P_ij u_j
//           S    = exp(cs_end) S0 + sum_j exp(cs_end - cs_j) k_j u_j^T
// P and T do not depend on the state: a first kernel makes them for all blocks and heads in parallel (entries between tokens of different
// runs are zero, so T is block-diagonal by itself), a second one goes along each run and carries the state from chunk to chunk. Entries of
// T are bounded: with unit keys and write rates below one, 1 - w k k^T does not lengthen a vector.
//
// Exactness. q, k and v are bfloat16 numbers (their unit norms are a float32 factor a row, applied behind the product), so q . k is a
// bfloat16 product with exact terms and a 32-bit sum. Every other product with a bfloat16 side has its 32-bit side (state, weights) split
// into three bfloat16 numbers that hold all its 24 bits, three products for one. Products with two 32-bit sides (T R, DELTA's P U, and those
// that make T) run on the 32-bit matrix instruction. Differences of running sums are taken in 64-bit: one fast decay must not cost the
// digits of the slow ones behind it.
//
// The matrix instruction leaves rows 4 (lane / 16) + r and column lane % 16 in register r of a lane; as the K order of a product is free as
// long as both sides agree, such registers feed the next product directly (k slot of lane group g, register r: row 4 g + r), also two tiles
// side by side for an instruction with K = 32. A 16 x 16 tile M as a left side is then M[lane % 16][4 (lane / 16) + r]; P and T are stored that
// way, [block][head][w (w + 1) / 2 + j][lane][4] for the tile of rows 16 w and columns 16 j, j <= w.
#include "state_recurrence.h"

typedef __attribute__((ext_vector_type(8))) __bf16 sc_bf16x8;
typedef __attribute__((ext_vector_type(4))) float sc_f32x4;
typedef __attribute__((ext_vector_type(4))) uint32_t sc_u32x4;
typedef __attribute__((ext_vector_type(2))) uint32_t sc_u32x2;

#define SC_Q 64   // tokens of a block
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
// the decays from tokens 4 grp + r of a tile to the token whose running sum is cs_i: zero for tokens of other runs and, in the token's own tile
// (`diagonal`), for those behind it (the condition goes into the exponent: around the exponential it would become a branch per element)
__device__ __forceinline__ sc_f32x4 sc_decays(double cs_i, const double* cs, const bool (&same)[4], bool valid, bool diagonal, int grp, int col) {
  typedef __attribute__((ext_vector_type(2))) double sc_f64x2;
  const sc_f64x2 a = *reinterpret_cast<const sc_f64x2*>(cs), b = *reinterpret_cast<const sc_f64x2*>(cs + 2);
  sc_f32x4 x = {(float)(cs_i - a[0]), (float)(cs_i - a[1]), (float)(cs_i - b[0]), (float)(cs_i - b[1])};
#pragma unroll
  for (int r = 0; r < 4; ++r) {
    x[r] = !valid || !same[r] || (diagonal && 4 * grp + r > col) ? -INFINITY : fminf(x[r], 0.f);
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

// ---- what does not depend on the state ---------------------------------------------------------------------------------------
// One workgroup of four waves per (block, head); wave w has the rows 16 w of the block's matrices.
template <int DKM, int RULE, bool VEC>
__global__ void __launch_bounds__(256)
sc_inner_kernel(const bf16_t* __restrict__ u, const float* __restrict__ scal, const int* __restrict__ token_slots, float* __restrict__ P_out,
                float* __restrict__ T_out, SrShape s) {
  constexpr int LDK = DKM + 8, KS = DKM / 32, QI = DKM / 32;
  constexpr bool DELTA = RULE == SR_DELTA;
  __shared__ __attribute__((aligned(16))) bf16_t s_q[SC_Q][LDK], s_k[SC_Q][LDK];
  __shared__ __attribute__((aligned(16))) double s_cs[SC_Q];
  __shared__ __attribute__((aligned(16))) float s_w[SC_Q], s_rk[SC_Q], s_rq[SC_Q];
  __shared__ __attribute__((aligned(16))) int s_slot[SC_Q];
  __shared__ __attribute__((aligned(16))) sc_f32x4 s_A[DELTA ? 6 : 1][64], s_T[DELTA ? 4 : 1][64];
  __shared__ __attribute__((aligned(16))) float s_At[DELTA ? 4 : 1][16][16], s_Tr[DELTA ? 4 : 1][16][20];
  const int h = blockIdx.x, tb = blockIdx.y * SC_Q;
  const int tid = threadIdx.x, lane = tid & 63, wave = __builtin_amdgcn_readfirstlane(tid >> 6), col = lane & 15, grp = lane >> 4;
  const int g = h / (s.H / s.G), n_scal = 2 * s.H + 2 * s.G, dk = s.dk;
#pragma unroll
  for (int n = 0; n < QI; ++n) {
    const int idx = tid + 256 * n, row = idx / (DKM / 8), i0 = (idx % (DKM / 8)) * 8;
    const bf16_t* ur = u + (size_t)min(tb + row, s.Tn - 1) * s.C + (size_t)g * dk;
    const sc_u32x4 q = sc_load8<VEC>(ur + s.q_off, i0, dk), k = sc_load8<VEC>(ur + s.k_off, i0, dk);
    *reinterpret_cast<sc_u32x4*>(&s_q[row][i0]) = VEC ? sc_mask8(q, i0, dk) : q;
    *reinterpret_cast<sc_u32x4*>(&s_k[row][i0]) = VEC ? sc_mask8(k, i0, dk) : k;
  }
  if (wave == 0) {
    const int t = min(tb + lane, s.Tn - 1), slot = tb + lane < s.Tn ? token_slots[t] : -1;
    const float* sc = scal + (size_t)t * n_scal;
    double cs = slot >= 0 ? (double)sc[h] : 0.0;
#pragma unroll
    for (int d = 1; d < 64; d <<= 1) {
      const double up = __shfl_up(cs, d, 64);
      if (lane >= d) cs += up;
    }
    s_cs[lane] = cs;
    s_slot[lane] = slot;
    s_w[lane] = sc[s.H + h];
    s_rk[lane] = sc[2 * s.H + g], s_rq[lane] = sc[2 * s.H + s.G + g];
  }
  __syncthreads();
  const double cs_i = s_cs[16 * wave + col];  // of the token that is this lane's row in the tiles below
  const int slot_i = s_slot[16 * wave + col];
  const float rq_i = s_rq[16 * wave + col], wk_i = DELTA ? s_w[16 * wave + col] * s_rk[16 * wave + col] : 0.f;
  const size_t tile0 = ((size_t)blockIdx.y * s.H + h) * 10;
  sc_u32x4 bq[KS], bk[KS];
#pragma unroll
  for (int ks = 0; ks < KS; ++ks) {
    bq[ks] = sc_read16(&s_q[16 * wave + col][32 * ks + 8 * grp]);
    if (DELTA) bk[ks] = sc_read16(&s_k[16 * wave + col][32 * ks + 8 * grp]);
  }
#pragma unroll
  for (int jt = 0; jt < 4; ++jt) {
    if (jt > wave) break;
    sc_f32x4 pq = {0.f, 0.f, 0.f, 0.f}, kk = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int ks = 0; ks < KS; ++ks) {
      const sc_u32x4 a = sc_read16(&s_k[16 * jt + col][32 * ks + 8 * grp]);
      pq = sc_mfma(a, bq[ks], pq);
      if (DELTA) kk = sc_mfma(a, bk[ks], kk);
    }
    const int4 slot_j = *reinterpret_cast<const int4*>(&s_slot[16 * jt + 4 * grp]);
    const bool same[4] = {slot_j.x == slot_i, slot_j.y == slot_i, slot_j.z == slot_i, slot_j.w == slot_i};
    sc_f32x4 dec = sc_decays(cs_i, &s_cs[16 * jt + 4 * grp], same, slot_i >= 0, jt == wave, grp, col);
    dec *= *reinterpret_cast<const sc_f32x4*>(DELTA ? &s_rk[16 * jt + 4 * grp] : &s_w[16 * jt + 4 * grp]);
    pq *= dec * rq_i;
    *reinterpret_cast<sc_f32x4*>(P_out + ((tile0 + wave * (wave + 1) / 2 + jt) * 64 + lane) * 4) = pq;
    if (DELTA) {
      kk *= dec * wk_i;
      if (jt < wave) {
        s_A[wave * (wave - 1) / 2 + jt][lane] = sc_f32x4{-kk[0], -kk[1], -kk[2], -kk[3]};
      } else {
#pragma unroll
        for (int r = 0; r < 4; ++r) s_At[wave][4 * grp + r][col] = 4 * grp + r == col ? 0.f : kk[r];  // column 4 grp + r of the diagonal tile
        __builtin_amdgcn_wave_barrier();
        // row `col` of its inverse: y (1 + A) = e_col, from the last column back
        float y[16];
#pragma unroll
        for (int c = 15; c >= 0; --c) {
          float acc[4] = {c == col ? 1.f : 0.f, 0.f, 0.f, 0.f};
#pragma unroll
          for (int q4 = 0; q4 < 4; ++q4) {
            if (4 * q4 + 3 <= c) continue;
            const sc_f32x4 a4 = *reinterpret_cast<const sc_f32x4*>(&s_At[wave][c][4 * q4]);
#pragma unroll
            for (int e = 0; e < 4; ++e)
              if (4 * q4 + e > c) acc[e] = fmaf(-a4[e], y[4 * q4 + e], acc[e]);
          }
          y[c] = (acc[0] + acc[1]) + (acc[2] + acc[3]);
        }
        sc_f32x4 T;
#pragma unroll
        for (int r = 0; r < 4; ++r) T[r] = grp == 0 ? y[r] : grp == 1 ? y[4 + r] : grp == 2 ? y[8 + r] : y[12 + r];
        s_T[wave][lane] = T;
        *reinterpret_cast<sc_f32x4*>(&s_Tr[wave][col][4 * grp]) = T;  // the same by rows, for the product below
        *reinterpret_cast<sc_f32x4*>(T_out + ((tile0 + wave * (wave + 1) / 2 + wave) * 64 + lane) * 4) = T;
      }
    }
  }
  if (!DELTA) return;
  __syncthreads();
  // wave j: the tiles below the diagonal of column tile j of the inverse, T_ij = -T_ii sum_k A_ik T_kj
  sc_f32x4 Tc[4];
#pragma unroll
  for (int i = 0; i < 4; ++i) {
    if (i < wave) continue;
    if (i == wave) {
#pragma unroll
      for (int r = 0; r < 4; ++r) Tc[i][r] = s_Tr[wave][4 * grp + r][col];
      continue;
    }
    sc_f32x4 acc = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int k = 0; k < 4; ++k) {
      if (k < wave || k >= i) continue;
      acc = sc_mfma32(s_A[i * (i - 1) / 2 + k][lane], Tc[k], acc);
    }
    Tc[i] = sc_mfma32(s_T[i][lane], acc, sc_f32x4{0.f, 0.f, 0.f, 0.f});
    float* dst = T_out + (tile0 + i * (i + 1) / 2 + wave) * 256;
#pragma unroll
    for (int r = 0; r < 4; ++r) dst[((col >> 2) * 16 + 4 * grp + r) * 4 + (col & 3)] = Tc[i][r];
  }
}

// ---- along the runs -------------------------------------------------------------------------------------------------------------
// One workgroup of four waves per (run, head, 16 value columns); wave w has the tokens 16 w .. of the block as rows of the result and a quarter
// of the state's key channels, in accumulator registers.
template <int DKM, int RULE, bool VEC>
__global__ void __launch_bounds__(256)
sc_chunk_kernel(const bf16_t* __restrict__ u, const float* __restrict__ scal, const float* __restrict__ P_in, const float* __restrict__ T_in,
                float* __restrict__ state, const int* __restrict__ token_slots, float* __restrict__ o, SrShape s) {
  constexpr int LDK = DKM + 8, KS = DKM / 32, NTW = DKM / 64, KI = DKM / 64, QI = DKM / 32;
  constexpr bool DELTA = RULE == SR_DELTA;
  __shared__ __attribute__((aligned(16))) bf16_t s_q[SC_Q][LDK], s_k[DELTA ? SC_Q : 1][LDK], s_kt[DKM][SC_LDT], s_S[3][SC_VB][LDK];
  __shared__ __attribute__((aligned(16))) bf16_t s_x[DELTA ? 1 : SC_VB][SC_LDT];
  __shared__ __attribute__((aligned(16))) float s_ecs[SC_Q], s_wend[SC_Q], s_w[SC_Q], s_rk[SC_Q], s_rq[SC_Q];
  __shared__ float s_end;
  __shared__ __attribute__((aligned(16))) sc_f32x4 s_R[DELTA ? 4 : 1][64], s_U[DELTA ? 4 : 1][64];
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
  const int jc = live ? j : 0;
  float* sp = state + (size_t)slot * s.slot_stride + (size_t)s.K * s.C + (size_t)h * dk * dv + jc;

  // the state: key channels 16 (wave * NTW + n) + 4 grp + r of column j
  sc_f32x4 S[NTW];
#pragma unroll
  for (int n = 0; n < NTW; ++n)
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int i = 16 * (wave * NTW + n) + 4 * grp + r;
      S[n][r] = live && i < dk ? sp[(size_t)i * dv] : 0.f;
    }

  // what of the next block is on its way: keys (two neighbouring tokens, eight channels), queries, values, scalars, this wave's rows of P and T.
  // Raw loads only, under no condition: whatever is computed from them here would wait for their way through the memory.
  sc_u32x4 nk[KI][2], nq[QI];
  bf16_t nv[4];
  sc_f32x4 nP[4], nT[4];
  float n_ld = 0.f, n_w = 0.f, n_rk = 0.f, n_rq = 0.f;
  auto fetch = [&](int tb) {
#pragma unroll
    for (int n = 0; n < KI; ++n) {
      const int idx = tid + 256 * n, pair = idx & 31, i0 = (idx >> 5) * 8;
#pragma unroll
      for (int e = 0; e < 2; ++e) nk[n][e] = sc_load8<VEC>(uk + (size_t)min(tb + 2 * pair + e, s.Tn - 1) * s.C, i0, dk);
    }
#pragma unroll
    for (int n = 0; n < QI; ++n) {
      const int idx = tid + 256 * n, row = idx / (DKM / 8), i0 = (idx % (DKM / 8)) * 8;
      nq[n] = sc_load8<VEC>(uq + (size_t)min(tb + row, s.Tn - 1) * s.C, i0, dk);
    }
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      // DELTA: the rows and the column of this lane's part of R; SSD: 16 columns of four tokens per thread, for the transposed copy
      const int t = DELTA ? tb + 16 * wave + 4 * grp + r : tb + (tid >> 4) + 16 * r;
      nv[r] = uv[(size_t)min(t, s.Tn - 1) * s.C + jc];
    }
    const size_t tile = ((size_t)(tb / SC_Q) * s.H + h) * 10 + wave * (wave + 1) / 2;
#pragma unroll
    for (int jt = 0; jt < 4; ++jt) {
      const size_t at = ((tile + min(jt, wave)) * 64 + lane) * 4;
      nP[jt] = *reinterpret_cast<const sc_f32x4*>(P_in + at);
      if (DELTA) nT[jt] = *reinterpret_cast<const sc_f32x4*>(T_in + at);
    }
    if (wave == 0) {
      const float* sc = scal + (size_t)min(tb + lane, s.Tn - 1) * n_scal;
      n_ld = sc[h], n_w = sc[s.H + h];
      if (DELTA) n_rk = sc[2 * s.H + g], n_rq = sc[2 * s.H + s.G + g];
    }
  };
  auto stage = [&](int tb) {
#pragma unroll
    for (int n = 0; n < KI; ++n) {
      const int idx = tid + 256 * n, pair = idx & 31, i0 = (idx >> 5) * 8;
#pragma unroll
      for (int e = 0; e < 2; ++e) {
        if (VEC) nk[n][e] = sc_mask8(nk[n][e], i0, dk);
        if (DELTA) *reinterpret_cast<sc_u32x4*>(&s_k[2 * pair + e][i0]) = nk[n][e];
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
      const float in = tb + lane >= t0 && tb + lane < t_end ? 1.f : 0.f;  // the block's tokens of other runs: no decay, no weight
      n_ld *= in, n_w *= in, n_rk *= in, n_rq *= in;
      double cs = (double)n_ld;
#pragma unroll
      for (int d = 1; d < 64; d <<= 1) {
        const double up = __shfl_up(cs, d, 64);
        if (lane >= d) cs += up;
      }
      const double end = __shfl(cs, 63, 64);
      s_ecs[lane] = expf((float)cs);
      s_wend[lane] = expf((float)(end - cs)) * (DELTA ? n_rk : n_w);
      s_w[lane] = n_w, s_rk[lane] = n_rk, s_rq[lane] = n_rq;
      if (lane == 0) s_end = expf((float)end);
    }
  };

  const int first = t0 / SC_Q * SC_Q;
  fetch(first);
  for (int tb = first; tb < t_end; tb += SC_Q) {
    float v_now[4];
    sc_f32x4 P[4], T[4];
    stage(tb);
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      v_now[r] = live ? to_float<bf16_t>(nv[r]) : 0.f;
      P[r] = nP[r];
      if (DELTA) T[r] = nT[r];
    }
    lds_barrier();  // the loads and stores in flight are the thread's own and are not waited for
    if (tb + SC_Q < t_end) fetch(tb + SC_Q);

    // rows of the result: tokens 16 wave + .. ; S0^T q and (DELTA) S0^T k, two sums each
    sc_f32x4 oq = {0.f, 0.f, 0.f, 0.f}, ok = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int ks = 0; ks < KS; ++ks) {
      const sc_u32x4 aq = sc_read16(&s_q[16 * wave + col][32 * ks + 8 * grp]);
      sc_u32x4 ak;
      if (DELTA) ak = sc_read16(&s_k[DELTA ? 16 * wave + col : 0][32 * ks + 8 * grp]);
#pragma unroll
      for (int p = 2; p >= 0; --p) {
        const sc_u32x4 b = sc_read16(&s_S[p][col][32 * ks + 8 * grp]);
        oq = sc_mfma(aq, b, oq);
        if (DELTA) ok = sc_mfma(ak, b, ok);
      }
    }
    const sc_f32x4 ecs_rows = *reinterpret_cast<const sc_f32x4*>(&s_ecs[16 * wave + 4 * grp]);
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
      lds_barrier();
      sc_f32x4 U0 = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int jt = 0; jt < 4; ++jt) {
        if (jt > wave) break;
        U0 = sc_mfma32(T[jt], s_R[jt][lane], U0);
      }
      s_U[wave][lane] = U0;
      lds_barrier();
      sc_f32x4 U[4];
#pragma unroll
      for (int jt = 0; jt < 4; ++jt) U[jt] = s_U[jt][lane];
#pragma unroll
      for (int jt = 0; jt < 4; ++jt) {
        if (jt > wave) break;
        oq = sc_mfma32(P[jt], U[jt], oq);
      }
      const float dend = s_end;
#pragma unroll
      for (int n = 0; n < NTW; ++n) S[n] = S[n] * dend;
#pragma unroll
      for (int half = 0; half < 2; ++half) {
        const sc_f32x4 w0 = *reinterpret_cast<const sc_f32x4*>(&s_wend[32 * half + 4 * grp]), w1 = *reinterpret_cast<const sc_f32x4*>(&s_wend[32 * half + 16 + 4 * grp]);
        float w8[8];
#pragma unroll
        for (int e = 0; e < 4; ++e) w8[e] = U[2 * half][e] * w0[e], w8[4 + e] = U[2 * half + 1][e] * w1[e];
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
      oq = oq * ecs_rows;
      const float dend = s_end;
#pragma unroll
      for (int n = 0; n < NTW; ++n) S[n] = S[n] * dend;
#pragma unroll
      for (int half = 0; half < 2; ++half) {
        const sc_u32x4 x8 = sc_read8x2(&s_x[DELTA ? 0 : col][32 * half + 4 * grp], &s_x[DELTA ? 0 : col][32 * half + 16 + 4 * grp]);
        float v8[8];
        sc_u32x4 b[3];
        if (2 * half <= wave) {
          const float second = 2 * half + 1 <= wave ? 1.f : 0.f;
#pragma unroll
          for (int e = 0; e < 4; ++e) v8[e] = P[2 * half][e], v8[4 + e] = P[2 * half + 1][e] * second;
          sc_split(v8, b);
#pragma unroll
          for (int p = 2; p >= 0; --p) oq = sc_mfma(b[p], x8, oq);
        }
        const sc_f32x4 w0 = *reinterpret_cast<const sc_f32x4*>(&s_wend[32 * half + 4 * grp]), w1 = *reinterpret_cast<const sc_f32x4*>(&s_wend[32 * half + 16 + 4 * grp]);
#pragma unroll
        for (int e = 0; e < 8; ++e) {
          const float xv = __uint_as_float((e & 1) ? x8[e >> 1] & 0xffff0000u : x8[e >> 1] << 16);
          v8[e] = xv * (e < 4 ? w0[e] : w1[e - 4]);
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
      if (live && t >= t0 && t < t_end) o[((size_t)t * s.H + h) * dv + j] = oq[r];
    }
    lds_barrier();  // the block's tiles have been read by every wave
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

long sr_chunks_workspace(int rule, int Tn, int H) { return (long)((Tn + SC_Q - 1) / SC_Q) * H * 10 * 256 * (rule == SR_DELTA ? 2 : 1); }

int sr_chunks_launch(int rule, const bf16_t* u, const float* scal, float* state, const int* token_slots, float* o, float* workspace, int max_runs,
                     const SrShape& s, hipStream_t stream) {
  const int vec = s.C % 8 == 0 && s.dk % 8 == 0 && s.k_off % 8 == 0 && s.q_off % 8 == 0 && ((uintptr_t)u & 15) == 0;
  const int n_blocks = (s.Tn + SC_Q - 1) / SC_Q;
  LEV_REQUIRE(max_runs <= 65535 && n_blocks <= 65535 && ((uintptr_t)workspace & 15) == 0, "state recurrence: too many runs (%d) or tokens (%d)", max_runs, s.Tn);
  float* P = workspace;
  float* T = workspace + (size_t)n_blocks * s.H * 10 * 256;
  const dim3 inner(s.H, n_blocks), grid(s.H * ((s.dv + SC_VB - 1) / SC_VB), max_runs);
#define SC_RUN(DKM, RULE, VEC)                                                                                   \
  do {                                                                                                           \
    sc_inner_kernel<DKM, RULE, VEC><<<inner, 256, 0, stream>>>(u, scal, token_slots, P, T, s);                    \
    if (lev_check_launch("state recurrence (blocks)")) return -1;                                                \
    sc_chunk_kernel<DKM, RULE, VEC><<<grid, 256, 0, stream>>>(u, scal, P, T, state, token_slots, o, s);           \
  } while (0)
#define SC_GO(DKM)                                          \
  do {                                                      \
    if (rule == SR_DELTA && vec) SC_RUN(DKM, SR_DELTA, true);   \
    else if (rule == SR_DELTA) SC_RUN(DKM, SR_DELTA, false);    \
    else if (vec) SC_RUN(DKM, SR_SSD, true);                    \
    else SC_RUN(DKM, SR_SSD, false);                            \
  } while (0)
  if (s.dk <= 64) SC_GO(64);
  else if (s.dk <= 128) SC_GO(128);
  else SC_GO(256);
#undef SC_GO
#undef SC_RUN
  return lev_check_launch("state recurrence (chunks)");
}
