// A feed-forward made of many small experts of which every token uses a few (a mixture of experts), steered from the device:
// no count ever goes to the host, so the launches depend on the number of tokens alone.
//
//   route     per token: scores s of the router's logits z (float32 [T][E]): sigmoid(z) (scoring 0), the softmax of z over all E outputs
//             (1) or z itself (2: the weights are then the softmax over the winners' s alone); the choice goes by c = s + correction;
//             the experts form G equal groups of neighbours, a group's score is the sum of its `group_top` largest c, only the
//             experts of the `keep` best groups can be chosen (the others count as -inf); the `top` largest c win (ties: the
//             lower index); the weights are the winners' s (times 1 / their sum if `renormalize`), in the order of falling c.
//   sort      the T * top (token, choice) pairs by expert: sorted[pos] = pair, pos_of[pair] = pos, and a list of row tiles
//             (expert, first position, rows <= tile_rows) that covers every expert's stretch; n_tiles on the device.
//             tile_rows is 16, or 128 for steps with many rows an expert.
//   linear    for every tile: out[pos][o] = sum_k w[expert][o][k] a[row(pos)][k], row(pos) = the pair's token (gather) or pos
//             itself, through the activation (none for the second product); with glu the expert's matrix is [gate ; up] (2F rows) and
//             out[pos][f] = act(gate_f) * up_f.
//             bfloat16 on the matrix cores (16x16x32): few tiles of 16 rows with K split over a workgroup's waves, many with a
//             wave per tile, tiles of 128 rows with both operands staged through LDS; float32 in plain arithmetic. Workgroups
//             beyond n_tiles return at once.
//             with limit > 0 the gate sum is capped at limit and the up sum clamped to +-limit first, and up_shift is added to
//             the up sum: act(min(gate, limit)) * (clamp(up) + up_shift).
//   combine   y[t] = sum_c weight[t][c] * out[pos_of[t * top + c]], c in order, float32; with `accumulate` added to what y holds.
//   identity  router outputs n_real .. E-1 may stand for experts without weights whose result is their input: sort gives their pairs
//             places but no tiles (the products never see them), and combine takes the token's own row of `identity_in` for them.
#include "common.h"

#define MOE_TM 16          // rows of a matrix-core row tile, and of a tile of the list in steps of few tokens
#define MOE_BIG 128        // rows of a tile of the list in the others
#define MOE_MAX_E 1024     // experts (at most 32 a lane)
#define MOE_MAX_TOP 32

// ---- route ------------------------------------------------------------------------------------
// One wave routes one token; s_s, c_s (and g_s with groups) are E (G) numbers of its own in LDS. Every wave of
// the workgroup passes the same barriers. `extra`: a further choice behind the `top` ones, expert E with weight 1 (an expert that runs for
// every token). store: the wave's token is one of the step's.
struct MoeRouteArgs {
  const float* z;
  long z_stride;
  const float* correction;
  int E, G, keep, group_top, top, renormalize, scoring, extra;
  int* chosen;
  float* weights;
};
__device__ __forceinline__ void moe_route_token(const MoeRouteArgs& a, int t, bool store, float* s_s, float* c_s, float* g_s) {
  const int lane = threadIdx.x & 63, E = a.E, G = a.G, top = a.top;
  const int per = E / G;
  const float* zt = a.z + (size_t)t * a.z_stride;
  float z_max = 0.f, inv_sum = 1.0f;
  if (a.scoring == 1) {
    float mx = -INFINITY;
    for (int e = lane; e < E; e += 64) mx = fmaxf(mx, zt[e]);
    z_max = wave_max(mx);
    float sum = 0.f;
    for (int e = lane; e < E; e += 64) sum += expf(zt[e] - z_max);
    inv_sum = 1.0f / wave_sum(sum);
  }
  for (int e = lane; e < E; e += 64) {
    const float ze = zt[e];
    const float s = a.scoring == 2 ? ze : a.scoring == 1 ? expf(ze - z_max) * inv_sum : 1.0f / (1.0f + expf(-ze));
    s_s[e] = s;
    c_s[e] = s + (a.correction ? a.correction[e] : 0.f);
  }
  __syncthreads();
  if (G > 1) {
    for (int g = lane; g < G; g += 64) {  // the sum of the group's largest choice scores
      float sum = 0.f;
      float last = INFINITY;
      int last_i = -1;
      for (int n = 0; n < min(a.group_top, per); ++n) {  // the next largest: below (last, last_i) in the order (value falling, index rising)
        float best = -INFINITY;
        int best_i = -1;
        for (int i = 0; i < per; ++i) {
          const float c = c_s[g * per + i];
          const bool after = c < last || (c == last && i > last_i);
          if (after && (best_i < 0 || c > best)) best = c, best_i = i;
        }
        sum += best;
        last = best, last_i = best_i;
      }
      g_s[g] = sum;
    }
    __syncthreads();
    for (int e = lane; e < E; e += 64) {
      const int g = e / per;
      const float mine = g_s[g];
      int ahead = 0;  // groups that come before this one
      for (int o = 0; o < G; ++o) ahead += (g_s[o] > mine || (g_s[o] == mine && o < g)) ? 1 : 0;
      if (ahead >= a.keep) c_s[e] = -INFINITY;
    }
    __syncthreads();
  }
  // the next largest, `top` times: every lane looks through its own experts (e % 64 == lane), the lanes compare; lane n keeps the n-th
  float wsum = 0.f;
  int mine = 0;
  uint32_t taken = 0;  // of this lane's experts: bit e / 64
  for (int n = 0; n < top; ++n) {
    float best = -INFINITY;
    int best_e = 0x7fffffff;
    for (int e = lane, i = 0; e < E; e += 64, ++i) {
      const float c = c_s[e];
      if (!(taken >> i & 1u) && (c > best || (c == best && e < best_e))) best = c, best_e = e;
    }
#pragma unroll
    for (int o = 32; o > 0; o >>= 1) {
      const float ob = __shfl_xor(best, o, 64);
      const int oe = __shfl_xor(best_e, o, 64);
      if (ob > best || (ob == best && oe < best_e)) best = ob, best_e = oe;
    }
    if (best_e >= E) best_e = 0;  // nothing left to choose from (a configuration that keeps fewer experts than it uses)
    if ((best_e & 63) == lane) taken |= 1u << (best_e >> 6);
    if (lane == n) mine = best_e;
    wsum += s_s[best_e];
  }
  const size_t at = (size_t)t * (top + a.extra);
  float weight = s_s[mine];
  if (a.scoring == 2) {
    const float mx = wave_max(lane < top ? weight : -INFINITY);
    weight = lane < top ? expf(weight - mx) : 0.f;
    weight /= wave_sum(weight);
  } else if (a.renormalize) {
    weight /= wsum;
  }
  if (!store) return;
  if (lane < top) {
    a.chosen[at + lane] = mine;
    a.weights[at + lane] = weight;
  } else if (lane == top && a.extra) {
    a.chosen[at + top] = E;
    a.weights[at + top] = 1.0f;
  }
}

__global__ void __launch_bounds__(64)
moe_route_kernel(const MoeRouteArgs a) {
  __shared__ float s_s[MOE_MAX_E], c_s[MOE_MAX_E], g_s[MOE_MAX_E];
  moe_route_token(a, blockIdx.x, true, s_s, c_s, g_s);
}

// ---- sort --------------------------------------------------------------------------------------
// One workgroup. meta: [0] = n_tiles; tiles: (expert, first position, rows) per tile. The order of an expert's pairs among
// themselves is whatever the atomic counters give: a pair's results do not depend on its place in a tile.
#define MOE_SORT_NT 1024
struct MoeSortLds {
  int count[MOE_MAX_E + 1], start[MOE_MAX_E + 1], tile_start[MOE_MAX_E + 2], cursor[MOE_MAX_E + 1];
};
__device__ __forceinline__ void moe_sort_pairs(MoeSortLds& l, const int* chosen, int P, int E, int n_real, int tile_rows, int* __restrict__ sorted,
                                               int* __restrict__ pos_of, int* __restrict__ tiles, int* __restrict__ meta) {
  const int tid = threadIdx.x;
  for (int e = tid; e < E; e += MOE_SORT_NT) l.count[e] = 0, l.cursor[e] = 0;
  __syncthreads();
  for (int p = tid; p < P; p += MOE_SORT_NT) atomicAdd(&l.count[chosen[p]], 1);
  __syncthreads();
  if (tid < 64) {  // running sums over the experts: each lane a stretch of neighbours, then across the lanes
    const int c = (E + 63) / 64, lo = min(E, tid * c), hi = min(E, lo + c);
    int n = 0, nt = 0;
    for (int e = lo; e < hi; ++e) {
      n += l.count[e];
      if (e < n_real) nt += (l.count[e] + tile_rows - 1) / tile_rows;  // experts without weights get places and no tiles
    }
    int at = n, tile = nt;
#pragma unroll
    for (int o = 1; o < 64; o <<= 1) {
      const int a = __shfl_up(at, o, 64), b = __shfl_up(tile, o, 64);
      if (tid >= o) at += a, tile += b;
    }
    if (tid == 63) l.tile_start[E] = tile, meta[0] = tile;
    at -= n, tile -= nt;
    for (int e = lo; e < hi; ++e) {
      l.start[e] = at;
      l.tile_start[e] = tile;
      at += l.count[e];
      if (e < n_real) tile += (l.count[e] + tile_rows - 1) / tile_rows;
    }
  }
  __syncthreads();
  for (int p = tid; p < P; p += MOE_SORT_NT) {
    const int e = chosen[p];
    const int pos = l.start[e] + atomicAdd(&l.cursor[e], 1);
    sorted[pos] = p;
    pos_of[p] = pos;
  }
  for (int e = tid; e < E; e += MOE_SORT_NT) {
    const int n = l.tile_start[e + 1] - l.tile_start[e];
    for (int i = 0; i < n; ++i) {
      int* tl = tiles + 3 * (size_t)(l.tile_start[e] + i);
      tl[0] = e;
      tl[1] = l.start[e] + i * tile_rows;
      tl[2] = min(tile_rows, l.count[e] - i * tile_rows);
    }
  }
}

__global__ void __launch_bounds__(MOE_SORT_NT)
moe_sort_kernel(const int* __restrict__ chosen, int P, int E, int n_real, int tile_rows, int* __restrict__ sorted, int* __restrict__ pos_of,
                int* __restrict__ tiles, int* __restrict__ meta) {
  __shared__ MoeSortLds l;
  moe_sort_pairs(l, chosen, P, E, n_real, tile_rows, sorted, pos_of, tiles, meta);
}

// Both for a step of few tokens, in one workgroup: a wave routes a token, then all of them sort.
#define MOE_SMALL_T (MOE_SORT_NT / 64)
#define MOE_SMALL_E 256
__global__ void __launch_bounds__(MOE_SORT_NT)
moe_route_sort_kernel(const MoeRouteArgs a, int T, int n_real, int tile_rows, int* __restrict__ sorted, int* __restrict__ pos_of, int* __restrict__ tiles,
                      int* __restrict__ meta) {
  __shared__ MoeSortLds l;
  __shared__ float s_s[MOE_SMALL_T][MOE_SMALL_E], c_s[MOE_SMALL_T][MOE_SMALL_E];
  const int wave = threadIdx.x >> 6;
  // the groups' scores take the place of the sort's counters, which nobody needs before the routing is done
  float* g_s = reinterpret_cast<float*>(l.count) + (size_t)wave * MOE_SMALL_E / 4;
  moe_route_token(a, min(wave, T - 1), wave < T, s_s[wave], c_s[wave], g_s);
  __syncthreads();  // the choices, in global memory, are the whole workgroup's
  moe_sort_pairs(l, a.chosen, T * (a.top + a.extra), a.E + a.extra, n_real, tile_rows, sorted, pos_of, tiles, meta);
}

static int moe_route_check(const MoeRouteArgs& a, int T) {
  LEV_REQUIRE(a.scoring >= 0 && a.scoring <= 2, "experts: unknown scoring %d", a.scoring);
  LEV_REQUIRE(T >= 0 && a.E > 0 && a.E <= MOE_MAX_E, "experts: %d experts (at most %d)", a.E, MOE_MAX_E);
  LEV_REQUIRE(a.G > 0 && a.E % a.G == 0 && a.keep > 0 && a.keep <= a.G && a.group_top > 0, "experts: %d groups of %d experts, %d kept", a.G, a.E, a.keep);
  LEV_REQUIRE(a.top > 0 && a.top <= MOE_MAX_TOP && a.top <= a.keep * (a.E / a.G), "experts: %d experts a token out of %d that can be chosen (at most %d)", a.top,
              a.keep * (a.E / a.G), MOE_MAX_TOP);
  LEV_REQUIRE(a.extra == 0 || a.extra == 1, "experts: one further choice at most");
  LEV_REQUIRE(a.z && a.chosen && a.weights && a.z_stride >= a.E, "experts: a tensor is missing");
  return 0;
}

extern "C" int lev_moe_route(const float* z, long z_stride, const float* correction, int T, int E, int G, int keep, int group_top, int top,
                             int renormalize, int scoring, int extra, int* chosen, float* weights, hipStream_t stream) {
  const MoeRouteArgs a{z, z_stride, correction, E, G, keep, group_top, top, renormalize, scoring, extra, chosen, weights};
  if (moe_route_check(a, T)) return -1;
  if (T == 0) return 0;
  moe_route_kernel<<<T, 64, 0, stream>>>(a);
  return lev_check_launch("moe_route");
}

extern "C" int lev_moe_max_tiles(int P, int E, int tile_rows) { return P / tile_rows + E + 1; }

static int moe_sort_check(const void* chosen, int P, int E, int n_real, int tile_rows, const void* sorted, const void* pos_of, const void* tiles, const void* meta) {
  LEV_REQUIRE(P >= 0 && E > 0 && E <= MOE_MAX_E + 1, "experts: %d experts (at most %d)", E, MOE_MAX_E + 1);
  LEV_REQUIRE(tile_rows == MOE_TM || tile_rows == MOE_BIG, "experts: tiles of %d rows (%d or %d)", tile_rows, MOE_TM, MOE_BIG);
  LEV_REQUIRE(chosen && sorted && pos_of && tiles && meta, "experts: a tensor is missing");
  LEV_REQUIRE(n_real >= 0 && n_real <= E, "experts: %d of %d experts have weights", n_real, E);
  return 0;
}

extern "C" int lev_moe_sort(const int* chosen, int P, int E, int n_real, int tile_rows, int* sorted, int* pos_of, int* tiles, int* meta, hipStream_t stream) {
  if (moe_sort_check(chosen, P, E, n_real, tile_rows, sorted, pos_of, tiles, meta)) return -1;
  moe_sort_kernel<<<1, MOE_SORT_NT, 0, stream>>>(chosen, P, E, n_real, tile_rows, sorted, pos_of, tiles, meta);
  return lev_check_launch("moe_sort");
}

// 1: not for these sizes (nothing has been launched); else as the two above, one after the other
extern "C" int lev_moe_route_sort(const float* z, long z_stride, const float* correction, int T, int E, int G, int keep, int group_top, int top,
                                  int renormalize, int scoring, int extra, int* chosen, float* weights, int n_real, int tile_rows, int* sorted, int* pos_of,
                                  int* tiles, int* meta, hipStream_t stream) {
  const MoeRouteArgs a{z, z_stride, correction, E, G, keep, group_top, top, renormalize, scoring, extra, chosen, weights};
  if (moe_route_check(a, T) || moe_sort_check(chosen, T * (top + extra), E + extra, n_real, tile_rows, sorted, pos_of, tiles, meta)) return -1;
  if (T == 0 || T > MOE_SMALL_T || E > MOE_SMALL_E || G > MOE_SMALL_E / 4) return 1;
  moe_route_sort_kernel<<<1, MOE_SORT_NT, 0, stream>>>(a, T, n_real, tile_rows, sorted, pos_of, tiles, meta);
  return lev_check_launch("moe_route_sort");
}

// ---- the experts' products ------------------------------------------------------------------------
__device__ __forceinline__ float moe_act(float gate, float up, int act, float limit, float up_shift) {
  if (limit > 0.f) gate = fminf(gate, limit), up = fminf(fmaxf(up, -limit), limit);
  return lev_activate(gate, act) * (up + up_shift);
}

// float32: a thread per (row of the tile, output); 16 x 16 a workgroup
template <typename T, typename TO>
__global__ void __launch_bounds__(256)
moe_linear_plain_kernel(const T* __restrict__ a, long a_stride, const T* __restrict__ w, TO* __restrict__ out, long o_stride,
                        const int* __restrict__ tiles, const int* __restrict__ meta, const int* __restrict__ sorted, int top, int gather,
                        int K, int N, int F, int glu, int act, float limit, float up_shift) {
  const int tile = blockIdx.x;
  if (tile >= meta[0]) return;
  const int e = tiles[3 * tile], first = tiles[3 * tile + 1], rows = tiles[3 * tile + 2];
  const int o = blockIdx.y * 16 + (threadIdx.x & 15);
  if (o >= F) return;
  for (int rr = threadIdx.x >> 4; rr < rows; rr += 16) {  // a tile may have more rows than the workgroup has row threads
    const int pos = first + rr;
    const T* ar = a + (size_t)(gather ? sorted[pos] / top : pos) * a_stride;
    const T* wg = w + ((size_t)e * N + o) * K;
    float acc = 0.f, acc_up = 0.f;
    for (int kk = 0; kk < K; ++kk) acc = fmaf(to_float<T>(wg[kk]), to_float<T>(ar[kk]), acc);
    if (glu) {
      const T* wu = wg + (size_t)F * K;
      for (int kk = 0; kk < K; ++kk) acc_up = fmaf(to_float<T>(wu[kk]), to_float<T>(ar[kk]), acc_up);
      acc = moe_act(acc, acc_up, act, limit, up_shift);
    } else {
      acc = lev_activate(acc, act);
    }
    out[(size_t)pos * o_stride + o] = from_float<TO>(acc);
  }
}

typedef __attribute__((ext_vector_type(8))) __bf16 moe_bf16x8;
typedef __attribute__((ext_vector_type(4))) float moe_f32x4;
typedef __attribute__((ext_vector_type(4))) uint32_t moe_u32x4;
__device__ __forceinline__ moe_bf16x8 moe_as_bf16x8(moe_u32x4 v) {
  union { moe_u32x4 u; moe_bf16x8 b; } c;
  c.u = v;
  return c.b;
}

// bfloat16 on the matrix cores: a wave owns the tile's rows (RT row tiles of 16) and NT tiles of 16 outputs (with glu: of gate
// and of up); the transposed product out^T = w a^T leaves each lane with four neighbouring outputs of one row. Every weight
// fragment a wave loads is used for all its row tiles.
template <typename TO, int NT, bool GLU, int RT>
__global__ void __launch_bounds__(256)
moe_linear_mfma_kernel(const bf16_t* __restrict__ a, long a_stride, const bf16_t* __restrict__ w, TO* __restrict__ out, long o_stride,
                       const int* __restrict__ tiles, const int* __restrict__ meta, const int* __restrict__ sorted, int top, int gather,
                       int K, int N, int F, int act, float limit, float up_shift) {
  const int tile = blockIdx.x;
  if (tile >= meta[0]) return;
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6, col = lane & 15, g = lane >> 4;
  const int o0 = (blockIdx.y * 4 + wave) * 16 * NT;
  if (o0 >= F) return;  // the whole wave
  const int e = tiles[3 * tile], first = tiles[3 * tile + 1], rows = tiles[3 * tile + 2];
  const bf16_t* ar[RT];
#pragma unroll
  for (int rt = 0; rt < RT; ++rt) {
    const int pos = first + min(16 * rt + col, rows - 1);  // rows beyond the tile: read again, never stored
    ar[rt] = a + (size_t)(gather ? sorted[pos] / top : pos) * a_stride;
  }
  const bf16_t* we = w + (size_t)e * N * K;
  const bf16_t* wr[NT];
#pragma unroll
  for (int nt = 0; nt < NT; ++nt) wr[nt] = we + (size_t)min(o0 + 16 * nt + col, F - 1) * K;
  moe_f32x4 acc[RT][NT], acc_up[RT][NT];
#pragma unroll
  for (int rt = 0; rt < RT; ++rt)
#pragma unroll
    for (int nt = 0; nt < NT; ++nt) acc[rt][nt] = acc_up[rt][nt] = moe_f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll 4
  for (int k0 = 0; k0 < K; k0 += 32) {
    const int kk = k0 + 8 * g, kc = min(kk, K - 8);  // loads stand under no condition; a chunk beyond the row counts as zeros
    const uint32_t keep = kk < K ? 0xffffffffu : 0u;
    moe_u32x4 av[RT];
#pragma unroll
    for (int rt = 0; rt < RT; ++rt) {
      const moe_u32x4 x = *reinterpret_cast<const moe_u32x4*>(ar[rt] + kc);
      av[rt] = moe_u32x4{x[0] & keep, x[1] & keep, x[2] & keep, x[3] & keep};
    }
    moe_u32x4 wv[NT], wu[NT];
#pragma unroll
    for (int nt = 0; nt < NT; ++nt) {
      wv[nt] = *reinterpret_cast<const moe_u32x4*>(wr[nt] + kc);
      if (GLU) wu[nt] = *reinterpret_cast<const moe_u32x4*>(wr[nt] + (size_t)F * K + kc);
    }
#pragma unroll
    for (int rt = 0; rt < RT; ++rt)
#pragma unroll
      for (int nt = 0; nt < NT; ++nt) {
        acc[rt][nt] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(moe_as_bf16x8(wv[nt]), moe_as_bf16x8(av[rt]), acc[rt][nt], 0, 0, 0);
        if (GLU) acc_up[rt][nt] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(moe_as_bf16x8(wu[nt]), moe_as_bf16x8(av[rt]), acc_up[rt][nt], 0, 0, 0);
      }
  }
#pragma unroll
  for (int rt = 0; rt < RT; ++rt) {
    if (16 * rt + col >= rows) continue;
#pragma unroll
    for (int nt = 0; nt < NT; ++nt)
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int o = o0 + 16 * nt + 4 * g + r;
        if (o < F)
          out[(size_t)(first + 16 * rt + col) * o_stride + o] = from_float<TO>(GLU ? moe_act(acc[rt][nt][r], acc_up[rt][nt][r], act, limit, up_shift) : lev_activate(acc[rt][nt][r], act));
      }
  }
}

// Few tiles (a step of single tokens): the products are bound by reading the chosen experts' weights, and a tile's 16 rows give
// the chip too few waves. A workgroup of MOE_KS waves owns one tile of 16 rows and 16 outputs; its waves split K, every wave has
// all loads of its share in flight, and the partial sums are added through LDS in wave order.
#define MOE_KS 8
template <typename TO, bool GLU>
__global__ void __launch_bounds__(64 * MOE_KS)
moe_linear_splitk_kernel(const bf16_t* __restrict__ a, long a_stride, const bf16_t* __restrict__ w, TO* __restrict__ out, long o_stride,
                         const int* __restrict__ tiles, const int* __restrict__ meta, const int* __restrict__ sorted, int top, int gather,
                         int K, int N, int F, int act, float limit, float up_shift) {
  __shared__ float part[MOE_KS][2][4][64];
  const int tile = blockIdx.x;
  if (tile >= meta[0]) return;
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6, col = lane & 15, g = lane >> 4;
  const int o0 = blockIdx.y * 16;
  const int e = tiles[3 * tile], first = tiles[3 * tile + 1], rows = tiles[3 * tile + 2];
  const int pos = first + min(col, rows - 1);  // rows beyond the tile: read again, never stored
  const bf16_t* ar = a + (size_t)(gather ? sorted[pos] / top : pos) * a_stride;
  const bf16_t* wr = w + (size_t)e * N * K + (size_t)min(o0 + col, F - 1) * K;
  const int share = ((K + MOE_KS * 32 - 1) / (MOE_KS * 32)) * 32;  // k steps of 32 a wave
  const int k_lo = wave * share, k_hi = min(K, k_lo + share);
  moe_f32x4 acc = moe_f32x4{0.f, 0.f, 0.f, 0.f}, acc_up = acc;
#pragma unroll 4
  for (int k0 = k_lo; k0 < k_hi; k0 += 32) {
    const int kk = k0 + 8 * g, kc = min(kk, K - 8);  // loads stand under no condition; a chunk beyond the row counts as zeros
    const uint32_t keep = kk < K ? 0xffffffffu : 0u;
    const moe_u32x4 x = *reinterpret_cast<const moe_u32x4*>(ar + kc);
    const moe_u32x4 av = moe_u32x4{x[0] & keep, x[1] & keep, x[2] & keep, x[3] & keep};
    const moe_u32x4 wv = *reinterpret_cast<const moe_u32x4*>(wr + kc);
    acc = __builtin_amdgcn_mfma_f32_16x16x32_bf16(moe_as_bf16x8(wv), moe_as_bf16x8(av), acc, 0, 0, 0);
    if (GLU) {
      const moe_u32x4 wu = *reinterpret_cast<const moe_u32x4*>(wr + (size_t)F * K + kc);
      acc_up = __builtin_amdgcn_mfma_f32_16x16x32_bf16(moe_as_bf16x8(wu), moe_as_bf16x8(av), acc_up, 0, 0, 0);
    }
  }
#pragma unroll
  for (int r = 0; r < 4; ++r) {
    part[wave][0][r][lane] = acc[r];
    if (GLU) part[wave][1][r][lane] = acc_up[r];
  }
  __syncthreads();
  if (wave != 0 || col >= rows) return;
#pragma unroll
  for (int r = 0; r < 4; ++r) {
    float sum = 0.f, sum_up = 0.f;
#pragma unroll
    for (int q = 0; q < MOE_KS; ++q) {
      sum += part[q][0][r][lane];
      if (GLU) sum_up += part[q][1][r][lane];
    }
    const int o = o0 + 4 * g + r;
    if (o < F) out[(size_t)(first + col) * o_stride + o] = from_float<TO>(GLU ? moe_act(sum, sum_up, act, limit, up_shift) : lev_activate(sum, act));
  }
}

// Tiles of 128 rows (prompts, large batches): a workgroup of four waves owns 128 rows and 128 weight rows (with glu: 64 outputs' gate
// rows and the same outputs' up rows), a wave 64 x 64 of them, so that a fragment from LDS feeds four products. K goes by in steps of 64,
// two steps on their way in registers and two buffers in LDS (rows 72 elements apart), one barrier a step. Rows beyond the tile are
// read again and never stored; a wave whose 64 rows all lie beyond it does not compute. The workgroups of a tile and of its neighbours
// in the list (an expert's rows, its weights) follow each other on one of the eight chiplets (workgroups are dealt to them in turn).
#define MOE_BIG_K 64
#define MOE_BIG_LD (MOE_BIG_K + 8)
#define MOE_BIG_LDS (2 * 2 * MOE_BIG * MOE_BIG_LD * (int)sizeof(bf16_t))
template <typename TO>
__device__ __forceinline__ void moe_store4(TO* p, const float (&v)[4], int n, bool vec);
template <>
__device__ __forceinline__ void moe_store4<float>(float* p, const float (&v)[4], int n, bool vec) {
  if (vec && n >= 4) *reinterpret_cast<float4*>(p) = make_float4(v[0], v[1], v[2], v[3]);
  else
#pragma unroll
    for (int r = 0; r < 4; ++r)
      if (r < n) p[r] = v[r];
}
template <>
__device__ __forceinline__ void moe_store4<bf16_t>(bf16_t* p, const float (&v)[4], int n, bool vec) {
  if (vec && n >= 4) *reinterpret_cast<uint2*>(p) = make_uint2(float2_to_bf16x2(v[0], v[1]), float2_to_bf16x2(v[2], v[3]));
  else
#pragma unroll
    for (int r = 0; r < 4; ++r)
      if (r < n) p[r] = float_to_bf16(v[r]);
}

template <typename TO, bool GLU>
__global__ void __launch_bounds__(256, 2)
moe_linear_big_kernel(const bf16_t* __restrict__ a, long a_stride, const bf16_t* __restrict__ w, TO* __restrict__ out, long o_stride,
                      const int* __restrict__ tiles, const int* __restrict__ meta, const int* __restrict__ sorted, int top, int gather,
                      int K, int N, int F, int act, float limit, float up_shift, int n_cols, int vec) {
  extern __shared__ __attribute__((aligned(16))) unsigned char moe_smem[];
  bf16_t* sa = reinterpret_cast<bf16_t*>(moe_smem);    // [2][128][72]
  bf16_t* sw = sa + 2 * MOE_BIG * MOE_BIG_LD;          // [2][128][72]
  constexpr int BN = GLU ? MOE_BIG / 2 : MOE_BIG;      // outputs of a workgroup
  const int n_tiles = meta[0], per = (n_tiles + 7) / 8;
  if (per == 0) return;
  const int slot = blockIdx.x >> 3, tile = (blockIdx.x & 7) * per + slot % per, ycol = slot / per;
  if (ycol >= n_cols || tile >= n_tiles) return;  // the whole workgroup
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, col = lane & 15, g = lane >> 4;
  const int wr = wave >> 1, wc = wave & 1;
  const int o0 = ycol * BN;
  const int e = tiles[3 * tile], first = tiles[3 * tile + 1], rows = tiles[3 * tile + 2];
  // what this thread fetches: a chunk of 8 elements of four activation rows and of four weight rows per step
  const int lrow = tid >> 3, lk = (tid & 7) * 8;
  const bf16_t *ap[4], *wp[4];
#pragma unroll
  for (int i = 0; i < 4; ++i) {
    const int r = lrow + 32 * i;
    const int pos = first + min(r, rows - 1);
    ap[i] = a + (size_t)(gather ? sorted[pos] / top : pos) * a_stride;
    const int o = min(o0 + (r % BN), F - 1) + (r >= BN ? F : 0);
    wp[i] = w + ((size_t)e * N + o) * K;
  }
  moe_f32x4 acc[4][4];
#pragma unroll
  for (int rt = 0; rt < 4; ++rt)
#pragma unroll
    for (int nt = 0; nt < 4; ++nt) acc[rt][nt] = moe_f32x4{0.f, 0.f, 0.f, 0.f};
  moe_u32x4 ra0[4], rw0[4], ra1[4], rw1[4];
  auto fetch = [&](int k0, moe_u32x4 (&ra)[4], moe_u32x4 (&rw)[4]) {
    const int kk = k0 + lk, kc = min(kk, K - 8);  // loads stand under no condition; a chunk beyond the row counts as zeros
    const uint32_t keep = kk < K ? 0xffffffffu : 0u;
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const moe_u32x4 x = *reinterpret_cast<const moe_u32x4*>(ap[i] + kc);
      ra[i] = moe_u32x4{x[0] & keep, x[1] & keep, x[2] & keep, x[3] & keep};
      rw[i] = *reinterpret_cast<const moe_u32x4*>(wp[i] + kc);
    }
  };
  auto stage = [&](int buf, const moe_u32x4 (&ra)[4], const moe_u32x4 (&rw)[4]) {
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      *reinterpret_cast<moe_u32x4*>(sa + ((size_t)buf * MOE_BIG + lrow + 32 * i) * MOE_BIG_LD + lk) = ra[i];
      *reinterpret_cast<moe_u32x4*>(sw + ((size_t)buf * MOE_BIG + lrow + 32 * i) * MOE_BIG_LD + lk) = rw[i];
    }
  };
  const bool active = wr * 64 < rows;
  auto multiply = [&](int buf) {
    if (!active) return;  // the whole wave
#pragma unroll
    for (int ks = 0; ks < MOE_BIG_K; ks += 32) {
      moe_u32x4 av[4], wv[4];
#pragma unroll
      for (int rt = 0; rt < 4; ++rt)
        av[rt] = *reinterpret_cast<const moe_u32x4*>(sa + ((size_t)buf * MOE_BIG + wr * 64 + 16 * rt + col) * MOE_BIG_LD + ks + 8 * g);
#pragma unroll
      for (int nt = 0; nt < 4; ++nt) {
        const int r = GLU ? (nt < 2 ? wc * 32 + 16 * nt : BN + wc * 32 + 16 * (nt - 2)) : wc * 64 + 16 * nt;
        wv[nt] = *reinterpret_cast<const moe_u32x4*>(sw + ((size_t)buf * MOE_BIG + r + col) * MOE_BIG_LD + ks + 8 * g);
      }
#pragma unroll
      for (int rt = 0; rt < 4; ++rt)
#pragma unroll
        for (int nt = 0; nt < 4; ++nt)
          acc[rt][nt] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(moe_as_bf16x8(wv[nt]), moe_as_bf16x8(av[rt]), acc[rt][nt], 0, 0, 0);
    }
  };
  const int steps = (K + MOE_BIG_K - 1) / MOE_BIG_K;
  fetch(0, ra0, rw0);
  fetch(MOE_BIG_K, ra1, rw1);  // beyond K: clamped and zero
  stage(0, ra0, rw0);
  lds_barrier();
  for (int st = 0; st < steps; st += 2) {  // the buffers and the register sets take turns; conditions are uniform over the workgroup
    if (st + 2 < steps) fetch((st + 2) * MOE_BIG_K, ra0, rw0);
    multiply(0);
    if (st + 1 >= steps) break;
    stage(1, ra1, rw1);  // nobody reads that buffer: every wave has passed the barrier behind the step that did
    lds_barrier();
    if (st + 3 < steps) fetch((st + 3) * MOE_BIG_K, ra1, rw1);
    multiply(1);
    if (st + 2 < steps) stage(0, ra0, rw0);
    lds_barrier();
  }
#pragma unroll
  for (int rt = 0; rt < 4; ++rt) {
    const int row = wr * 64 + 16 * rt + col;
    if (row >= rows) continue;
#pragma unroll
    for (int nt = 0; nt < (GLU ? 2 : 4); ++nt) {
      const int o = o0 + wc * (GLU ? 32 : 64) + 16 * nt + 4 * g;
      if (o >= F) continue;
      float v[4];
#pragma unroll
      for (int r = 0; r < 4; ++r) v[r] = GLU ? moe_act(acc[rt][nt][r], acc[rt][(nt + 2) & 3][r], act, limit, up_shift) : lev_activate(acc[rt][nt][r], act);
      moe_store4<TO>(out + (size_t)(first + row) * o_stride + o, v, F - o, vec);
    }
  }
}

// a [rows][K]; w [E][N][K] with N = F outputs, or with glu N = 2F: gate rows then up rows; out [P][F]
extern "C" int lev_moe_linear(const void* a, long a_stride, const void* w, void* out, long o_stride, const int* tiles, const int* meta,
                              const int* sorted, int max_tiles, int tile_rows, int top, int gather, int K, int N, int glu, int act, float limit,
                              float up_shift, int dtype, int out_dtype, int use_mfma, hipStream_t stream) {
  LEV_REQUIRE(a && w && out && tiles && meta && sorted, "experts: a tensor is missing");
  LEV_REQUIRE(K > 0 && N > 0 && (!glu || N % 2 == 0) && top > 0 && max_tiles >= 0, "experts: bad sizes K=%d N=%d", K, N);
  LEV_REQUIRE(act >= 0 && act <= LEV_ACT_LAST, "experts: unknown activation %d", act);
  LEV_REQUIRE(tile_rows == MOE_TM || tile_rows == MOE_BIG, "experts: tiles of %d rows (%d or %d)", tile_rows, MOE_TM, MOE_BIG);
  LEV_REQUIRE(dtype == LEV_F32 || dtype == LEV_BF16, "experts: unknown dtype %d", dtype);
  LEV_REQUIRE(dtype == LEV_BF16 || out_dtype == LEV_F32, "experts: float32 inputs give float32 outputs");
  const int F = glu ? N / 2 : N;
  LEV_REQUIRE(a_stride >= K && o_stride >= F, "experts: row strides are smaller than the rows");
  if (max_tiles == 0) return 0;
  if (dtype == LEV_BF16 && use_mfma && K % 8 == 0 && a_stride % 8 == 0 && ((uintptr_t)a & 15) == 0 && ((uintptr_t)w & 15) == 0) {
    if (tile_rows == MOE_TM && max_tiles <= 96) {  // a step of single tokens: K split over the waves of a workgroup
      dim3 grid_k(max_tiles, (F + 15) / 16);
#define MOE_SPLITK(TO)                                                                                                                           \
  do {                                                                                                                                           \
    if (glu)                                                                                                                                     \
      moe_linear_splitk_kernel<TO, true><<<grid_k, 64 * MOE_KS, 0, stream>>>((const bf16_t*)a, a_stride, (const bf16_t*)w, (TO*)out, o_stride, tiles, \
                                                                            meta, sorted, top, gather, K, N, F, act, limit, up_shift);                            \
    else                                                                                                                                         \
      moe_linear_splitk_kernel<TO, false><<<grid_k, 64 * MOE_KS, 0, stream>>>((const bf16_t*)a, a_stride, (const bf16_t*)w, (TO*)out, o_stride, tiles, \
                                                                             meta, sorted, top, gather, K, N, F, act, limit, up_shift);                           \
  } while (0)
      if (out_dtype == LEV_F32) MOE_SPLITK(float); else MOE_SPLITK(bf16_t);
#undef MOE_SPLITK
      return lev_check_launch("moe_linear (matrix cores, K split)");
    }
    if (tile_rows == MOE_BIG) {
      const int bn = glu ? MOE_BIG / 2 : MOE_BIG, n_cols = (F + bn - 1) / bn;
      const long blocks = (long)((max_tiles + 7) / 8) * 8 * n_cols;
      LEV_REQUIRE(blocks <= 0x7fffffffL, "experts: too many tiles (%ld)", blocks);
      const int vec = o_stride % 4 == 0 && ((uintptr_t)out & (out_dtype == LEV_F32 ? 15 : 7)) == 0;
#define MOE_BIG_CASE(TO, G)                                                                                                                       \
  do {                                                                                                                                            \
    hipError_t e = hipFuncSetAttribute((const void*)moe_linear_big_kernel<TO, G>, hipFuncAttributeMaxDynamicSharedMemorySize, MOE_BIG_LDS);        \
    LEV_REQUIRE(e == hipSuccess, "experts: %d bytes of LDS a workgroup: %s", MOE_BIG_LDS, hipGetErrorString(e));                                   \
    moe_linear_big_kernel<TO, G><<<(unsigned)blocks, 256, MOE_BIG_LDS, stream>>>((const bf16_t*)a, a_stride, (const bf16_t*)w, (TO*)out, o_stride, tiles, \
                                                                                meta, sorted, top, gather, K, N, F, act, limit, up_shift, n_cols, vec); \
  } while (0)
      if (out_dtype == LEV_F32) {
        if (glu) MOE_BIG_CASE(float, true); else MOE_BIG_CASE(float, false);
      } else {
        if (glu) MOE_BIG_CASE(bf16_t, true); else MOE_BIG_CASE(bf16_t, false);
      }
#undef MOE_BIG_CASE
      return lev_check_launch("moe_linear (matrix cores, tiles of 128 rows)");
    }
    // many tiles of 16 rows: a wave per tile and 32 outputs, both operands straight from global memory
    const int nt = 2;
    dim3 grid(max_tiles, (F + 64 * nt - 1) / (64 * nt));
#define MOE_CASE(TO)                                                                                                                             \
  do {                                                                                                                                           \
    if (glu)                                                                                                                                     \
      moe_linear_mfma_kernel<TO, 2, true, 1><<<grid, 256, 0, stream>>>((const bf16_t*)a, a_stride, (const bf16_t*)w, (TO*)out, o_stride, tiles, meta, \
                                                                      sorted, top, gather, K, N, F, act, limit, up_shift);                                        \
    else                                                                                                                                         \
      moe_linear_mfma_kernel<TO, 2, false, 1><<<grid, 256, 0, stream>>>((const bf16_t*)a, a_stride, (const bf16_t*)w, (TO*)out, o_stride, tiles,  \
                                                                       meta, sorted, top, gather, K, N, F, act, limit, up_shift);                                 \
  } while (0)
    if (out_dtype == LEV_F32) MOE_CASE(float); else MOE_CASE(bf16_t);
#undef MOE_CASE
    return lev_check_launch("moe_linear (matrix cores)");
  }
  dim3 grid(max_tiles, (F + 15) / 16);
  if (dtype == LEV_F32)
    moe_linear_plain_kernel<float, float><<<grid, 256, 0, stream>>>((const float*)a, a_stride, (const float*)w, (float*)out, o_stride, tiles, meta,
                                                                    sorted, top, gather, K, N, F, glu, act, limit, up_shift);
  else if (out_dtype == LEV_F32)
    moe_linear_plain_kernel<bf16_t, float><<<grid, 256, 0, stream>>>((const bf16_t*)a, a_stride, (const bf16_t*)w, (float*)out, o_stride, tiles, meta,
                                                                     sorted, top, gather, K, N, F, glu, act, limit, up_shift);
  else
    moe_linear_plain_kernel<bf16_t, bf16_t><<<grid, 256, 0, stream>>>((const bf16_t*)a, a_stride, (const bf16_t*)w, (bf16_t*)out, o_stride, tiles,
                                                                      meta, sorted, top, gather, K, N, F, glu, act, limit, up_shift);
  return lev_check_launch("moe_linear");
}

// ---- combine -------------------------------------------------------------------------------------
__global__ void __launch_bounds__(256)
moe_combine_kernel(const float* __restrict__ expert_out, const int* __restrict__ pos_of, const float* __restrict__ weights, float* __restrict__ y,
                   int D, int top, int accumulate, const int* __restrict__ chosen, int n_real, const void* __restrict__ identity_in, long id_stride,
                   int id_dtype) {
  __shared__ int pos_s[MOE_MAX_TOP];
  __shared__ float w_s[MOE_MAX_TOP];
  const int t = blockIdx.x;
  if (threadIdx.x < top) {
    const bool own = identity_in != nullptr && chosen[(size_t)t * top + threadIdx.x] >= n_real;  // an expert that returns its input
    pos_s[threadIdx.x] = own ? -1 : pos_of[(size_t)t * top + threadIdx.x];
    w_s[threadIdx.x] = weights[(size_t)t * top + threadIdx.x];
  }
  __syncthreads();
  for (int d = threadIdx.x; d < D; d += 256) {
    float acc = accumulate ? y[(size_t)t * D + d] : 0.f;
    float own = 0.f;
    if (identity_in != nullptr)
      own = id_dtype == LEV_F32 ? ((const float*)identity_in)[(size_t)t * id_stride + d] : bf16_to_float(((const bf16_t*)identity_in)[(size_t)t * id_stride + d]);
    for (int c = 0; c < top; ++c) acc = fmaf(w_s[c], pos_s[c] < 0 ? own : expert_out[(size_t)pos_s[c] * D + d], acc);
    y[(size_t)t * D + d] = acc;
  }
}

extern "C" int lev_moe_combine(const float* expert_out, const int* pos_of, const float* weights, float* y, int T, int D, int top, int accumulate,
                               const int* chosen, int n_real, const void* identity_in, long id_stride, int id_dtype, hipStream_t stream) {
  LEV_REQUIRE(expert_out && pos_of && weights && y && T >= 0 && D > 0 && top > 0 && top <= MOE_MAX_TOP, "experts: bad arguments of the weighted sum");
  LEV_REQUIRE(identity_in == nullptr || (chosen && id_stride >= D && (id_dtype == LEV_F32 || id_dtype == LEV_BF16)), "experts: experts that return their input need the choices and the input's rows");
  if (T == 0) return 0;
  moe_combine_kernel<<<T, 256, 0, stream>>>(expert_out, pos_of, weights, y, D, top, accumulate, chosen, n_real, identity_in, id_stride, id_dtype);
  return lev_check_launch("moe_combine");
}
