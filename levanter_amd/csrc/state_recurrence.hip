// Recurrences with a matrix state per head, one decay per head and token, and a short convolution ahead of them. Two rules, with
// key channels i < dk and value channels j < dv; head h of H reads the keys and queries of group h / (H / G):
//     sp = softplus(a + a_bias_h),  d = exp(-rate_h sp)                       the decay, in (0, 1]
//   rule SSD (state-space duality):   S <- d S + sp k v^T,                                          o = S^T q + skip_h v
//   rule DELTA (gated delta rule):    S <- d S,  u = sigmoid(b) (v - S^T k),  S <- S + k u^T,       o = S^T q
//     with k and q unit vectors per head (divided by sqrt(sum of squares + key_eps)), q also times q_scale.
// q, k and v are channels of one tensor: u = silu(conv(x)), conv a causal convolution per channel with K taps (the last tap is the
// current token's; zeros before the sequence starts). Behind the recurrence a norm and a gate:
//   SSD:    y = o * silu(gate), divided by its root mean square in `norm_groups` equal parts of a token's row, times a weight;
//   DELTA:  o divided by its root mean square per head, times a weight, times silu(gate).
// The convolution's output is of the compute dtype; everything between it and the result is 32-bit.
//
// What a request carries lives in its state slot, float32: [K][C] the convolution's inputs, the one of position p in row p mod K, and
// behind them S, [H][dk][dv]. token_slots [T]: the slot of each token's request (-1: a token of nobody, zeros). The tokens of a request
// stand next to each other in a step, in the order of their positions.
//
// Steps of single tokens: one kernel per (token, head) does convolution, recurrence and (DELTA) norm and gate. A row of the ring of
// inputs is written by the token of its position and read by the K - 1 tokens after it, so the workgroups of a token that share
// channels need no order among them. Steps with runs: convolution; decays, step sizes, key norms and the ring (written by a
// kernel behind the one that reads it); the recurrence (bfloat16: in chunks on the matrix cores, state_chunks.hip; float32, or without the
// matrix cores: token by token); norm and gate.
#include "state_recurrence.h"

// the activation behind the convolution: what is rounded to bfloat16 takes the hardware's exponential and reciprocal (about 1 ulp each)
template <typename T>
__device__ __forceinline__ float sr_conv_silu(float x) { return sizeof(T) == 2 ? lev_sigmoid_mul(x, -1.4426950408889634f * x) : sr_silu(x); }

// ---- the convolution of a step with runs ----------------------------------------------------------------------------------
// A thread takes SR_CT tokens of one channel; with K <= 4 their inputs and the three before them are held in registers.
#define SR_CT 8
template <typename T>
__global__ void __launch_bounds__(256)
sr_conv_kernel(const T* __restrict__ x, const float* __restrict__ taps, const float* __restrict__ bias, const float* __restrict__ state,
               const int* __restrict__ token_slots, const int* __restrict__ positions, T* __restrict__ u, SrShape s) {
  const int c = blockIdx.y * 256 + threadIdx.x, t0 = blockIdx.x * SR_CT;
  const int C = s.C, K = s.K;
  if (c >= C) return;
  const float b = bias ? bias[c] : 0.f;
  if (K <= 4) {
    float tap[4], xv[SR_CT + 3];
#pragma unroll
    for (int k = 0; k < 4; ++k) tap[k] = k < K ? taps[(size_t)c * K + K - 1 - k] : 0.f;  // tap[k]: of the input k tokens back
#pragma unroll
    for (int i = 0; i < SR_CT + 3; ++i) xv[i] = to_float<T>(x[(size_t)min(max(t0 + i - 3, 0), s.Tn - 1) * s.x_stride + c]);
#pragma unroll
    for (int i = 0; i < SR_CT; ++i) {
      const int t = t0 + i;
      if (t >= s.Tn) break;
      const int slot = token_slots[t], pos = positions[t];
      float acc = b;
#pragma unroll
      for (int k = 0; k < 4; ++k) {
        if (k >= K || slot < 0) continue;
        float v = xv[i + 3 - k];
        if (k > 0 && !(t - k >= 0 && token_slots[t - k] == slot))
          v = pos - k >= 0 ? state[(size_t)slot * s.slot_stride + (size_t)((pos - k) % K) * C + c] : 0.f;
        acc = fmaf(tap[k], v, acc);
      }
      u[(size_t)t * C + c] = from_float<T>(slot < 0 ? 0.f : sr_conv_silu<T>(acc));
    }
  } else {
    for (int i = 0; i < SR_CT && t0 + i < s.Tn; ++i) {
      const int t = t0 + i, slot = token_slots[t], pos = positions[t];
      float acc = b;
      for (int k = 0; k < K && slot >= 0; ++k) {
        float v = 0.f;
        if (t - k >= 0 && token_slots[t - k] == slot) v = to_float<T>(x[(size_t)(t - k) * s.x_stride + c]);
        else if (pos - k >= 0) v = state[(size_t)slot * s.slot_stride + (size_t)((pos - k) % K) * C + c];
        acc = fmaf(taps[(size_t)c * K + K - 1 - k], v, acc);
      }
      u[(size_t)t * C + c] = from_float<T>(slot < 0 ? 0.f : sr_conv_silu<T>(acc));
    }
  }
}

// four neighbouring elements: 8 bytes of bfloat16 or 16 of float32
template <typename T>
struct __attribute__((aligned(4 * sizeof(T)))) SrQuad {
  T v[4];
};

// The same for up to four taps with four channels a thread (8-byte or 16-byte loads; C and the row stride multiples of 4).
template <typename T>
__global__ void __launch_bounds__(256)
sr_conv_quad_kernel(const T* __restrict__ x, const float* __restrict__ taps, const float* __restrict__ bias, const float* __restrict__ state,
                    const int* __restrict__ token_slots, const int* __restrict__ positions, T* __restrict__ u, SrShape s) {
  const int c = (blockIdx.y * 256 + threadIdx.x) * 4, t0 = blockIdx.x * SR_CT;
  const int C = s.C, K = s.K;
  if (c >= C) return;
  float b[4], tap[4][4];
#pragma unroll
  for (int e = 0; e < 4; ++e) {
    b[e] = bias ? bias[c + e] : 0.f;
#pragma unroll
    for (int k = 0; k < 4; ++k) tap[k][e] = k < K ? taps[(size_t)(c + e) * K + max(K - 1 - k, 0)] : 0.f;
  }
  SrQuad<T> xv[SR_CT + 3];
#pragma unroll
  for (int i = 0; i < SR_CT + 3; ++i) xv[i] = *reinterpret_cast<const SrQuad<T>*>(x + (size_t)min(max(t0 + i - 3, 0), s.Tn - 1) * s.x_stride + c);
#pragma unroll
  for (int i = 0; i < SR_CT; ++i) {
    const int t = t0 + i;
    if (t >= s.Tn) break;
    const int slot = token_slots[t], pos = positions[t];
    float acc[4] = {b[0], b[1], b[2], b[3]};
#pragma unroll
    for (int k = 0; k < 4; ++k) {
      if (k >= K || slot < 0) continue;
      if (k == 0 || (t - k >= 0 && token_slots[t - k] == slot)) {
#pragma unroll
        for (int e = 0; e < 4; ++e) acc[e] = fmaf(tap[k][e], to_float<T>(xv[i + 3 - k].v[e]), acc[e]);
      } else if (pos - k >= 0) {
        const float* row = state + (size_t)slot * s.slot_stride + (size_t)((pos - k) % K) * C + c;
#pragma unroll
        for (int e = 0; e < 4; ++e) acc[e] = fmaf(tap[k][e], row[e], acc[e]);
      }
    }
    SrQuad<T> w;
#pragma unroll
    for (int e = 0; e < 4; ++e) w.v[e] = from_float<T>(slot < 0 ? 0.f : sr_conv_silu<T>(acc[e]));
    *reinterpret_cast<SrQuad<T>*>(u + (size_t)t * C + c) = w;
  }
}

// ---- per token: log decay and write rate of every head, inverse norms of keys and queries, the ring of inputs ----------------
// scal: [Tn][2 H + 2 G] = log decays | write rates | 1 / |k| | q_scale / |q|  (SSD: ones)
template <typename T, int RULE>
__global__ void __launch_bounds__(256)
sr_prepare_kernel(const T* __restrict__ x, const T* __restrict__ u, const T* __restrict__ a, const T* __restrict__ b, const float* __restrict__ a_bias,
                  const float* __restrict__ rate, float* __restrict__ state, const int* __restrict__ token_slots, const int* __restrict__ positions,
                  float* __restrict__ scal, SrShape s) {
  const int t = blockIdx.x, tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
  const int slot = token_slots[t];
  const int H = s.H, G = s.G;
  float* sc = scal + (size_t)t * (2 * H + 2 * G);
  if (slot < 0) {
    for (int i = tid; i < 2 * H + 2 * G; i += 256) sc[i] = 0.f;
    return;
  }
  // one of the run's last K - 1 tokens: its inputs stay for the tokens of the next step
  if (t + s.K - 1 >= s.Tn || token_slots[t + s.K - 1] != slot) {
    float* row = state + (size_t)slot * s.slot_stride + (size_t)(positions[t] % s.K) * s.C;
    for (int c = tid; c < s.C; c += 256) row[c] = to_float<T>(x[(size_t)t * s.x_stride + c]);
  }
  for (int h = tid; h < H; h += 256) {
    const float sp = sr_softplus(to_float<T>(a[(size_t)t * s.a_stride + h]) + a_bias[h]);
    sc[h] = -rate[h] * sp;
    sc[H + h] = RULE == SR_DELTA ? sr_sigmoid(to_float<T>(b[(size_t)t * s.b_stride + h])) : sp;
  }
  for (int g = wave; g < 2 * G; g += 4) {
    float r = 1.0f;
    if (RULE == SR_DELTA) {
      const bool is_q = g >= G;
      const T* row = u + (size_t)t * s.C + (is_q ? s.q_off + (size_t)(g - G) * s.dk : s.k_off + (size_t)g * s.dk);
      float ss = 0.f;
      for (int i = lane; i < s.dk; i += 64) {
        const float v = to_float<T>(row[i]);
        ss = fmaf(v, v, ss);
      }
      ss = wave_sum(ss);
      r = (is_q ? s.q_scale : 1.0f) / sqrtf(ss + s.key_eps);
    }
    if (lane == 0) sc[2 * H + g] = r;
  }
}

// ---- the recurrence of a step with runs, token by token ------------------------------------------------------------------------
// One workgroup per (run, head, SR_WC state columns): 8 neighbouring lanes share a column, each with DKM / 8 key channels of it in
// registers; sums over the key channels go across the 8 lanes. Keys and queries of SR_WT tokens at a time are staged through LDS.
#define SR_WC 32
#define SR_WT 16
template <typename T, int DKM, int RULE>
__global__ void __launch_bounds__(256)
sr_walk_kernel(const T* __restrict__ u, const float* __restrict__ scal, float* __restrict__ state, const int* __restrict__ token_slots,
               float* __restrict__ o, SrShape s) {
  constexpr int IP = DKM / 8;
  __shared__ float s_k[SR_WT][DKM], s_q[SR_WT][DKM];
  __shared__ int tmp[256 + 2];
  const int h = blockIdx.x, tid = threadIdx.x, part = tid & 7, j = blockIdx.y * SR_WC + (tid >> 3);
  const int g = h / (s.H / s.G), n_scal = 2 * s.H + 2 * s.G;
  int t0, t_end, slot;
  if (!sr_find_run<256>(blockIdx.z, token_slots, s.Tn, tmp, t0, t_end, slot)) return;
  const bool live = j < s.dv;
  float* sp = state + (size_t)slot * s.slot_stride + (size_t)s.K * s.C + (size_t)h * s.dk * s.dv + (live ? j : 0);
  float S[IP];
#pragma unroll
  for (int ii = 0; ii < IP; ++ii) {
    const int i = ii * 8 + part;
    S[ii] = live && i < s.dk ? sp[(size_t)i * s.dv] : 0.f;
  }
  for (int tb = t0; tb < t_end; tb += SR_WT) {
    __syncthreads();
    for (int idx = tid; idx < SR_WT * DKM; idx += 256) {
      const int tt = idx / DKM, i = idx - tt * DKM, t = min(tb + tt, t_end - 1);
      const bool in = i < s.dk;
      const T* row = u + (size_t)t * s.C + (size_t)g * s.dk + (in ? i : 0);
      s_k[tt][i] = in ? to_float<T>(row[s.k_off]) * scal[(size_t)t * n_scal + 2 * s.H + g] : 0.f;
      s_q[tt][i] = in ? to_float<T>(row[s.q_off]) * scal[(size_t)t * n_scal + 2 * s.H + s.G + g] : 0.f;
    }
    __syncthreads();
    const int n = min(SR_WT, t_end - tb);
    for (int tt = 0; tt < n; ++tt) {
      const int t = tb + tt;
      const float d = expf(scal[(size_t)t * n_scal + h]), w = scal[(size_t)t * n_scal + s.H + h];
      const float v = live ? to_float<T>(u[(size_t)t * s.C + s.v_off + (size_t)h * s.dv + j]) : 0.f;
      float add = w * v;
      if (RULE == SR_DELTA) {
        float ks = 0.f;
#pragma unroll
        for (int ii = 0; ii < IP; ++ii) ks = fmaf(s_k[tt][ii * 8 + part], S[ii], ks);
        ks += __shfl_xor(ks, 1, 64);
        ks += __shfl_xor(ks, 2, 64);
        ks += __shfl_xor(ks, 4, 64);
        add = w * (v - d * ks);
      }
      float out = 0.f;
#pragma unroll
      for (int ii = 0; ii < IP; ++ii) {
        S[ii] = fmaf(s_k[tt][ii * 8 + part], add, d * S[ii]);
        out = fmaf(s_q[tt][ii * 8 + part], S[ii], out);
      }
      out += __shfl_xor(out, 1, 64);
      out += __shfl_xor(out, 2, 64);
      out += __shfl_xor(out, 4, 64);
      if (live && part == 0) o[((size_t)t * s.H + h) * s.dv + j] = out;
    }
  }
  if (live) {
#pragma unroll
    for (int ii = 0; ii < IP; ++ii) {
      const int i = ii * 8 + part;
      if (i < s.dk) sp[(size_t)i * s.dv] = S[ii];
    }
  }
}

// ---- norm and gate ----------------------------------------------------------------------------------------------------------------
// One workgroup per (token, part of its row): SSD: parts of H * dv / norm_groups numbers, y = (o + skip_h v) silu(gate) first and then the
// norm; DELTA: a head a part, the norm and then the gate. v (SSD): the values in u, null if `o` holds the skip already.
template <typename T, int RULE, int NT>
__global__ void __launch_bounds__(NT)
sr_finish_kernel(const float* __restrict__ o, const T* __restrict__ u, const float* __restrict__ skip, const T* __restrict__ gate,
                 const float* __restrict__ norm_w, const int* __restrict__ token_slots, T* __restrict__ out, int len, SrShape s) {
  __shared__ float red[NT / 64];
  const int t = blockIdx.x, c0 = blockIdx.y * len, tid = threadIdx.x;
  T* orow = out + (size_t)t * s.o_stride + c0;
  if (token_slots[t] < 0) {
    for (int c = tid; c < len; c += NT) orow[c] = from_float<T>(0.f);
    return;
  }
  const float* orw = o + (size_t)t * s.H * s.dv + c0;
  const T* grow = gate + (size_t)t * s.gate_stride + c0;
  constexpr int KEEP = 4;  // numbers a thread keeps between the two passes; what lies beyond is computed again
  float kept[KEEP];
  auto value = [&](int c) {
    float y = orw[c];
    if (RULE == SR_SSD) {
      if (u) y = fmaf(skip[(c0 + c) / s.dv], to_float<T>(u[(size_t)t * s.C + s.v_off + c0 + c]), y);
      y *= sr_silu(to_float<T>(grow[c]));
    }
    return y;
  };
  float ss = 0.f;
#pragma unroll
  for (int i = 0; i < KEEP; ++i) {
    const int c = tid + NT * i;
    kept[i] = c < len ? value(c) : 0.f;
    ss = fmaf(kept[i], kept[i], ss);
  }
  for (int c = tid + NT * KEEP; c < len; c += NT) {
    const float y = value(c);
    ss = fmaf(y, y, ss);
  }
  ss = block_sum<NT>(ss, red);
  const float r = 1.0f / sqrtf(ss / (float)len + s.norm_eps);
  auto store = [&](int c, float y) {
    y *= r * norm_w[c0 + c];
    if (RULE == SR_DELTA) y *= sr_silu(to_float<T>(grow[c]));
    orow[c] = from_float<T>(y);
  };
#pragma unroll
  for (int i = 0; i < KEEP; ++i)
    if (tid + NT * i < len) store(tid + NT * i, kept[i]);
  for (int c = tid + NT * KEEP; c < len; c += NT) store(c, value(c));
}

// The same with four neighbouring numbers a lane, NV of them: LANES lanes share a part (a wave or less: several parts a workgroup; 256: the
// whole workgroup). Everything is a multiple of 4 and aligned; LANES * NV * 4 >= len.
template <typename T, int RULE, int LANES, int NV>
__global__ void __launch_bounds__(256)
sr_finish_quad_kernel(const float* __restrict__ o, const T* __restrict__ u, const float* __restrict__ skip, const T* __restrict__ gate,
                      const float* __restrict__ norm_w, const int* __restrict__ token_slots, T* __restrict__ out, int len, int parts, SrShape s) {
  __shared__ float red[4];
  const int t = blockIdx.x, lane = threadIdx.x % LANES;
  const int part = min((int)(blockIdx.y * (256 / LANES) + threadIdx.x / LANES), parts - 1);  // the last workgroup's surplus lanes repeat the last part
  const int c0 = part * len;
  const bool nobody = token_slots[t] < 0;
  float y[NV][4];
  SrQuad<T> gv[NV];
  float4 wv[NV];
  float ss = 0.f;
#pragma unroll
  for (int i = 0; i < NV; ++i) {
    const int c = min((lane + LANES * i) * 4, len - 4);
    const float4 ov = *reinterpret_cast<const float4*>(o + (size_t)t * s.H * s.dv + c0 + c);
    gv[i] = *reinterpret_cast<const SrQuad<T>*>(gate + (size_t)t * s.gate_stride + c0 + c);
    wv[i] = *reinterpret_cast<const float4*>(norm_w + c0 + c);
    y[i][0] = ov.x, y[i][1] = ov.y, y[i][2] = ov.z, y[i][3] = ov.w;
    if (RULE == SR_SSD && u) {
      const SrQuad<T> x = *reinterpret_cast<const SrQuad<T>*>(u + (size_t)t * s.C + s.v_off + c0 + c);
      const float sk = skip[(c0 + c) / s.dv];
#pragma unroll
      for (int e = 0; e < 4; ++e) y[i][e] = fmaf(sk, to_float<T>(x.v[e]), y[i][e]);
    }
  }
#pragma unroll
  for (int i = 0; i < NV; ++i)
#pragma unroll
    for (int e = 0; e < 4; ++e) {
      if (RULE == SR_SSD) y[i][e] *= sr_silu(to_float<T>(gv[i].v[e]));
      if ((lane + LANES * i) * 4 < len) ss = fmaf(y[i][e], y[i][e], ss);
    }
  if (LANES == 256) {
    ss = block_sum<256>(ss, red);
  } else {
#pragma unroll
    for (int d = LANES / 2; d > 0; d >>= 1) ss += __shfl_xor(ss, d, 64);
  }
  const float r = 1.0f / sqrtf(ss / (float)len + s.norm_eps);
#pragma unroll
  for (int i = 0; i < NV; ++i) {
    const int c = (lane + LANES * i) * 4;
    if (c >= len) continue;
    const float w4[4] = {wv[i].x, wv[i].y, wv[i].z, wv[i].w};
    SrQuad<T> w;
#pragma unroll
    for (int e = 0; e < 4; ++e) {
      float z = y[i][e] * r * w4[e];
      if (RULE == SR_DELTA) z *= sr_silu(to_float<T>(gv[i].v[e]));
      w.v[e] = from_float<T>(nobody ? 0.f : z);
    }
    *reinterpret_cast<SrQuad<T>*>(out + (size_t)t * s.o_stride + c0 + c) = w;
  }
}

// ---- steps of single tokens ----------------------------------------------------------------------------------------------------------
// One workgroup per (token, head). Thread (rg, c4) of 16 x DVM / 4 takes the four columns 4 c4 .. of the key channels rg, rg + 16, ..:
// the state is asked for first, the convolution and the scalars run while it is on its way.
template <typename T, int DKM, int DVM, int RULE>
__global__ void __launch_bounds__(DVM * 4)
sr_token_kernel(const T* __restrict__ x, const float* __restrict__ taps, const float* __restrict__ conv_bias, const T* __restrict__ a,
                const T* __restrict__ b, const float* __restrict__ a_bias, const float* __restrict__ rate, const float* __restrict__ skip,
                const T* __restrict__ gate, const float* __restrict__ norm_w, float* __restrict__ state, const int* __restrict__ token_slots,
                const int* __restrict__ positions, float* __restrict__ y_out, T* __restrict__ out, int vec, SrShape s) {
  constexpr int NT = DVM * 4, QD = DVM / 4, RPT = DKM / 16;
  __shared__ float s_k[DKM], s_q[DKM], red[NT / 64];
  __shared__ __attribute__((aligned(16))) float s_v[DVM];
  __shared__ __attribute__((aligned(16))) float s_po[16][DVM], s_pk[RULE == SR_DELTA ? 16 : 1][DVM];
  const int t = blockIdx.x, h = blockIdx.y, tid = threadIdx.x, c4 = tid % QD, rg = tid / QD;
  const int dk = s.dk, dv = s.dv, C = s.C, K = s.K, rep = s.H / s.G, g = h / rep;
  const int slot = token_slots[t], pos = positions[t];
  const size_t vcol = (size_t)h * dv;
  if (slot < 0) {  // a token of nobody (the whole workgroup)
    for (int j = tid; j < dv; j += NT) {
      if (RULE == SR_SSD) y_out[(size_t)t * s.H * dv + vcol + j] = 0.f;
      else out[(size_t)t * s.o_stride + vcol + j] = from_float<T>(0.f);
    }
    return;
  }
  float* ring = state + (size_t)slot * s.slot_stride;
  float* sp = ring + (size_t)K * C + (size_t)h * dk * dv;
  float4 S[RPT];
#pragma unroll
  for (int r = 0; r < RPT; ++r) {
    const int i = rg + 16 * r;
    S[r] = make_float4(0.f, 0.f, 0.f, 0.f);
    if (i < dk) {
      const float* p = sp + (size_t)i * dv + 4 * c4;
      if (vec) {
        if (4 * c4 < dv) S[r] = *reinterpret_cast<const float4*>(p);
      } else {
        if (4 * c4 < dv) S[r].x = p[0];
        if (4 * c4 + 1 < dv) S[r].y = p[1];
        if (4 * c4 + 2 < dv) S[r].z = p[2];
        if (4 * c4 + 3 < dv) S[r].w = p[3];
      }
    }
  }
  // convolution of this head's values and its group's keys and queries; the shared channels' ring row is the first head's to write
  {
    constexpr int NIT = (DVM + 2 * DKM + NT - 1) / NT;
    // the channel of a thread's n-th item (clamped: loads stand under no condition) and whether there is one
    auto item = [&](int n, int& which, int& i, bool& in) {
      const int idx = min(tid + NT * n, DVM + 2 * DKM - 1);
      which = idx < DVM ? 0 : idx < DVM + DKM ? 1 : 2;
      i = which == 0 ? idx : which == 1 ? idx - DVM : idx - DVM - DKM;
      in = i < (which == 0 ? dv : dk);
      const int ic = in ? i : 0;
      return which == 0 ? s.v_off + h * dv + ic : which == 1 ? s.k_off + g * dk + ic : s.q_off + g * dk + ic;
    };
    T cur[NIT];
    float acc[NIT], tap[NIT][4], old[NIT][3];
#pragma unroll
    for (int n = 0; n < NIT; ++n) {
      int which, i;
      bool in;
      const int c = item(n, which, i, in);
      cur[n] = x[(size_t)t * s.x_stride + c];
      acc[n] = conv_bias ? conv_bias[c] : 0.f;
#pragma unroll
      for (int k = 0; k < 4; ++k) tap[n][k] = taps[(size_t)c * K + max(K - 1 - k, 0)];
#pragma unroll
      for (int k = 1; k < 4; ++k) old[n][k - 1] = ring[(size_t)((pos + 4 * K - k) % K) * C + c];
    }
#pragma unroll
    for (int n = 0; n < NIT; ++n) {
      int which, i;
      bool in;
      const int c = item(n, which, i, in);
      const float cf = to_float<T>(cur[n]);
      acc[n] = fmaf(tap[n][0], cf, acc[n]);
#pragma unroll
      for (int k = 1; k < 4; ++k)
        if (k < K && pos - k >= 0) acc[n] = fmaf(tap[n][k], old[n][k - 1], acc[n]);
      for (int k = 4; k < K; ++k)
        if (pos - k >= 0) acc[n] = fmaf(taps[(size_t)c * K + K - 1 - k], ring[(size_t)((pos - k) % K) * C + c], acc[n]);
      const float val = in ? to_float<T>(from_float<T>(sr_conv_silu<T>(acc[n]))) : 0.f;
      if (tid + NT * n < DVM + 2 * DKM) {
        if (in && (which == 0 || h % rep == 0)) ring[(size_t)(pos % K) * C + c] = cf;
        if (which == 0) s_v[i] = val;
        else if (which == 1) s_k[i] = val;
        else s_q[i] = val;
      }
    }
  }
  const float sft = sr_softplus(to_float<T>(a[(size_t)t * s.a_stride + h]) + a_bias[h]);
  const float d = expf(-rate[h] * sft);
  const float w = RULE == SR_DELTA ? sr_sigmoid(to_float<T>(b[(size_t)t * s.b_stride + h])) : sft;
  float gt = 0.f, nw = 0.f;
  if (RULE == SR_DELTA && tid < dv) gt = to_float<T>(gate[(size_t)t * s.gate_stride + vcol + tid]), nw = norm_w[vcol + tid];
  __syncthreads();
  float rk = 1.f, rq = 1.f, qk = 0.f;
  if (RULE == SR_DELTA) {
    float kk = 0.f, qq = 0.f;  // every wave for itself: no barrier
#pragma unroll
    for (int i = tid & 63; i < DKM; i += 64) kk = fmaf(s_k[i], s_k[i], kk), qq = fmaf(s_q[i], s_q[i], qq), qk = fmaf(s_k[i], s_q[i], qk);
    kk = wave_sum(kk);
    qq = wave_sum(qq);
    qk = wave_sum(qk);
    rk = 1.0f / sqrtf(kk + s.key_eps);
    rq = s.q_scale / sqrtf(qq + s.key_eps);
    qk *= rk * rq;
  }
  const float4 v4 = *reinterpret_cast<const float4*>(&s_v[4 * c4]);
  float4 po = make_float4(0.f, 0.f, 0.f, 0.f);
  if (RULE == SR_SSD) {
#pragma unroll
    for (int r = 0; r < RPT; ++r) {
      const float kw = s_k[rg + 16 * r] * w, q = s_q[rg + 16 * r];
      S[r].x = fmaf(kw, v4.x, d * S[r].x), S[r].y = fmaf(kw, v4.y, d * S[r].y), S[r].z = fmaf(kw, v4.z, d * S[r].z), S[r].w = fmaf(kw, v4.w, d * S[r].w);
      po.x = fmaf(q, S[r].x, po.x), po.y = fmaf(q, S[r].y, po.y), po.z = fmaf(q, S[r].z, po.z), po.w = fmaf(q, S[r].w, po.w);
    }
    *reinterpret_cast<float4*>(&s_po[rg][4 * c4]) = po;
    __syncthreads();
  } else {
    // the two sums over the old state, S^T k and S^T q, cross the threads together; o = d S^T q + (k . q) u is the read-out behind the write
    float4 pk = make_float4(0.f, 0.f, 0.f, 0.f);
#pragma unroll
    for (int r = 0; r < RPT; ++r) {
      const float k = s_k[rg + 16 * r], q = s_q[rg + 16 * r];
      pk.x = fmaf(k, S[r].x, pk.x), pk.y = fmaf(k, S[r].y, pk.y), pk.z = fmaf(k, S[r].z, pk.z), pk.w = fmaf(k, S[r].w, pk.w);
      po.x = fmaf(q, S[r].x, po.x), po.y = fmaf(q, S[r].y, po.y), po.z = fmaf(q, S[r].z, po.z), po.w = fmaf(q, S[r].w, po.w);
    }
    *reinterpret_cast<float4*>(&s_pk[rg][4 * c4]) = pk;
    *reinterpret_cast<float4*>(&s_po[rg][4 * c4]) = po;
    __syncthreads();
    float4 ks = make_float4(0.f, 0.f, 0.f, 0.f);
#pragma unroll
    for (int i = 0; i < 16; ++i) {
      const float4 p = *reinterpret_cast<const float4*>(&s_pk[i][4 * c4]);
      ks.x += p.x, ks.y += p.y, ks.z += p.z, ks.w += p.w;
    }
    const float4 add = make_float4(w * (v4.x - d * rk * ks.x), w * (v4.y - d * rk * ks.y), w * (v4.z - d * rk * ks.z), w * (v4.w - d * rk * ks.w));
#pragma unroll
    for (int r = 0; r < RPT; ++r) {
      const float k = s_k[rg + 16 * r] * rk;
      S[r].x = fmaf(k, add.x, d * S[r].x), S[r].y = fmaf(k, add.y, d * S[r].y), S[r].z = fmaf(k, add.z, d * S[r].z), S[r].w = fmaf(k, add.w, d * S[r].w);
    }
  }
#pragma unroll
  for (int r = 0; r < RPT; ++r) {
    const int i = rg + 16 * r;
    if (i < dk) {
      float* p = sp + (size_t)i * dv + 4 * c4;
      if (vec) {
        if (4 * c4 < dv) *reinterpret_cast<float4*>(p) = S[r];
      } else {
        if (4 * c4 < dv) p[0] = S[r].x;
        if (4 * c4 + 1 < dv) p[1] = S[r].y;
        if (4 * c4 + 2 < dv) p[2] = S[r].z;
        if (4 * c4 + 3 < dv) p[3] = S[r].w;
      }
    }
  }
  if (DVM == 64 && tid >= 64) return;  // one wave has the columns, and no barrier follows
  float o = 0.f;
  const bool mine = tid < dv;
  if (mine) {
#pragma unroll
    for (int i = 0; i < 16; ++i) o += s_po[i][tid];
  }
  if (RULE == SR_SSD) {
    if (mine) y_out[(size_t)t * s.H * dv + vcol + tid] = fmaf(skip[h], s_v[tid], o);
    return;
  }
  if (mine) {
    float ks = 0.f;
#pragma unroll
    for (int i = 0; i < 16; ++i) ks += s_pk[i][tid];
    o = fmaf(qk, w * (s_v[tid] - d * rk * ks), d * rq * o);
  }
  const float ss = block_sum<DVM == 64 ? 64 : NT>(mine ? o * o : 0.f, red);
  if (mine) out[(size_t)t * s.o_stride + vcol + tid] = from_float<T>(o / sqrtf(ss / (float)dv + s.norm_eps) * nw * sr_silu(gt));
}

// ---- entry points ----------------------------------------------------------------------------------------------------------------------
static int sr_check(const SrShape& s, int rule, int norm_groups, int dtype) {
  LEV_REQUIRE(rule == SR_SSD || rule == SR_DELTA, "state recurrence: unknown rule %d", rule);
  LEV_REQUIRE(s.Tn >= 0 && s.H > 0 && s.G > 0 && s.H % s.G == 0 && s.H <= 65535, "state recurrence: %d heads over %d groups", s.H, s.G);
  LEV_REQUIRE(s.dk > 0 && s.dk <= 256 && s.dv > 0 && s.dv <= 256, "state recurrence: heads of %d key and %d value channels (at most 256 each)", s.dk, s.dv);
  LEV_REQUIRE(s.K >= 1 && s.C > 0 && (s.C + 255) / 256 <= 65535, "state recurrence: %d channels with %d taps", s.C, s.K);
  LEV_REQUIRE(s.q_off >= 0 && s.k_off >= 0 && s.v_off >= 0 && s.q_off + s.G * s.dk <= s.C && s.k_off + s.G * s.dk <= s.C && s.v_off + s.H * s.dv <= s.C,
              "state recurrence: queries, keys and values do not fit the %d channels", s.C);
  LEV_REQUIRE(s.x_stride >= s.C && s.a_stride >= s.H && s.b_stride >= s.H && s.gate_stride >= (long)s.H * s.dv && s.o_stride >= (long)s.H * s.dv,
              "state recurrence: row strides are smaller than the rows");
  LEV_REQUIRE(s.slot_stride >= (long)s.K * s.C + (long)s.H * s.dk * s.dv, "state recurrence: a slot of %ld floats is too small", s.slot_stride);
  LEV_REQUIRE(norm_groups > 0 && norm_groups <= 65535 && (s.H * s.dv) % norm_groups == 0, "state recurrence: %d numbers do not split into %d equal parts", s.H * s.dv, norm_groups);
  LEV_REQUIRE(dtype == LEV_F32 || dtype == LEV_BF16, "state recurrence: unknown dtype %d", dtype);
  return 0;
}

template <typename T, int RULE>
static void sr_finish_launch(const float* o, const T* u, const float* skip, const T* gate, const float* norm_w, const int* token_slots, T* out,
                             int norm_groups, const SrShape& s, hipStream_t stream) {
  const int parts = RULE == SR_DELTA ? s.H : norm_groups, len = s.H * s.dv / parts;
  const uintptr_t a4 = 4 * sizeof(T) - 1;
  const bool quad = len % 4 == 0 && s.dv % 4 == 0 && s.C % 4 == 0 && s.v_off % 4 == 0 && s.gate_stride % 4 == 0 && s.o_stride % 4 == 0 &&
                    (((uintptr_t)o | (uintptr_t)norm_w) & 15) == 0 && (((uintptr_t)u | (uintptr_t)gate | (uintptr_t)out) & a4) == 0;
#define SR_FQ(LANES, NV)                                                                                                                         \
  do {                                                                                                                                           \
    sr_finish_quad_kernel<T, RULE, LANES, NV><<<dim3(s.Tn, (parts + 256 / LANES - 1) / (256 / LANES)), 256, 0, stream>>>(o, u, skip, gate, norm_w,  \
                                                                                                                        token_slots, out, len, parts, s); \
    return;                                                                                                                                      \
  } while (0)
  if (quad && len <= 64) SR_FQ(16, 1);
  if (quad && len <= 128) SR_FQ(32, 1);
  if (quad && len <= 256) SR_FQ(64, 1);
  if (quad && len <= 1024) SR_FQ(256, 1);
  if (quad && len <= 2048) SR_FQ(256, 2);
  if (quad && len <= 4096) SR_FQ(256, 4);
#undef SR_FQ
  if (len <= 128) sr_finish_kernel<T, RULE, 64><<<dim3(s.Tn, parts), 64, 0, stream>>>(o, u, skip, gate, norm_w, token_slots, out, len, s);
  else if (len <= 1024) sr_finish_kernel<T, RULE, 256><<<dim3(s.Tn, parts), 256, 0, stream>>>(o, u, skip, gate, norm_w, token_slots, out, len, s);
  else sr_finish_kernel<T, RULE, 1024><<<dim3(s.Tn, parts), 1024, 0, stream>>>(o, u, skip, gate, norm_w, token_slots, out, len, s);
}

template <typename T, int RULE>
static int sr_tokens_launch(const T* x, const float* taps, const float* conv_bias, const T* a, const T* b, const float* a_bias, const float* rate,
                            const float* skip, const T* gate, const float* norm_w, float* state, const int* token_slots, const int* positions,
                            float* y, T* out, int norm_groups, const SrShape& s, hipStream_t stream) {
  const int vec = s.dv % 4 == 0 && s.slot_stride % 4 == 0 && ((long)s.K * s.C) % 4 == 0 && ((uintptr_t)state & 15) == 0;
  const dim3 grid(s.Tn, s.H);
#define SR_TOK(DKM, DVM)                                                                                                                             \
  sr_token_kernel<T, DKM, DVM, RULE><<<grid, DVM * 4, 0, stream>>>(x, taps, conv_bias, a, b, a_bias, rate, skip, gate, norm_w, state, token_slots,     \
                                                                   positions, y, out, vec, s)
#define SR_TOK_DV(DKM)                           \
  do {                                           \
    if (s.dv <= 64) SR_TOK(DKM, 64);             \
    else if (s.dv <= 128) SR_TOK(DKM, 128);      \
    else SR_TOK(DKM, 256);                       \
  } while (0)
  if (s.dk <= 64) SR_TOK_DV(64);
  else if (s.dk <= 128) SR_TOK_DV(128);
  else SR_TOK_DV(256);
#undef SR_TOK_DV
#undef SR_TOK
  if (lev_check_launch("state recurrence (single tokens)")) return -1;
  if (RULE == SR_SSD) {
    sr_finish_launch<T, RULE>(y, nullptr, skip, gate, norm_w, token_slots, out, norm_groups, s, stream);
    return lev_check_launch("state recurrence (norm)");
  }
  return 0;
}

static long sr_pad8(long n) { return (n + 7) / 8 * 8; }
static long sr_pad4(long n) { return (n + 3) / 4 * 4; }  // parts of the scratch memory start at 16-byte boundaries

template <typename T, int RULE>
static int sr_runs_launch(const T* x, const float* taps, const float* conv_bias, const T* a, const T* b, const float* a_bias, const float* rate,
                          const float* skip, const T* gate, const float* norm_w, float* state, const int* token_slots, const int* positions,
                          float* ws, T* out, int norm_groups, int max_runs, int use_mfma, const SrShape& s, hipStream_t stream) {
  float* o = ws;
  float* scal = o + sr_pad4((long)s.Tn * s.H * s.dv);
  T* u = reinterpret_cast<T*>(scal + sr_pad4((long)s.Tn * (2 * s.H + 2 * s.G)));
  const uintptr_t a4 = 4 * sizeof(T) - 1;
  if (s.K <= 4 && s.C % 4 == 0 && s.x_stride % 4 == 0 && (((uintptr_t)x | (uintptr_t)u) & a4) == 0)
    sr_conv_quad_kernel<T><<<dim3((s.Tn + SR_CT - 1) / SR_CT, (s.C / 4 + 255) / 256), 256, 0, stream>>>(x, taps, conv_bias, state, token_slots, positions, u, s);
  else
    sr_conv_kernel<T><<<dim3((s.Tn + SR_CT - 1) / SR_CT, (s.C + 255) / 256), 256, 0, stream>>>(x, taps, conv_bias, state, token_slots, positions, u, s);
  if (lev_check_launch("state recurrence (convolution)")) return -1;
  sr_prepare_kernel<T, RULE><<<s.Tn, 256, 0, stream>>>(x, u, a, b, a_bias, rate, state, token_slots, positions, scal, s);
  if (lev_check_launch("state recurrence (prepare)")) return -1;
  if (sizeof(T) == 2 && use_mfma) {
    if (sr_chunks_launch(RULE, (const bf16_t*)(const void*)u, scal, state, token_slots, o, reinterpret_cast<float*>(u + sr_pad8((long)s.Tn * s.C)), max_runs, s, stream)) return -1;
    sr_finish_launch<T, RULE>(o, u, skip, gate, norm_w, token_slots, out, norm_groups, s, stream);
    return lev_check_launch("state recurrence (norm)");
  }
  LEV_REQUIRE(max_runs <= 65535, "state recurrence: too many runs (%d)", max_runs);
  const dim3 walk(s.H, (s.dv + SR_WC - 1) / SR_WC, max_runs);
  if (s.dk <= 64) sr_walk_kernel<T, 64, RULE><<<walk, 256, 0, stream>>>(u, scal, state, token_slots, o, s);
  else if (s.dk <= 128) sr_walk_kernel<T, 128, RULE><<<walk, 256, 0, stream>>>(u, scal, state, token_slots, o, s);
  else sr_walk_kernel<T, 256, RULE><<<walk, 256, 0, stream>>>(u, scal, state, token_slots, o, s);
  if (lev_check_launch("state recurrence (walk)")) return -1;
  sr_finish_launch<T, RULE>(o, u, skip, gate, norm_w, token_slots, out, norm_groups, s, stream);
  return lev_check_launch("state recurrence (norm)");
}

// scratch memory in bytes. Steps with runs: o [Tn][H][dv], the scalars, the convolution's output, bfloat16: the chunks' matrices; steps of single tokens: o of the rule SSD
extern "C" long lev_state_recurrence_workspace(int rule, int Tn, int H, int G, int dv, int C, int runs, int dtype) {
  const long o = sr_pad4((long)Tn * H * dv) * 4;
  return runs ? o + sr_pad4((long)Tn * (2L * H + 2L * G)) * 4 + sr_pad8((long)Tn * C) * (dtype == LEV_F32 ? 4 : 2) +
                    (dtype == LEV_F32 ? 0 : sr_chunks_workspace(rule, Tn, H) * 4)
              : o;
}

extern "C" int lev_state_recurrence(int rule, const void* x, long x_stride, const float* taps, const float* conv_bias, const void* a, long a_stride,
                                    const void* b, long b_stride, const float* a_bias, const float* rate, const float* skip, const void* gate,
                                    long gate_stride, const float* norm_w, float* state, long slot_stride, const int* token_slots,
                                    const int* positions, void* out, long o_stride, float* workspace, int T, int max_runs, int H, int G, int dk,
                                    int dv, int C, int K, int q_off, int k_off, int v_off, int norm_groups, float norm_eps, float key_eps,
                                    float q_scale, int use_mfma, int dtype, hipStream_t stream) {
  SrShape s{T, H, G, dk, dv, C, K, q_off, k_off, v_off, x_stride, a_stride, b_stride, gate_stride, o_stride, slot_stride, key_eps, q_scale, norm_eps};
  if (sr_check(s, rule, norm_groups, dtype)) return -1;
  LEV_REQUIRE(x && taps && a && a_bias && rate && gate && norm_w && state && token_slots && positions && out && workspace, "state recurrence: a tensor is missing");
  LEV_REQUIRE(rule == SR_DELTA ? b != nullptr : skip != nullptr, "state recurrence: the write rate (delta) or the skip weights (SSD) are missing");
  LEV_REQUIRE(max_runs >= 0 && max_runs <= T, "state recurrence: %d runs of %d tokens", max_runs, T);
  if (T == 0) return 0;
#define SR_GO(TT, RULE)                                                                                                                              \
  (max_runs ? sr_runs_launch<TT, RULE>((const TT*)x, taps, conv_bias, (const TT*)a, (const TT*)b, a_bias, rate, skip, (const TT*)gate, norm_w, state,   \
                                       token_slots, positions, workspace, (TT*)out, norm_groups, max_runs, use_mfma, s, stream)                              \
            : sr_tokens_launch<TT, RULE>((const TT*)x, taps, conv_bias, (const TT*)a, (const TT*)b, a_bias, rate, skip, (const TT*)gate, norm_w, state, \
                                         token_slots, positions, workspace, (TT*)out, norm_groups, s, stream))
  if (dtype == LEV_F32) return rule == SR_SSD ? SR_GO(float, SR_SSD) : SR_GO(float, SR_DELTA);
  return rule == SR_SSD ? SR_GO(bf16_t, SR_SSD) : SR_GO(bf16_t, SR_DELTA);
#undef SR_GO
}
