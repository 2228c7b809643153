// What the kernels of the recurrences with a matrix state per head share (state_recurrence.hip, state_chunks.hip).
#pragma once
#include "common.h"

#define SR_SSD 0
#define SR_DELTA 1

__device__ __forceinline__ float sr_softplus(float x) { return fmaxf(x, 0.f) + log1pf(expf(-fabsf(x))); }
__device__ __forceinline__ float sr_sigmoid(float x) { return 1.0f / (1.0f + expf(-x)); }
__device__ __forceinline__ float sr_silu(float x) { return x / (1.0f + expf(-x)); }

// sizes and places, the same for every kernel of the file
struct SrShape {
  int Tn, H, G, dk, dv, C, K;
  int q_off, k_off, v_off;  // first channel of the queries, keys and values among the C
  long x_stride;            // row stride of the convolution's inputs
  long a_stride, b_stride;  // of the decay's and the write rate's sums
  long gate_stride, o_stride;
  long slot_stride;         // floats of a slot
  float key_eps, q_scale, norm_eps;
};

// ---- the run-th run of a step: its first token, the token behind its last, its slot; false: there are fewer ------------------
// A token starts a run if it has a slot and the token before it has another. Each thread counts the starts of its stretch of
// tokens; the thread whose stretch holds the run-th one finds it. `tmp`: NT + 2 ints of LDS.
template <int NT>
__device__ __forceinline__ bool sr_find_run(int run, const int* __restrict__ token_slots, int Tn, int* tmp, int& t0, int& t_end, int& slot) {
  const int tid = threadIdx.x;
  const int per = (Tn + NT - 1) / NT, lo = min(Tn, tid * per), hi = min(Tn, lo + per);
  int mine = 0;
  for (int t = lo; t < hi; ++t) mine += (token_slots[t] >= 0 && (t == 0 || token_slots[t - 1] != token_slots[t])) ? 1 : 0;
  if (tid == 0) tmp[NT] = -1, tmp[NT + 1] = Tn;
  // the starts in the stretches before this thread's: across the lanes of its wave, then the waves before it
  int upto = mine;
#pragma unroll
  for (int d = 1; d < 64; d <<= 1) {
    const int up = __shfl_up(upto, d, 64);
    if ((tid & 63) >= d) upto += up;
  }
  if ((tid & 63) == 63) tmp[tid >> 6] = upto;
  __syncthreads();
  int before = upto - mine;
  for (int i = 0; i < (tid >> 6); ++i) before += tmp[i];
  if (run >= before && run < before + mine) {
    int seen = before;
    for (int t = lo; t < hi; ++t)
      if (token_slots[t] >= 0 && (t == 0 || token_slots[t - 1] != token_slots[t])) {
        if (seen == run) tmp[NT] = t;
        ++seen;
      }
  }
  __syncthreads();
  t0 = tmp[NT];
  if (t0 < 0) return false;  // the whole workgroup
  slot = token_slots[t0];
  int end = Tn;  // the first later token of another slot
#pragma unroll 8
  for (int t = tid; t < Tn; t += NT)
    if (t > t0 && token_slots[t] != slot) end = min(end, t);
  if (end < Tn) atomicMin(&tmp[NT + 1], end);
  __syncthreads();
  t_end = tmp[NT + 1];
  return true;
}

// Steps with runs, bfloat16: the recurrence in chunks of up to 64 tokens on the matrix cores (state_chunks.hip); the same inputs and outputs as
// the walk token by token. workspace: sr_chunks_workspace floats at a 16-byte boundary.
int sr_chunks_launch(int rule, const bf16_t* u, const float* scal, float* state, const int* token_slots, float* o, float* workspace, int max_runs,
                     const SrShape& s, hipStream_t stream);
long sr_chunks_workspace(int rule, int Tn, int H);
