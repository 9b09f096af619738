// Selective scan: per channel c and state n, with a step size per token and channel,
//   dt = softplus(raw + bias),  S[n, c] <- exp(dt A[n, c]) S[n, c] + dt x_c B_n,  y_c = sum_n S[n, c] C_n + D_c x_c,
//   out_c = y_c silu(z_c)
// over the tokens of one request, from the float32 state [slots, SSM_STATE, C] its slot holds.  B and C are columns
// of a token's float32 row and the same for all channels; A = -exp(.) comes with the factor log2(e) in it, so that a
// decay is one base-2 exponential.  Compiled per state size (-DSSM_STATE=...).
//
// A thread owns a channel and all of its states (in registers); B and C are read at addresses that are the same for
// the whole wave.  More than 32 states are shared by four waves, whose sums of y meet in LDS.  Long runs are cut
// into chunks that are scanned side by side: from zero states (which needs only the chunk's last state and the sum
// of its step sizes: the product of its decays is exp(A sum dt)), then the states are carried from chunk to chunk, then
// every chunk is scanned once more from the state before it.
#include "common.h"

#ifndef SSM_STATE
#define SSM_STATE 16
#endif
#if SSM_STATE < 1 || SSM_STATE > 256
#error "state sizes 1 to 256"
#endif
#define SP (SSM_STATE > 32 ? 4 : 1)               // waves that share a channel's states
#define NW ((SSM_STATE + SP - 1) / SP)            // states of a wave
#define CH_BLOCK (256 / SP)                       // channels of a block
#define TB 8                                      // tokens whose loads are issued together

enum { SCAN_WHOLE = 0, SCAN_STATE = 1, SCAN_FROM = 2 };   // all of a run / a chunk's last state only / a chunk's outputs

struct ScanArgs {
  const void* x;              // [N, C] of TX: the convolved input
  const float* dt;            // [N, C] before bias and softplus
  const float* dt_bias;       // [C]
  const float* a2;            // [SSM_STATE, C]: -exp(A_log) log2(e)
  const float* bc;            // rows of bc_stride values: B from b_off, C from c_off
  long long bc_stride;
  int b_off, c_off;
  const float* d;             // [C]
  const void* z;              // rows of z_stride values of TX
  long long z_stride;
  void* out;                  // [N, C] of TX
  float* state;               // [rows, SSM_STATE, C]
  float* dt_sum;              // SCAN_STATE: [rows, C]
  const int* bounds;          // token bounds of run (or chunk) i: bounds[i] .. bounds[i + 1]
  const int* row_of;          // [runs] its row of state (null: row i)
  int C;
};

// max(z, 0) + log(1 + e) with e = exp(-|z|), the logarithm as 2 atanh(s), s = e / (2 + e) <= 1/3, by its power series
// up to s^15 (the rest is below 2e-8 of the sum).
__device__ __forceinline__ float softplus_f(float z) {
  const float e = __builtin_amdgcn_exp2f(-1.4426950408889634f * fabsf(z));
  const float s = e * __builtin_amdgcn_rcpf(2.0f + e), q = s * s;
  float p = 1.0f / 15.0f;
  p = p * q + 1.0f / 13.0f;
  p = p * q + 1.0f / 11.0f;
  p = p * q + 1.0f / 9.0f;
  p = p * q + 1.0f / 7.0f;
  p = p * q + 1.0f / 5.0f;
  p = p * q + 1.0f / 3.0f;
  p = p * q + 1.0f;
  return fmaxf(z, 0.f) + 2.0f * s * p;
}
// z sigmoid(z); exp(-z) that overflows gives zero
__device__ __forceinline__ float silu_f(float z) {
  return z * __builtin_amdgcn_rcpf(1.0f + __builtin_amdgcn_exp2f(-1.4426950408889634f * z));
}

template <typename TX, int MODE>
__global__ __launch_bounds__(256) void selective_scan_kernel(ScanArgs a) {
  __shared__ float part[SP > 1 && MODE != SCAN_STATE ? SP : 1][TB][64];
  const int share = SP > 1 ? __builtin_amdgcn_readfirstlane(threadIdx.x >> 6) : 0;
  const int lane = SP > 1 ? threadIdx.x & 63 : threadIdx.x;
  const int ch = blockIdx.x * CH_BLOCK + lane;
  const bool live = ch < a.C;
  const int c = live ? ch : 0;                      // a thread past the last channel reads the first and writes nothing
  const int run = blockIdx.y;
  const int begin = a.bounds[run], end = a.bounds[run + 1];
  if (begin >= end) return;
  const size_t srow = (size_t)(a.row_of ? a.row_of[run] : run) * SSM_STATE;
  const int n0 = share * NW;
  float S[NW], A[NW];
#pragma unroll
  for (int i = 0; i < NW; ++i) {
    const int n = n0 + i < SSM_STATE ? n0 + i : SSM_STATE - 1;
    A[i] = a.a2[(size_t)n * a.C + c];
    S[i] = (MODE == SCAN_STATE || n0 + i >= SSM_STATE) ? 0.f : a.state[(srow + n) * a.C + c];
  }
  const float bias = a.dt_bias[c], skip = a.d[c];
  const TX* x = reinterpret_cast<const TX*>(a.x);
  const TX* z = reinterpret_cast<const TX*>(a.z);
  TX* out = reinterpret_cast<TX*>(a.out);
  float total = 0.f;
  for (int t0 = begin; t0 < end; t0 += TB) {
    const int nt = end - t0 < TB ? end - t0 : TB;
    float dtr[TB], xv[TB], zv[TB];
#pragma unroll
    for (int k = 0; k < TB; ++k) {
      const size_t t = t0 + (k < nt ? k : 0);
      dtr[k] = a.dt[t * a.C + c];
      xv[k] = ldf<TX>(x + t * a.C + c);
      zv[k] = MODE == SCAN_STATE ? 0.f : ldf<TX>(z + t * a.z_stride + c);
    }
#pragma unroll
    for (int k = 0; k < TB; ++k) {
      if (k < nt) {                                 // the same for the whole block
        const float dt = softplus_f(dtr[k] + bias), dx = dt * xv[k];
        const float* row = a.bc + (size_t)(t0 + k) * a.bc_stride;
        float y = 0.f;
#pragma unroll
        for (int i = 0; i < NW; ++i) {
          const bool in = SSM_STATE % SP == 0 || n0 + i < SSM_STATE;
          const int n = in ? n0 + i : 0;
          const float b = in ? row[a.b_off + n] : 0.f;
          S[i] = __builtin_amdgcn_exp2f(dt * A[i]) * S[i] + dx * b;
          if (MODE != SCAN_STATE) y += S[i] * (in ? row[a.c_off + n] : 0.f);
        }
        if (MODE == SCAN_STATE) total += dt;
        else if (SP > 1) part[share][k][lane] = y;
        else if (live) {
          y += skip * xv[k];
          stf<TX>(out + (size_t)(t0 + k) * a.C + c, y * silu_f(zv[k]));
        }
      }
    }
    if (SP > 1 && MODE != SCAN_STATE) {
      __syncthreads();
#pragma unroll
      for (int k = 0; k < TB; ++k) {
        if (k < nt && k % SP == share && live) {
          float y = part[0][k][lane];
#pragma unroll
          for (int s = 1; s < SP; ++s) y += part[s][k][lane];
          y += skip * xv[k];
          stf<TX>(out + (size_t)(t0 + k) * a.C + c, y * silu_f(zv[k]));
        }
      }
      __syncthreads();
    }
  }
  if (!live || MODE == SCAN_FROM) return;
#pragma unroll
  for (int i = 0; i < NW; ++i)
    if (n0 + i < SSM_STATE) a.state[(srow + n0 + i) * a.C + c] = S[i];
  if (MODE == SCAN_STATE && share == 0) a.dt_sum[(size_t)run * a.C + c] = total;
}

// One thread per (state, channel) of a request: scratch[chunk] (the chunk's own last state) is replaced by the state
// before the chunk, and the request's slot gets the state after its last chunk.
__global__ __launch_bounds__(256) void selective_carry_kernel(float* __restrict__ scratch, const float* __restrict__ dt_sum,
                                                              const float* __restrict__ a2, float* __restrict__ state,
                                                              const int* __restrict__ req_first,
                                                              const int* __restrict__ req_slots, int C) {
  const int req = blockIdx.y;
  const long long per_row = (long long)SSM_STATE * C;
  const long long e = (long long)blockIdx.x * blockDim.x + threadIdx.x;
  if (e >= per_row) return;
  const int c = (int)(e % C);
  const float a = a2[e];
  float* mine = state + (size_t)req_slots[req] * per_row + e;
  float S = *mine;
  const int first = req_first[req], last = req_first[req + 1];
  for (int k0 = first; k0 < last; k0 += 8) {
    float u[8], dt[8];
#pragma unroll
    for (int k = 0; k < 8; ++k) {                   // the loads of eight chunks are on their way together
      const int at = k0 + k < last ? k0 + k : k0;
      u[k] = scratch[(size_t)at * per_row + e];
      dt[k] = dt_sum[(size_t)at * C + c];
    }
#pragma unroll
    for (int k = 0; k < 8; ++k) {
      if (k0 + k < last) {
        scratch[(size_t)(k0 + k) * per_row + e] = S;
        S = __builtin_amdgcn_exp2f(dt[k] * a) * S + u[k];
      }
    }
  }
  *mine = S;
}

extern "C" int qvl_selective_state_size() { return SSM_STATE; }

// mode 0: runs of requests (bounds = cu_q, row_of = req_slots), outputs and states; 1: chunks from zero states, last
// states and sums of step sizes; 2: chunks from the states in `state`, outputs.  dtype: of x, z and out.
extern "C" int qvl_selective_scan(int mode, const void* x, const void* dt, const void* dt_bias, const void* a2, const void* bc,
                                  long long bc_stride, int b_off, int c_off, const void* d, const void* z,
                                  long long z_stride, void* out, void* state, void* dt_sum, const void* bounds,
                                  const void* row_of, int runs, int C, int states, int dtype, hipStream_t stream) {
  if (runs <= 0) return QVL_OK;
  if (states != SSM_STATE || C <= 0 || !x || !dt || !dt_bias || !a2 || !bc || !d || !state || !bounds) return QVL_ERR_SHAPE;
  if (b_off < 0 || c_off < 0 || bc_stride < b_off + SSM_STATE || bc_stride < c_off + SSM_STATE) return QVL_ERR_SHAPE;
  if ((mode != SCAN_STATE && (!z || !out)) || (mode == SCAN_STATE && !dt_sum)) return QVL_ERR_SHAPE;
  if (runs > 65535) return QVL_ERR_LIMIT;
  ScanArgs a;
  a.x = x; a.dt = (const float*)dt; a.dt_bias = (const float*)dt_bias; a.a2 = (const float*)a2; a.bc = (const float*)bc;
  a.bc_stride = bc_stride; a.b_off = b_off; a.c_off = c_off; a.d = (const float*)d; a.z = z; a.z_stride = z_stride;
  a.out = out; a.state = (float*)state; a.dt_sum = (float*)dt_sum; a.bounds = (const int*)bounds;
  a.row_of = (const int*)row_of; a.C = C;
  const dim3 grid((C + CH_BLOCK - 1) / CH_BLOCK, runs);
#define LAUNCH(TX, MODE) hipLaunchKernelGGL((selective_scan_kernel<TX, MODE>), grid, dim3(256), 0, stream, a)
#define BY_MODE(TX)                                    \
  if (mode == SCAN_WHOLE) LAUNCH(TX, SCAN_WHOLE);      \
  else if (mode == SCAN_STATE) LAUNCH(TX, SCAN_STATE); \
  else if (mode == SCAN_FROM) LAUNCH(TX, SCAN_FROM);   \
  else return QVL_ERR_SHAPE;
  if (dtype == 0) { BY_MODE(float) }
  else if (dtype == 1) { BY_MODE(bf16_t) }
  else return QVL_ERR_DTYPE;
#undef BY_MODE
#undef LAUNCH
  return qvl_launch_status();
}

// scratch [chunks, SSM_STATE, C], dt_sum [chunks, C], state [slots, SSM_STATE, C]; request r has the chunks
// req_first[r] .. req_first[r + 1].
extern "C" int qvl_selective_carry(void* scratch, const void* dt_sum, const void* a2, void* state, const void* req_first,
                                   const void* req_slots, int R, int C, int states, hipStream_t stream) {
  if (R <= 0) return QVL_OK;
  if (states != SSM_STATE || C <= 0) return QVL_ERR_SHAPE;
  if (R > 65535) return QVL_ERR_LIMIT;
  const long long per_row = (long long)SSM_STATE * C;
  hipLaunchKernelGGL(selective_carry_kernel, dim3((unsigned)((per_row + 255) / 256), R), dim3(256), 0, stream,
                     (float*)scratch, (const float*)dt_sum, (const float*)a2, (float*)state, (const int*)req_first,
                     (const int*)req_slots, C);
  return qvl_launch_status();
}
