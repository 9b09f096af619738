// Recurrences over outer products with one decay per head and token, a_t = exp(A_h softplus(raw_t + bias_h)):
//   plain   S <- a S + step k v^T,                              o = S^T q (+ D v)      (step = the softplus)
//   delta   S <- a S;  u = beta (v - S^T k);  S <- S + k u^T;   o = S^T q              (beta = sigmoid of another raw column)
// S is [HS_DIM, vdim] float32 per (request slot, head).  q and k belong to groups of heads (head h reads group
// h / (H / G)) and may be made unit vectors first, x / sqrt(sum x^2 + unit_eps); q is scaled.  q, k and v are columns of
// float32 or bfloat16 rows; raw columns, decays, step sizes, unit lengths, states and outputs are float32.
// Compiled per key size (-DHS_DIM=...).
//
// Runs of few tokens: hs_scan_kernel walks a request's tokens in order.  A block of four waves owns 64 value channels of
// one head; lane = value channel, each wave keeps a quarter of the rows of S in registers.
//
// Long runs are cut into chunks of 64 tokens.  With L_ij = a_(j+1) ... a_i (i >= j, from logarithms summed in float64)
// and S' the state before a chunk
//   delta: (I + strict lower(diag(beta) L o K K^T)) [Wv | Wk] = diag(beta) [V | diag(L_i0) K],   U = Wv - Wk S'
//   plain: U = diag(step) V
//   O = (L o Q K^T) U + diag(L_i0) Q S',     S_end = L_n0 S' + sum_j L_nj k_j u_j^T
// (L_i0: from the chunk's start up to i.)  Everything but the carry of S runs over chunks side by side, the products
// through v_mfma_f32_16x16x4_f32 (float32 operands, float32 sums):
//   hs_prep    sums of logarithms and gates per (chunk, head)
//   hs_score   Q K^T (and K K^T) per (chunk, group), unit lengths folded in
//   hs_solve   [Wv | Wk] per (chunk, head), a triangular system in blocks of 16 rows        (delta)
//   hs_carry   the states, chunk after chunk; a block per (request, head, 16 value channels); leaves S' (delta: and U) of every chunk
//   hs_out     O per (chunk, head)
//
// Matrix fragments.  Lane l of a wave stands for row (or column) l % 16 and the four inner indices 4 (l / 16) .. + 3 of a
// block of 16: instruction j of four takes inner index 4 (l / 16) + j of both operands.  A result's lane holds rows
// 4 (l / 16) .. + 3 of column l % 16, which is the right operand's layout with rows as the inner index, so results
// are multiplied again without moving.  U and S' lie in memory in that layout: [.., block of 16 rows, lane, 4].
#include "common.h"

#ifndef HS_DIM
#define HS_DIM 64
#endif
#if HS_DIM < 1 || HS_DIM > 512
#error "key sizes 1 to 512"
#endif
#define HS_ROWS ((HS_DIM + 3) / 4)              // rows of S a wave keeps in hs_scan_kernel
#define HS_TB (HS_DIM > 256 ? 2 : (HS_DIM > 128 ? 4 : 8))
#define HS_CHUNK 64
#define HS_KB ((HS_DIM + 15) / 16)              // blocks of 16 key channels
#define HS_DIMP (HS_KB * 16)
#define HS_LD (HS_DIMP + 4)                     // a row of staged keys: columns read down a row block hit different banks
#define HS_CHUNKED (HS_DIMP <= 256)

struct HeadScan {
  const void* x;             // rows of x_stride values of TX
  long long x_stride;
  int q_off, k_off, v_off;
  const float* raw;          // rows of raw_stride values: step inputs from a_off, beta inputs from b_off
  long long raw_stride;
  int a_off, b_off;
  const float* bias;         // [H]
  const float* a_neg;        // [H], -exp(A_log)
  const float* skip;         // [H] or null: D
  float q_scale, unit_eps;   // unit_eps < 0: q and k are taken as they are
  float* state;              // [slots, H, HS_DIM, vdim]
  const int* bounds;         // [runs + 1] tokens of a run (or chunk)
  const int* row_of;         // [runs] a request's slot
  float* out;                // [N, H * vdim]
  int H, G, vdim;
  // chunks
  const int* req_first;      // [R + 1] a request's chunks
  double* lsum;              // [chunks, H, 64]: sum of the decays' logarithms from the chunk's start, token included
  float* gate;               // [chunks, H, 64]: beta or step
  float* head;               // [chunks, H, 64]: the decays' product from the chunk's start, token included
  float* tail;               // [chunks, H, 64]: the decays' product behind the token to the chunk's end
  float* qk;                 // [chunks, G, 64, 64]
  float* kk;                 // [chunks, G, 64, 64]
  void* kt;                  // [chunks, G, HS_KB, 4, 64, 4] of TX: K as left operand with channels as rows
  float* unit;               // [chunks, G, 2, 64]: factors on q (its scale included) and k
  float* wk;                 // [chunks, H, 64, HS_DIMP]
  float* u;                  // [chunks, H, vtiles, 4, 64, 4] (delta)
  float* s0;                 // [chunks, H, vtiles, HS_KB, 64, 4]
};

__device__ __forceinline__ float hs_softplus(float z) { return fmaxf(z, 0.f) + log1pf(expf(-fabsf(z))); }
__device__ __forceinline__ float hs_sigmoid(float z) { return 1.0f / (1.0f + expf(-z)); }

// ---------------------------------------------------------------------------------------
// few tokens: one after the other
// ---------------------------------------------------------------------------------------
template <typename TX, bool DELTA>
__global__ __launch_bounds__(256) void hs_scan_kernel(HeadScan a) {
  __shared__ float qs[HS_TB][4 * HS_ROWS];
  __shared__ float ks[HS_TB][4 * HS_ROWS];
  __shared__ float fq[HS_TB], fk[HS_TB], dec[HS_TB], gate[HS_TB];
  __shared__ float seen[2][4][64];              // a token's S^T k by wave
  __shared__ float po[HS_TB][4][64];
  const int tid = threadIdx.x, wave = tid >> 6, lane = tid & 63;
  const int head = blockIdx.y, run = blockIdx.z, grp = head / (a.H / a.G);
  const int vcol = blockIdx.x * 64 + lane;
  const bool live = vcol < a.vdim;
  const int begin = a.bounds[run], end = a.bounds[run + 1];
  if (begin >= end) return;
  const TX* x = reinterpret_cast<const TX*>(a.x);
  const int d0 = wave * HS_ROWS;
  float* srow = a.state + (((size_t)a.row_of[run] * a.H + head) * HS_DIM + d0) * a.vdim + (live ? vcol : 0);
  float S[HS_ROWS];
#pragma unroll
  for (int i = 0; i < HS_ROWS; ++i) S[i] = live && d0 + i < HS_DIM ? srow[(size_t)i * a.vdim] : 0.f;
  const float bias = a.bias[head], a_neg = a.a_neg[head], skip = a.skip ? a.skip[head] : 0.f;

  for (int t0 = begin; t0 < end; t0 += HS_TB) {
    const int nt = end - t0 < HS_TB ? end - t0 : HS_TB;
    for (int idx = tid; idx < nt * 4 * HS_ROWS; idx += 256) {
      const int t = idx / (4 * HS_ROWS), d = idx % (4 * HS_ROWS);
      const TX* row = x + (size_t)(t0 + t) * a.x_stride + (size_t)grp * HS_DIM + d;
      qs[t][d] = d < HS_DIM ? ldf<TX>(row + a.q_off) : 0.f;
      ks[t][d] = d < HS_DIM ? ldf<TX>(row + a.k_off) : 0.f;
    }
    float vt[HS_TB];
#pragma unroll
    for (int t = 0; t < HS_TB; ++t)
      vt[t] = ldf<TX>(x + (size_t)(t0 + (t < nt ? t : 0)) * a.x_stride + a.v_off + (size_t)head * a.vdim + (live ? vcol : 0));
    if (tid < nt) {
      const float* r = a.raw + (size_t)(t0 + tid) * a.raw_stride;
      const float step = hs_softplus(r[a.a_off + head] + bias);
      dec[tid] = expf(a_neg * step);
      gate[tid] = DELTA ? hs_sigmoid(r[a.b_off + head]) : step;
    }
    __syncthreads();
    for (int t = wave; t < nt; t += 4) {        // a wave's token: its factors on q and k
      float sq = 0.f, sk = 0.f;
      if (a.unit_eps >= 0.f) {
        for (int d = lane; d < HS_DIM; d += 64) {
          sq += qs[t][d] * qs[t][d];
          sk += ks[t][d] * ks[t][d];
        }
        sq = wave_sum(sq);
        sk = wave_sum(sk);
      }
      if (lane == 0) {
        fq[t] = a.unit_eps >= 0.f ? a.q_scale / sqrtf(sq + a.unit_eps) : a.q_scale;
        fk[t] = a.unit_eps >= 0.f ? 1.0f / sqrtf(sk + a.unit_eps) : 1.0f;
      }
    }
    __syncthreads();
#pragma unroll
    for (int t = 0; t < HS_TB; ++t) {
      if (t < nt) {                             // the same for the whole block
        const float g = dec[t], kf = fk[t];
        float w;                                // what the key writes, its factor included
        if (DELTA) {
          float acc = 0.f;
#pragma unroll
          for (int i = 0; i < HS_ROWS; ++i) {
            S[i] *= g;
            acc += S[i] * ks[t][d0 + i];
          }
          seen[t & 1][wave][lane] = acc;
          __syncthreads();
          const float sum = (seen[t & 1][0][lane] + seen[t & 1][1][lane]) + (seen[t & 1][2][lane] + seen[t & 1][3][lane]);
          w = gate[t] * (vt[t] - kf * sum) * kf;
        } else {
          w = gate[t] * vt[t] * kf;
        }
        float acc = 0.f;
#pragma unroll
        for (int i = 0; i < HS_ROWS; ++i) {
          S[i] = (DELTA ? S[i] : g * S[i]) + ks[t][d0 + i] * w;
          acc += S[i] * qs[t][d0 + i];
        }
        po[t][wave][lane] = acc;
      }
    }
    __syncthreads();
    for (int t = wave; t < nt; t += 4) {        // vt[t] with t not known at compile time: the value is read again
      if (live) {
        float o = ((po[t][0][lane] + po[t][1][lane]) + (po[t][2][lane] + po[t][3][lane])) * fq[t];
        if (a.skip) o += skip * ldf<TX>(x + (size_t)(t0 + t) * a.x_stride + a.v_off + (size_t)head * a.vdim + vcol);
        a.out[((size_t)(t0 + t) * a.H + head) * a.vdim + vcol] = o;
      }
    }
    __syncthreads();
  }
  if (live) {
#pragma unroll
    for (int i = 0; i < HS_ROWS; ++i)
      if (d0 + i < HS_DIM) srow[(size_t)i * a.vdim] = S[i];
  }
}

#if HS_CHUNKED
typedef float f32x4 __attribute__((ext_vector_type(4)));

// exp(l) of a difference of sums of logarithms, which is not positive where it counts.  Formed whether or not it is
// used: a branch around it would wait for its operands one by one.
__device__ __forceinline__ float decay_of(double l) {
  float e = expf(fminf((float)l, 0.f));
  asm volatile("" : "+v"(e));
  return e;
}

// acc += A B over one block of 16 inner indices
__device__ __forceinline__ f32x4 mma16(const f32x4 p, const f32x4 q, f32x4 acc) {
#pragma unroll
  for (int j = 0; j < 4; ++j) acc = __builtin_amdgcn_mfma_f32_16x16x4f32(p[j], q[j], acc, 0, 0, 0);
  return acc;
}

// ---------------------------------------------------------------------------------------
// a wave per (chunk, head), a lane per token
// ---------------------------------------------------------------------------------------
template <bool DELTA>
__global__ __launch_bounds__(256) void hs_prep_kernel(HeadScan a) {
  const int c = blockIdx.x, head = blockIdx.y * 4 + (threadIdx.x >> 6), t = threadIdx.x & 63;
  if (head >= a.H) return;
  const int begin = a.bounds[c], n = a.bounds[c + 1] - begin;
  double l = 0.0;
  float g = 0.f;
  if (t < n) {
    const float* r = a.raw + (size_t)(begin + t) * a.raw_stride;
    const float step = hs_softplus(r[a.a_off + head] + a.bias[head]);
    l = (double)(a.a_neg[head] * step);
    g = DELTA ? hs_sigmoid(r[a.b_off + head]) : step;
  }
#pragma unroll
  for (int o = 1; o < 64; o <<= 1) {
    const double up = __shfl_up(l, o, 64);
    if (t >= o) l += up;
  }
  const size_t at = ((size_t)c * a.H + head) * HS_CHUNK + t;
  a.lsum[at] = l;                               // tokens past the chunk's end keep the last sum
  a.gate[at] = g;
  a.head[at] = expf((float)l);
  a.tail[at] = expf((float)(__shfl(l, 63, 64) - l));
}

// Four channels of a row as they lie in memory.  VEC: HS_DIM, strides and offsets are multiples of four and rows lie on
// boundaries of four values, so that one load fetches them.
// `at`: where channel d lies, or channel 0 with d past the last one.
template <typename TX, bool VEC> struct Four {
  TX v[4];
  __device__ __forceinline__ void fetch_at(const TX* at, int d) {
#pragma unroll
    for (int j = 0; j < 4; ++j) v[j] = at[d + j < HS_DIM ? j : 0];
  }
  __device__ __forceinline__ void fetch(const TX* row, int d) { fetch_at(row + (d < HS_DIM ? d : 0), d); }
  __device__ __forceinline__ f32x4 value(int d, bool live) const {
    f32x4 o;
#pragma unroll
    for (int j = 0; j < 4; ++j) o[j] = live && d + j < HS_DIM ? ldf<TX>(v + j) : 0.f;
    return o;
  }
};
template <> struct Four<bf16_t, true> {
  uint2 v;
  // of values that are bfloat16 already
  __device__ __forceinline__ void set(const f32x4& w) {
    v.x = (__float_as_uint(w[0]) >> 16) | (__float_as_uint(w[1]) & 0xffff0000u);
    v.y = (__float_as_uint(w[2]) >> 16) | (__float_as_uint(w[3]) & 0xffff0000u);
  }
  __device__ __forceinline__ f32x4 all() const {
    return f32x4{__uint_as_float(v.x << 16), __uint_as_float(v.x & 0xffff0000u), __uint_as_float(v.y << 16),
                 __uint_as_float(v.y & 0xffff0000u)};
  }
  __device__ __forceinline__ void store(bf16_t* at) const { *reinterpret_cast<uint2*>(at) = v; }
  __device__ __forceinline__ void fetch_at(const bf16_t* at, int) { v = *reinterpret_cast<const uint2*>(at); }
  __device__ __forceinline__ void fetch(const bf16_t* row, int d) { fetch_at(row + (d < HS_DIM ? d : 0), d); }
  __device__ __forceinline__ f32x4 value(int d, bool live) const {
    if (!live || d >= HS_DIM) return f32x4{0.f, 0.f, 0.f, 0.f};
    return all();
  }
};
template <> struct Four<float, true> {
  f32x4 v;
  __device__ __forceinline__ void set(const f32x4& w) { v = w; }
  __device__ __forceinline__ f32x4 all() const { return v; }
  __device__ __forceinline__ void store(float* at) const { *reinterpret_cast<f32x4*>(at) = v; }
  __device__ __forceinline__ void fetch_at(const float* at, int) { v = *reinterpret_cast<const f32x4*>(at); }
  __device__ __forceinline__ void fetch(const float* row, int d) { fetch_at(row + (d < HS_DIM ? d : 0), d); }
  __device__ __forceinline__ f32x4 value(int d, bool live) const { return live && d < HS_DIM ? v : f32x4{0.f, 0.f, 0.f, 0.f}; }
};

// ---------------------------------------------------------------------------------------
// Q K^T and K K^T of a (chunk, group), lower triangle's tiles; factors of the unit lengths folded in
// ---------------------------------------------------------------------------------------
template <typename TX, bool DELTA, bool VEC>
__global__ __launch_bounds__(256) void hs_score_kernel(HeadScan a) {
  __shared__ __attribute__((aligned(16))) float q[HS_CHUNK * HS_LD], k[HS_CHUNK * HS_LD];
  __shared__ float f[2][HS_CHUNK];
  const int c = blockIdx.x, grp = blockIdx.y, tid = threadIdx.x, wave = tid >> 6, lane = tid & 63;
  const int begin = a.bounds[c], n = a.bounds[c + 1] - begin;
  const TX* x = reinterpret_cast<const TX*>(a.x) + (size_t)begin * a.x_stride + (size_t)grp * HS_DIM;
#pragma unroll 4
  for (int i = 0; i < HS_KB; ++i) {             // 64 tokens of HS_KB * 4 groups of four channels
    const int idx = tid + 256 * i, t = idx / (HS_DIMP / 4), d = idx % (HS_DIMP / 4) * 4;
    Four<TX, VEC> qv, kv;
    const TX* row = x + (size_t)(t < n ? t : 0) * a.x_stride;
    qv.fetch(row + a.q_off, d);
    kv.fetch(row + a.k_off, d);
    *reinterpret_cast<f32x4*>(q + t * HS_LD + d) = qv.value(d, t < n);
    *reinterpret_cast<f32x4*>(k + t * HS_LD + d) = kv.value(d, t < n);
  }
  __syncthreads();
  {                                             // four threads a token
    const int t = tid >> 2, part = tid & 3;
    float sq = 0.f, sk = 0.f;
    if (a.unit_eps >= 0.f) {
      for (int d = part * 4; d < HS_DIMP; d += 16) {
        const f32x4 qv = *reinterpret_cast<const f32x4*>(q + t * HS_LD + d), kv = *reinterpret_cast<const f32x4*>(k + t * HS_LD + d);
        sq += qv[0] * qv[0] + qv[1] * qv[1] + qv[2] * qv[2] + qv[3] * qv[3];
        sk += kv[0] * kv[0] + kv[1] * kv[1] + kv[2] * kv[2] + kv[3] * kv[3];
      }
      sq += __shfl_xor(sq, 1, 64); sq += __shfl_xor(sq, 2, 64);
      sk += __shfl_xor(sk, 1, 64); sk += __shfl_xor(sk, 2, 64);
    }
    if (part == 0) {
      f[0][t] = a.unit_eps >= 0.f ? a.q_scale / sqrtf(sq + a.unit_eps) : a.q_scale;
      f[1][t] = a.unit_eps >= 0.f ? 1.0f / sqrtf(sk + a.unit_eps) : 1.0f;
    }
  }
  __syncthreads();
  if (tid < 2 * HS_CHUNK) a.unit[((size_t)c * a.G + grp) * 2 * HS_CHUNK + tid] = f[tid >> 6][tid & 63];
  const int col = lane & 15, lg = lane >> 4;
  const size_t base = ((size_t)c * a.G + grp) * HS_CHUNK * HS_CHUNK;
  TX* kt = reinterpret_cast<TX*>(a.kt) + (((size_t)c * a.G + grp) * HS_KB * 4 * 64 + lane) * 4;
#pragma unroll 4
  for (int i = wave; i < HS_KB * 4; i += 4) {   // a block of 16 channels and a block of 16 tokens
    Four<TX, true> o;
    f32x4 v;
#pragma unroll
    for (int j = 0; j < 4; ++j) v[j] = k[((i & 3) * 16 + 4 * lg + j) * HS_LD + (i >> 2) * 16 + col];
    o.set(v);
    o.store(kt + (size_t)i * 256);
  }
  // ten tiles on or below the diagonal: tile number i is (row, column) of the list, shared among the waves
  for (int i = wave; i < 10; i += 4) {
    const int rt = i < 1 ? 0 : (i < 3 ? 1 : (i < 6 ? 2 : 3)), ct = i - rt * (rt + 1) / 2;
    f32x4 s = {0.f, 0.f, 0.f, 0.f}, w = s;
#pragma unroll 4
    for (int b = 0; b < HS_KB; ++b) {
      const f32x4 kb = *reinterpret_cast<const f32x4*>(k + (ct * 16 + col) * HS_LD + b * 16 + 4 * lg);
      s = mma16(*reinterpret_cast<const f32x4*>(q + (rt * 16 + col) * HS_LD + b * 16 + 4 * lg), kb, s);
      if (DELTA) w = mma16(*reinterpret_cast<const f32x4*>(k + (rt * 16 + col) * HS_LD + b * 16 + 4 * lg), kb, w);
    }
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int row = rt * 16 + 4 * lg + r;
      const size_t at = base + (size_t)row * HS_CHUNK + ct * 16 + col;
      a.qk[at] = s[r] * f[0][row] * f[1][ct * 16 + col];
      if (DELTA) a.kk[at] = w[r] * f[1][row] * f[1][ct * 16 + col];
    }
  }
}

// ---------------------------------------------------------------------------------------
// [Wv | Wk] of a (chunk, head): a wave owns 16 columns of the right side at a time
// ---------------------------------------------------------------------------------------
template <typename TX>
__global__ __launch_bounds__(256) void hs_solve_kernel(HeadScan a) {
  __shared__ __attribute__((aligned(16))) float A[HS_CHUNK][HS_CHUNK + 4];   // strictly below the diagonal
  __shared__ __attribute__((aligned(16))) float T[4][16][20];                // inverses of the diagonal blocks
  __shared__ __attribute__((aligned(16))) float rv[HS_CHUNK], rk[HS_CHUNK];                               // factors on the rows of V and K
  __shared__ double ls[HS_CHUNK];
  const int c = blockIdx.x, head = blockIdx.y, grp = head / (a.H / a.G);
  const int tid = threadIdx.x, wave = __builtin_amdgcn_readfirstlane(tid >> 6), lane = tid & 63, col = lane & 15, lg = lane >> 4;
  const int begin = a.bounds[c], n = a.bounds[c + 1] - begin;
  const size_t ch = (size_t)c * a.H + head;
  const float* kk = a.kk + ((size_t)c * a.G + grp) * HS_CHUNK * HS_CHUNK;
  f32x4 prod[4];                                // a thread has four neighbouring columns of the rows tid / 16 + 16 i
#pragma unroll
  for (int i = 0; i < 4; ++i)
    prod[i] = (tid & 15) * 4 < 16 * i + 16 ? *reinterpret_cast<const f32x4*>(kk + (tid + 256 * i) * 4) : f32x4{0.f, 0.f, 0.f, 0.f};
  if (tid < HS_CHUNK) {
    const float beta = a.gate[ch * HS_CHUNK + tid];
    ls[tid] = a.lsum[ch * HS_CHUNK + tid];
    rv[tid] = beta;
    rk[tid] = beta * a.head[ch * HS_CHUNK + tid] * a.unit[((size_t)c * a.G + grp) * 2 * HS_CHUNK + HS_CHUNK + tid];
  }
  __syncthreads();
#pragma unroll
  for (int i = 0; i < 4; ++i) {
    const int row = (tid >> 4) + 16 * i, j0 = (tid & 15) * 4;
    f32x4 v;
#pragma unroll
    for (int j = 0; j < 4; ++j)
      v[j] = j0 + j < row ? rv[row] * decay_of(ls[row] - ls[j0 + j]) * prod[i][j] : 0.f;
    *reinterpret_cast<f32x4*>(&A[row][j0]) = v;
  }
  __syncthreads();
  if (lane < 16) {                              // wave w inverts diagonal block w, a lane per column
    float xcol[16];
#pragma unroll
    for (int i = 0; i < 16; ++i) {
      float v = i == lane ? 1.f : 0.f;
#pragma unroll
      for (int j = 0; j < i; ++j) v -= A[wave * 16 + i][wave * 16 + j] * xcol[j];
      xcol[i] = v;
    }
#pragma unroll
    for (int i = 0; i < 16; ++i) T[wave][i][lane] = xcol[i];
  }
  __syncthreads();
  f32x4 inv[4], low[6];                         // low[i (i - 1) / 2 + j] = -A's block (i, j)
#pragma unroll
  for (int i = 0; i < 4; ++i) {
    inv[i] = *reinterpret_cast<const f32x4*>(&T[i][col][4 * lg]);
#pragma unroll
    for (int j = 0; j < i; ++j) low[i * (i - 1) / 2 + j] = -*reinterpret_cast<const f32x4*>(&A[i * 16 + col][j * 16 + 4 * lg]);
  }
  const TX* x = reinterpret_cast<const TX*>(a.x) + (size_t)begin * a.x_stride;
  const int vtiles = (a.vdim + 15) / 16, tiles = vtiles + HS_KB;
  // a tile's values as they lie in memory, asked for a tile ahead; what lies outside is read from inside and not counted
  TX raw[16];
  auto ask = [&](int tile) {
    const bool values = tile < vtiles;
    const int cc = (values ? tile : tile - vtiles) * 16 + col;
    const TX* src = x + (values ? a.v_off + (size_t)head * a.vdim : a.k_off + (size_t)grp * HS_DIM) +
                    (cc < (values ? a.vdim : HS_DIM) ? cc : 0);
#pragma unroll
    for (int i = 0; i < 16; ++i) {
      const int t = (i >> 2) * 16 + 4 * lg + (i & 3);
      raw[i] = src[(size_t)(t < n ? t : 0) * a.x_stride];
    }
  };
  if (wave < tiles) ask(wave);
  for (int tile = wave; tile < tiles; tile += 4) {
    const bool values = tile < vtiles;
    const int cc = (values ? tile : tile - vtiles) * 16 + col;
    const bool in = cc < (values ? a.vdim : HS_DIM);
    const float* factor = values ? rv : rk;
    f32x4 y[4];
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      y[i] = *reinterpret_cast<const f32x4*>(factor + i * 16 + 4 * lg);
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const float v = y[i][r] * ldf<TX>(raw + i * 4 + r);
        y[i][r] = in && i * 16 + 4 * lg + r < n ? v : 0.f;
      }
    }
    if (tile + 4 < tiles) ask(tile + 4);
#pragma unroll
    for (int i = 0; i < 4; ++i) {
#pragma unroll
      for (int j = 0; j < i; ++j) y[i] = mma16(low[i * (i - 1) / 2 + j], y[j], y[i]);
      y[i] = mma16(inv[i], y[i], f32x4{0.f, 0.f, 0.f, 0.f});
    }
    if (values) {
      float* dst = a.u + ((ch * vtiles + tile) * 4 * 64 + lane) * 4;
#pragma unroll
      for (int i = 0; i < 4; ++i) *reinterpret_cast<f32x4*>(dst + i * 256) = y[i];
    } else {
      float* dst = a.wk + ch * HS_CHUNK * HS_DIMP + cc;
#pragma unroll
      for (int i = 0; i < 4; ++i)
#pragma unroll
        for (int r = 0; r < 4; ++r) dst[(size_t)(i * 16 + 4 * lg + r) * HS_DIMP] = y[i][r];
    }
  }
}

// ---------------------------------------------------------------------------------------
// The states from chunk to chunk: a block per (16 value channels, head, request)
// ---------------------------------------------------------------------------------------
#define HS_MT ((HS_KB + 3) / 4)                 // row blocks of S a wave keeps: wave w has blocks w, w + 4, ...

// What a block reads of a chunk, asked for two chunks ahead: nothing here is waited for before it is used.
template <typename TX, bool DELTA> struct CarryLoads {
  Four<TX, true> k[HS_MT][4];
  f32x4 wk[DELTA ? HS_KB : 1];
  f32x4 u;
  TX v[4];
  f32x4 gate, tail, unit;
  float end;
  int n;
};

template <typename TX, bool DELTA>
__global__ __launch_bounds__(256) void hs_carry_kernel(HeadScan a) {
  __shared__ f32x4 us_place[2][4 * 64];         // U, weighted by what is left of it at the chunk's end; two places, taken in turn
  __shared__ f32x4 s[DELTA ? HS_KB * 64 : 1];   // S as right operand
  __shared__ float left[2];                     // what a chunk leaves of the state before it
  // Workgroups go to the 8 XCDs in turn: numbered so that an XCD gets neighbouring tiles and heads, whose blocks read the
  // same keys and Wk.
  const int vtiles = (a.vdim + 15) / 16;
  const int item = (blockIdx.x & 7) * (gridDim.x >> 3) + (blockIdx.x >> 3);
  if (item >= vtiles * a.H) return;
  const int head = item / vtiles, vtile = item % vtiles, req = blockIdx.y, grp = head / (a.H / a.G);
  const int tid = threadIdx.x, wave = __builtin_amdgcn_readfirstlane(tid >> 6), lane = tid & 63, col = lane & 15, lg = lane >> 4;
  const int first = __builtin_amdgcn_readfirstlane(a.req_first[req]), last = __builtin_amdgcn_readfirstlane(a.req_first[req + 1]);
  if (first >= last) return;
  // a run's chunks follow one another and all but the last are full
  const int run_begin = __builtin_amdgcn_readfirstlane(a.bounds[first]), run_end = __builtin_amdgcn_readfirstlane(a.bounds[last]);
  const int vcol = vtile * 16 + col;
  const bool in = vcol < a.vdim;
  float* slot = a.state + ((size_t)a.row_of[req] * a.H + head) * HS_DIM * a.vdim + (in ? vcol : 0);
  f32x4 S[HS_MT];
#pragma unroll
  for (int m = 0; m < HS_MT; ++m) {
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int d = (wave + 4 * m) * 16 + 4 * lg + r;
      S[m][r] = in && d < HS_DIM ? slot[(size_t)d * a.vdim] : 0.f;
    }
  }
  const TX* x = reinterpret_cast<const TX*>(a.x);
  const int t_own = wave * 16 + 4 * lg;         // the first of this lane's four rows of U
  typedef CarryLoads<TX, DELTA> Loads;
  // places of values within a chunk, in bytes from its first token's: the same for every chunk
  unsigned v_at[4];
#pragma unroll
  for (int r = 0; r < 4; ++r) v_at[r] = (unsigned)(((t_own + r) * (int)a.x_stride + (in ? vcol : 0)) * (int)sizeof(TX));
  auto ask_keys = [&](Loads& l, int c) {
    const TX* kt = reinterpret_cast<const TX*>(a.kt) + (((size_t)c * a.G + grp) * HS_KB * 4 * 64 + lane) * 4;
#pragma unroll
    for (int m = 0; m < HS_MT; ++m) {
      const int b = wave + 4 * m;
#pragma unroll
      for (int tb = 0; tb < 4; ++tb) l.k[m][tb].fetch_at(kt + (size_t)((HS_KB % 4 == 0 || b < HS_KB ? b : 0) * 4 + tb) * 256, 0);
    }
  };
  auto ask_rest = [&](Loads& l, int c) {
    const size_t ch = (size_t)c * a.H + head;
    l.tail = *reinterpret_cast<const f32x4*>(a.tail + ch * HS_CHUNK + t_own);
    l.unit = *reinterpret_cast<const f32x4*>(a.unit + (((size_t)c * a.G + grp) * 2 + 1) * HS_CHUNK + t_own);
    l.end = a.head[ch * HS_CHUNK + HS_CHUNK - 1];
    if (DELTA) {
      const float* wk = a.wk + (ch * HS_CHUNK + wave * 16 + col) * HS_DIMP + 4 * lg;
#pragma unroll
      for (int b = 0; b < HS_KB; ++b) l.wk[DELTA ? b : 0] = *reinterpret_cast<const f32x4*>(wk + b * 16);
      l.u = *reinterpret_cast<const f32x4*>(a.u + ((ch * vtiles + vtile) * 4 + wave) * 256 + lane * 4);
    } else {
      l.gate = *reinterpret_cast<const f32x4*>(a.gate + ch * HS_CHUNK + t_own);
      const int begin = run_begin + (c - first) * HS_CHUNK;
      l.n = run_end - begin < HS_CHUNK ? run_end - begin : HS_CHUNK;
      const char* base = reinterpret_cast<const char*>(x + (size_t)begin * a.x_stride + a.v_off + (size_t)head * a.vdim);
#pragma unroll
      for (int r = 0; r < 4; ++r) l.v[r] = *reinterpret_cast<const TX*>(base + (t_own + r < l.n ? v_at[r] : 0u));
    }
  };
  // The order of a step's memory operations is that in which they are waited for: what the next step needs first is asked
  // for first, and the stores, which nobody waits for, come behind what the next but one waits for.
  auto step = [&](Loads& l, int c) {
    const size_t ch = (size_t)c * a.H + head;
    const int next = c + 2 < last ? c + 2 : last - 1;      // the last two ask for the last chunk again
    f32x4* us = us_place[c & 1];
    f32x4 u;
    if (DELTA) {
#pragma unroll
      for (int m = 0; m < HS_MT; ++m)
        if (HS_KB % 4 == 0 || wave + 4 * m < HS_KB) s[DELTA ? (wave + 4 * m) * 64 + lane : 0] = S[m];
      __syncthreads();
      f32x4 p0 = {0.f, 0.f, 0.f, 0.f}, p1 = p0;
#pragma unroll
      for (int b = 0; b < HS_KB; b += 2) {
        p0 = mma16(l.wk[DELTA ? b : 0], s[DELTA ? b * 64 + lane : 0], p0);
        if (b + 1 < HS_KB) p1 = mma16(l.wk[DELTA ? b + 1 : 0], s[DELTA ? (b + 1) * 64 + lane : 0], p1);
      }
      u = l.u - (p0 + p1);
    } else {
#pragma unroll
      for (int r = 0; r < 4; ++r) u[r] = in && t_own + r < l.n ? l.gate[r] * ldf<TX>(l.v + r) : 0.f;
    }
    us[wave * 64 + lane] = u * l.tail * l.unit;
    if (tid == 0) left[c & 1] = l.end;
    ask_rest(l, next);
    float* s0 = a.s0 + ((ch * vtiles + vtile) * HS_KB * 64 + lane) * 4;
#pragma unroll
    for (int m = 0; m < HS_MT; ++m)
      if (HS_KB % 4 == 0 || wave + 4 * m < HS_KB) *reinterpret_cast<f32x4*>(s0 + (size_t)(wave + 4 * m) * 256) = S[m];
    if (DELTA) *reinterpret_cast<f32x4*>(a.u + ((ch * vtiles + vtile) * 4 + wave) * 256 + lane * 4) = u;
    __syncthreads();
    f32x4 ur[4];
#pragma unroll
    for (int tb = 0; tb < 4; ++tb) ur[tb] = us[tb * 64 + lane];
    const float g = left[c & 1];
#pragma unroll
    for (int m = 0; m < HS_MT; ++m) S[m] *= g;
#pragma unroll
    for (int tb = 0; tb < 4; ++tb) {
      f32x4 kt[HS_MT];
#pragma unroll
      for (int m = 0; m < HS_MT; ++m) kt[m] = l.k[m][tb].all();
#pragma unroll
      for (int j = 0; j < 4; ++j)
#pragma unroll
        for (int m = 0; m < HS_MT; ++m) S[m] = __builtin_amdgcn_mfma_f32_16x16x4f32(kt[m][j], ur[tb][j], S[m], 0, 0, 0);
    }
    ask_keys(l, next);
  };
  Loads even, odd;
  ask_keys(even, first);
  ask_rest(even, first);
  ask_keys(odd, first + 1 < last ? first + 1 : first);
  ask_rest(odd, first + 1 < last ? first + 1 : first);
  for (int c = first; c < last; c += 2) {
    step(even, c);
    if (c + 1 >= last) break;
    step(odd, c + 1);
  }
  if (in) {
#pragma unroll
    for (int m = 0; m < HS_MT; ++m) {
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int d = (wave + 4 * m) * 16 + 4 * lg + r;
        if (d < HS_DIM) slot[(size_t)d * a.vdim] = S[m][r];
      }
    }
  }
}

// ---------------------------------------------------------------------------------------
// O of a (chunk, head): wave w forms the tiles of 16 value channels w, w + 4, ... of all 64 tokens, so that S' and U are
// read once; the left operands, the same for all tiles, lie in LDS as fragments.
// ---------------------------------------------------------------------------------------
template <typename TX, bool DELTA, bool VEC>
__global__ __launch_bounds__(256, HS_DIMP <= 128 ? 3 : 2) void hs_out_kernel(HeadScan a) {
  __shared__ f32x4 qf[4][HS_KB][64];            // diag(L_i0) Q
  __shared__ f32x4 pf[10][64];                  // L o Q K^T, tile (row, column) at row (row + 1) / 2 + column
  __shared__ double ls[HS_CHUNK];
  const int c = blockIdx.x, head = blockIdx.y, grp = head / (a.H / a.G);
  const int wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6), lane = threadIdx.x & 63, col = lane & 15, lg = lane >> 4;
  const int begin = a.bounds[c], n = a.bounds[c + 1] - begin;
  const size_t ch = (size_t)c * a.H + head;
  const int vtiles = (a.vdim + 15) / 16, row_tiles = (n + 15) / 16;
  const f32x4* s0 = reinterpret_cast<const f32x4*>(a.s0) + ch * vtiles * HS_KB * 64 + lane;
  const f32x4* ug = reinterpret_cast<const f32x4*>(a.u) + ch * vtiles * 4 * 64 + lane;
  const TX* xr = reinterpret_cast<const TX*>(a.x) + (size_t)begin * a.x_stride;
  const float* gate = a.gate + ch * HS_CHUNK;
  constexpr int AHEAD = HS_KB <= 4 ? HS_KB : 4; // blocks of S' asked for together
  f32x4 sv[AHEAD];
#pragma unroll
  for (int b = 0; b < AHEAD; ++b) sv[b] = s0[((wave < vtiles ? wave : 0) * HS_KB + b) * 64];
  {
    const int row = wave * 16 + col;
    const TX* qr = xr + (size_t)(row < n ? row : 0) * a.x_stride + a.q_off + (size_t)grp * HS_DIM;
    Four<TX, VEC> qraw[HS_KB];
#pragma unroll
    for (int b = 0; b < HS_KB; ++b) qraw[b].fetch(qr, b * 16 + 4 * lg);
    const float f = a.head[ch * HS_CHUNK + row] * a.unit[((size_t)c * a.G + grp) * 2 * HS_CHUNK + row];
    const float* qk = a.qk + (((size_t)c * a.G + grp) * HS_CHUNK + row) * HS_CHUNK + 4 * lg;
    f32x4 sc[4];
#pragma unroll
    for (int jb = 0; jb < 4; ++jb) sc[jb] = *reinterpret_cast<const f32x4*>(qk + (jb <= wave ? jb : 0) * 16);
    if (threadIdx.x < HS_CHUNK) ls[threadIdx.x] = a.lsum[ch * HS_CHUNK + threadIdx.x];
    __syncthreads();
    const double mine = ls[row];
#pragma unroll
    for (int jb = 0; jb < 4; ++jb) {
      if (jb <= wave) {
        f32x4 p;
#pragma unroll
        for (int j = 0; j < 4; ++j) {
          const int t = jb * 16 + 4 * lg + j;
          p[j] = t <= row ? sc[jb][j] * decay_of(mine - ls[t]) : 0.f;
        }
        pf[wave * (wave + 1) / 2 + jb][lane] = p;
      }
    }
#pragma unroll
    for (int b = 0; b < HS_KB; ++b) qf[wave][b][lane] = qraw[b].value(b * 16 + 4 * lg, row < n) * f;
  }
  const float skip = a.skip ? a.skip[head] : 0.f;
  __syncthreads();
  for (int vt = wave; vt < vtiles; vt += 4) {
    asm volatile("" ::: "memory");              // the fragments are read from LDS for every tile, not kept in registers
    const int vcol = vt * 16 + col;
    const bool in = vcol < a.vdim;
    const TX* vr = xr + a.v_off + (size_t)head * a.vdim + (in ? vcol : 0);
    f32x4 u[4], v[4], o[4];
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      o[i] = f32x4{0.f, 0.f, 0.f, 0.f};
      v[i] = o[i];
      if (DELTA) u[i] = ug[(vt * 4 + i) * 64];
      if (!DELTA || a.skip) {
#pragma unroll
        for (int r = 0; r < 4; ++r) {
          const int t = i * 16 + 4 * lg + r;
          const float x = ldf<TX>(vr + (size_t)(t < n ? t : 0) * a.x_stride);
          v[i][r] = in && t < n ? x : 0.f;
        }
      }
      if (!DELTA) u[i] = v[i] * *reinterpret_cast<const f32x4*>(gate + i * 16 + 4 * lg);
    }
#pragma unroll
    for (int b = 0; b < HS_KB; ++b) {
      const f32x4 sb = sv[b % AHEAD];
      if (b + AHEAD < HS_KB) sv[b % AHEAD] = s0[(vt * HS_KB + b + AHEAD) * 64];
      else if (vt + 4 < vtiles) sv[b % AHEAD] = s0[((vt + 4) * HS_KB + b + AHEAD - HS_KB) * 64];
      f32x4 q[4];
#pragma unroll
      for (int i = 0; i < 4; ++i) q[i] = qf[i][b][lane];
#pragma unroll
      for (int j = 0; j < 4; ++j)
#pragma unroll
        for (int i = 0; i < 4; ++i) o[i] = __builtin_amdgcn_mfma_f32_16x16x4f32(q[i][j], sb[j], o[i], 0, 0, 0);
    }
#pragma unroll
    for (int jb = 0; jb < 4; ++jb)
#pragma unroll
      for (int i = jb; i < 4; ++i) o[i] = mma16(pf[i * (i + 1) / 2 + jb][lane], u[jb], o[i]);
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      if (i < row_tiles && in) {
#pragma unroll
        for (int r = 0; r < 4; ++r) {
          const int t = i * 16 + 4 * lg + r;
          if (t < n) a.out[((size_t)(begin + t) * a.H + head) * a.vdim + vcol] = o[i][r] + skip * v[i][r];
        }
      }
    }
  }
}
#endif  // HS_CHUNKED

extern "C" int qvl_head_scan_key_size() { return HS_DIM; }
extern "C" int qvl_head_scan_chunked() { return HS_CHUNKED; }

static int fill_args(HeadScan& a, const void* x, long long x_stride, int q_off, int k_off, int v_off, const void* raw,
                     long long raw_stride, int a_off, int b_off, const void* bias, const void* a_neg, const void* skip,
                     float q_scale, float unit_eps, void* state, const void* bounds, const void* row_of, void* out, int H,
                     int G, int dim, int vdim) {
  if (dim != HS_DIM || H <= 0 || G <= 0 || H % G || vdim <= 0) return QVL_ERR_SHAPE;
  if (!x || !raw || !bias || !a_neg || !state || !bounds || !row_of || !out) return QVL_ERR_SHAPE;
  if (q_off < 0 || k_off < 0 || v_off < 0 || a_off < 0) return QVL_ERR_SHAPE;
  if (x_stride < (long long)q_off + (long long)G * HS_DIM || x_stride < (long long)k_off + (long long)G * HS_DIM ||
      x_stride < (long long)v_off + (long long)H * vdim || x_stride > 0x7fffffffLL / (HS_CHUNK * 8) || raw_stride < (long long)a_off + H || raw_stride < (long long)b_off + H)
    return QVL_ERR_SHAPE;
  if (H > 65535) return QVL_ERR_LIMIT;
  a = HeadScan{};
  a.x = x; a.x_stride = x_stride; a.q_off = q_off; a.k_off = k_off; a.v_off = v_off; a.raw = (const float*)raw;
  a.raw_stride = raw_stride; a.a_off = a_off; a.b_off = b_off; a.bias = (const float*)bias; a.a_neg = (const float*)a_neg;
  a.skip = (const float*)skip; a.q_scale = q_scale; a.unit_eps = unit_eps; a.state = (float*)state;
  a.bounds = (const int*)bounds; a.row_of = (const int*)row_of; a.out = (float*)out; a.H = H; a.G = G; a.vdim = vdim;
  return QVL_OK;
}

// x rows hold q (G * HS_DIM columns from q_off), k (from k_off) and v (H * vdim columns from v_off); raw rows the step
// inputs (from a_off) and, with the delta rule (b_off >= 0), the beta inputs.  unit_eps < 0: no unit vectors.  bounds
// [R + 1], row_of [R] (the request's slot); out float32 [N, H * vdim].  dtype: of x.
extern "C" int qvl_head_scan(const void* x, long long x_stride, int q_off, int k_off, int v_off, const void* raw,
                             long long raw_stride, int a_off, int b_off, const void* bias, const void* a_neg,
                             const void* skip, float q_scale, float unit_eps, void* state, const void* bounds,
                             const void* row_of, void* out, int R, int H, int G, int dim, int vdim, int dtype,
                             hipStream_t stream) {
  if (R <= 0) return QVL_OK;
  if (R > 65535) return QVL_ERR_LIMIT;
  HeadScan a;
  const int bad = fill_args(a, x, x_stride, q_off, k_off, v_off, raw, raw_stride, a_off, b_off, bias, a_neg, skip, q_scale,
                            unit_eps, state, bounds, row_of, out, H, G, dim, vdim);
  if (bad) return bad;
  const dim3 grid((vdim + 63) / 64, H, R);
  const bool delta = b_off >= 0;
#define LAUNCH(TX, D) hipLaunchKernelGGL((hs_scan_kernel<TX, D>), grid, dim3(256), 0, stream, a)
  if (dtype == 0) { if (delta) LAUNCH(float, true); else LAUNCH(float, false); }
  else if (dtype == 1) { if (delta) LAUNCH(bf16_t, true); else LAUNCH(bf16_t, false); }
  else return QVL_ERR_DTYPE;
#undef LAUNCH
  return qvl_launch_status();
}

// Floats of scratch memory that qvl_head_scan_chunks needs.
extern "C" long long qvl_head_scan_scratch(int chunks, int H, int G, int vdim, int delta) {
  const long long vtiles = (vdim + 15) / 16, c = chunks;
  return c * H * HS_CHUNK * 5 + c * G * (2 * HS_CHUNK + HS_CHUNK * HS_DIMP + (delta ? 2 : 1) * HS_CHUNK * HS_CHUNK) +
         (delta ? c * H * HS_CHUNK * HS_DIMP : 0) + c * H * vtiles * ((delta ? 4 : 0) + HS_KB) * 256;
}

// The same in chunks of at most 64 tokens: chunk_cu [chunks + 1], req_first [R + 1] (the first chunk of each request);
// scratch 16-byte aligned.
extern "C" int qvl_head_scan_chunks(const void* x, long long x_stride, int q_off, int k_off, int v_off, const void* raw,
                                    long long raw_stride, int a_off, int b_off, const void* bias, const void* a_neg,
                                    const void* skip, float q_scale, float unit_eps, void* state, const void* chunk_cu,
                                    const void* req_first, const void* row_of, void* out, void* scratch, int chunks, int R,
                                    int H, int G, int dim, int vdim, int dtype, hipStream_t stream) {
#if HS_CHUNKED
  if (R <= 0 || chunks <= 0) return QVL_OK;
  if (R > 65535) return QVL_ERR_LIMIT;
  HeadScan a;
  const int bad = fill_args(a, x, x_stride, q_off, k_off, v_off, raw, raw_stride, a_off, b_off, bias, a_neg, skip, q_scale,
                            unit_eps, state, chunk_cu, row_of, out, H, G, dim, vdim);
  if (bad) return bad;
  if (!req_first || !scratch || ((uintptr_t)scratch & 15)) return QVL_ERR_SHAPE;
  const bool delta = b_off >= 0;
  const int vtiles = (vdim + 15) / 16;
  a.req_first = (const int*)req_first;
  const long long c = chunks;
  float* at = (float*)scratch;
  a.lsum = (double*)at; at += c * H * HS_CHUNK * 2;
  a.gate = at; at += c * H * HS_CHUNK;
  a.head = at; at += c * H * HS_CHUNK;
  a.tail = at; at += c * H * HS_CHUNK;
  a.unit = at; at += c * G * 2 * HS_CHUNK;
  a.kt = at; at += c * G * HS_CHUNK * HS_DIMP;
  a.qk = at; at += c * G * HS_CHUNK * HS_CHUNK;
  if (delta) { a.kk = at; at += c * G * HS_CHUNK * HS_CHUNK; }
  if (delta) { a.wk = at; at += c * H * HS_CHUNK * HS_DIMP; }
  if (delta) { a.u = at; at += c * H * vtiles * 4 * 256; }
  a.s0 = at;
  const bool vec = HS_DIM % 4 == 0 && x_stride % 4 == 0 && q_off % 4 == 0 && k_off % 4 == 0 && ((uintptr_t)x & 15) == 0;
#define LAUNCH(TX, D, V)                                                                                             \
  {                                                                                                                  \
    hipLaunchKernelGGL((hs_prep_kernel<D>), dim3(chunks, (H + 3) / 4), dim3(256), 0, stream, a);                     \
    hipLaunchKernelGGL((hs_score_kernel<TX, D, V>), dim3(chunks, G), dim3(256), 0, stream, a);                       \
    if (D) hipLaunchKernelGGL((hs_solve_kernel<TX>), dim3(chunks, H), dim3(256), 0, stream, a);                      \
    hipLaunchKernelGGL((hs_carry_kernel<TX, D>), dim3((vtiles * H + 7) / 8 * 8, R), dim3(256), 0, stream, a);          \
    hipLaunchKernelGGL((hs_out_kernel<TX, D, V>), dim3(chunks, H), dim3(256), 0, stream, a);                            \
  }
#define BY_VEC(TX, D) { if (vec) LAUNCH(TX, D, true) else LAUNCH(TX, D, false) }
  if (dtype == 0) { if (delta) BY_VEC(float, true) else BY_VEC(float, false) }
  else if (dtype == 1) { if (delta) BY_VEC(bf16_t, true) else BY_VEC(bf16_t, false) }
  else return QVL_ERR_DTYPE;
#undef BY_VEC
#undef LAUNCH
  return qvl_launch_status();
#else
  return QVL_ERR_LIMIT;
#endif
}
