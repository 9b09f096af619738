// The residual sum of layers whose norm stands behind the sum, joined by one or two terms:
//   x = alpha h[n] + c1 f1(t1[n]) + c2 f2(t2[n]),      f(t) = t, or t / sqrt(mean(t^2) + eps_t) * gain
//   h[n] = (x - mean(x)) / sqrt(mean((x - mean(x))^2) + eps) * w + b,   or h[n] = x without w
// and, if asked for, a copy of the new row in another type.  A term is float32 or bfloat16 [N, H], or float32 slabs
// of it that are added in order.  All arithmetic is float32; the deviations are formed from the mean (two passes).
// A block owns a row and keeps it in registers between the passes: PER groups of VEC neighbouring values a thread.
#include "common.h"

#define SUM_NORM_MANY 512       // rows from which blocks are narrow

template <typename T, int VEC> struct Row;
template <typename T> struct Row<T, 1> {
  static __device__ __forceinline__ void load(float* v, const T* p) { v[0] = ldf<T>(p); }
  static __device__ __forceinline__ void store(T* p, const float* v) { stf<T>(p, v[0]); }
};
template <> struct Row<float, 4> {
  static __device__ __forceinline__ void load(float* v, const float* p) {
    const float4 t = *reinterpret_cast<const float4*>(p);
    v[0] = t.x; v[1] = t.y; v[2] = t.z; v[3] = t.w;
  }
  static __device__ __forceinline__ void store(float* p, const float* v) { *reinterpret_cast<float4*>(p) = float4{v[0], v[1], v[2], v[3]}; }
};
template <> struct Row<bf16_t, 4> {
  static __device__ __forceinline__ void load(float* v, const bf16_t* p) {
    const uint2 t = *reinterpret_cast<const uint2*>(p);
    v[0] = __uint_as_float(t.x << 16); v[1] = __uint_as_float(t.x & 0xffff0000u);
    v[2] = __uint_as_float(t.y << 16); v[3] = __uint_as_float(t.y & 0xffff0000u);
  }
  static __device__ __forceinline__ void store(bf16_t* p, const float* v) {
    uint2 o;
    o.x = (uint32_t)f32_to_bf16(v[0]) | ((uint32_t)f32_to_bf16(v[1]) << 16);
    o.y = (uint32_t)f32_to_bf16(v[2]) | ((uint32_t)f32_to_bf16(v[3]) << 16);
    *reinterpret_cast<uint2*>(p) = o;
  }
};

struct Term {
  const void* t;
  int nslabs;
  long long slab_stride;
  const float* gain;        // null: the term is taken as it is
  float eps, factor;
};

template <typename T, int VEC, int PER>
__device__ __forceinline__ void load_term(float* v, const Term& a, size_t row, int H) {
  const T* p = reinterpret_cast<const T*>(a.t) + row * H;
#pragma unroll
  for (int i = 0; i < PER; ++i) {
    const int c = (threadIdx.x + i * blockDim.x) * VEC;
    Row<T, VEC>::load(v + i * VEC, p + (c < H ? c : 0));       // past the row's end: its start, counted as zero
  }
  for (int s = 1; s < a.nslabs; ++s) {
    float w[PER * VEC];
#pragma unroll
    for (int i = 0; i < PER; ++i) {
      const int c = (threadIdx.x + i * blockDim.x) * VEC;
      Row<T, VEC>::load(w + i * VEC, p + (size_t)s * a.slab_stride + (c < H ? c : 0));
    }
#pragma unroll
    for (int i = 0; i < PER * VEC; ++i) v[i] += w[i];
  }
#pragma unroll
  for (int i = 0; i < PER; ++i)
    if ((threadIdx.x + i * blockDim.x) * VEC >= H) {
#pragma unroll
      for (int j = 0; j < VEC; ++j) v[i * VEC + j] = 0.f;
    }
}

template <int VEC, int PER>
__device__ __forceinline__ void normed_term(float* v, const Term& a, int H, float* red) {
  float g[PER * VEC];
#pragma unroll
  for (int i = 0; i < PER; ++i) {
    const int c = (threadIdx.x + i * blockDim.x) * VEC;
    Row<float, VEC>::load(g + i * VEC, a.gain + (c < H ? c : 0));
  }
  float ss = 0.f;
#pragma unroll
  for (int i = 0; i < PER * VEC; ++i) ss += v[i] * v[i];
  const float rs = 1.0f / sqrtf(block_sum(ss, red) / (float)H + a.eps);
#pragma unroll
  for (int i = 0; i < PER * VEC; ++i) v[i] = (v[i] * rs) * g[i];
}

template <typename TA, typename TB, typename TC, int TERMS, int VEC, int PER>
__global__ __launch_bounds__(1024) void sum_norm_kernel(float* __restrict__ h, float alpha, Term a, Term b,
                                                        const float* __restrict__ w, const float* __restrict__ bias,
                                                        float eps, TC* __restrict__ copy, int H) {
  __shared__ float red[17];
  const size_t n = blockIdx.x;
  float* hr = h + n * H;
  float x[PER * VEC], t1[PER * VEC], t2[TERMS > 1 ? PER * VEC : 1], wv[PER * VEC], bv[PER * VEC];
  load_term<TA, VEC, PER>(t1, a, n, H);
  if (TERMS > 1) load_term<TB, VEC, PER>(t2, b, n, H);
#pragma unroll
  for (int i = 0; i < PER; ++i) {
    const int c = (threadIdx.x + i * blockDim.x) * VEC, cc = c < H ? c : 0;
    Row<float, VEC>::load(x + i * VEC, hr + cc);
    if (w) {
      Row<float, VEC>::load(wv + i * VEC, w + cc);
      Row<float, VEC>::load(bv + i * VEC, bias + cc);
    }
    if (c >= H) {
#pragma unroll
      for (int j = 0; j < VEC; ++j) x[i * VEC + j] = 0.f;
    }
  }
  if (a.gain) normed_term<VEC, PER>(t1, a, H, red);
  if (TERMS > 1 && b.gain) normed_term<VEC, PER>(t2, b, H, red);
  float sum = 0.f;
#pragma unroll
  for (int i = 0; i < PER * VEC; ++i) {
    x[i] = alpha * x[i] + a.factor * t1[i];
    if (TERMS > 1) x[i] += b.factor * t2[TERMS > 1 ? i : 0];
    sum += x[i];
  }
  if (w) {
    const float mean = block_sum(sum, red) / (float)H;
    float sq = 0.f;
#pragma unroll
    for (int i = 0; i < PER; ++i) {
      const bool in = (threadIdx.x + i * blockDim.x) * VEC < H;
#pragma unroll
      for (int j = 0; j < VEC; ++j) {
        x[i * VEC + j] -= mean;
        sq += in ? x[i * VEC + j] * x[i * VEC + j] : 0.f;
      }
    }
    const float inv = 1.0f / sqrtf(block_sum(sq, red) / (float)H + eps);
#pragma unroll
    for (int i = 0; i < PER * VEC; ++i) x[i] = x[i] * inv * wv[i] + bv[i];
  }
#pragma unroll
  for (int i = 0; i < PER; ++i) {
    const int c = (threadIdx.x + i * blockDim.x) * VEC;
    if (c < H) {
      Row<float, VEC>::store(hr + c, x + i * VEC);
      if (copy) Row<TC, VEC>::store(copy + n * H + c, x + i * VEC);
    }
  }
}

static inline bool on16(const void* p) { return ((uintptr_t)p & 15) == 0; }

// h float32 [N, H], in place.  t1 (and t2, or null): dtype 0 float32, 1 bfloat16; slabs float32.  gain1, gain2: float32
// [H] or null.  w and bias: float32 [H], both or neither.  copy: [N, H] of copy_dtype, or null.
extern "C" int qvl_sum_norm(void* h, float alpha, const void* t1, int dtype1, int nslabs1, const void* gain1, float eps1,
                            float factor1, const void* t2, int dtype2, int nslabs2, const void* gain2, float eps2,
                            float factor2, const void* w, const void* bias, float eps, void* copy, int copy_dtype, int N,
                            int H, hipStream_t stream) {
  if (N <= 0) return QVL_OK;
  if (H <= 0 || !h || !t1 || nslabs1 < 1 || (nslabs1 > 1 && dtype1 != 0) || (!w != !bias)) return QVL_ERR_SHAPE;
  if (t2 && (nslabs2 < 1 || (nslabs2 > 1 && dtype2 != 0))) return QVL_ERR_SHAPE;
  if (dtype1 < 0 || dtype1 > 1 || dtype2 < 0 || dtype2 > 1 || copy_dtype < 0 || copy_dtype > 1) return QVL_ERR_DTYPE;
  const Term a{t1, nslabs1, (long long)N * H, (const float*)gain1, eps1, factor1};
  const Term b{t2, t2 ? nslabs2 : 1, (long long)N * H, (const float*)gain2, eps2, factor2};
  const bool vec = H % 4 == 0 && H <= 4 * 8 * 1024 && on16(h) && on16(t1) && on16(t2) && on16(gain1) && on16(gain2) && on16(w) && on16(bias) && on16(copy);
  const int units = vec ? H / 4 : H;
  if (units > 1024 * 32) return QVL_ERR_LIMIT;
  // few rows: a thread has little of a row (short chains of waits); many: narrow blocks, whose barriers hold up fewer waves
  // (2,048 rows of 3,584, two terms: 23 us with blocks of 512 threads, 34 with 1,024)
  const int most = N < SUM_NORM_MANY || units > 512 * 8 ? 1024 : (units <= 512 ? 256 : 512);
  const int per = (units + most - 1) / most;
  const int slots = per <= 1 ? 1 : (per <= 2 ? 2 : (per <= 4 ? 4 : (per <= 8 ? 8 : 32)));
  const int threads = ((units + slots - 1) / slots + 63) / 64 * 64;
#define LAUNCH(TA, TB, TC, TERMS, VEC, PER)                                                                             \
  hipLaunchKernelGGL((sum_norm_kernel<TA, TB, TC, TERMS, VEC, PER>), dim3(N), dim3(threads), 0, stream, (float*)h, alpha, \
                     a, b, (const float*)w, (const float*)bias, eps, (TC*)copy, H)
#define BY_PER(TA, TB, TC, TERMS, VEC)                         \
  {                                                            \
    if (slots == 1) LAUNCH(TA, TB, TC, TERMS, VEC, 1);         \
    else if (slots == 2) LAUNCH(TA, TB, TC, TERMS, VEC, 2);    \
    else if (slots == 4) LAUNCH(TA, TB, TC, TERMS, VEC, 4);    \
    else if (slots == 8) LAUNCH(TA, TB, TC, TERMS, VEC, 8);    \
    else LAUNCH(TA, TB, TC, TERMS, 1, 32);                     \
  }
#define BY_VEC(TA, TB, TC, TERMS) { if (vec) BY_PER(TA, TB, TC, TERMS, 4) else BY_PER(TA, TB, TC, TERMS, 1) }
#define BY_TERMS(TC)                                                              \
  {                                                                               \
    if (!t2) { if (dtype1 == 0) BY_VEC(float, float, TC, 1) else BY_VEC(bf16_t, float, TC, 1) } \
    else if (dtype1 == 0 && dtype2 == 0) BY_VEC(float, float, TC, 2)              \
    else if (dtype1 == 0) BY_VEC(float, bf16_t, TC, 2)                            \
    else if (dtype2 == 0) BY_VEC(bf16_t, float, TC, 2)                            \
    else BY_VEC(bf16_t, bf16_t, TC, 2)                                            \
  }
  if (copy_dtype == 1) BY_TERMS(bf16_t) else BY_TERMS(float)
#undef BY_TERMS
#undef BY_VEC
#undef BY_PER
#undef LAUNCH
  return qvl_launch_status();
}

// ---------------------------------------------------------------------------------------
// out[n, c] = gelu(z[n, c]) * table[ids[n], first + c]    (gelu in its tanh form)
// ---------------------------------------------------------------------------------------
template <typename TZ, typename TT>
__global__ __launch_bounds__(256) void gelu_rows_kernel(const TZ* __restrict__ z, long long z_stride,
                                                        const TT* __restrict__ table, long long table_stride, int first,
                                                        const int* __restrict__ ids, TT* __restrict__ out, long long total,
                                                        int C) {
  const long long i = (long long)blockIdx.x * blockDim.x + threadIdx.x;
  if (i >= total) return;
  const long long n = i / C;
  const int c = (int)(i % C);
  stf<TT>(out + i, gate_act(ldf<TZ>(z + n * z_stride + c), 1) * ldf<TT>(table + (size_t)ids[n] * table_stride + first + c));
}

extern "C" int qvl_gelu_rows(const void* z, int z_dtype, long long z_stride, const void* table, int dtype,
                             long long table_stride, int first, const void* ids, void* out, int N, int C,
                             hipStream_t stream) {
  if (N <= 0) return QVL_OK;
  if (C <= 0 || first < 0 || z_stride < C || table_stride < first + C || !z || !table || !ids || !out) return QVL_ERR_SHAPE;
  const long long total = (long long)N * C;
  if ((total + 255) / 256 > 0x7fffffffLL) return QVL_ERR_LIMIT;
#define LAUNCH(TZ, TT)                                                                                             \
  hipLaunchKernelGGL((gelu_rows_kernel<TZ, TT>), dim3((unsigned)((total + 255) / 256)), dim3(256), 0, stream,      \
                     (const TZ*)z, z_stride, (const TT*)table, table_stride, first, (const int*)ids, (TT*)out, total, C)
  if (z_dtype == 0 && dtype == 0) LAUNCH(float, float);
  else if (z_dtype == 0 && dtype == 1) LAUNCH(float, bf16_t);
  else if (z_dtype == 1 && dtype == 1) LAUNCH(bf16_t, bf16_t);
  else return QVL_ERR_DTYPE;
#undef LAUNCH
  return qvl_launch_status();
}
