// A residual stream of several copies that every sublayer mixes anew (hyper-connections), and the norm of what the
// next sublayer reads.  One pass over a token's row:
//   y   = the pending addend, or factor * (rms(y1) g1 + rms(y2) g2) of two of them (each normed over the row)
//   x_t = sum_s mix[s, t] x_s + out[t] y          every copy from the copies as they were (skipped without `mix`)
//   u   = sum_t read[t] x_t                       (`read` null: the plain sum of the copies)
//   h   = norm(u): every one of `groups` consecutive parts of the row divided by its own root mean square
//         (eps inside the root), times w
// The copies are float32 [N, copies, W]; while they all equal the embedding's output the source is that [N, W] with a
// copy stride of zero.  Compiled per number of copies (-DHC_S=...).
//
// For a step of single tokens (one per request) the kernel also takes h the rest of the way (`shift` or `mu`
// given): h <- h + (h' - h) shift with h' the request's previous h, and, per row m of mu,
// out_m = h + (h'' - h) mu_m with h'' the previous value of the h so shifted; both come from the request's state
// rows and replace them.  Longer runs go through csrc/previous_token.hip, which does the same arithmetic.
//
// One block per row.  The order of every sum depends on the sizes alone.
#include "common.h"

#ifndef HC_S
#define HC_S 4
#endif

struct JoinArgs {
  const float* src;            // copies (or the embedding's output) before
  long long src_row, src_copy; // strides in values
  float* dst;                  // [N, HC_S, W] the copies afterwards (may be src), or null
  const float* mix;            // [HC_S, HC_S] (from, to), or null: nothing joins
  const float* out;            // [HC_S]
  const void* y1;
  const void* y2;              // null: y1 is added as it is
  int y1_dtype, y2_dtype, y1_slabs, y2_slabs;
  long long slab_stride;
  const float* g1;
  const float* g2;
  float eps_pair, factor;
  const float* read;           // [HC_S] or null
  const float* w;              // [W]
  int groups;
  float eps;
  void* h;                     // [M, W], or [mixes, M, W]
  const int* rows;             // row m is made from token rows[m] (then dst is null), or null
  int W;
  const float* shift;          // [W] or null
  float* prev;                 // [slots, W]
  const float* mu;             // [mixes, W] or null
  int mixes;
  float* prev_shifted;         // [slots, W]
  const int* req_slots;        // [N]: token n is request n's only one
  long long mix_stride;
};

template <int VEC> struct Cols { float v[VEC]; };
template <int VEC> __device__ __forceinline__ Cols<VEC> ldc(const float* p) {
  Cols<VEC> o;
  if constexpr (VEC == 4) {
    const float4 t = *reinterpret_cast<const float4*>(p);
    o.v[0] = t.x; o.v[1] = t.y; o.v[2] = t.z; o.v[3] = t.w;
  } else {
    o.v[0] = *p;
  }
  return o;
}
template <int VEC> __device__ __forceinline__ void stc(float* p, const Cols<VEC>& a) {
  if constexpr (VEC == 4) *reinterpret_cast<float4*>(p) = float4{a.v[0], a.v[1], a.v[2], a.v[3]};
  else *p = a.v[0];
}
template <int VEC> __device__ __forceinline__ Cols<VEC> ldc16(const bf16_t* p) {
  Cols<VEC> o;
  if constexpr (VEC == 4) {
    const uint2 t = *reinterpret_cast<const uint2*>(p);
    o.v[0] = __uint_as_float(t.x << 16); o.v[1] = __uint_as_float(t.x & 0xffff0000u);
    o.v[2] = __uint_as_float(t.y << 16); o.v[3] = __uint_as_float(t.y & 0xffff0000u);
  } else {
    o.v[0] = bf16_to_f32(*p);
  }
  return o;
}
template <int VEC, typename T> __device__ __forceinline__ void st_as(T* p, const Cols<VEC>& a) {
  if constexpr (sizeof(T) == 4) {
    stc<VEC>(reinterpret_cast<float*>(p), a);
  } else if constexpr (VEC == 4) {
    uint2 o;
    o.x = (uint32_t)f32_to_bf16(a.v[0]) | ((uint32_t)f32_to_bf16(a.v[1]) << 16);
    o.y = (uint32_t)f32_to_bf16(a.v[2]) | ((uint32_t)f32_to_bf16(a.v[3]) << 16);
    *reinterpret_cast<uint2*>(p) = o;
  } else {
    *p = f32_to_bf16(a.v[0]);
  }
}
// columns c .. of an addend: float32 slabs added in order, or bfloat16
template <int VEC>
__device__ __forceinline__ Cols<VEC> ld_addend(const void* y, int dtype, int slabs, long long slab_stride, size_t at) {
  if (dtype) return ldc16<VEC>(reinterpret_cast<const bf16_t*>(y) + at);
  const float* p = reinterpret_cast<const float*>(y) + at;
  Cols<VEC> a = ldc<VEC>(p);
  // eight slabs' loads are on their way together (past the last: slab 0 again, not counted); the sum keeps the order
  for (int s0 = 1; s0 < slabs; s0 += 8) {
    Cols<VEC> b[8];
#pragma unroll
    for (int s = 0; s < 8; ++s) b[s] = ldc<VEC>(p + (size_t)(s0 + s < slabs ? s0 + s : 0) * slab_stride);
#pragma unroll
    for (int s = 0; s < 8; ++s)
#pragma unroll
      for (int k = 0; k < VEC; ++k) a.v[k] += s0 + s < slabs ? b[s].v[k] : 0.f;
  }
  return a;
}

// VPT vectors of VEC neighbouring columns a thread.  lds: one partial sum per vector, then one value per group.
template <int VEC, int VPT, typename TO>
__global__ __launch_bounds__(1024) void join_norm_kernel(JoinArgs a) {
  extern __shared__ float lds[];
  __shared__ float red[17];
  const int m = blockIdx.x, n = a.rows ? a.rows[m] : m;
  const int tid = threadIdx.x, nvec = a.W / VEC;
  const size_t row = (size_t)n * a.W;
  // a vector past the row's end reads its start and counts as nothing
  int col[VPT];
  bool ok[VPT];
#pragma unroll
  for (int j = 0; j < VPT; ++j) {
    const int i = tid + j * blockDim.x;
    ok[j] = i < nvec;
    col[j] = ok[j] ? i * VEC : 0;
  }
  // with one vector a thread the copies are asked for before anything is waited for
  constexpr bool EARLY = VPT == 1 && HC_S * VEC <= 32;
  Cols<VEC> early[EARLY ? HC_S : 1];
  if constexpr (EARLY) {
#pragma unroll
    for (int s = 0; s < HC_S; ++s) early[s] = ldc<VEC>(a.src + (size_t)n * a.src_row + (size_t)s * a.src_copy + col[0]);
  }
  Cols<VEC> y[VPT];
  if (a.mix) {
#pragma unroll
    for (int j = 0; j < VPT; ++j) y[j] = ld_addend<VEC>(a.y1, a.y1_dtype, a.y1_slabs, a.slab_stride, row + col[j]);
    if (a.y2) {
      Cols<VEC> z[VPT];
      float s1 = 0.f, s2 = 0.f;
#pragma unroll
      for (int j = 0; j < VPT; ++j) {
        z[j] = ld_addend<VEC>(a.y2, a.y2_dtype, a.y2_slabs, a.slab_stride, row + col[j]);
#pragma unroll
        for (int k = 0; k < VEC; ++k) {
          s1 += ok[j] ? y[j].v[k] * y[j].v[k] : 0.f;
          s2 += ok[j] ? z[j].v[k] * z[j].v[k] : 0.f;
        }
      }
      const float r1 = 1.0f / sqrtf(block_sum(s1, red) / (float)a.W + a.eps_pair);
      const float r2 = 1.0f / sqrtf(block_sum(s2, red) / (float)a.W + a.eps_pair);
#pragma unroll
      for (int j = 0; j < VPT; ++j) {
        const Cols<VEC> w1 = ldc<VEC>(a.g1 + col[j]), w2 = ldc<VEC>(a.g2 + col[j]);
#pragma unroll
        for (int k = 0; k < VEC; ++k) y[j].v[k] = a.factor * ((y[j].v[k] * r1) * w1.v[k] + (z[j].v[k] * r2) * w2.v[k]);
      }
    }
  }
  Cols<VEC> u[VPT];
#pragma unroll
  for (int j = 0; j < VPT; ++j) {
    Cols<VEC> x[HC_S];
#pragma unroll
    for (int s = 0; s < HC_S; ++s) {
      if constexpr (EARLY) x[s] = early[s];
      else x[s] = ldc<VEC>(a.src + (size_t)n * a.src_row + (size_t)s * a.src_copy + col[j]);
    }
#pragma unroll
    for (int k = 0; k < VEC; ++k) u[j].v[k] = 0.f;
#pragma unroll
    for (int t = 0; t < HC_S; ++t) {
      Cols<VEC> xt = x[t];
      if (a.mix) {
        const float share = a.out[t];
#pragma unroll
        for (int k = 0; k < VEC; ++k) {
          float v = a.mix[t] * x[0].v[k];
#pragma unroll
          for (int s = 1; s < HC_S; ++s) v += a.mix[s * HC_S + t] * x[s].v[k];
          xt.v[k] = v + share * y[j].v[k];
        }
        if (a.dst && ok[j]) stc<VEC>(a.dst + ((size_t)n * HC_S + t) * a.W + col[j], xt);
      }
      const float weight = a.read ? a.read[t] : 1.0f;
#pragma unroll
      for (int k = 0; k < VEC; ++k) u[j].v[k] += weight * xt.v[k];
    }
  }
  // sums of squares of the groups: a vector lies in one group; a wave adds up a group's vectors
  float* gsum = lds + nvec;
#pragma unroll
  for (int j = 0; j < VPT; ++j) {
    float ss = 0.f;
#pragma unroll
    for (int k = 0; k < VEC; ++k) ss += u[j].v[k] * u[j].v[k];
    if (ok[j]) lds[col[j] / VEC] = ss;
  }
  __syncthreads();
  const int per = nvec / a.groups;
  for (int g = tid >> 6; g < a.groups; g += blockDim.x >> 6) {
    float ss = 0.f;
    for (int i = tid & 63; i < per; i += 64) ss += lds[g * per + i];
    ss = wave_sum(ss);
    if ((tid & 63) == 0) gsum[g] = 1.0f / sqrtf(ss / (float)(per * VEC) + a.eps);
  }
  __syncthreads();
  const size_t slot = (a.shift || a.mu) ? (size_t)a.req_slots[n] * a.W : 0;
#pragma unroll
  for (int j = 0; j < VPT; ++j) {
    if (!ok[j]) continue;
    const int c = col[j];
    const float rs = gsum[(c / VEC) / per];
    const Cols<VEC> w = ldc<VEC>(a.w + c);
    Cols<VEC> h;
#pragma unroll
    for (int k = 0; k < VEC; ++k) h.v[k] = (u[j].v[k] * rs) * w.v[k];
    if (a.shift) {
      const Cols<VEC> p = ldc<VEC>(a.prev + slot + c), sh = ldc<VEC>(a.shift + c);
      stc<VEC>(a.prev + slot + c, h);
#pragma unroll
      for (int k = 0; k < VEC; ++k) h.v[k] = h.v[k] + (p.v[k] - h.v[k]) * sh.v[k];
    }
    TO* o = reinterpret_cast<TO*>(a.h) + (size_t)m * a.W + c;
    if (a.mu) {
      const Cols<VEC> p = ldc<VEC>(a.prev_shifted + slot + c);
      stc<VEC>(a.prev_shifted + slot + c, h);
      for (int i = 0; i < a.mixes; ++i) {
        const Cols<VEC> mu = ldc<VEC>(a.mu + (size_t)i * a.W + c);
        Cols<VEC> q;
#pragma unroll
        for (int k = 0; k < VEC; ++k) q.v[k] = h.v[k] + (p.v[k] - h.v[k]) * mu.v[k];
        st_as<VEC, TO>(o + (size_t)i * a.mix_stride, q);
      }
    } else {
      st_as<VEC, TO>(o, h);
    }
  }
}

extern "C" int qvl_hyper_copies() { return HC_S; }

// M rows of W values (W / groups whole).  y*_dtype 0 float32 (slabs `slab_stride` values apart), 1 bfloat16;
// out_dtype 0 float32, 1 bfloat16.  A step through `shift` or `mu` has one token per request and no `rows`.
extern "C" int qvl_hyper_join_norm(const void* src, long long src_row, long long src_copy, void* dst, const void* mix,
                                   const void* out, const void* y1, int y1_dtype, int y1_slabs, const void* y2,
                                   int y2_dtype, int y2_slabs, long long slab_stride, const void* g1, const void* g2,
                                   float eps_pair, float factor, const void* read, const void* w, int groups, float eps,
                                   void* h, int out_dtype, const void* rows, int M, int W, const void* shift, void* prev,
                                   const void* mu, int mixes, void* prev_shifted, const void* req_slots,
                                   long long mix_stride, hipStream_t stream) {
  if (M <= 0) return QVL_OK;
  if (!src || !w || !h || W <= 0 || groups <= 0 || W % groups) return QVL_ERR_SHAPE;
  if (mix && (!out || !y1 || y1_slabs < 1 || (y1_slabs > 1 && y1_dtype))) return QVL_ERR_SHAPE;
  if (y2 && (!mix || !g1 || !g2 || y2_slabs < 1 || (y2_slabs > 1 && y2_dtype))) return QVL_ERR_SHAPE;
  if ((dst && (!mix || rows)) || (mu && mixes < 1) || ((shift || mu) && (rows || !req_slots)) || (shift && !prev) ||
      (mu && !prev_shifted))
    return QVL_ERR_SHAPE;
  JoinArgs a;
  a.src = (const float*)src; a.src_row = src_row; a.src_copy = src_copy; a.dst = (float*)dst; a.mix = (const float*)mix;
  a.out = (const float*)out; a.y1 = y1; a.y2 = y2; a.y1_dtype = y1_dtype; a.y2_dtype = y2_dtype; a.y1_slabs = y1_slabs;
  a.y2_slabs = y2_slabs; a.slab_stride = slab_stride; a.g1 = (const float*)g1; a.g2 = (const float*)g2;
  a.eps_pair = eps_pair; a.factor = factor; a.read = (const float*)read; a.w = (const float*)w; a.groups = groups;
  a.eps = eps; a.h = h; a.rows = (const int*)rows; a.W = W; a.shift = (const float*)shift; a.prev = (float*)prev;
  a.mu = (const float*)mu; a.mixes = mixes; a.prev_shifted = (float*)prev_shifted; a.req_slots = (const int*)req_slots;
  a.mix_stride = mix_stride;
  const uintptr_t addresses = (uintptr_t)src | (uintptr_t)dst | (uintptr_t)y1 | (uintptr_t)y2 | (uintptr_t)g1 | (uintptr_t)g2 |
                              (uintptr_t)w | (uintptr_t)h | (uintptr_t)shift | (uintptr_t)prev | (uintptr_t)mu | (uintptr_t)prev_shifted;
  const bool vec = (W / groups) % 4 == 0 && src_row % 4 == 0 && src_copy % 4 == 0 && slab_stride % 4 == 0 &&
                   mix_stride % 4 == 0 && addresses % 16 == 0;
  const int nvec = vec ? W / 4 : W;
  if (nvec > (vec ? 4096 : 8192)) return QVL_ERR_LIMIT;
  const size_t bytes = (size_t)(nvec + groups) * 4;
#define LAUNCH(VEC, VPT)                                                                                             \
  {                                                                                                                  \
    const int threads = ((nvec + VPT - 1) / VPT + 63) / 64 * 64;                                                     \
    if (out_dtype == 0) hipLaunchKernelGGL((join_norm_kernel<VEC, VPT, float>), dim3(M), dim3(threads), bytes, stream, a); \
    else if (out_dtype == 1) hipLaunchKernelGGL((join_norm_kernel<VEC, VPT, bf16_t>), dim3(M), dim3(threads), bytes, stream, a); \
    else return QVL_ERR_DTYPE;                                                                                       \
    return qvl_launch_status();                                                                                      \
  }
  if (vec && nvec <= 1024) LAUNCH(4, 1)
  if (vec) LAUNCH(4, 4)
  if (nvec <= 1024) LAUNCH(1, 1)
  LAUNCH(1, 8)
#undef LAUNCH
}
