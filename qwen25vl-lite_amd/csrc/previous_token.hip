// What a token takes from the one before it in its sequence: a table row picked by both their ids, and mixes
// of their rows.  A request's last id (plus one; zero: no token yet) and last rows are its state, read by the first
// tokens of its next run and replaced at the end of this one.
//
// Grids have N + R rows: below N a token that stands far enough into its run to need nothing of the state; the last R
// rows are requests, whose threads form the run's first tokens from the old state and then write the new one, so
// nobody else reads or writes a request's state in this launch.
#include "common.h"

// ---------------------------------------------------------------------------------------
// out[n, :] = table[id[n], :] + pairs[row, :],  row = (id[n-1] mul_prev + id[n] mul_cur) mod buckets, or row number
// `buckets` for a sequence's first token
// ---------------------------------------------------------------------------------------
template <typename T>
__global__ __launch_bounds__(256) void bigram_gather_kernel(const int* __restrict__ ids, const T* __restrict__ table,
                                                            const T* __restrict__ pairs, int* __restrict__ last_id,
                                                            const int* __restrict__ cu_q, const int* __restrict__ req_slots,
                                                            const int* __restrict__ token_req, float* __restrict__ out,
                                                            int N, int H, int V, int buckets, long long mul_prev,
                                                            long long mul_cur) {
  int t, prev;      // prev: the id before, or -1
  int req = -1;
  if ((int)blockIdx.x < N) {
    t = blockIdx.x;
    if (t == cu_q[token_req[t]]) return;      // the request's row forms it
    prev = ids[t - 1];
  } else {
    req = blockIdx.x - N;
    t = cu_q[req];
    if (t >= cu_q[req + 1]) return;
    prev = last_id[req_slots[req]] - 1;
  }
  __syncthreads();                            // everybody has read the state before it is replaced
  if (req >= 0 && threadIdx.x == 0) last_id[req_slots[req]] = ids[cu_q[req + 1] - 1] + 1;
  int id = ids[t];
  id = id < 0 ? 0 : (id >= V ? V - 1 : id);   // ids are validated on the host; never read outside the table
  long long row = buckets;
  if (prev >= 0) {
    row = ((long long)prev * mul_prev + (long long)id * mul_cur) % buckets;
    if (row < 0) row += buckets;
  }
  const T* a = table + (size_t)id * H;
  const T* b = pairs + (size_t)row * H;
  float* o = out + (size_t)t * H;
  for (int i = threadIdx.x; i < H; i += blockDim.x) o[i] = ldf<T>(a + i) + ldf<T>(b + i);
}

// table [V, H], pairs [buckets + 1, H] of dtype (0 float32, 1 bfloat16); last_id int32 [slots]; out float32 [N, H].
extern "C" int qvl_bigram_gather(const void* ids, const void* table, const void* pairs, void* last_id, const void* cu_q,
                                 const void* req_slots, const void* token_req, void* out, int N, int R, int H, int V,
                                 int buckets, long long mul_prev, long long mul_cur, int dtype, hipStream_t stream) {
  if (N <= 0) return QVL_OK;
  if (R <= 0 || H <= 0 || V <= 0 || buckets <= 0 || !last_id || !cu_q || !req_slots || !token_req) return QVL_ERR_SHAPE;
  const dim3 grid((unsigned)(N + R));
#define LAUNCH(T)                                                                                                    \
  hipLaunchKernelGGL(bigram_gather_kernel<T>, grid, dim3(256), 0, stream, (const int*)ids, (const T*)table,           \
                     (const T*)pairs, (int*)last_id, (const int*)cu_q, (const int*)req_slots, (const int*)token_req, \
                     (float*)out, N, H, V, buckets, mul_prev, mul_cur)
  if (dtype == 0) LAUNCH(float);
  else if (dtype == 1) LAUNCH(bf16_t);
  else return QVL_ERR_DTYPE;
#undef LAUNCH
  return qvl_launch_status();
}

// ---------------------------------------------------------------------------------------
// Mixes of a token's row with the one before it, h' (zeros before the first):
//   g = h + (h' - h) shift                      (without `shift`: g = h)
//   out_m = g + (g' - g) mu_m  for every row m of mu, or, without mu, out = g
// state rows: prev [slots, W] (the last h, with `shift`), prev_mixed [slots, W] (the last g, with `mu`).
// A thread owns VEC neighbouring columns of a token (or of a request).
// ---------------------------------------------------------------------------------------
template <int VEC> struct Vals { float v[VEC]; };
template <int VEC, typename T> __device__ __forceinline__ Vals<VEC> ld_vals(const T* p) {
  Vals<VEC> o;
  if constexpr (VEC == 4 && sizeof(T) == 4) {
    const float4 t = *reinterpret_cast<const float4*>(p);
    o.v[0] = t.x; o.v[1] = t.y; o.v[2] = t.z; o.v[3] = t.w;
  } else if constexpr (VEC == 4) {
    const uint2 t = *reinterpret_cast<const uint2*>(p);
    o.v[0] = __uint_as_float(t.x << 16); o.v[1] = __uint_as_float(t.x & 0xffff0000u);
    o.v[2] = __uint_as_float(t.y << 16); o.v[3] = __uint_as_float(t.y & 0xffff0000u);
  } else {
    o.v[0] = ldf<T>(p);
  }
  return o;
}
template <int VEC, typename T> __device__ __forceinline__ void st_vals(T* p, const Vals<VEC>& a) {
  if constexpr (VEC == 4 && sizeof(T) == 4) {
    *reinterpret_cast<float4*>(p) = float4{a.v[0], a.v[1], a.v[2], a.v[3]};
  } else if constexpr (VEC == 4) {
    uint2 o;
    o.x = (uint32_t)f32_to_bf16(a.v[0]) | ((uint32_t)f32_to_bf16(a.v[1]) << 16);
    o.y = (uint32_t)f32_to_bf16(a.v[2]) | ((uint32_t)f32_to_bf16(a.v[3]) << 16);
    *reinterpret_cast<uint2*>(p) = o;
  } else {
    stf<T>(p, a.v[0]);
  }
}
template <int VEC> __device__ __forceinline__ Vals<VEC> towards(const Vals<VEC>& h, const Vals<VEC>& p, const Vals<VEC>& w) {
  Vals<VEC> o;
#pragma unroll
  for (int k = 0; k < VEC; ++k) o.v[k] = h.v[k] + (p.v[k] - h.v[k]) * w.v[k];
  return o;
}

template <int VEC, typename TI, typename TO>
__global__ __launch_bounds__(256) void token_mix_kernel(const TI* __restrict__ h, const float* __restrict__ shift,
                                                        float* __restrict__ prev, const float* __restrict__ mu, int mixes,
                                                        float* __restrict__ prev_mixed, const int* __restrict__ cu_q,
                                                        const int* __restrict__ req_slots, const int* __restrict__ token_req,
                                                        TO* __restrict__ out, long long mix_stride, int N, int W) {
  const int c = (blockIdx.y * blockDim.x + threadIdx.x) * VEC;
  if (c >= W) return;
  const int keep = (shift ? 1 : 0) + (mu ? 1 : 0);    // tokens of a run that need the state
  Vals<VEC> sh;
#pragma unroll
  for (int k = 0; k < VEC; ++k) sh.v[k] = 0.f;
  if (shift) sh = ld_vals<VEC>(shift + c);
  auto emit = [&](int t, const Vals<VEC>& g, const Vals<VEC>& before) {
    TO* o = out + (size_t)t * W + c;
    if (!mu) {
      st_vals<VEC, TO>(o, g);
      return;
    }
    for (int i = 0; i < mixes; ++i)
      st_vals<VEC, TO>(o + (size_t)i * mix_stride, towards<VEC>(g, before, ld_vals<VEC>(mu + (size_t)i * W + c)));
  };
  if ((int)blockIdx.x < N) {
    const int t = blockIdx.x;
    if (t - cu_q[token_req[t]] < keep) return;
    const TI* p = h + (size_t)t * W + c;
    const Vals<VEC> h0 = ld_vals<VEC>(p), h1 = ld_vals<VEC>(keep ? p - W : p), h2 = ld_vals<VEC>(keep == 2 ? p - 2 * (size_t)W : p);
    emit(t, shift ? towards<VEC>(h0, h1, sh) : h0, shift ? towards<VEC>(h1, h2, sh) : h1);
    return;
  }
  const int r = blockIdx.x - N, begin = cu_q[r], n = cu_q[r + 1] - begin;
  if (n <= 0) return;
  const size_t slot = (size_t)req_slots[r] * W + c;
  Vals<VEC> p, g_before;
#pragma unroll
  for (int k = 0; k < VEC; ++k) p.v[k] = g_before.v[k] = 0.f;
  if (shift) p = ld_vals<VEC>(prev + slot);
  if (mu) g_before = ld_vals<VEC>(prev_mixed + slot);
  const int first = n < keep ? n : keep;
  for (int i = 0; i < first; ++i) {
    const Vals<VEC> hi = ld_vals<VEC>(h + (size_t)(begin + i) * W + c);
    const Vals<VEC> g = shift ? towards<VEC>(hi, p, sh) : hi;
    emit(begin + i, g, g_before);
    p = hi;
    g_before = g;
  }
  if (n > first) {
    const Vals<VEC> last = ld_vals<VEC>(h + (size_t)(begin + n - 1) * W + c);
    if (mu) g_before = shift ? towards<VEC>(last, ld_vals<VEC>(h + (size_t)(begin + n - 2) * W + c), sh) : last;
    p = last;
  }
  if (shift) st_vals<VEC, float>(prev + slot, p);
  if (mu) st_vals<VEC, float>(prev_mixed + slot, g_before);
}

// h [N, W] of in_dtype; out [N, W], or [mixes, N, W] with mu, of out_dtype (0 float32, 1 bfloat16).
extern "C" int qvl_token_mix(const void* h, int in_dtype, const void* shift, void* prev, const void* mu, int mixes,
                             void* prev_mixed, const void* cu_q, const void* req_slots, const void* token_req, void* out,
                             int out_dtype, long long mix_stride, int N, int R, int W, hipStream_t stream) {
  if (N <= 0) return QVL_OK;
  if (R <= 0 || W <= 0 || !h || !out || !cu_q || !req_slots || !token_req || (!shift && !mu)) return QVL_ERR_SHAPE;
  if ((shift && !prev) || (mu && (!prev_mixed || mixes < 1))) return QVL_ERR_SHAPE;
  const uintptr_t addresses = (uintptr_t)h | (uintptr_t)shift | (uintptr_t)prev | (uintptr_t)mu | (uintptr_t)prev_mixed | (uintptr_t)out;
  const bool vec = W % 4 == 0 && mix_stride % 4 == 0 && addresses % 16 == 0;
  const int cols = vec ? 1024 : 256;
  if ((W + cols - 1) / cols > 65535) return QVL_ERR_LIMIT;
  const dim3 grid((unsigned)(N + R), (W + cols - 1) / cols);
#define LAUNCH(VEC, TI, TO)                                                                                          \
  hipLaunchKernelGGL((token_mix_kernel<VEC, TI, TO>), grid, dim3(256), 0, stream, (const TI*)h, (const float*)shift,  \
                     (float*)prev, (const float*)mu, mixes, (float*)prev_mixed, (const int*)cu_q,                     \
                     (const int*)req_slots, (const int*)token_req, (TO*)out, mix_stride, N, W)
#define BY_VEC(TI, TO) { if (vec) LAUNCH(4, TI, TO); else LAUNCH(1, TI, TO); }
  if (in_dtype == 0 && out_dtype == 0) BY_VEC(float, float)
  else if (in_dtype == 0 && out_dtype == 1) BY_VEC(float, bf16_t)
  else if (in_dtype == 1 && out_dtype == 1) BY_VEC(bf16_t, bf16_t)
  else return QVL_ERR_DTYPE;
#undef BY_VEC
#undef LAUNCH
  return qvl_launch_status();
}
