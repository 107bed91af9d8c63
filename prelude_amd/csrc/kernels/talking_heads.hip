// What stands in front of attention whose heads' scores are mixed, score_h <- sum_g T[h, g] score_g.
//
// With G key heads (query head g reads key head kv(g)), sum_g T[h, g] (q_g . k_kv(g)) = sum_c (sum_{g: kv(g) = c} T[h, g] q_g)
// . k_c: the mixing moves to the query side.  Head h gets one query over the keys of ALL key heads side by side,
// q'_h = [q'_(h,0) | .. | q'_(h,G-1)], and the attention behind it has one key head of width G * dim, shared by all query
// heads, beside G value heads.
//
//   pa_talking_prepare   a token's queries, keys and values out of the merged projection: biases; queries and keys over
//                        their own root mean square per head, times a weight shared by the heads; the first `rot`
//                        dimensions turned in pairs by position; the queries mixed (all of this in 32-bit, rounded once)
//                        -> q_out [T, nh, nkv * hd]; keys -> K [page, offset, nkv * hd]; values, over their own root mean
//                        square when `value_norm`, -> V [page, nkv, vd, offset].
#include "common.h"
#include "api.h"

namespace pa {

constexpr int kTalkThreads = 256;
constexpr int kTalkWaves = kTalkThreads / kWave;
constexpr int kTalkMaxHead = 256;                 // widest key or value head
constexpr int kTalkPer = kTalkMaxHead / kWave;    // elements of a head a lane holds

// A workgroup a (token, key head c): the queries of the heads that read c, key head c and value head c; then the columns c of
// every head's mixed query.  LDS: those queries, normed and rotated [nh / nkv, hd], and their columns of the mixing matrix.
template <typename T>
__global__ __launch_bounds__(kTalkThreads) void talking_prepare_kernel(
    const T* __restrict__ p, size_t stride, int q_off, int k_off, int v_off, const float* __restrict__ q_bias,
    const float* __restrict__ k_bias, const float* __restrict__ v_bias, const float* __restrict__ q_weight,
    const float* __restrict__ k_weight, const float* __restrict__ inv_freq, const int* __restrict__ positions,
    const float* __restrict__ talk, const int* __restrict__ slots, T* __restrict__ q_out, T* __restrict__ k_cache,
    T* __restrict__ v_cache, int nh, int nkv, int hd, int vd, int rot, int value_norm, int page_size, float eps) {
  extern __shared__ float qs[];
  const int group = nh / nkv, kd = nkv * hd;
  float* ts = qs + group * hd;                    // [group][nh]
  const int wave = threadIdx.x / kWave, lane = threadIdx.x % kWave;
  const size_t t = blockIdx.x;
  const int c = blockIdx.y;
  const T* row = p + t * stride;
  const int slot = slots ? slots[t] : -1;
  const float pos = (float)positions[t];
  const size_t page = slot >= 0 ? slot / page_size : 0, off = slot >= 0 ? slot % page_size : 0;
  for (int i = threadIdx.x; i < group * nh; i += kTalkThreads) ts[i] = talk[(size_t)(i % nh) * nh + c * group + i / nh];
  for (int u = wave; u < group + 2; u += kTalkWaves) {      // a wavefront a head; a lane holds two neighbouring elements at a time
    if (u >= group && slot < 0) break;
    const bool is_q = u < group, is_v = u == group + 1;
    const int h = is_q ? c * group + u : c;
    const int width = is_v ? vd : hd;
    const T* src = row + (is_q ? q_off : is_v ? v_off : k_off) + (size_t)h * width;
    const float* bias = is_q ? q_bias : is_v ? v_bias : k_bias;
    const float* w = is_q ? q_weight : is_v ? nullptr : k_weight;
    float x[kTalkPer];
    float ss = 0.f;
#pragma unroll
    for (int e = 0; e < kTalkPer / 2; ++e)
#pragma unroll
      for (int b = 0; b < 2; ++b) {
        const int i = 2 * (lane + kWave * e) + b;
        float v = 0.f;
        if (i < width) {
          v = to_f32(src[i]);
          if (bias) v += bias[(size_t)h * width + i];
        }
        x[2 * e + b] = v;
        ss += v * v;
      }
    const bool normed = is_v ? value_norm != 0 : w != nullptr;
    const float inv = normed ? 1.0f / sqrtf(wave_sum(ss) / (float)width + eps) : 1.0f;
#pragma unroll
    for (int e = 0; e < kTalkPer / 2; ++e) {
      const int i = 2 * (lane + kWave * e);
      if (i >= width) continue;
      const bool two = i + 1 < width;
      float u0 = x[2 * e] * inv, u1 = x[2 * e + 1] * inv;
      if (w) {
        u0 *= w[i];
        if (two) u1 *= w[i + 1];
      }
      if (is_v) {
        T* dst = v_cache + ((page * nkv + c) * vd + i) * page_size + off;
        dst[0] = from_f32<T>(u0);
        if (two) dst[page_size] = from_f32<T>(u1);
        continue;
      }
      if (i < rot) {                                        // rot is even: the pair turns whole
        float sn, cs;
        sincosf(pos * inv_freq[i / 2], &sn, &cs);
        const float v0 = u0 * cs - u1 * sn;
        u1 = u1 * cs + u0 * sn;
        u0 = v0;
      }
      if (is_q) {
        qs[u * hd + i] = u0;
        if (two) qs[u * hd + i + 1] = u1;
      } else {
        T* dst = k_cache + (page * page_size + off) * (size_t)kd + (size_t)c * hd + i;
        dst[0] = from_f32<T>(u0);
        if (two) dst[1] = from_f32<T>(u1);
      }
    }
  }
  __syncthreads();
  T* dst = q_out + t * (size_t)nh * kd + (size_t)c * hd;
  if (hd % 8 == 0) {                                        // sixteen or thirty-two bytes a thread
    typedef T vec8 __attribute__((ext_vector_type(8)));
    for (int i = threadIdx.x; i < nh * hd / 8; i += kTalkThreads) {
      const int h = i / (hd / 8), d = 8 * (i % (hd / 8));
      float acc[8] = {};
      for (int g = 0; g < group; ++g) {
        const float m = ts[g * nh + h];
#pragma unroll
        for (int e = 0; e < 8; ++e) acc[e] = fmaf(m, qs[g * hd + d + e], acc[e]);
      }
      vec8 v;
#pragma unroll
      for (int e = 0; e < 8; ++e) v[e] = from_f32<T>(acc[e]);
      *reinterpret_cast<vec8*>(dst + (size_t)h * kd + d) = v;
    }
    return;
  }
  for (int i = threadIdx.x; i < nh * hd; i += kTalkThreads) {
    const int h = i / hd, d = i % hd;
    float acc = 0.f;
    for (int g = 0; g < group; ++g) acc = fmaf(ts[g * nh + h], qs[g * hd + d], acc);
    dst[(size_t)h * kd + d] = from_f32<T>(acc);
  }
}

}  // namespace pa

using namespace pa;

extern "C" int pa_talking_prepare(void* stream, int dtype, const void* p, long stride, int q_off, int k_off, int v_off,
                                  const float* q_bias, const float* k_bias, const float* v_bias, const float* q_weight,
                                  const float* k_weight, const float* inv_freq, const int* positions, const float* talk,
                                  const int* slots, void* q_out, void* k_cache, void* v_cache, int tokens, int nh, int nkv, int hd,
                                  int vd, int rot, int value_norm, int page_size, float eps) {
  if (tokens == 0) return 0;
  PA_REQUIRE(tokens > 0 && nh > 0 && nkv > 0 && nh % nkv == 0 && hd > 0 && vd > 0, "talking_prepare: bad sizes tokens=%d heads=%d over "
             "%d of %d and %d", tokens, nh, nkv, hd, vd);
  PA_REQUIRE(rot >= 0 && rot <= hd && rot % 2 == 0 && (rot == 0 || inv_freq) && positions && talk && q_out,
             "talking_prepare: %d rotated dimensions of %d, or a tensor is missing", rot, hd);
  PA_REQUIRE(q_off >= 0 && k_off >= 0 && v_off >= 0 && q_off + (long)nh * hd <= stride && k_off + (long)nkv * hd <= stride &&
             v_off + (long)nkv * vd <= stride, "talking_prepare: the columns do not fit the row of %ld", stride);
  PA_REQUIRE(!slots || (k_cache && v_cache && page_size > 0), "talking_prepare: slots without caches");
  PA_REQUIRE(hd <= kTalkMaxHead && vd <= kTalkMaxHead, "talking_prepare: heads of %d or values of %d are wider than %d", hd, vd, kTalkMaxHead);
  const size_t lds = (size_t)(nh / nkv) * (hd + nh) * sizeof(float);
  PA_REQUIRE(lds <= 65536, "talking_prepare: %d heads of %d take %zu bytes of LDS, more than 65536", nh, hd, lds);
  hipStream_t st = (hipStream_t)stream;
#define PA_TALK(T)                                                                                                              \
  hipLaunchKernelGGL(talking_prepare_kernel<T>, dim3(tokens, nkv), dim3(kTalkThreads), lds, st, (const T*)p, (size_t)stride, q_off,   \
                     k_off, v_off, q_bias, k_bias, v_bias, q_weight, k_weight, inv_freq, positions, talk, slots, (T*)q_out,      \
                     (T*)k_cache, (T*)v_cache, nh, nkv, hd, vd, rot, value_norm, page_size, eps)
  if (dtype == kF32) PA_TALK(float);
  else if (dtype == kBF16) PA_TALK(bf16);
  else return pa::fail("talking_prepare: unknown element type code %d", dtype);
#undef PA_TALK
  return check_launch("talking_prepare");
}
