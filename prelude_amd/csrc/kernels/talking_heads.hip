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

// A workgroup a token.  LDS: the normed, rotated queries [nh, hd] and the mixing matrix [nh, nh].
template <typename T>
__global__ __launch_bounds__(kTalkThreads) void talking_prepare_kernel(
    const T* __restrict__ p, size_t stride, int q_off, int k_off, int v_off, const float* __restrict__ q_bias,
    const float* __restrict__ k_bias, const float* __restrict__ v_bias, const float* __restrict__ q_weight,
    const float* __restrict__ k_weight, const float* __restrict__ inv_freq, const int* __restrict__ positions,
    const float* __restrict__ talk, const int* __restrict__ slots, T* __restrict__ q_out, T* __restrict__ k_cache,
    T* __restrict__ v_cache, int nh, int nkv, int hd, int vd, int rot, int value_norm, int page_size, float eps) {
  extern __shared__ float qs[];
  float* ts = qs + nh * hd;
  const int wave = threadIdx.x / kWave, lane = threadIdx.x % kWave;
  const size_t t = blockIdx.x;
  const T* row = p + t * stride;
  const int slot = slots ? slots[t] : -1;
  const float pos = (float)positions[t];
  const size_t page = slot >= 0 ? slot / page_size : 0, off = slot >= 0 ? slot % page_size : 0;
  for (int i = threadIdx.x; i < nh * nh; i += kTalkThreads) ts[i] = talk[i];
  for (int u = wave; u < nh + 2 * nkv; u += kTalkWaves) {   // a wavefront a head
    if (u >= nh && slot < 0) break;
    if (u >= nh + nkv) {                                    // a value head
      const int c = u - nh - nkv;
      const T* src = row + v_off + (size_t)c * vd;
      const float* b = v_bias ? v_bias + (size_t)c * vd : nullptr;
      float inv = 1.f;
      if (value_norm) {
        float ss = 0.f;
        for (int i = lane; i < vd; i += kWave) {
          const float v = to_f32(src[i]) + (b ? b[i] : 0.f);
          ss += v * v;
        }
        inv = 1.0f / sqrtf(wave_sum(ss) / (float)vd + eps);
      }
      T* dst = v_cache + ((page * nkv + c) * vd) * page_size + off;
      for (int i = lane; i < vd; i += kWave) dst[(size_t)i * page_size] = from_f32<T>((to_f32(src[i]) + (b ? b[i] : 0.f)) * inv);
      continue;
    }
    const bool is_q = u < nh;
    const int h = is_q ? u : u - nh;
    const T* src = row + (is_q ? q_off : k_off) + (size_t)h * hd;
    const float* bias = is_q ? q_bias : k_bias;
    const float* b = bias ? bias + (size_t)h * hd : nullptr;
    const float* w = is_q ? q_weight : k_weight;
    float inv = 1.f;
    if (w) {
      float ss = 0.f;
      for (int i = lane; i < hd; i += kWave) {
        const float v = to_f32(src[i]) + (b ? b[i] : 0.f);
        ss += v * v;
      }
      inv = 1.0f / sqrtf(wave_sum(ss) / (float)hd + eps);
    }
    auto value = [&](int i) {
      const float v = (to_f32(src[i]) + (b ? b[i] : 0.f)) * inv;
      return w ? v * w[i] : v;
    };
    T* kdst = is_q ? nullptr : k_cache + (page * page_size + off) * ((size_t)nkv * hd) + (size_t)h * hd;
    auto put = [&](int i, float v) {
      if (is_q) qs[h * hd + i] = v;
      else kdst[i] = from_f32<T>(v);
    };
    for (int i = lane; i < rot / 2; i += kWave) {           // a lane a pair
      float s, c;
      sincosf(pos * inv_freq[i], &s, &c);
      const float x = value(2 * i), y = value(2 * i + 1);
      put(2 * i, x * c - y * s);
      put(2 * i + 1, y * c + x * s);
    }
    for (int i = rot + lane; i < hd; i += kWave) put(i, value(i));
  }
  __syncthreads();
  const int group = nh / nkv, kd = nkv * hd;
  T* dst = q_out + t * (size_t)nh * kd;
  for (int i = threadIdx.x; i < nh * kd; i += kTalkThreads) {
    const int h = i / kd, c = (i % kd) / hd, d = i % hd;
    float acc = 0.f;
    for (int g = 0; g < group; ++g) acc = fmaf(ts[h * nh + c * group + g], qs[(c * group + g) * hd + d], acc);
    dst[i] = from_f32<T>(acc);
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
  const size_t lds = ((size_t)nh * hd + (size_t)nh * nh) * sizeof(float);
  PA_REQUIRE(lds <= 65536, "talking_prepare: %d heads of %d take %zu bytes of LDS, more than 65536", nh, hd, lds);
  hipStream_t st = (hipStream_t)stream;
#define PA_TALK(T)                                                                                                              \
  hipLaunchKernelGGL(talking_prepare_kernel<T>, dim3(tokens), dim3(kTalkThreads), lds, st, (const T*)p, (size_t)stride, q_off,   \
                     k_off, v_off, q_bias, k_bias, v_bias, q_weight, k_weight, inv_freq, positions, talk, slots, (T*)q_out,      \
                     (T*)k_cache, (T*)v_cache, nh, nkv, hd, vd, rot, value_norm, page_size, eps)
  if (dtype == kF32) PA_TALK(float);
  else if (dtype == kBF16) PA_TALK(bf16);
  else return pa::fail("talking_prepare: unknown element type code %d", dtype);
#undef PA_TALK
  return check_launch("talking_prepare");
}
