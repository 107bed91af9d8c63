// A gated linear recurrence on every channel by itself (the real-gated linear recurrent unit of Griffin):
//
//   r = sigmoid(Wr[n] u_n + br), i = sigmoid(Wi[n] u_n + bi)      per block n of `size` channels
//   log a = -r rate,   S_t = a S_(t-1) + sqrt(1 - a^2) i u         rate = 8 softplus(lambda), one a channel
//   out = S * act(y + y_bias)                                      y the other branch, inside the merged projection
//
// u [tokens, width] of the engine's type; gates, decays and state are 32-bit; the state [slots, width] is zero at a
// request's start and carried from step to step.
//
//   pa_lru_gates   a and sqrt(1 - a^2) i u for every token; a sequence that brings one token is finished here (it is the only
//                  reader of its slot).  bfloat16: the blocks' products on the matrix cores, a wavefront 16 channels of both
//                  gates against up to 64 tokens, so that a lane holds both gates of its channels.
//   pa_lru_scan    the sequences of several tokens.  Chunks of 32 tokens run side by side: (1) where a sequence has more than one,
//                  every chunk makes its product of decays and its end from zero; (2) every chunk folds the chunks before it
//                  into the state it starts from, in order, and makes its outputs.
#include "common.h"
#include "api.h"
#include "attention_mfma_core.h"

namespace pa {

constexpr int kLruChunk = 32;
constexpr int kLruBatch = 16;    // tokens asked for together
constexpr int kLruThreads = 256;

// 1 - e^-x for x >= 0: below a quarter as its series (an alternating one whose eighth term is below 2^-30 of the first), which
// loses nothing where a is close to one
__device__ __forceinline__ float lru_one_minus_exp(float x, float e) {
  if (x > 0.25f) return 1.0f - e;
  float p = 1.0f - x * (1.0f / 8.0f);
  p = 1.0f - x * (1.0f / 7.0f) * p;
  p = 1.0f - x * (1.0f / 6.0f) * p;
  p = 1.0f - x * (1.0f / 5.0f) * p;
  p = 1.0f - x * (1.0f / 4.0f) * p;
  p = 1.0f - x * (1.0f / 3.0f) * p;
  p = 1.0f - x * (1.0f / 2.0f) * p;
  return x * p;
}

// a, and the factor of u
template <typename T>
__device__ __forceinline__ float2 lru_gate(float zr, float zi, float rate) {
  const float x = rate * sigmoid_of<T>(zr);
  const float a = sizeof(T) == 2 ? __builtin_amdgcn_exp2f(-1.4426950408889634f * x) : expf(-x);
  return float2{a, sqrtf(lru_one_minus_exp(2.0f * x, a * a)) * sigmoid_of<T>(zi)};
}

template <typename T>
struct LruArgs {
  const T* u;              // [tokens, width]
  const float* rate;       // [width]
  float* state;            // [slots, width]
  const int* slots;
  const int* cu_q;
  const T* y;              // rows of stride y_ld: the other branch's columns
  size_t y_ld;
  const float* y_bias;     // [width], or null
  int act;                 // of the other branch (GateActivation)
  float* a;                // [tokens, width]
  float* x;                // [tokens, width]
  T* out;                  // rows of stride out_ld
  size_t out_ld;
  float out_scale;
  int tokens, width;
  __device__ __forceinline__ T output(float s, size_t t, int c) const {
    const float z = to_f32(y[t * y_ld + c]) + (y_bias ? y_bias[c] : 0.f);
    return from_f32<T>(s * gate_activation_of<T>(z, act) * out_scale);
  }
  // what a (token, channel)'s gates lead to; ut: the token's u; slot: of a sequence that brings this token alone, else -1
  __device__ __forceinline__ void finish(float zr, float zi, float ut, int t, int c, int slot) const {
    const size_t at = (size_t)t * width + c;
    const float2 g = lru_gate<T>(zr, zi, rate[c]);
    const float in = g.y * ut;
    if (slot < 0) {
      a[at] = g.x;
      x[at] = in;
    } else {
      float* sp = state + (size_t)slot * width + c;
      const float s = fmaf(g.x, *sp, in);
      *sp = s;
      out[(size_t)t * out_ld + c] = output(s, t, c);
    }
  }
  __device__ __forceinline__ int single_slot(int seq) const { return cu_q[seq + 1] - cu_q[seq] == 1 ? slots[seq] : -1; }
};

// A thread a (token, channel).
template <typename T>
__global__ __launch_bounds__(kLruThreads) void lru_gates_kernel(LruArgs<T> p, const T* __restrict__ wr, const T* __restrict__ wi,
                                                                const float* __restrict__ br, const float* __restrict__ bi,
                                                                const int* __restrict__ seq_of_token, int size) {
  const int t = blockIdx.x, c = blockIdx.y * kLruThreads + threadIdx.x;
  if (c >= p.width) return;
  const T* un = p.u + (size_t)t * p.width + c / size * size;
  const T* r = wr + (size_t)c * size;
  const T* i = wi + (size_t)c * size;
  float zr = 0.f, zi = 0.f;
  for (int k = 0; k < size; ++k) {
    const float v = to_f32(un[k]);
    zr = fmaf(to_f32(r[k]), v, zr);
    zi = fmaf(to_f32(i[k]), v, zi);
  }
  p.finish(zr + br[c], zi + bi[c], to_f32(p.u[(size_t)t * p.width + c]), t, c, p.single_slot(seq_of_token[t]));
}

// Grid (runs of 16 * MT tokens, runs of 64 channels of a block, blocks); a wavefront 16 channels, of which a lane holds four
// neighbouring ones of one token.  MT = 4: the tokens' u go through LDS, 128 channels of the block at a time.
constexpr int kLruPanel = 128;

template <int MT>
__global__ __launch_bounds__(kLruThreads) void lru_gates_mfma_kernel(LruArgs<bf16> p, const bf16* __restrict__ wr,
                                                                     const bf16* __restrict__ wi, const float* __restrict__ br,
                                                                     const float* __restrict__ bi, const int* __restrict__ seq_of_token,
                                                                     int size) {
  constexpr bool STAGED = MT == 4;
  constexpr int kRow = kLruPanel + 8;           // 16-byte reads of sixteen rows fall into different banks
  constexpr int kPieces = 16 * MT * kLruPanel / 8 / kLruThreads;
  __shared__ __align__(16) bf16 us[STAGED ? 16 * MT * kRow : 8];
  __shared__ int slot_of[16 * MT];
  const int wave = threadIdx.x / kWave, lane = threadIdx.x % kWave;
  const int g = lane / 16, r = lane % 16;
  const int t0 = blockIdx.x * 16 * MT;
  const int o0 = blockIdx.y * 64 + 16 * wave;   // may lie past the block's end: such a wavefront only helps to stage
  const int base = blockIdx.z * size;
  const int o = o0 + r < size ? o0 + r : size - 1;
  const bf16* rr = wr + (size_t)(base + o) * size;
  const bf16* ri = wi + (size_t)(base + o) * size;
  if ((int)threadIdx.x < 16 * MT) {
    const int t = t0 + threadIdx.x;
    slot_of[threadIdx.x] = t < p.tokens ? p.single_slot(seq_of_token[t]) : -1;
  }
  const bf16* ur[MT];
#pragma unroll
  for (int m = 0; m < MT; ++m) {
    const int t = t0 + 16 * m + r;
    ur[m] = p.u + (size_t)(t < p.tokens ? t : p.tokens - 1) * p.width + base;
  }
  f32x4 ar[MT], ai[MT];
#pragma unroll
  for (int m = 0; m < MT; ++m) ar[m] = ai[m] = f32x4{0.f, 0.f, 0.f, 0.f};
  if (STAGED) {
    bf16x8 raw[kPieces > 0 ? kPieces : 1];
    auto fetch = [&](int k0) {
#pragma unroll
      for (int i = 0; i < kPieces; ++i) {
        const int piece = i * kLruThreads + threadIdx.x;
        const int row = piece / (kLruPanel / 8), k = k0 + 8 * (piece % (kLruPanel / 8));
        const int t = t0 + row < p.tokens ? t0 + row : p.tokens - 1;
        const bf16x8 v = *reinterpret_cast<const bf16x8*>(p.u + (size_t)t * p.width + base + (k < size ? k : 0));
        raw[i] = k < size ? v : zero8();        // (a multiple of 8: a piece lies inside or outside whole)
      }
    };
    fetch(0);
    for (int k0 = 0; k0 < size; k0 += kLruPanel) {
      bf16x8 fr[kLruPanel / 32], fi[kLruPanel / 32];
#pragma unroll
      for (int ks = 0; ks < kLruPanel / 32; ++ks) {
        const int k = k0 + 32 * ks + 8 * g < size ? k0 + 32 * ks + 8 * g : 0;
        fr[ks] = *reinterpret_cast<const bf16x8*>(rr + k);
        fi[ks] = *reinterpret_cast<const bf16x8*>(ri + k);
      }
      __syncthreads();
#pragma unroll
      for (int i = 0; i < kPieces; ++i) {
        const int piece = i * kLruThreads + threadIdx.x;
        *reinterpret_cast<bf16x8*>(us + (piece / (kLruPanel / 8)) * kRow + 8 * (piece % (kLruPanel / 8))) = raw[i];
      }
      __syncthreads();
      if (k0 + kLruPanel < size) fetch(k0 + kLruPanel);
#pragma unroll
      for (int ks = 0; ks < kLruPanel / 32; ++ks)
#pragma unroll
        for (int m = 0; m < MT; ++m) {
          const bf16x8 f = *reinterpret_cast<const bf16x8*>(us + (16 * m + r) * kRow + 32 * ks + 8 * g);
          ar[m] = mfma16(fr[ks], f, ar[m]);
          ai[m] = mfma16(fi[ks], f, ai[m]);
        }
    }
  } else {
#pragma unroll 4
    for (int k0 = 0; k0 < size; k0 += 32) {
      const bool in = k0 + 8 * g < size;
      const int k = in ? k0 + 8 * g : 0;
      const bf16x8 fr = *reinterpret_cast<const bf16x8*>(rr + k), fi = *reinterpret_cast<const bf16x8*>(ri + k);
#pragma unroll
      for (int m = 0; m < MT; ++m) {
        const bf16x8 v = *reinterpret_cast<const bf16x8*>(ur[m] + k);
        const bf16x8 f = in ? v : zero8();
        ar[m] = mfma16(fr, f, ar[m]);
        ai[m] = mfma16(fi, f, ai[m]);
      }
    }
    __syncthreads();                            // slot_of
  }
  if (o0 + 4 * g >= size) return;
  const int c = base + o0 + 4 * g;
  const f32x4 b0 = *reinterpret_cast<const f32x4*>(br + c), b1 = *reinterpret_cast<const f32x4*>(bi + c);
  const f32x4 rate = *reinterpret_cast<const f32x4*>(p.rate + c);
#pragma unroll
  for (int m = 0; m < MT; ++m) {
    const int t = t0 + 16 * m + r;
    if (t >= p.tokens) continue;
    const size_t at = (size_t)t * p.width + c;
    const bf16x4 ut = *reinterpret_cast<const bf16x4*>(p.u + at);
    f32x4 a4, x4;
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const float2 f = lru_gate<bf16>(ar[m][i] + b0[i], ai[m][i] + b1[i], rate[i]);
      a4[i] = f.x;
      x4[i] = f.y * (float)ut[i];
    }
    const int slot = slot_of[16 * m + r];
    if (slot < 0) {
      *reinterpret_cast<f32x4*>(p.a + at) = a4;
      *reinterpret_cast<f32x4*>(p.x + at) = x4;
    } else {
      f32x4* sp = reinterpret_cast<f32x4*>(p.state + (size_t)slot * p.width + c);
      f32x4 s4 = *sp;
#pragma unroll
      for (int i = 0; i < 4; ++i) s4[i] = fmaf(a4[i], s4[i], x4[i]);
      *sp = s4;
#pragma unroll
      for (int i = 0; i < 4; ++i) p.out[(size_t)t * p.out_ld + c + i] = p.output(s4[i], t, c + i);
    }
  }
}

// Where chunk j of the z-th listed sequence keeps its sums (a different place for every chunk of the launch).
__device__ __forceinline__ size_t lru_chunk_index(int row0, int z, int j) { return (size_t)(row0 / kLruChunk + z + j); }

// work: products of decays [chunks, width], ends from zero [chunks, width], the states before the step [listed, width].
// (1) A thread a channel of a chunk of a sequence of more than one chunk.
template <typename T>
__global__ __launch_bounds__(kLruThreads) void lru_chunk_kernel(LruArgs<T> p, const int* __restrict__ seq_ids, float* __restrict__ wa,
                                                                float* __restrict__ wu, float* __restrict__ w0, int max_chunks) {
  const int z = blockIdx.y / max_chunks, j = blockIdx.y % max_chunks;
  const int c = blockIdx.x * kLruThreads + threadIdx.x;
  const int seq = seq_ids[z];
  const int row0 = p.cu_q[seq], row1 = p.cu_q[seq + 1];
  if (c >= p.width || p.slots[seq] < 0 || row1 - row0 <= kLruChunk || row0 + j * kLruChunk >= row1) return;
  if (j == 0) w0[(size_t)z * p.width + c] = p.state[(size_t)p.slots[seq] * p.width + c];
  const int t0 = row0 + j * kLruChunk, t1 = t0 + kLruChunk < row1 ? t0 + kLruChunk : row1;
  float A = 1.f, U = 0.f;
  for (int t = t0; t < t1; t += kLruBatch) {
    float av[kLruBatch], xv[kLruBatch];
#pragma unroll
    for (int k = 0; k < kLruBatch; ++k) {
      const size_t at = (size_t)(t + k < t1 ? t + k : t1 - 1) * p.width + c;
      av[k] = p.a[at];
      xv[k] = p.x[at];
    }
#pragma unroll
    for (int k = 0; k < kLruBatch; ++k)
      if (t + k < t1) {
        A *= av[k];
        U = fmaf(av[k], U, xv[k]);
      }
  }
  const size_t at = lru_chunk_index(row0, z, j) * p.width + c;
  wa[at] = A;
  wu[at] = U;
}

// (2)
template <typename T>
__global__ __launch_bounds__(kLruThreads) void lru_out_kernel(LruArgs<T> p, const int* __restrict__ seq_ids, const float* __restrict__ wa,
                                                              const float* __restrict__ wu, const float* __restrict__ w0, int max_chunks) {
  const int z = blockIdx.y / max_chunks, j = blockIdx.y % max_chunks;
  const int c = blockIdx.x * kLruThreads + threadIdx.x;
  const int seq = seq_ids[z];
  const int row0 = p.cu_q[seq], row1 = p.cu_q[seq + 1];
  const int slot = p.slots[seq];
  if (c >= p.width || slot < 0 || row0 + j * kLruChunk >= row1) return;
  float* sp = p.state + (size_t)slot * p.width + c;
  // one chunk: its thread is the only one that touches the slot's place; several: they start from the copy (1) made
  float S = row1 - row0 <= kLruChunk ? *sp : w0[(size_t)z * p.width + c];
  const size_t first = lru_chunk_index(row0, z, 0) * p.width + c;
  for (int k0 = 0; k0 < j; k0 += kLruBatch) {
    float A[kLruBatch], U[kLruBatch];
#pragma unroll
    for (int k = 0; k < kLruBatch; ++k) {
      const size_t at = first + (size_t)(k0 + k < j ? k0 + k : j - 1) * p.width;
      A[k] = wa[at];
      U[k] = wu[at];
    }
#pragma unroll
    for (int k = 0; k < kLruBatch; ++k)
      if (k0 + k < j) S = fmaf(A[k], S, U[k]);
  }
  const int t0 = row0 + j * kLruChunk, t1 = t0 + kLruChunk < row1 ? t0 + kLruChunk : row1;
  for (int t = t0; t < t1; t += kLruBatch) {
    float av[kLruBatch], xv[kLruBatch];
    T yv[kLruBatch];
#pragma unroll
    for (int k = 0; k < kLruBatch; ++k) {
      const size_t tt = t + k < t1 ? t + k : t1 - 1;
      av[k] = p.a[tt * p.width + c];
      xv[k] = p.x[tt * p.width + c];
      yv[k] = p.y[tt * p.y_ld + c];
    }
    const float yb = p.y_bias ? p.y_bias[c] : 0.f;
#pragma unroll
    for (int k = 0; k < kLruBatch; ++k)
      if (t + k < t1) {
        S = fmaf(av[k], S, xv[k]);
        p.out[(size_t)(t + k) * p.out_ld + c] = from_f32<T>(S * gate_activation_of<T>(to_f32(yv[k]) + yb, p.act) * p.out_scale);
      }
  }
  if (t1 == row1) *sp = S;
}

template <typename T>
static int lru_args(const char* what, LruArgs<T>& p, const void* u, const float* rate, float* state, const int* slots, const int* cu_q,
                    const void* y, long y_ld, const float* y_bias, int act, float* a, float* x, void* out, long out_ld, float out_scale,
                    int tokens, int width) {
  PA_REQUIRE(tokens > 0 && width > 0 && y_ld >= width && out_ld >= width && (width + 255) / 256 <= 65535, "%s: bad sizes tokens=%d width=%d "
             "strides %ld and %ld", what, tokens, width, y_ld, out_ld);
  PA_REQUIRE(u && rate && state && slots && cu_q && y && a && x && out && act >= 0 && act < kActCount, "%s: a tensor is missing, or activation "
             "code %d", what, act);
  p = LruArgs<T>{(const T*)u, rate, state, slots, cu_q, (const T*)y, (size_t)y_ld, y_bias, act, a, x, (T*)out, (size_t)out_ld, out_scale,
                 tokens, width};
  return 0;
}

}  // namespace pa

using namespace pa;

extern "C" int pa_lru_gates(void* stream, int dtype, const void* u, const void* wr, const void* wi, const float* br, const float* bi,
                            const float* rate, float* state, const int* seq_of_token, const int* state_slots, const int* cu_q,
                            const void* y, long y_ld, const float* y_bias, int act, float* a, float* x, void* out, long out_ld,
                            float out_scale, int tokens, int width, int blocks) {
  if (tokens == 0) return 0;
  PA_REQUIRE(blocks > 0 && blocks <= 65535 && width % blocks == 0, "lru_gates: %d blocks do not divide a width of %d", blocks, width);
  const int size = width / blocks;
  hipStream_t st = (hipStream_t)stream;
  if (dtype == kF32) {
    LruArgs<float> p;
    if (int rc = lru_args("lru_gates", p, u, rate, state, state_slots, cu_q, y, y_ld, y_bias, act, a, x, out, out_ld, out_scale, tokens, width)) return rc;
    hipLaunchKernelGGL(lru_gates_kernel<float>, dim3(tokens, (width + 255) / 256), dim3(kLruThreads), 0, st, p, (const float*)wr,
                       (const float*)wi, br, bi, seq_of_token, size);
  } else if (dtype == kBF16) {
    LruArgs<bf16> p;
    if (int rc = lru_args("lru_gates", p, u, rate, state, state_slots, cu_q, y, y_ld, y_bias, act, a, x, out, out_ld, out_scale, tokens, width)) return rc;
    const uintptr_t all = reinterpret_cast<uintptr_t>(u) | reinterpret_cast<uintptr_t>(wr) | reinterpret_cast<uintptr_t>(wi) | reinterpret_cast<uintptr_t>(br) |
                          reinterpret_cast<uintptr_t>(bi) | reinterpret_cast<uintptr_t>(rate) | reinterpret_cast<uintptr_t>(state) |
                          reinterpret_cast<uintptr_t>(a) | reinterpret_cast<uintptr_t>(x);
    const bool pieces = size % 8 == 0 && (all & 15) == 0;
    if (!pieces)
      hipLaunchKernelGGL(lru_gates_kernel<bf16>, dim3(tokens, (width + 255) / 256), dim3(kLruThreads), 0, st, p, (const bf16*)wr,
                         (const bf16*)wi, br, bi, seq_of_token, size);
    else if (tokens <= 32)
      hipLaunchKernelGGL(lru_gates_mfma_kernel<1>, dim3((tokens + 15) / 16, (size + 63) / 64, blocks), dim3(kLruThreads), 0, st, p,
                         (const bf16*)wr, (const bf16*)wi, br, bi, seq_of_token, size);
    else
      hipLaunchKernelGGL(lru_gates_mfma_kernel<4>, dim3((tokens + 63) / 64, (size + 63) / 64, blocks), dim3(kLruThreads), 0, st, p,
                         (const bf16*)wr, (const bf16*)wi, br, bi, seq_of_token, size);
  } else {
    return pa::fail("lru_gates: unknown element type code %d", dtype);
  }
  return check_launch("lru_gates");
}

// 32-bit words of workspace
extern "C" long pa_lru_scan_workspace(int nlisted, int tokens, int width) {
  return (2 * ((long)tokens / kLruChunk + nlisted) + nlisted) * width;
}

// The listed sequences (of more than one token, at most max_len).
extern "C" int pa_lru_scan(void* stream, int dtype, const void* u, const float* rate, float* state, const int* state_slots, const int* cu_q,
                           const int* seq_ids, const void* y, long y_ld, const float* y_bias, int act, float* a, float* x, void* out,
                           long out_ld, float out_scale, float* work, int nlisted, int tokens, int max_len, int width) {
  if (nlisted == 0 || tokens == 0) return 0;
  const int max_chunks = (max_len + kLruChunk - 1) / kLruChunk;
  PA_REQUIRE(max_len > 0 && nlisted > 0 && (long)nlisted * max_chunks <= 65535 && seq_ids && work, "lru_scan: %d sequences of up to %d tokens",
             nlisted, max_len);
  const long chunks = (long)tokens / kLruChunk + nlisted;
  float* wa = work;
  float* wu = wa + chunks * width;
  float* w0 = wu + chunks * width;
  const dim3 grid((width + kLruThreads - 1) / kLruThreads, nlisted * max_chunks);
  hipStream_t st = (hipStream_t)stream;
#define PA_LRU(T)                                                                                                              \
  do {                                                                                                                         \
    LruArgs<T> p;                                                                                                              \
    if (int rc = lru_args("lru_scan", p, u, rate, state, state_slots, cu_q, y, y_ld, y_bias, act, a, x, out, out_ld, out_scale, tokens, width)) return rc; \
    if (max_chunks > 1)                                                                                                        \
      hipLaunchKernelGGL(lru_chunk_kernel<T>, grid, dim3(kLruThreads), 0, st, p, seq_ids, wa, wu, w0, max_chunks);              \
    hipLaunchKernelGGL(lru_out_kernel<T>, grid, dim3(kLruThreads), 0, st, p, seq_ids, wa, wu, w0, max_chunks);                  \
  } while (0)
  if (dtype == kF32) PA_LRU(float);
  else if (dtype == kBF16) PA_LRU(bf16);
  else return pa::fail("lru_scan: unknown element type code %d", dtype);
#undef PA_LRU
  return check_launch("lru_scan");
}
