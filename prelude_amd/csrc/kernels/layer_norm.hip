// Layer norm around a 32-bit residual stream, and the small sums such a stream takes between layers:
//
//   pa_layer_norm_step   residual += y (a branch's output, as a tensor or as the 32-bit partial sums of a product cut along
//                        its inner size; absent: nothing is added), then out = (x - mean) / sqrt(mean((x - mean)^2) + eps)
//                        * w + b of the new row.  With `rows` only those rows are normed and the residual is read only.
//   pa_branches_norm_step   residual += sum_b c_b norm_b(y_b) over one or two branches' outputs (each over its own root mean
//                        square, times its weight), then out = the RMS norm of the new row times w; `rows` as above
//   pa_stream_sum        out = x + y + extra + row, any of the last three absent; out may be x
//   pa_embed_scaled      out[t] = table[id] * scale, 32-bit
//   pa_activate          out = act(x) * scale on columns of wider rows: act GELU in its tanh form or SiLU
//
// All arithmetic is 32-bit; the order of every sum follows the thread layout alone, so a row's result never depends on
// what else the launch holds.
#include "common.h"
#include "api.h"

namespace pa {

constexpr int kLnThreads = 256;

__device__ __forceinline__ void ln_load8(const float* p, float* v) {
  const float4 a = *reinterpret_cast<const float4*>(p), b = *reinterpret_cast<const float4*>(p + 4);
  v[0] = a.x; v[1] = a.y; v[2] = a.z; v[3] = a.w; v[4] = b.x; v[5] = b.y; v[6] = b.z; v[7] = b.w;
}
__device__ __forceinline__ void ln_load8(const bf16* p, float* v) {
  const bf16x8 a = *reinterpret_cast<const bf16x8*>(p);
#pragma unroll
  for (int i = 0; i < 8; ++i) v[i] = (float)a[i];
}
__device__ __forceinline__ void ln_store8(float* p, const float* v) {
  *reinterpret_cast<float4*>(p) = float4{v[0], v[1], v[2], v[3]};
  *reinterpret_cast<float4*>(p + 4) = float4{v[4], v[5], v[6], v[7]};
}
__device__ __forceinline__ void ln_store8(bf16* p, const float* v) {
  bf16x8 a;
#pragma unroll
  for (int i = 0; i < 8; ++i) a[i] = (bf16)v[i];
  *reinterpret_cast<bf16x8*>(p) = a;
}

// What is added to the stream: a tensor of the engine's type, or `slices` partial sums, or nothing.
template <typename T>
struct Pending {
  const T* y;
  const float* parts;
  int slices;
  size_t slice_stride;
  __device__ __forceinline__ float at(size_t i) const {
    if (y) return to_f32(y[i]);
    float s = 0.f;
    for (int k = 0; k < slices; ++k) s += parts[k * slice_stride + i];
    return s;
  }
  __device__ __forceinline__ bool any() const { return y || slices > 0; }
};

// A workgroup a row of up to 8 * 256 * VPT elements, the row in registers in pieces of eight.
template <typename T, int VPT>
__global__ __launch_bounds__(kLnThreads) void layer_norm_step_vec_kernel(Pending<T> add, float* __restrict__ residual,
                                                                         const float* __restrict__ w, const float* __restrict__ b,
                                                                         T* __restrict__ out, const int* __restrict__ rows, int hidden,
                                                                         float eps) {
  __shared__ float scratch[16];
  const size_t r = blockIdx.x;
  const size_t src = rows ? (size_t)rows[r] : r;
  float* res = residual + src * hidden;
  const int pieces = hidden / 8;
  float x[VPT][8], wv[VPT][8], bv[VPT][8];
  float sum = 0.f;
#pragma unroll
  for (int v = 0; v < VPT; ++v) {
    const int piece = v * kLnThreads + threadIdx.x;
#pragma unroll
    for (int i = 0; i < 8; ++i) x[v][i] = 0.f;
    if (piece < pieces) {
      ln_load8(res + 8 * piece, x[v]);
      ln_load8(w + 8 * piece, wv[v]);
      ln_load8(b + 8 * piece, bv[v]);
      float yv[8];
      if (add.y) {
        ln_load8(add.y + src * hidden + 8 * piece, yv);
#pragma unroll
        for (int i = 0; i < 8; ++i) x[v][i] += yv[i];
      } else if (add.slices > 0) {
        float ys[8];
        ln_load8(add.parts + src * hidden + 8 * piece, yv);
        for (int k = 1; k < add.slices; ++k) {
          ln_load8(add.parts + k * add.slice_stride + src * hidden + 8 * piece, ys);
#pragma unroll
          for (int i = 0; i < 8; ++i) yv[i] += ys[i];
        }
#pragma unroll
        for (int i = 0; i < 8; ++i) x[v][i] += yv[i];
      }
      if (!rows && add.any()) ln_store8(res + 8 * piece, x[v]);
#pragma unroll
      for (int i = 0; i < 8; ++i) sum += x[v][i];
    }
  }
  const float mean = block_sum(sum, scratch) / (float)hidden;
  float ss = 0.f;
#pragma unroll
  for (int v = 0; v < VPT; ++v)
    if (v * kLnThreads + (int)threadIdx.x < pieces) {
#pragma unroll
      for (int i = 0; i < 8; ++i) {
        const float d = x[v][i] - mean;
        ss += d * d;
      }
    }
  const float inv = 1.0f / sqrtf(block_sum(ss, scratch) / (float)hidden + eps);
#pragma unroll
  for (int v = 0; v < VPT; ++v) {
    const int piece = v * kLnThreads + threadIdx.x;
    if (piece < pieces) {
      float o[8];
#pragma unroll
      for (int i = 0; i < 8; ++i) o[i] = (x[v][i] - mean) * inv * wv[v][i] + bv[v][i];
      ln_store8(out + r * hidden + 8 * piece, o);
    }
  }
}

// Rows of any width, read element by element (a thread comes back to its own elements alone).
template <typename T>
__global__ __launch_bounds__(kLnThreads) void layer_norm_step_kernel(Pending<T> add, float* __restrict__ residual,
                                                                     const float* __restrict__ w, const float* __restrict__ b,
                                                                     T* __restrict__ out, const int* __restrict__ rows, int hidden,
                                                                     float eps) {
  __shared__ float scratch[16];
  const size_t r = blockIdx.x;
  const size_t src = rows ? (size_t)rows[r] : r;
  float* res = residual + src * hidden;
  const bool stored = !rows && add.any();
  auto value = [&](int i) { return res[i] + (!stored && add.any() ? add.at(src * hidden + i) : 0.f); };
  float sum = 0.f;
  for (int i = threadIdx.x; i < hidden; i += kLnThreads) {
    float v;
    if (stored) {
      v = res[i] + add.at(src * hidden + i);
      res[i] = v;
    } else {
      v = value(i);
    }
    sum += v;
  }
  const float mean = block_sum(sum, scratch) / (float)hidden;
  float ss = 0.f;
  for (int i = threadIdx.x; i < hidden; i += kLnThreads) {
    const float d = value(i) - mean;
    ss += d * d;
  }
  const float inv = 1.0f / sqrtf(block_sum(ss, scratch) / (float)hidden + eps);
  for (int i = threadIdx.x; i < hidden; i += kLnThreads) out[r * hidden + i] = from_f32<T>((value(i) - mean) * inv * w[i] + b[i]);
}

// One or two branches beside each other in front of a 32-bit stream.
template <typename T>
struct NormedBranches {
  Pending<T> y[2];           // the second may be empty
  const float* w[2];
  float c[2];
  float eps;
};

template <typename T>
__device__ __forceinline__ void pending_load8(const Pending<T>& p, size_t at, float* v) {
  if (p.y) {
    ln_load8(p.y + at, v);
    return;
  }
  ln_load8(p.parts + at, v);
  for (int k = 1; k < p.slices; ++k) {
    float u[8];
    ln_load8(p.parts + k * p.slice_stride + at, u);
#pragma unroll
    for (int i = 0; i < 8; ++i) v[i] += u[i];
  }
}

// A workgroup a row of up to 8 * 256 * VPT elements, everything in registers in pieces of eight.
template <typename T, int VPT>
__global__ __launch_bounds__(kLnThreads) void branches_norm_step_vec_kernel(NormedBranches<T> nb, float* __restrict__ residual,
                                                                            const float* __restrict__ w, T* __restrict__ out,
                                                                            const int* __restrict__ rows, int hidden, float eps) {
  __shared__ float scratch[16], scratch2[16];
  const size_t r = blockIdx.x;
  const size_t src = rows ? (size_t)rows[r] : r;
  float* res = residual + src * hidden;
  const int pieces = hidden / 8;
  const bool two = nb.y[1].any();
  float x[VPT][8], a[VPT][8], b[VPT][8];
  float sa = 0.f, sb = 0.f;
#pragma unroll
  for (int v = 0; v < VPT; ++v) {
    const int piece = v * kLnThreads + threadIdx.x;
#pragma unroll
    for (int i = 0; i < 8; ++i) x[v][i] = a[v][i] = b[v][i] = 0.f;
    if (piece < pieces) {
      ln_load8(res + 8 * piece, x[v]);
      pending_load8(nb.y[0], src * hidden + 8 * piece, a[v]);
      if (two) pending_load8(nb.y[1], src * hidden + 8 * piece, b[v]);
#pragma unroll
      for (int i = 0; i < 8; ++i) {
        sa += a[v][i] * a[v][i];
        sb += b[v][i] * b[v][i];
      }
    }
  }
  const float fa = nb.c[0] / sqrtf(block_sum(sa, scratch) / (float)hidden + nb.eps);
  const float fb = two ? nb.c[1] / sqrtf(block_sum(sb, scratch2) / (float)hidden + nb.eps) : 0.f;
  float ss = 0.f;
#pragma unroll
  for (int v = 0; v < VPT; ++v) {
    const int piece = v * kLnThreads + threadIdx.x;
    if (piece < pieces) {
      float wa[8], wb[8];
      ln_load8(nb.w[0] + 8 * piece, wa);
      if (two) ln_load8(nb.w[1] + 8 * piece, wb);
#pragma unroll
      for (int i = 0; i < 8; ++i) {
        float y = a[v][i] * fa * wa[i];
        if (two) y += b[v][i] * fb * wb[i];
        x[v][i] += y;
        ss += x[v][i] * x[v][i];
      }
      if (!rows) ln_store8(res + 8 * piece, x[v]);
    }
  }
  const float inv = 1.0f / sqrtf(block_sum(ss, scratch) / (float)hidden + eps);
#pragma unroll
  for (int v = 0; v < VPT; ++v) {
    const int piece = v * kLnThreads + threadIdx.x;
    if (piece < pieces) {
      float o[8], wv[8];
      ln_load8(w + 8 * piece, wv);
#pragma unroll
      for (int i = 0; i < 8; ++i) o[i] = x[v][i] * inv * wv[i];
      ln_store8(out + r * hidden + 8 * piece, o);
    }
  }
}

// Rows of any width up to 16384, the new row in LDS.
template <typename T>
__global__ __launch_bounds__(kLnThreads) void branches_norm_step_kernel(NormedBranches<T> nb, float* __restrict__ residual,
                                                                        const float* __restrict__ w, T* __restrict__ out,
                                                                        const int* __restrict__ rows, int hidden, float eps) {
  extern __shared__ float new_row[];
  __shared__ float scratch[16];
  const size_t r = blockIdx.x;
  const size_t src = rows ? (size_t)rows[r] : r;
  float* res = residual + src * hidden;
  for (int i = threadIdx.x; i < hidden; i += kLnThreads) new_row[i] = res[i];
  for (int b = 0; b < 2; ++b) {
    if (!nb.y[b].any()) continue;
    float ss = 0.f;
    for (int i = threadIdx.x; i < hidden; i += kLnThreads) {
      const float v = nb.y[b].at(src * hidden + i);
      ss += v * v;
    }
    const float f = nb.c[b] / sqrtf(block_sum(ss, scratch) / (float)hidden + nb.eps);
    for (int i = threadIdx.x; i < hidden; i += kLnThreads) new_row[i] += nb.y[b].at(src * hidden + i) * f * nb.w[b][i];
  }
  float ss = 0.f;
  for (int i = threadIdx.x; i < hidden; i += kLnThreads) {   // (a thread comes back to its own elements alone)
    const float v = new_row[i];
    if (!rows) res[i] = v;
    ss += v * v;
  }
  const float inv = 1.0f / sqrtf(block_sum(ss, scratch) / (float)hidden + eps);
  for (int i = threadIdx.x; i < hidden; i += kLnThreads) out[r * hidden + i] = from_f32<T>(new_row[i] * inv * w[i]);
}

// V elements a thread (V = 4 where the row width allows).
template <typename T, int V>
__global__ void stream_sum_kernel(const float* __restrict__ x, const T* __restrict__ y, const float* __restrict__ extra,
                                  const float* __restrict__ row, float* __restrict__ out, size_t total, int hidden) {
  typedef T vec_t __attribute__((ext_vector_type(V)));
  typedef float fvec_t __attribute__((ext_vector_type(V)));
  const size_t i = ((size_t)blockIdx.x * blockDim.x + threadIdx.x) * V;
  if (i >= total) return;
  fvec_t v = *reinterpret_cast<const fvec_t*>(x + i);
  if (y) {
    const vec_t yv = *reinterpret_cast<const vec_t*>(y + i);
#pragma unroll
    for (int e = 0; e < V; ++e) v[e] += to_f32(yv[e]);
  }
  if (extra) {
    const fvec_t ev = *reinterpret_cast<const fvec_t*>(extra + i);
#pragma unroll
    for (int e = 0; e < V; ++e) v[e] += ev[e];
  }
  if (row) {
    const fvec_t rv = *reinterpret_cast<const fvec_t*>(row + i % hidden);
#pragma unroll
    for (int e = 0; e < V; ++e) v[e] += rv[e];
  }
  *reinterpret_cast<fvec_t*>(out + i) = v;
}

template <typename T>
__global__ __launch_bounds__(256) void embed_scaled_kernel(const int* __restrict__ ids, const T* __restrict__ table,
                                                           float* __restrict__ out, int hidden, int vocab, float scale) {
  const int t = blockIdx.x;
  int id = ids[t];
  id = id < 0 ? 0 : (id >= vocab ? vocab - 1 : id);
  const T* src = table + (size_t)id * hidden;
  float* dst = out + (size_t)t * hidden;
  if (hidden % 8 == 0) {
    for (int i = threadIdx.x; i < hidden / 8; i += blockDim.x) {
      float v[8];
      ln_load8(src + 8 * i, v);
#pragma unroll
      for (int e = 0; e < 8; ++e) v[e] *= scale;
      ln_store8(dst + 8 * i, v);
    }
  } else {
    for (int i = threadIdx.x; i < hidden; i += blockDim.x) dst[i] = to_f32(src[i]) * scale;
  }
}

// V consecutive columns a thread.
template <typename T, int V>
__global__ __launch_bounds__(256) void activate_kernel(const T* __restrict__ x, size_t x_stride, T* __restrict__ out, size_t out_stride,
                                                       int rows, int width, int act, float scale) {
  typedef T vec_t __attribute__((ext_vector_type(V)));
  const size_t i = ((size_t)blockIdx.x * blockDim.x + threadIdx.x) * V;
  if (i >= (size_t)rows * width) return;
  const size_t r = i / width, c = i % width;
  const vec_t v = *reinterpret_cast<const vec_t*>(x + r * x_stride + c);
  vec_t o;
#pragma unroll
  for (int e = 0; e < V; ++e) o[e] = from_f32<T>(gate_activation_of<T>(to_f32(v[e]), act) * scale);
  *reinterpret_cast<vec_t*>(out + r * out_stride + c) = o;
}

}  // namespace pa

using namespace pa;

static bool aligned16(const void* p) { return (reinterpret_cast<uintptr_t>(p) & 15) == 0; }

template <typename T>
static void launch_layer_norm(hipStream_t st, const Pending<T>& add, float* residual, const float* w, const float* b, T* out,
                              const int* rows, int nrows, int hidden, float eps) {
  const bool vec = hidden % 8 == 0 && hidden <= 8 * kLnThreads * 4 && aligned16(add.y) && aligned16(add.parts) &&
                   add.slice_stride % 4 == 0 && aligned16(residual) && aligned16(w) && aligned16(b) && aligned16(out);
  const dim3 grid(nrows), block(kLnThreads);
#define PA_LN(V) hipLaunchKernelGGL((layer_norm_step_vec_kernel<T, V>), grid, block, 0, st, add, residual, w, b, out, rows, hidden, eps)
  if (!vec)
    hipLaunchKernelGGL(layer_norm_step_kernel<T>, grid, block, 0, st, add, residual, w, b, out, rows, hidden, eps);
  else if (hidden <= 8 * kLnThreads) PA_LN(1);
  else if (hidden <= 16 * kLnThreads) PA_LN(2);
  else PA_LN(4);
#undef PA_LN
}

extern "C" int pa_layer_norm_step(void* stream, int dtype, const void* y, const float* parts, int slices, long slice_stride,
                                  float* residual, const float* w, const float* b, void* out, const int* rows, int nrows,
                                  int hidden, float eps) {
  if (nrows == 0) return 0;
  PA_REQUIRE(nrows > 0 && hidden > 0 && residual && w && b && out, "layer_norm_step: bad sizes rows=%d hidden=%d or a missing tensor",
             nrows, hidden);
  PA_REQUIRE(slices >= 0 && (slices == 0 || (parts && !y)), "layer_norm_step: a branch is a tensor or %d partial sums, not both", slices);
  hipStream_t st = (hipStream_t)stream;
  if (dtype == kF32)
    launch_layer_norm<float>(st, Pending<float>{(const float*)y, parts, slices, (size_t)slice_stride}, residual, w, b, (float*)out,
                             rows, nrows, hidden, eps);
  else if (dtype == kBF16)
    launch_layer_norm<bf16>(st, Pending<bf16>{(const bf16*)y, parts, slices, (size_t)slice_stride}, residual, w, b, (bf16*)out, rows,
                            nrows, hidden, eps);
  else
    return pa::fail("layer_norm_step: unknown element type code %d", dtype);
  return check_launch("layer_norm_step");
}

extern "C" int pa_stream_sum(void* stream, int dtype, const float* x, const void* y, const float* extra, const float* row, float* out,
                             int tokens, int hidden) {
  if (tokens == 0) return 0;
  PA_REQUIRE(tokens > 0 && hidden > 0 && x && out, "stream_sum: bad sizes tokens=%d hidden=%d", tokens, hidden);
  const size_t total = (size_t)tokens * hidden;
  const bool vec = hidden % 4 == 0 && aligned16(x) && aligned16(y) && aligned16(extra) && aligned16(row) && aligned16(out);
  const size_t threads = vec ? total / 4 : total;
  dim3 grid((unsigned)((threads + 255) / 256));
  hipStream_t st = (hipStream_t)stream;
#define PA_SUM(T, V) hipLaunchKernelGGL((stream_sum_kernel<T, V>), grid, dim3(256), 0, st, x, (const T*)y, extra, row, out, total, hidden)
  if (dtype == kF32) {
    if (vec) PA_SUM(float, 4);
    else PA_SUM(float, 1);
  } else if (dtype == kBF16) {
    if (vec) PA_SUM(bf16, 4);
    else PA_SUM(bf16, 1);
  } else {
    return pa::fail("stream_sum: unknown element type code %d", dtype);
  }
#undef PA_SUM
  return check_launch("stream_sum");
}

extern "C" int pa_embed_scaled(void* stream, int dtype, const int* ids, const void* table, float* out, int tokens, int hidden,
                               int vocab, float scale) {
  if (tokens == 0) return 0;
  PA_REQUIRE(tokens > 0 && hidden > 0 && vocab > 0, "embed_scaled: bad sizes tokens=%d hidden=%d vocab=%d", tokens, hidden, vocab);
  hipStream_t st = (hipStream_t)stream;
  if (dtype == kF32)
    hipLaunchKernelGGL(embed_scaled_kernel<float>, dim3(tokens), dim3(256), 0, st, ids, (const float*)table, out, hidden, vocab, scale);
  else if (dtype == kBF16)
    hipLaunchKernelGGL(embed_scaled_kernel<bf16>, dim3(tokens), dim3(256), 0, st, ids, (const bf16*)table, out, hidden, vocab, scale);
  else
    return pa::fail("embed_scaled: unknown element type code %d", dtype);
  return check_launch("embed_scaled");
}

extern "C" int pa_activate(void* stream, int dtype, const void* x, long x_stride, void* out, long out_stride, int rows, int width,
                           int act, float scale) {
  if (rows == 0) return 0;
  PA_REQUIRE(rows > 0 && width > 0 && x_stride >= width && out_stride >= width, "activate: bad sizes rows=%d width=%d", rows, width);
  PA_REQUIRE(act >= 0 && act < kActCount, "activate: unknown activation code %d", act);
  hipStream_t st = (hipStream_t)stream;
  const long per16 = dtype == kBF16 ? 8 : 4;
  const bool vec = width % per16 == 0 && x_stride % per16 == 0 && out_stride % per16 == 0 && aligned16(x) && aligned16(out);
  const size_t threads = (size_t)rows * width / (vec ? per16 : 1);
  dim3 grid((unsigned)((threads + 255) / 256));
#define PA_ACT(T, V) hipLaunchKernelGGL((activate_kernel<T, V>), grid, dim3(256), 0, st, (const T*)x, (size_t)x_stride, (T*)out, \
                                        (size_t)out_stride, rows, width, act, scale)
  if (dtype == kF32) {
    if (vec) PA_ACT(float, 4);
    else PA_ACT(float, 1);
  } else if (dtype == kBF16) {
    if (vec) PA_ACT(bf16, 8);
    else PA_ACT(bf16, 1);
  } else {
    return pa::fail("activate: unknown element type code %d", dtype);
  }
#undef PA_ACT
  return check_launch("activate");
}

template <typename T>
static void launch_branches_norm(hipStream_t st, const NormedBranches<T>& nb, float* residual, const float* w, T* out, const int* rows,
                                 int nrows, int hidden, float eps) {
  bool vec = hidden % 8 == 0 && hidden <= 8 * kLnThreads * 4 && aligned16(residual) && aligned16(w) && aligned16(out);
  for (int b = 0; b < 2; ++b)
    vec = vec && aligned16(nb.y[b].y) && aligned16(nb.y[b].parts) && nb.y[b].slice_stride % 4 == 0 && aligned16(nb.w[b]);
  const dim3 grid(nrows), block(kLnThreads);
#define PA_BNORM(V) hipLaunchKernelGGL((branches_norm_step_vec_kernel<T, V>), grid, block, 0, st, nb, residual, w, out, rows, hidden, eps)
  if (!vec)
    hipLaunchKernelGGL(branches_norm_step_kernel<T>, grid, block, hidden * sizeof(float), st, nb, residual, w, out, rows, hidden, eps);
  else if (hidden <= 8 * kLnThreads) PA_BNORM(1);
  else if (hidden <= 8 * kLnThreads * 2) PA_BNORM(2);
  else PA_BNORM(4);
#undef PA_BNORM
}

extern "C" int pa_branches_norm_step(void* stream, int dtype, const void* y0, const float* parts0, int slices0, const float* w0, float c0,
                                     const void* y1, const float* parts1, int slices1, const float* w1, float c1, long slice_stride,
                                     float branch_eps, float* residual, const float* w, void* out, const int* rows, int nrows, int hidden,
                                     float eps) {
  if (nrows == 0) return 0;
  PA_REQUIRE(nrows > 0 && hidden > 0 && hidden <= 16384 && residual && w && out, "branches_norm_step: bad sizes rows=%d hidden=%d", nrows, hidden);
  PA_REQUIRE((y0 != nullptr) != (slices0 > 0) && (slices0 == 0 || parts0) && w0 && !(y1 && slices1 > 0) && (slices1 == 0 || parts1) &&
             (!(y1 || slices1 > 0) || w1), "branches_norm_step: a branch is a tensor or partial sums, with a weight");
  hipStream_t st = (hipStream_t)stream;
#define PA_BRANCHES(T)                                                                                                            \
  launch_branches_norm<T>(st, NormedBranches<T>{{{(const T*)y0, parts0, slices0, (size_t)slice_stride}, {(const T*)y1, parts1, slices1, (size_t)slice_stride}}, \
                                                {w0, w1}, {c0, c1}, branch_eps}, residual, w, (T*)out, rows, nrows, hidden, eps)
  if (dtype == kF32) PA_BRANCHES(float);
  else if (dtype == kBF16) PA_BRANCHES(bf16);
  else return pa::fail("branches_norm_step: unknown element type code %d", dtype);
#undef PA_BRANCHES
  return check_launch("branches_norm_step");
}
