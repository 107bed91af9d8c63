// Recurrent mixers whose state is a matrix per (request, head) that decays by one number a token:
//
//   S_t = a_t S_(t-1) + b_t k_t v_t^T          S [dim, vdim], 32-bit, one per (request, head), kept in a state slot
//   n_t = a_t n_(t-1) + b_t k_t                n [dim], where the design keeps one
//   o_t = S_t^T q_t + skip_h v_t,   den_t = n_t . q_t        (q times a constant on its way in), 32-bit
//
// with a_t = exp(la_t) and b_t one number per token and head, made in 32-bit from the projections by
//   ssd gates     b = softplus(z + bias), la = -exp(a_log) b                                            (Mamba-2)
//   mlstm gates   i = c tanh((z_i + bias_i) / c), f = log sigmoid(c tanh((z_f + bias_f) / c)), and a running maximum m (zero
//                 at a request's start): m_t = max(f + m_(t-1), i), la = f + m_(t-1) - m_t, b = exp(i - m_t); the reader of
//                 den also gets exp(-m_t)                                                                (xLSTM's mLSTM)
//
// q, k [tokens, heads / group, dim] (head h reads q/k head h / group) and v [tokens, heads, vdim] lie inside one row per
// token (stride ld).  A request's portions may be cut anywhere; the state carries over.
//
//   pa_decay_scan          the recurrence as it stands, token by token, on the vector ALU, for any sizes and both types
//   pa_decay_scan_step     single tokens, gates included
//   pa_decay_scan_chunked  portions, bfloat16, on the matrix cores, in chunks of 64 tokens.  With c_i the sum of la up to
//                          token i of a chunk and S_b the state in front of it,
//
//                            o_i  = sum_{j <= i} e^(c_i - c_j) b_j (q_i . k_j) v_j  +  e^(c_i) S_b^T q_i
//                            S_b' = e^(c_n) S_b + U,    U = sum_j e^(c_n - c_j) b_j k_j v_j^T
//
//                          (1) every chunk makes its U; (2) one pass over the chunks of a sequence turns the U into the
//                          S_b and leaves the end in the slot; (3) every chunk makes its outputs.  The sums c are 64-bit,
//                          so a difference of two of them is exact to 32-bit whatever came before.  What is not a stored
//                          bfloat16 number already -- the weights of the first sum, the scaled keys of U, the state -- takes
//                          part as the sum of two bfloat16 numbers (a product with 16 bits of mantissa, added up in 32-bit).
#include "common.h"
#include "api.h"
#include "attention_mfma_core.h"

namespace pa {

constexpr int kScanCols = 64;      // value columns a workgroup of the token-by-token kernels
constexpr int kScanTokens = 16;    // tokens staged at a time
constexpr int kScanThreads = 256;
constexpr int kScanChunk = 64;
constexpr int kScanMaxTiles = 16;  // tiles of 16 value columns a workgroup of the chunked kernels at most

template <typename T>
struct ScanArgs {
  const T* p;
  size_t ld;
  int q_off, k_off, v_off;
  int heads, group, dim, vdim;
  const float* la;     // [tokens, heads]
  const float* b;      // [tokens, heads]
  float* s;            // [slots, heads, dim, vdim]
  float* n;            // [slots, heads, dim], or null
  const float* skip;   // [heads], or null
  float q_scale;
  const int* slots;
  const int* cu_q;
  float* out;          // [tokens, heads, vdim]
  float* den;          // [tokens, heads], or null
};

__device__ __forceinline__ float scan_softplus(float z) { return fmaxf(z, 0.f) + log1pf(expf(-fabsf(z))); }
__device__ __forceinline__ float scan_log_sigmoid(float z) { return fminf(z, 0.f) - log1pf(expf(-fabsf(z))); }
__device__ __forceinline__ float scan_capped(float z, float cap) { return cap * tanhf(z / cap); }

// ---- gates of portions -------------------------------------------------------------------------------------------------
template <typename T>
__global__ __launch_bounds__(256) void ssd_gates_kernel(const T* __restrict__ p, size_t ld, int off, const float* __restrict__ bias,
                                                        const float* __restrict__ a_log, float* __restrict__ la,
                                                        float* __restrict__ b, size_t total, int heads) {
  const size_t i = (size_t)blockIdx.x * 256 + threadIdx.x;
  if (i >= total) return;
  const size_t t = i / heads;
  const int h = (int)(i % heads);
  const float dt = scan_softplus(to_f32(p[t * ld + off + h]) + bias[h]);
  b[i] = dt;
  la[i] = -expf(a_log[h]) * dt;
}

// A workgroup a (head, sequence of at least min_len tokens), 1,024 tokens at a time, a thread a token.  A token is the map
// m -> max(f + m, i), and maps compose: (f1, i1) and then (f2, i2) is (f1 + f2, max(i1 + f2, i2)).
constexpr int kGateThreads = 1024;

template <typename T>
__global__ __launch_bounds__(kGateThreads) void mlstm_gates_kernel(const T* __restrict__ p, size_t ld, int i_off, int f_off,
                                                                   const float* __restrict__ i_bias, const float* __restrict__ f_bias,
                                                                   float cap, float* __restrict__ m_state, int copies,
                                                                   const int* __restrict__ state_slots, const int* __restrict__ cu_q,
                                                                   float* __restrict__ la, float* __restrict__ b,
                                                                   float* __restrict__ floor_out, int heads, int min_len) {
  constexpr int kWaves = kGateThreads / kWave;
  __shared__ float wave_f[2][kWaves], wave_i[2][kWaves];
  const int h = blockIdx.x, seq = blockIdx.y, lane = threadIdx.x % kWave, wave = threadIdx.x / kWave;
  const int row0 = cu_q[seq], row1 = cu_q[seq + 1];
  const int slot = state_slots[seq];
  if (slot < 0 || row1 - row0 < min_len || row1 <= row0) return;   // the same for the whole workgroup
  float* ms = m_state + ((size_t)slot * heads + h) * copies;
  float m = ms[0];
  const float ib = i_bias[h], fb = f_bias[h];
  int buf = 0;
  for (int t0 = row0; t0 < row1; t0 += kGateThreads, buf ^= 1) {
    const int t = t0 + threadIdx.x;
    const bool live = t < row1;
    const T* z = p + (size_t)(live ? t : row1 - 1) * ld + h;
    const float zi = to_f32(z[i_off]), zf = to_f32(z[f_off]);
    const float ig = live ? scan_capped(zi + ib, cap) : -INFINITY;
    const float fg = live ? scan_log_sigmoid(scan_capped(zf + fb, cap)) : 0.f;
    float A = fg, B = ig;
#pragma unroll
    for (int o = 1; o < kWave; o <<= 1) {
      const float Ao = __shfl_up(A, o, kWave), Bo = __shfl_up(B, o, kWave);
      if (lane >= o) {
        B = fmaxf(Bo + A, B);
        A += Ao;
      }
    }
    if (lane == kWave - 1) {
      wave_f[buf][wave] = A;
      wave_i[buf][wave] = B;
    }
    __syncthreads();               // (two buffers: the next block's sums do not meet this one's readers)
    float mine = m;                // the maximum in front of this wavefront's tokens, and behind the block's
    for (int w = 0; w < kWaves; ++w) {
      if (w == wave) mine = m;
      m = fmaxf(wave_f[buf][w] + m, wave_i[buf][w]);
    }
    const float mt = fmaxf(A + mine, B);
    float before = __shfl_up(mt, 1, kWave);
    if (lane == 0) before = mine;
    if (live) {
      const size_t at = (size_t)t * heads + h;
      la[at] = fg + before - mt;
      b[at] = expf(ig - mt);
      floor_out[at] = expf(-mt);
    }
  }
  __syncthreads();                 // every thread has read the slot
  for (int i = threadIdx.x; i < copies; i += kGateThreads) ms[i] = m;
}

// ---- token by token ----------------------------------------------------------------------------------------------------
// Grid (tiles of 64 value columns, and one more for n where there is one; heads; sequences of at least min_len tokens).  A lane
// keeps a quarter of the rows of S (R of them) for one column in registers: the 16-lane rows of a wavefront are the
// quarters, whose dot products are added across them.
template <typename T, int R>
__global__ __launch_bounds__(kScanThreads) void decay_scan_kernel(ScanArgs<T> a, int min_len) {
  constexpr int kQuarter = R + 4;
  __shared__ __align__(16) float qs[kScanTokens][4 * kQuarter];
  __shared__ __align__(16) float ks[kScanTokens][4 * kQuarter];
  __shared__ float vs[kScanTokens][kScanCols];
  __shared__ float as[kScanTokens], bs[kScanTokens];
  const int w = threadIdx.x / kWave, lane = threadIdx.x % kWave;
  const int dp = lane / 16, cl = 16 * w + lane % 16;
  const int h = blockIdx.y, seq = blockIdx.z;
  const int row0 = a.cu_q[seq], row1 = a.cu_q[seq + 1];
  const int slot = a.slots[seq];
  if (slot < 0 || row1 - row0 < min_len || row1 <= row0) return;   // the same for the whole workgroup
  const int vt = (a.vdim + kScanCols - 1) / kScanCols;
  const bool is_n = (int)blockIdx.x == vt;
  const int c0 = is_n ? 0 : blockIdx.x * kScanCols;
  const int width = is_n ? 1 : a.vdim;
  const int col = c0 + cl;
  const bool live = col < width;
  float* sp = is_n ? a.n + ((size_t)slot * a.heads + h) * a.dim : a.s + ((size_t)slot * a.heads + h) * a.dim * a.vdim;
  float S[R];
#pragma unroll
  for (int r = 0; r < R; ++r) {
    const int d = dp * R + r;
    S[r] = (live && d < a.dim) ? sp[(size_t)d * width + col] : 0.f;
  }
  const T* qp = a.p + a.q_off + (size_t)(h / a.group) * a.dim;
  const T* kp = a.p + a.k_off + (size_t)(h / a.group) * a.dim;
  const T* vp = a.p + a.v_off + (size_t)h * a.vdim;
  const float skip = (a.skip && !is_n) ? a.skip[h] : 0.f;
  for (int t0 = row0; t0 < row1; t0 += kScanTokens) {
    const int n = row1 - t0 < kScanTokens ? row1 - t0 : kScanTokens;
    __syncthreads();
    for (int e = threadIdx.x; e < kScanTokens * 4 * R; e += kScanThreads) {
      const int t = e / (4 * R), d = e % (4 * R);
      const bool on = t < n && d < a.dim;
      const size_t at = (size_t)(t0 + t) * a.ld + d;
      const int to = (d / R) * kQuarter + d % R;
      qs[t][to] = on ? to_f32(qp[at]) * a.q_scale : 0.f;
      ks[t][to] = on ? to_f32(kp[at]) : 0.f;
    }
    for (int e = threadIdx.x; e < kScanTokens * kScanCols; e += kScanThreads) {
      const int t = e / kScanCols, c = e % kScanCols;
      const bool on = t < n && c0 + c < width;
      vs[t][c] = on ? (is_n ? 1.f : to_f32(vp[(size_t)(t0 + t) * a.ld + c0 + c])) : 0.f;
    }
    if ((int)threadIdx.x < n) {
      const size_t at = (size_t)(t0 + threadIdx.x) * a.heads + h;
      as[threadIdx.x] = expf(a.la[at]);
      bs[threadIdx.x] = a.b[at];
    }
    __syncthreads();
    for (int t = 0; t < n; ++t) {
      const float al = as[t], v = vs[t][cl], bv = bs[t] * v;
      float acc = 0.f;
#pragma unroll
      for (int r = 0; r < R; r += 4) {
        const f32x4 q4 = *reinterpret_cast<const f32x4*>(&qs[t][dp * kQuarter + r]);
        const f32x4 k4 = *reinterpret_cast<const f32x4*>(&ks[t][dp * kQuarter + r]);
#pragma unroll
        for (int e = 0; e < 4; ++e) {
          S[r + e] = fmaf(al, S[r + e], k4[e] * bv);
          acc = fmaf(S[r + e], q4[e], acc);
        }
      }
      const float sum = xor_sum16_32(acc);
      if (dp == 0 && live) {
        const size_t at = (size_t)(t0 + t) * a.heads + h;
        if (is_n) a.den[at] = sum;
        else a.out[at * a.vdim + col] = fmaf(skip, v, sum);
      }
    }
  }
#pragma unroll
  for (int r = 0; r < R; ++r) {
    const int d = dp * R + r;
    if (live && d < a.dim) sp[(size_t)d * width + col] = S[r];
  }
}

// How a single token's gates are made on the way in.
template <typename T>
struct StepGates {
  const T* z;               // rows of stride z_ld that hold the heads' gate inputs
  size_t z_ld;
  int z_off, f_off;         // their columns (mlstm: of i and f)
  const float* bias;        // [heads] (mlstm: of i)
  const float* f_bias;      // mlstm
  const float* a_log;       // ssd
  float cap;                // mlstm
  float* m;                 // mlstm: [slots, heads, copies], a copy of the running maximum per column tile
  int copies;
  float* floor_out;         // mlstm: exp(-m) [tokens, heads]
};

// Sequences of exactly one token.  Grid as above; a wavefront owns a quarter of the rows, a lane a column: a row's 64 columns
// are one run of memory, and all of a lane's rows are asked for at once.
template <typename T, int R, bool MLSTM>
__global__ __launch_bounds__(kScanThreads) void decay_scan_step_kernel(ScanArgs<T> a, StepGates<T> g) {
  __shared__ float qs[4 * R], ks[4 * R];
  __shared__ float part[4][kScanCols];
  const int w = threadIdx.x / kWave, lane = threadIdx.x % kWave;
  const int h = blockIdx.y, seq = blockIdx.z;
  const int row = a.cu_q[seq];
  const int slot = a.slots[seq];
  if (slot < 0 || a.cu_q[seq + 1] - row != 1) return;   // the same for the whole workgroup
  const int vt = (a.vdim + kScanCols - 1) / kScanCols;
  const bool is_n = (int)blockIdx.x == vt;
  const int col = (is_n ? 0 : blockIdx.x * kScanCols) + lane;
  const int width = is_n ? 1 : a.vdim;
  const bool live = col < width;
  float* sp = (is_n ? a.n + ((size_t)slot * a.heads + h) * a.dim : a.s + ((size_t)slot * a.heads + h) * a.dim * a.vdim) + (live ? col : width - 1);
  float s[R];
#pragma unroll
  for (int r = 0; r < R; ++r) {
    const int d = w * R + r;
    s[r] = sp[(size_t)(d < a.dim ? d : a.dim - 1) * width];
  }
  const T* src = a.p + (size_t)row * a.ld;
  if ((int)threadIdx.x < 4 * R) {
    const int d = (int)threadIdx.x < a.dim ? threadIdx.x : a.dim - 1;
    qs[threadIdx.x] = to_f32(src[a.q_off + (size_t)(h / a.group) * a.dim + d]) * a.q_scale;
    ks[threadIdx.x] = to_f32(src[a.k_off + (size_t)(h / a.group) * a.dim + d]);
  }
  const float v = is_n ? 1.f : to_f32(src[a.v_off + (size_t)h * a.vdim + (live ? col : width - 1)]);
  float al, b, m_new = 0.f;
  float* mp = nullptr;
  const T* zr = g.z + (size_t)row * g.z_ld + h;
  if (MLSTM) {
    const float ig = scan_capped(to_f32(zr[g.z_off]) + g.bias[h], g.cap);
    const float fg = scan_log_sigmoid(scan_capped(to_f32(zr[g.f_off]) + g.f_bias[h], g.cap));
    mp = g.m + ((size_t)slot * a.heads + h) * g.copies + blockIdx.x;
    const float m = *mp;
    m_new = fmaxf(fg + m, ig);
    al = expf(fg + m - m_new);
    b = expf(ig - m_new);
  } else {
    b = scan_softplus(to_f32(zr[g.z_off]) + g.bias[h]);
    al = expf(-expf(g.a_log[h]) * b);
  }
  __syncthreads();
  if (MLSTM && threadIdx.x == 0) {   // behind the barrier: every thread has read its copy
    *mp = m_new;
    if (is_n) g.floor_out[(size_t)row * a.heads + h] = expf(-m_new);
  }
  const float bv = b * v;
  float acc = 0.f;
#pragma unroll
  for (int r = 0; r < R; ++r) {
    const int d = w * R + r;
    s[r] = fmaf(al, s[r], ks[d] * bv);
    if (d < a.dim) acc = fmaf(s[r], qs[d], acc);
  }
#pragma unroll
  for (int r = 0; r < R; ++r) {
    const int d = w * R + r;
    if (live && d < a.dim) sp[(size_t)d * width] = s[r];
  }
  part[w][lane] = acc;
  __syncthreads();
  if (w == 0 && live) {
    const float sum = (part[0][lane] + part[1][lane]) + (part[2][lane] + part[3][lane]);
    const size_t at = (size_t)row * a.heads + h;
    if (is_n) a.den[at] = sum;
    else a.out[at * a.vdim + col] = fmaf(a.skip ? a.skip[h] : 0.f, v, sum);
  }
}

// ---- portions in chunks, on the matrix cores ---------------------------------------------------------------------------
// Where chunk j of the z-th listed sequence, which starts at packed row row0, keeps its state: every sequence adds at most one
// partial chunk, so the index is different for every chunk of the launch and below tokens / 64 + sequences.
__device__ __forceinline__ size_t scan_chunk_index(int row0, int z, int j) { return (size_t)(row0 / kScanChunk + z + j); }

// Rows of 64 tokens in LDS, 128 bytes each, in eight pieces of eight tokens whose places are permuted by the row: sixteen
// rows' pieces of the same tokens (an operand) and eight rows' pairs of tokens (how they are written) lie in different banks.
__device__ __forceinline__ int scan_at(int row, int j) { return row * kScanChunk + ((((j >> 3) ^ row ^ (row >> 3)) & 7) << 3) + (j & 7); }

// src [token][columns] -> LDS [column][token] for `rows` columns from `first` on (a multiple of 8 each), columns from `width` on and
// tokens from n on zero; `ones`: column `width` is one for the tokens there are.  With `scale` (a factor a token): as the sum of
// hi and lo.
template <bool SCALED>
__device__ __forceinline__ void scan_stage(const bf16* __restrict__ src, size_t ld, int first, int rows, int width, int n, bool ones,
                                           const float* scale, bf16* hi, bf16* lo) {
  const int pieces = rows / 8;
  for (int u = threadIdx.x; u < 32 * pieces; u += kScanThreads) {
    const int piece = u % pieces, j = 2 * (u / pieces);
    const int c = first + 8 * piece;
    const bool in = c + 8 <= width;
    // (no load stands under a branch: what does not exist is read from where something does and not used)
    const bf16* at = src + (in ? c : 0);
    const bf16x8 v0 = *reinterpret_cast<const bf16x8*>(at + (size_t)(j < n ? j : n - 1) * ld);
    const bf16x8 v1 = *reinterpret_cast<const bf16x8*>(at + (size_t)(j + 1 < n ? j + 1 : n - 1) * ld);
    const bool on0 = in && j < n, on1 = in && j + 1 < n;
#pragma unroll
    for (int i = 0; i < 8; ++i) {
      float x0 = on0 ? (float)v0[i] : 0.f, x1 = on1 ? (float)v1[i] : 0.f;
      if (ones && i == 0 && c == width) {
        x0 = j < n ? 1.f : 0.f;
        x1 = j + 1 < n ? 1.f : 0.f;
      }
      if (SCALED) {
        x0 *= scale[j];
        x1 *= scale[j + 1];
      }
      bf16x2 h2;
      h2[0] = (bf16)x0;
      h2[1] = (bf16)x1;
      const int to = scan_at(8 * piece + i, j);
      *reinterpret_cast<bf16x2*>(hi + to) = h2;
      if (SCALED) {
        bf16x2 l2;
        l2[0] = (bf16)(x0 - (float)h2[0]);
        l2[1] = (bf16)(x1 - (float)h2[1]);
        *reinterpret_cast<bf16x2*>(lo + to) = l2;
      }
    }
  }
}

// The inclusive sums of la over the wavefront's 64 tokens, 64-bit.
__device__ __forceinline__ double scan_sums(double v) {
  const int lane = threadIdx.x % kWave;
#pragma unroll
  for (int o = 1; o < kWave; o <<= 1) {
    const double u = __shfl_up(v, o, kWave);
    if (lane >= o) v += u;
  }
  return v;
}

__device__ __forceinline__ bf16x8 scan_piece(const bf16* lds, int row, int j) { return *reinterpret_cast<const bf16x8*>(lds + scan_at(row, j)); }

// (1) work[chunk][head][column e][row d] = U^T, rows padded to dpad (zeros), columns to a multiple of 16; chunk_decay[chunk][head].
// Grid (heads, runs of `et_per` tiles of 16 columns, listed sequences x max_chunks).
template <int DP>
__global__ __launch_bounds__(kScanThreads) void scan_chunk_state_kernel(ScanArgs<bf16> a, const int* __restrict__ seq_ids,
                                                                        float* __restrict__ work, float* __restrict__ chunk_decay,
                                                                        int max_chunks, int et_per) {
  extern __shared__ __align__(16) unsigned char scan_lds[];
  __shared__ float cs[kScanChunk];
  const int h = blockIdx.x, z = blockIdx.z / max_chunks, j = blockIdx.z % max_chunks;
  const int seq = seq_ids[z];
  int row0 = a.cu_q[seq];
  const int row1 = a.cu_q[seq + 1];
  if (a.slots[seq] < 0 || row0 + j * kScanChunk >= row1) return;   // the same for the whole workgroup
  const size_t idx = scan_chunk_index(row0, z, j);
  row0 += j * kScanChunk;
  const int n = row1 - row0 < kScanChunk ? row1 - row0 : kScanChunk;
  const int tiles = (a.vdim + (a.n ? 1 : 0) + 15) / 16;
  const int et0 = blockIdx.y * et_per;
  const int etn = tiles - et0 < et_per ? tiles - et0 : et_per;
  const int dpad = (a.dim + 31) / 32 * 32;
  bf16* vt = reinterpret_cast<bf16*>(scan_lds);
  bf16* kh = vt + (size_t)et_per * 16 * kScanChunk;
  bf16* kl = kh + (size_t)dpad * kScanChunk;
  const int wave = threadIdx.x / kWave, lane = threadIdx.x % kWave;
  const int g = lane / 16, r = lane % 16;
  if (wave == 0) {
    const size_t at = (size_t)(row0 + (lane < n ? lane : n - 1)) * a.heads + h;
    const double c = scan_sums(lane < n ? (double)a.la[at] : 0.0);
    const double total = __shfl(c, kWave - 1, kWave);
    cs[lane] = lane < n ? expf((float)(total - c)) * a.b[at] : 0.f;
    if (lane == 0 && blockIdx.y == 0) chunk_decay[idx * a.heads + h] = expf((float)total);
  }
  scan_stage<false>(a.p + (size_t)row0 * a.ld + a.v_off + (size_t)h * a.vdim, a.ld, 16 * et0, 16 * etn, a.vdim, n, a.n != nullptr, nullptr, vt, nullptr);
  __syncthreads();
  scan_stage<true>(a.p + (size_t)row0 * a.ld + a.k_off + (size_t)(h / a.group) * a.dim, a.ld, 0, dpad, a.dim, n, false, cs, kh, kl);
  __syncthreads();
  float* wp = work + (idx * a.heads + h) * (size_t)(16 * tiles) * dpad;
  for (int et = wave; et < etn; et += kScanThreads / kWave) {
    const bf16x8 v0 = scan_piece(vt, 16 * et + r, 8 * g), v1 = scan_piece(vt, 16 * et + r, 32 + 8 * g);
#pragma unroll
    for (int dt = 0; dt < DP / 16; ++dt) {
      if (16 * dt >= dpad) break;
      const int row = 16 * dt + r;
      f32x4 acc{0.f, 0.f, 0.f, 0.f};
      acc = mfma16(v0, scan_piece(kl, row, 8 * g), acc);
      acc = mfma16(v1, scan_piece(kl, row, 32 + 8 * g), acc);
      acc = mfma16(v0, scan_piece(kh, row, 8 * g), acc);
      acc = mfma16(v1, scan_piece(kh, row, 32 + 8 * g), acc);
#pragma unroll
      for (int i = 0; i < 4; ++i) wp[(size_t)(16 * (et0 + et) + 4 * g + i) * dpad + row] = acc[i];
    }
  }
}

// (2) a thread an element of a head's state, a batch of chunks asked for together.
__global__ __launch_bounds__(256) void scan_chunk_carry_kernel(ScanArgs<bf16> a, const int* __restrict__ seq_ids,
                                                               float* __restrict__ work, const float* __restrict__ chunk_decay) {
  const int z = blockIdx.z, h = blockIdx.y;
  const int seq = seq_ids[z];
  const int row0 = a.cu_q[seq], len = a.cu_q[seq + 1] - row0;
  const int slot = a.slots[seq];
  if (slot < 0 || len <= 0) return;
  const int dpad = (a.dim + 31) / 32 * 32, columns = a.vdim + (a.n ? 1 : 0);
  const int i = blockIdx.x * 256 + threadIdx.x;
  if (i >= columns * dpad) return;
  const int e = i / dpad, d = i % dpad;
  const size_t chunk_size = (size_t)a.heads * ((columns + 15) / 16 * 16) * dpad;
  const size_t first = scan_chunk_index(row0, z, 0);
  float* wp = work + first * chunk_size + (size_t)h * (chunk_size / a.heads) + i;
  const float* dp = chunk_decay + first * a.heads + h;
  const bool real = d < a.dim;
  float* sp = e < a.vdim ? a.s + (((size_t)slot * a.heads + h) * a.dim + (real ? d : 0)) * a.vdim + e
                         : a.n + ((size_t)slot * a.heads + h) * a.dim + (real ? d : 0);
  float S = real ? *sp : 0.f;
  const int chunks = (len + kScanChunk - 1) / kScanChunk;
  constexpr int kBatch = 8;
  for (int j0 = 0; j0 < chunks; j0 += kBatch) {
    float U[kBatch], A[kBatch];
#pragma unroll
    for (int k = 0; k < kBatch; ++k) {
      const int j = j0 + k < chunks ? j0 + k : chunks - 1;
      U[k] = wp[(size_t)j * chunk_size];
      A[k] = dp[(size_t)j * a.heads];
    }
#pragma unroll
    for (int k = 0; k < kBatch; ++k)
      if (j0 + k < chunks) {
        wp[(size_t)(j0 + k) * chunk_size] = S;
        S = fmaf(A[k], S, U[k]);
      }
  }
  if (real) *sp = S;
}

// (3) Grid as (1).  Every wavefront makes the weights of one tile of 16 keys against the queries of the chunk, then all of
// them the outputs of their tiles of columns.
template <int DP>
__global__ __launch_bounds__(kScanThreads, DP <= 64 ? 3 : 1) void scan_chunk_out_kernel(ScanArgs<bf16> a, const int* __restrict__ seq_ids,
                                                                      const float* __restrict__ work, int max_chunks, int et_per) {
  constexpr int KS = DP / 32;
  extern __shared__ __align__(16) unsigned char scan_lds[];
  __shared__ double cum[kScanChunk];
  __shared__ float bj[kScanChunk], ec[kScanChunk];
  const int h = blockIdx.x, z = blockIdx.z / max_chunks, j = blockIdx.z % max_chunks;
  const int seq = seq_ids[z];
  int row0 = a.cu_q[seq];
  const int row1 = a.cu_q[seq + 1];
  if (a.slots[seq] < 0 || row0 + j * kScanChunk >= row1) return;   // the same for the whole workgroup
  const size_t idx = scan_chunk_index(row0, z, j);
  row0 += j * kScanChunk;
  const int n = row1 - row0 < kScanChunk ? row1 - row0 : kScanChunk;
  const int tiles = (a.vdim + (a.n ? 1 : 0) + 15) / 16;
  const int et0 = blockIdx.y * et_per;
  const int etn = tiles - et0 < et_per ? tiles - et0 : et_per;
  const int dpad = (a.dim + 31) / 32 * 32;
  bf16* wh = reinterpret_cast<bf16*>(scan_lds);       // [query][key]
  bf16* wl = wh + kScanChunk * kScanChunk;
  bf16* vt = wl + kScanChunk * kScanChunk;            // [column][key]
  const int wave = threadIdx.x / kWave, lane = threadIdx.x % kWave;
  const int g = lane / 16, r = lane % 16;
  if (wave == 0) {
    const size_t at = (size_t)(row0 + (lane < n ? lane : n - 1)) * a.heads + h;
    const double c = scan_sums(lane < n ? (double)a.la[at] : 0.0);
    cum[lane] = c;
    bj[lane] = lane < n ? a.b[at] * a.q_scale : 0.f;
    ec[lane] = expf((float)c) * a.q_scale;
  }
  const size_t qk = (size_t)(h / a.group) * a.dim;
  bf16x8 qf[4][KS], kf[KS];
#pragma unroll
  for (int it = 0; it < 4; ++it) {
    const int t = 16 * it + r;
    const bf16* qr = a.p + (size_t)(row0 + (t < n ? t : n - 1)) * a.ld + a.q_off + qk;
#pragma unroll
    for (int ks = 0; ks < KS; ++ks) {
      const bool in = 32 * ks + 8 * g < a.dim;
      const bf16x8 x = *reinterpret_cast<const bf16x8*>(qr + (in ? 32 * ks + 8 * g : 0));
      qf[it][ks] = in ? x : zero8();
    }
  }
  {
    const int t = 16 * wave + r;
    const bf16* kr = a.p + (size_t)(row0 + (t < n ? t : n - 1)) * a.ld + a.k_off + qk;
#pragma unroll
    for (int ks = 0; ks < KS; ++ks) kf[ks] = *reinterpret_cast<const bf16x8*>(kr + (32 * ks + 8 * g < a.dim ? 32 * ks + 8 * g : 0));
  }
  scan_stage<false>(a.p + (size_t)row0 * a.ld + a.v_off + (size_t)h * a.vdim, a.ld, 16 * et0, 16 * etn, a.vdim, n, a.n != nullptr, nullptr, vt, nullptr);
  __syncthreads();
#pragma unroll
  for (int it = 0; it < 4; ++it) {
    bf16x4 hi, lo;
#pragma unroll
    for (int i = 0; i < 4; ++i) hi[i] = lo[i] = (bf16)0.f;
    const int i = 16 * it + r, j0 = 16 * wave + 4 * g;
    if (it >= wave) {
      f32x4 acc{0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int ks = 0; ks < KS; ++ks)
        if (32 * ks < dpad) acc = mfma16(kf[ks], qf[it][ks], acc);
      const double ci = cum[i];
#pragma unroll
      for (int k = 0; k < 4; ++k) {
        const float x = j0 + k <= i ? acc[k] * (expf((float)(ci - cum[j0 + k])) * bj[j0 + k]) : 0.f;
        hi[k] = (bf16)x;
        lo[k] = (bf16)(x - (float)hi[k]);
      }
    }
    *reinterpret_cast<bf16x4*>(wh + scan_at(i, j0)) = hi;
    *reinterpret_cast<bf16x4*>(wl + scan_at(i, j0)) = lo;
  }
  __syncthreads();
  const float* wp = work + (idx * a.heads + h) * (size_t)(16 * tiles) * dpad;
  const float skip = a.skip ? a.skip[h] : 0.f;
#pragma unroll 1
  for (int et = wave; et < etn; et += kScanThreads / kWave) {
    const int e = 16 * (et0 + et) + r;
    f32x4 acc[4];
#pragma unroll
    for (int it = 0; it < 4; ++it) acc[it] = f32x4{0.f, 0.f, 0.f, 0.f};
    const float* srow = wp + (size_t)e * dpad + 8 * g;
#pragma unroll
    for (int ks = 0; ks < KS; ++ks) {
      if (32 * ks >= dpad) break;
      const f32x4 s0 = *reinterpret_cast<const f32x4*>(srow + 32 * ks), s1 = *reinterpret_cast<const f32x4*>(srow + 32 * ks + 4);
      bf16x8 sh, sl;
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        sh[i] = (bf16)s0[i];
        sl[i] = (bf16)(s0[i] - (float)sh[i]);
        sh[4 + i] = (bf16)s1[i];
        sl[4 + i] = (bf16)(s1[i] - (float)sh[4 + i]);
      }
#pragma unroll
      for (int it = 0; it < 4; ++it) {
        acc[it] = mfma16(qf[it][ks], sl, acc[it]);
        acc[it] = mfma16(qf[it][ks], sh, acc[it]);
      }
    }
#pragma unroll
    for (int it = 0; it < 4; ++it)
#pragma unroll
      for (int i = 0; i < 4; ++i) acc[it][i] *= ec[16 * it + 4 * g + i];
#pragma unroll
    for (int ks = 0; ks < 2; ++ks) {
      const bf16x8 v = scan_piece(vt, 16 * et + r, 32 * ks + 8 * g);
#pragma unroll
      for (int it = 2 * ks; it < 4; ++it) {
        acc[it] = mfma16(scan_piece(wl, 16 * it + r, 32 * ks + 8 * g), v, acc[it]);
        acc[it] = mfma16(scan_piece(wh, 16 * it + r, 32 * ks + 8 * g), v, acc[it]);
      }
    }
    // a column of S, or n's: from one base, a token a step
    const bool is_n = e == a.vdim && a.den;
    if (e >= a.vdim && !is_n) continue;
    const int step = is_n ? a.heads : a.heads * a.vdim;
    float* dst = is_n ? a.den + (size_t)row0 * a.heads + h : a.out + ((size_t)row0 * a.heads + h) * a.vdim + e;
#pragma unroll
    for (int it = 0; it < 4; ++it)
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        const int t = 16 * it + 4 * g + i;
        if (t >= n) continue;
        float o = acc[it][i];
        if (a.skip && !is_n) o = fmaf(skip, (float)vt[scan_at(16 * et + r, t)], o);
        dst[(size_t)t * step] = o;
      }
  }
}

static int scan_check(const char* what, int nseq, int tokens, int heads, int group, int dim, int vdim, long ld, int q_off, int k_off,
                      int v_off, const void* n, const void* den) {
  PA_REQUIRE(nseq > 0 && nseq <= 65535 && tokens > 0 && heads > 0 && heads <= 65535 && group > 0 && heads % group == 0 && vdim > 0,
             "%s: bad sizes seqs=%d tokens=%d heads=%d (groups of %d) vdim=%d", what, nseq, tokens, heads, group, vdim);
  PA_REQUIRE(dim > 0 && dim <= 256, "%s: a key width of %d is outside 1..256", what, dim);
  PA_REQUIRE(q_off >= 0 && k_off >= 0 && v_off >= 0 && q_off + (long)(heads / group) * dim <= ld &&
             k_off + (long)(heads / group) * dim <= ld && v_off + (long)heads * vdim <= ld, "%s: the columns do not fit the row of %ld", what, ld);
  PA_REQUIRE((n == nullptr) == (den == nullptr), "%s: a sum of keys and its product with the queries go together", what);
  return 0;
}

}  // namespace pa

using namespace pa;

extern "C" int pa_ssd_gates(void* stream, int dtype, const void* p, long ld, int off, const float* bias, const float* a_log, float* la,
                            float* b, int tokens, int heads) {
  if (tokens == 0) return 0;
  PA_REQUIRE(tokens > 0 && heads > 0 && off >= 0 && off + (long)heads <= ld, "ssd_gates: bad sizes tokens=%d heads=%d", tokens, heads);
  const size_t total = (size_t)tokens * heads;
  const dim3 grid((unsigned)((total + 255) / 256));
  hipStream_t st = (hipStream_t)stream;
  if (dtype == kF32)
    hipLaunchKernelGGL(ssd_gates_kernel<float>, grid, dim3(256), 0, st, (const float*)p, (size_t)ld, off, bias, a_log, la, b, total, heads);
  else if (dtype == kBF16)
    hipLaunchKernelGGL(ssd_gates_kernel<bf16>, grid, dim3(256), 0, st, (const bf16*)p, (size_t)ld, off, bias, a_log, la, b, total, heads);
  else
    return pa::fail("ssd_gates: unknown element type code %d", dtype);
  return check_launch("ssd_gates");
}

// copies of the running maximum: one per column tile of the step kernel, n's included
extern "C" int pa_mlstm_max_copies(int vdim) { return (vdim + kScanCols - 1) / kScanCols + 1; }

extern "C" int pa_mlstm_gates(void* stream, int dtype, const void* p, long ld, int i_off, int f_off, const float* i_bias,
                              const float* f_bias, float cap, float* m, const int* state_slots, const int* cu_q, float* la, float* b,
                              float* floor_out, int nseq, int heads, int vdim, int min_len) {
  if (nseq == 0) return 0;
  PA_REQUIRE(nseq > 0 && nseq <= 65535 && heads > 0 && cap > 0.f && i_off >= 0 && f_off >= 0 && i_off + (long)heads <= ld &&
             f_off + (long)heads <= ld, "mlstm_gates: bad sizes seqs=%d heads=%d cap=%g", nseq, heads, (double)cap);
  hipStream_t st = (hipStream_t)stream;
  const int copies = pa_mlstm_max_copies(vdim);
  if (dtype == kF32)
    hipLaunchKernelGGL(mlstm_gates_kernel<float>, dim3(heads, nseq), dim3(kGateThreads), 0, st, (const float*)p, (size_t)ld, i_off, f_off, i_bias,
                       f_bias, cap, m, copies, state_slots, cu_q, la, b, floor_out, heads, min_len);
  else if (dtype == kBF16)
    hipLaunchKernelGGL(mlstm_gates_kernel<bf16>, dim3(heads, nseq), dim3(kGateThreads), 0, st, (const bf16*)p, (size_t)ld, i_off, f_off, i_bias,
                       f_bias, cap, m, copies, state_slots, cu_q, la, b, floor_out, heads, min_len);
  else
    return pa::fail("mlstm_gates: unknown element type code %d", dtype);
  return check_launch("mlstm_gates");
}

extern "C" int pa_decay_scan(void* stream, int dtype, const void* p, long ld, int q_off, int k_off, int v_off, const float* la,
                             const float* b, float* s, float* n, const float* skip, float q_scale, const int* state_slots,
                             const int* cu_q, float* out, float* den, int nseq, int tokens, int heads, int group, int dim, int vdim,
                             int min_len) {
  if (nseq == 0 || tokens == 0) return 0;
  if (int rc = scan_check("decay_scan", nseq, tokens, heads, group, dim, vdim, ld, q_off, k_off, v_off, n, den)) return rc;
  const dim3 grid((vdim + kScanCols - 1) / kScanCols + (n ? 1 : 0), heads, nseq);
  hipStream_t st = (hipStream_t)stream;
#define PA_SCAN(T, R)                                                                                                         \
  hipLaunchKernelGGL((decay_scan_kernel<T, R>), grid, dim3(kScanThreads), 0, st,                                              \
                     (ScanArgs<T>{(const T*)p, (size_t)ld, q_off, k_off, v_off, heads, group, dim, vdim, la, b, s, n, skip, q_scale, \
                                  state_slots, cu_q, out, den}), min_len)
#define PA_SCAN_R(T)                     \
  do {                                   \
    if (dim <= 32) PA_SCAN(T, 8);        \
    else if (dim <= 64) PA_SCAN(T, 16);  \
    else if (dim <= 128) PA_SCAN(T, 32); \
    else PA_SCAN(T, 64);                 \
  } while (0)
  if (dtype == kF32) PA_SCAN_R(float);
  else if (dtype == kBF16) PA_SCAN_R(bf16);
  else return pa::fail("decay_scan: unknown element type code %d", dtype);
#undef PA_SCAN_R
#undef PA_SCAN
  return check_launch("decay_scan");
}

// a_log given: ssd gates (z_off, bias); else mlstm gates (z_off / bias of i, f_off / f_bias, cap, m, floor_out).
extern "C" int pa_decay_scan_step(void* stream, int dtype, const void* p, long ld, int q_off, int k_off, int v_off, const void* z, long z_ld,
                                  int z_off, int f_off, const float* bias, const float* f_bias, const float* a_log, float cap, float* m, float* floor_out,
                                  float* s, float* n, const float* skip, float q_scale, const int* state_slots, const int* cu_q,
                                  float* out, float* den, int nseq, int heads, int group, int dim, int vdim) {
  if (nseq == 0) return 0;
  if (int rc = scan_check("decay_scan_step", nseq, nseq, heads, group, dim, vdim, ld, q_off, k_off, v_off, n, den)) return rc;
  const bool mlstm = a_log == nullptr;
  PA_REQUIRE(z && z_off >= 0 && z_off + (long)heads <= z_ld && bias && (!mlstm || (f_off >= 0 && f_off + (long)heads <= z_ld && f_bias && cap > 0.f && m &&
             floor_out && n)), "decay_scan_step: a gate's columns do not fit the row of %ld, or a tensor is missing", z_ld);
  const dim3 grid((vdim + kScanCols - 1) / kScanCols + (n ? 1 : 0), heads, nseq);
  hipStream_t st = (hipStream_t)stream;
#define PA_STEP(T, R, M)                                                                                                      \
  hipLaunchKernelGGL((decay_scan_step_kernel<T, R, M>), grid, dim3(kScanThreads), 0, st,                                      \
                     (ScanArgs<T>{(const T*)p, (size_t)ld, q_off, k_off, v_off, heads, group, dim, vdim, nullptr, nullptr, s, n, skip, \
                                  q_scale, state_slots, cu_q, out, den}),                                              \
                     (StepGates<T>{(const T*)z, (size_t)z_ld, z_off, f_off, bias, f_bias, a_log, cap, m, pa_mlstm_max_copies(vdim), floor_out}))
#define PA_STEP_R(T, M)                     \
  do {                                      \
    if (dim <= 32) PA_STEP(T, 8, M);        \
    else if (dim <= 64) PA_STEP(T, 16, M);  \
    else if (dim <= 128) PA_STEP(T, 32, M); \
    else PA_STEP(T, 64, M);                 \
  } while (0)
#define PA_STEP_M(T)                  \
  do {                                \
    if (mlstm) PA_STEP_R(T, true);    \
    else PA_STEP_R(T, false);         \
  } while (0)
  if (dtype == kF32) PA_STEP_M(float);
  else if (dtype == kBF16) PA_STEP_M(bf16);
  else return pa::fail("decay_scan_step: unknown element type code %d", dtype);
#undef PA_STEP_M
#undef PA_STEP_R
#undef PA_STEP
  return check_launch("decay_scan_step");
}

extern "C" int pa_decay_scan_chunked_supports(const void* p, long ld, int q_off, int k_off, int v_off, int dim, int vdim) {
  return dim > 0 && dim <= 256 && dim % 8 == 0 && vdim > 0 && vdim % 8 == 0 && ld % 8 == 0 && q_off % 8 == 0 && k_off % 8 == 0 &&
         v_off % 8 == 0 && (reinterpret_cast<uintptr_t>(p) & 15) == 0;
}

// 32-bit words of workspace: the chunks' states, then their decays
extern "C" long pa_decay_scan_chunked_workspace(int nlisted, int tokens, int heads, int dim, int vdim, int with_n) {
  const long tiles = (vdim + (with_n ? 1 : 0) + 15) / 16, dpad = (dim + 31) / 32 * 32;
  return ((long)tokens / kScanChunk + nlisted) * heads * (tiles * 16 * dpad + 1);
}

// The listed sequences (at most max_len tokens each), bfloat16.
extern "C" int pa_decay_scan_chunked(void* stream, const void* p, long ld, int q_off, int k_off, int v_off, const float* la, const float* b,
                                     float* s, float* n, const float* skip, float q_scale, const int* state_slots, const int* cu_q,
                                     const int* seq_ids, float* out, float* den, float* work, int nlisted, int tokens, int max_len,
                                     int heads, int group, int dim, int vdim) {
  if (nlisted == 0 || tokens == 0 || max_len == 0) return 0;
  if (int rc = scan_check("decay_scan_chunked", nlisted, tokens, heads, group, dim, vdim, ld, q_off, k_off, v_off, n, den)) return rc;
  PA_REQUIRE(pa_decay_scan_chunked_supports(p, ld, q_off, k_off, v_off, dim, vdim), "decay_scan_chunked: widths %d and %d, or columns that "
             "are no whole 16-byte pieces", dim, vdim);
  PA_REQUIRE(seq_ids && work, "decay_scan_chunked: no list of sequences or no workspace");
  const int max_chunks = (max_len + kScanChunk - 1) / kScanChunk;
  PA_REQUIRE((long)nlisted * max_chunks <= 65535, "decay_scan_chunked: %d sequences x %d chunks exceed the grid", nlisted, max_chunks);
  const ScanArgs<bf16> a{(const bf16*)p, (size_t)ld, q_off, k_off, v_off, heads, group, dim, vdim, la, b, s, n, skip, q_scale, state_slots,
                         cu_q, out, den};
  const int tiles = (vdim + (n ? 1 : 0) + 15) / 16, dpad = (dim + 31) / 32 * 32, columns = vdim + (n ? 1 : 0);
  // tiles a workgroup: all of them where there are chunks and heads enough for the chip, fewer otherwise
  const long units = (long)nlisted * max_chunks * heads;
  int parts = units >= 256 ? 1 : (int)((256 + units - 1) / units);
  parts = parts > 4 ? 4 : parts;
  int et_per = (tiles + parts - 1) / parts;
  et_per = et_per > kScanMaxTiles ? kScanMaxTiles : et_per;
  const dim3 grid(heads, (tiles + et_per - 1) / et_per, nlisted * max_chunks);
  float* chunk_decay = work + ((long)tokens / kScanChunk + nlisted) * heads * (long)(tiles * 16) * dpad;
  hipStream_t st = (hipStream_t)stream;
  const size_t lds1 = ((size_t)et_per * 16 + 2 * (size_t)dpad) * kScanChunk * sizeof(bf16);
  const size_t lds3 = ((size_t)et_per * 16 + 2 * kScanChunk) * kScanChunk * sizeof(bf16);
#define PA_CHUNKED(DP)                                                                                                          \
  do {                                                                                                                          \
    constexpr int most = (kScanMaxTiles * 16 + 2 * DP) * kScanChunk * (int)sizeof(bf16);                                         \
    static const hipError_t allowed = hipFuncSetAttribute(reinterpret_cast<const void*>(&scan_chunk_state_kernel<DP>),           \
                                                          hipFuncAttributeMaxDynamicSharedMemorySize, most);                     \
    PA_REQUIRE(allowed == hipSuccess, "decay_scan_chunked: %d bytes of LDS refused: %s", most, hipGetErrorString(allowed));      \
    hipLaunchKernelGGL(scan_chunk_state_kernel<DP>, grid, dim3(kScanThreads), lds1, st, a, seq_ids, work, chunk_decay, max_chunks, et_per); \
    hipLaunchKernelGGL(scan_chunk_carry_kernel, dim3((columns * dpad + 255) / 256, heads, nlisted), dim3(256), 0, st, a, seq_ids, \
                       work, chunk_decay);                                                                                      \
    hipLaunchKernelGGL(scan_chunk_out_kernel<DP>, grid, dim3(kScanThreads), lds3, st, a, seq_ids, work, max_chunks, et_per);     \
  } while (0)
  if (dim <= 64) PA_CHUNKED(64);
  else if (dim <= 128) PA_CHUNKED(128);
  else PA_CHUNKED(256);
#undef PA_CHUNKED
  return check_launch("decay_scan_chunked");
}
