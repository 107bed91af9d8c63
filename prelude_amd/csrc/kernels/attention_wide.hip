// Paged causal attention on the matrix cores for keys and values of widths of their own that are not known when this is
// compiled: keys of `kd` elements (a multiple of 8 up to 512), values of `vd` (a multiple of 4 up to 256), `nkv` key heads and
// `nv` value heads (fewer value heads than key heads: key head k goes with value head k mod nv; more: the query heads are
// dealt out to them in runs as to the key heads), an optional window, optional chunks (a query sees the keys of its own chunk
// of `chunk` places alone), an optional sink per head and an optional gate (the output times sigmoid(gate), a number per value
// column of every head).  bfloat16 storage, 32-bit scores, sums and softmax.  The inner arithmetic and its operand layout are those of attention_mfma_core.h; the
// kernels are compiled for bounds of the widths; what lies between a width and its bound takes part in the products as
// zeros (a branch around it would end a basic block, and operands could no longer be asked for ahead of their use).
//
//   attn_wide_kernel     portions of several tokens.  A workgroup of eight wavefronts owns a tile of 64 * QT tokens of one
//                        head.  Blocks of 64 keys go through LDS (asked for a block ahead); wavefront w works on the tokens
//                        of group w % 4 (QT times 16 of them, which share every operand read from LDS) and on one half of
//                        every block's keys, w / 4; the halves' sums are merged through LDS at the end.  Which keys are
//                        added up in which order follows from their positions alone.
//   attn_shared_kernel   single tokens: up to sixteen query heads that read the same key head are the columns of a score
//                        tile, so every key is read once for all of them; the probabilities are masked per value head where
//                        their sums are formed.  The keys are cut into splits anchored at multiples
//                        of split_keys; attn_shared_merge_kernel adds the splits up.
#include "common.h"
#include "api.h"
#include "attention_mfma_core.h"

namespace pa {

constexpr int kWideKeys = 64;    // keys a block
constexpr int kWideWaves = 8;
constexpr int kWideThreads = kWideWaves * kWave;

struct WideArgs {
  const bf16* q;        // [tokens, nh, kd]
  const bf16* kc;       // [page, nkv, offset, kd]
  const bf16* vc;       // [page, nv, vd, offset]
  const int* block_table;
  int table_stride;
  const int* seq_ids;   // null: 0, 1, ..
  const int* cu_q;
  const int* context_lens;
  bf16* out;
  size_t out_stride;
  int nh, nkv, nv, kd, vd, page_shift, window;
  ScoreMap sm;
  int chunk;
  const bf16* gate;     // [tokens, gate_stride], a column per value column of every head; or null
  size_t gate_stride;
  __device__ __forceinline__ float gated(float v, size_t row, int h, int d) const {
    return gate ? v / (1.0f + __expf(-(float)gate[row * gate_stride + (size_t)h * vd + d])) : v;
  }
  __device__ __forceinline__ int value_head(int h) const { return nv <= nkv ? (h / (nh / nkv)) % nv : h / (nh / nv); }
};

// Rows are padded to 32 bytes past a multiple of 64, at which 16-byte reads of sixteen rows run at the full rate.
template <int KDM, int VDM, int QT, int NBUF>
struct WideLds {
  static constexpr int KROW = KDM + 16, VROW = kWideKeys + 16;   // elements
  static constexpr int kStage = NBUF * (kWideKeys * KROW + VDM * VROW) * 2;
  static constexpr int kPerLane = QT * (VDM / 4 + 2);           // floats a lane hands over when the halves are merged
  static constexpr int kMerge = 4 * kWave * kPerLane * 4;
  static constexpr int kBytes = kStage > kMerge ? kStage : kMerge;
};

template <int KDM, int VDM, int QT, int NBUF>
__global__ __launch_bounds__(kWideThreads) void attn_wide_kernel(WideArgs a) {
  typedef WideLds<KDM, VDM, QT, NBUF> L;
  constexpr int KS = KDM / 32, OT = VDM / 16;
  constexpr int NK = KDM / 64, NV = VDM / 64;     // 16-byte pieces of K and V^T a thread stages a block
  extern __shared__ __align__(16) unsigned char lds_raw[];
  bf16* lk = reinterpret_cast<bf16*>(lds_raw);                          // [NBUF][64][KROW]
  bf16* lv = lk + NBUF * kWideKeys * L::KROW;                           // [NBUF][VDM][VROW]
  const int tid = threadIdx.x, wave = tid / kWave, lane = tid % kWave;
  const int g = lane / 16, r = lane % 16;
  const int tg = wave % 4, half = wave / 4;
  const int h = blockIdx.x;
  const int seq = a.seq_ids ? a.seq_ids[blockIdx.z] : (int)blockIdx.z;
  const int row0 = a.cu_q[seq];
  const int q_len = a.cu_q[seq + 1] - row0;
  constexpr int kTile = 64 * QT;
  const int tile = (q_len + kTile - 1) / kTile - 1 - (int)blockIdx.y;   // late tiles first
  if (tile < 0) return;                                                // the same for the whole workgroup
  const int* table = a.block_table + (size_t)seq * a.table_stride;
  const int kvh = h / (a.nh / a.nkv), vh = a.value_head(h);
  const int start = a.context_lens[seq] - q_len, window = a.window;
  const int cpk = a.kd / 8;
  const int shift = a.page_shift, mask = (1 << shift) - 1;

  // what the workgroup stages, and what this wavefront's tokens see
  const int wg_first = start + tile * kTile;
  const int wg_last = start + (tile * kTile + kTile - 1 < q_len ? tile * kTile + kTile - 1 : q_len - 1);
  const int wg_lo = first_visible(wg_first, window, a.chunk);
  const int wg_hi = wg_last + 1;
  const int t0 = tile * kTile + tg * 16 * QT;
  const bool wave_on = t0 < q_len;
  const int last_valid = t0 + 16 * QT - 1 < q_len ? t0 + 16 * QT - 1 : q_len - 1;
  const int first_pos = start + t0, last_pos = start + last_valid;
  const int lo = first_visible(first_pos, window, a.chunk);
  const int hi = last_pos + 1;
  const int all_lo = first_visible(last_pos, window, a.chunk);
  const int all_hi = first_pos + 1;

  bf16x8 qf[QT][KS];
#pragma unroll
  for (int j = 0; j < QT; ++j) {
    const int t = t0 + 16 * j + r;
    const bf16* qrow = a.q + ((size_t)(row0 + (t < q_len ? t : 0)) * a.nh + h) * a.kd;
#pragma unroll
    for (int ks = 0; ks < KS; ++ks)
      qf[j][ks] = (t < q_len && 32 * ks + 8 * g < a.kd) ? *reinterpret_cast<const bf16x8*>(qrow + 32 * ks + 8 * g) : zero8();
  }
  HeadState<VDM> st[QT];

  // columns of K from kd and rows of V^T from vd on hold zeros throughout
  const int pad = KDM - a.kd;
  for (int i = tid; i < NBUF * kWideKeys * pad; i += kWideThreads) lk[(i / pad) * L::KROW + a.kd + i % pad] = (bf16)0.f;
  const int vpad = VDM - a.vd;
  for (int i = tid; i < NBUF * vpad * kWideKeys; i += kWideThreads) {
    const int b = i / (vpad * kWideKeys), e = i % (vpad * kWideKeys);
    lv[(b * VDM + a.vd + e / kWideKeys) * L::VROW + e % kWideKeys] = (bf16)0.f;
  }

  // a thread's pieces of a block: K piece i is 16 bytes of one key's row, V^T piece i the eight keys 8 (tid % 8) .. of one row
  int kkey[NK], kcol[NK];
  bool kon[NK];
#pragma unroll
  for (int i = 0; i < NK; ++i) {
    const int p = i * kWideThreads + tid;
    kon[i] = p < kWideKeys * cpk;
    kkey[i] = kon[i] ? p / cpk : 0;
    kcol[i] = kon[i] ? 8 * (p % cpk) : 0;
  }
  const int vd_row = tid / 8, v8 = 8 * (tid % 8);
  const int lo_page = wg_lo >> shift, hi_page = (wg_hi - 1) >> shift;
  int kpage[NK], vpage = 0, at = 0;
  bf16x8 kr[NK], vr[NV];
  auto load_pages = [&](int key0) {
    at = key0;
#pragma unroll
    for (int i = 0; i < NK; ++i) {
      int p = (key0 + kkey[i]) >> shift;
      p = p < lo_page ? lo_page : (p > hi_page ? hi_page : p);
      kpage[i] = table[p];
    }
    int p = (key0 + v8) >> shift;
    p = p < lo_page ? lo_page : (p > hi_page ? hi_page : p);
    vpage = table[p];
  };
  auto load = [&]() {
    // (no load stands under a branch: pieces and rows that do not exist are read from ones that do and not stored)
#pragma unroll
    for (int i = 0; i < NK; ++i)
      kr[i] = *reinterpret_cast<const bf16x8*>(a.kc + ((((size_t)kpage[i] * a.nkv + kvh) << shift) + ((at + kkey[i]) & mask)) * a.kd + kcol[i]);
#pragma unroll
    for (int i = 0; i < NV; ++i) {
      const int d = 64 * i + vd_row < a.vd ? 64 * i + vd_row : a.vd - 1;
      vr[i] = *reinterpret_cast<const bf16x8*>(a.vc + ((((size_t)vpage * a.nv + vh) * a.vd + d) << shift) + ((at + v8) & mask));
    }
  };
  auto store = [&](int buf) {
#pragma unroll
    for (int i = 0; i < NK; ++i)
      if (kon[i]) {
        const int key = kkey[i];   // 32 s + 8 a + 4 t + i  ->  row 32 s + 16 t + 4 a + i
        const int row = (key & 32) | ((key & 4) << 2) | ((key & 24) >> 1) | (key & 3);
        *reinterpret_cast<bf16x8*>(lk + (buf * kWideKeys + row) * L::KROW + kcol[i]) = kr[i];
      }
#pragma unroll
    for (int i = 0; i < NV; ++i) {
      const int d = 64 * i + vd_row;
      if (d < a.vd) *reinterpret_cast<bf16x8*>(lv + (buf * VDM + d) * L::VROW + v8) = vr[i];
    }
  };
  const float c = a.sm.c, over = kLazyLog2 / c;
  auto attend = [&](int buf, int key0) {
    const bf16* kb = lk + (buf * kWideKeys + 32 * half + r) * L::KROW + 8 * g;
    f32x4 acc[2][QT];
#pragma unroll
    for (int t = 0; t < 2; ++t)
#pragma unroll
      for (int j = 0; j < QT; ++j) acc[t][j] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int ks = 0; ks < KS; ++ks) {
      const bf16x8 k0 = *reinterpret_cast<const bf16x8*>(kb + 32 * ks);
      const bf16x8 k1 = *reinterpret_cast<const bf16x8*>(kb + 16 * L::KROW + 32 * ks);
#pragma unroll
      for (int j = 0; j < QT; ++j) {
        acc[0][j] = mfma16(k0, qf[j][ks], acc[0][j]);
        acc[1][j] = mfma16(k1, qf[j][ks], acc[1][j]);
      }
    }
    const bool masked = key0 < all_lo || key0 + 32 > all_hi;
    bf16x8 pb[QT];
#pragma unroll
    for (int j = 0; j < QT; ++j) {
      float s[8];
#pragma unroll
      for (int t = 0; t < 2; ++t)
#pragma unroll
        for (int i = 0; i < 4; ++i) s[4 * t + i] = acc[t][j][i];
      if (masked) {
        const int my_pos = first_pos + 16 * j + r;
        const int my_lo = first_visible(my_pos, window, a.chunk);
#pragma unroll
        for (int i = 0; i < 8; ++i) {
          const int key = key0 + 8 * g + i;
          if (!(key >= my_lo && key <= my_pos)) s[i] = -INFINITY;
        }
      }
      float mx = s[0];
#pragma unroll
      for (int i = 1; i < 8; ++i) mx = fmaxf(mx, s[i]);
      if (__any(mx > st[j].lim)) {
        asm volatile("" ::: "memory");
        move_reference<VDM>(st[j], mx, c, over);
      }
      pb[j] = probabilities(s, c, st[j].shift);
    }
    const bf16x8 ones = ones8();
#pragma unroll
    for (int j = 0; j < QT; ++j) st[j].l = mfma16(ones, pb[j], st[j].l);
    const bf16* vb = lv + (buf * VDM + r) * L::VROW + 32 * half + 8 * g;
#pragma unroll
    for (int t = 0; t < OT; ++t) {
      const bf16x8 va = *reinterpret_cast<const bf16x8*>(vb + 16 * t * L::VROW);
#pragma unroll
      for (int j = 0; j < QT; ++j) st[j].o[t] = mfma16(va, pb[j], st[j].o[t]);
    }
  };

  int key0 = (wg_lo / kWideKeys) * kWideKeys;
  load_pages(key0);
  load();
  if (NBUF == 2) {
    if (key0 + kWideKeys < wg_hi) load_pages(key0 + kWideKeys);
    store(0);
    if (key0 + kWideKeys < wg_hi) {
      load();
      if (key0 + 2 * kWideKeys < wg_hi) load_pages(key0 + 2 * kWideKeys);
    }
    __syncthreads();
    int buf = 0;
    for (; key0 < wg_hi; key0 += kWideKeys, buf ^= 1) {
      if (key0 + kWideKeys < wg_hi) {
        store(buf ^ 1);                          // the next block, asked for a block ago
        if (key0 + 2 * kWideKeys < wg_hi) {
          load();                                // the one after it, from the pages looked up a block ago
          if (key0 + 3 * kWideKeys < wg_hi) load_pages(key0 + 3 * kWideKeys);
        }
      }
      const int k32 = key0 + 32 * half;
      if (wave_on && k32 + 32 > lo && k32 < hi) attend(buf, k32);
      __syncthreads();
    }
  } else {
    for (; key0 < wg_hi; key0 += kWideKeys) {
      store(0);
      __syncthreads();
      if (key0 + kWideKeys < wg_hi) {
        load_pages(key0 + kWideKeys);
        load();
      }
      const int k32 = key0 + 32 * half;
      if (wave_on && k32 + 32 > lo && k32 < hi) attend(0, k32);
      __syncthreads();
    }
  }
  // the second half's sums to the first, lane to lane (the loop's last barrier leaves the buffers free)
  float* mg = reinterpret_cast<float*>(lds_raw) + (size_t)tg * L::kPerLane * kWave + lane;
  if (half == 1) {
#pragma unroll
    for (int j = 0; j < QT; ++j) {
      float* m = mg + j * (VDM / 4 + 2) * kWave;
      m[0] = st[j].reference();
      m[kWave] = st[j].l[0];
#pragma unroll
      for (int t = 0; t < OT; ++t)
#pragma unroll
        for (int i = 0; i < 4; ++i) m[(2 + 4 * t + i) * kWave] = st[j].o[t][i];
    }
  }
  __syncthreads();
  if (half == 1 || !wave_on) return;
#pragma unroll
  for (int j = 0; j < QT; ++j) {
    const int t = t0 + 16 * j + r;
    if (t >= q_len) continue;
    const float* m = mg + j * (VDM / 4 + 2) * kWave;
    const float ra = st[j].reference(), rb = m[0];
    const float ref = fmaxf(ra, rb);
    const float fa = ra == -INFINITY ? 0.f : exp2f(ra - ref), fb = rb == -INFINITY ? 0.f : exp2f(rb - ref);
    const float inv = 1.0f / (st[j].l[0] * fa + m[kWave] * fb + a.sm.sink_term(h, ref));
    bf16* orow = a.out + (size_t)(row0 + t) * a.out_stride + (size_t)h * a.vd;
#pragma unroll
    for (int tt = 0; tt < OT; ++tt)
      if (16 * tt + 4 * g < a.vd) {
        bf16x4 v;
#pragma unroll
        for (int i = 0; i < 4; ++i)
          v[i] = (bf16)a.gated((st[j].o[tt][i] * fa + m[(2 + 4 * tt + i) * kWave] * fb) * inv, row0 + t, h, 16 * tt + 4 * g + i);
        *reinterpret_cast<bf16x4*>(orow + 16 * tt + 4 * g) = v;
      }
  }
}

// ---- single tokens: the heads over one key head together ------------------------------------------------------------------------
constexpr int kSharedWaves = 8;
constexpr int kSharedBlock = 128;   // keys a block: a wavefront a tile of 16 of them

// Grid (key heads x tiles of 16 of a key head's query heads, splits, sequences).  A block's scores are eight tiles of 16 keys x 16 heads, one a wavefront; they
// share one reference maximum per head through LDS, and their probabilities lie in LDS as the operands of the second
// product.  That product's units, (value head, 32 keys), are dealt out to the wavefronts; the V^T of a wavefront's first two
// units is asked for together with the keys, so that a short context is one trip to memory.
template <int KDM, int VDM>
__global__ __launch_bounds__(kSharedWaves* kWave) void attn_shared_kernel(WideArgs a, float* __restrict__ part_o,
                                                                         float* __restrict__ part_ml, int split_keys, int max_splits) {
  constexpr int KS = KDM / 32, OT = VDM / 16;
  extern __shared__ float lds_o[];                    // [waves][16 heads][vd + 1]
  __shared__ float lds_max[kSharedWaves][16];
  __shared__ float lds_l[4][16];
  __shared__ __align__(16) bf16 lds_p[kSharedBlock / 32][16][32 + 8];
  const int tid = threadIdx.x, wave = tid / kWave, lane = tid % kWave;
  const int g = lane / 16, r = lane % 16;
  const int seq = a.seq_ids ? a.seq_ids[blockIdx.z] : (int)blockIdx.z;
  const int row = a.cu_q[seq];
  const int ctx = a.context_lens[seq];
  const int pos = ctx - 1;
  const int lo = first_visible(pos, a.window, a.chunk);
  const int first_split = lo / split_keys;
  const int nsplit = (ctx + split_keys - 1) / split_keys - first_split;
  if ((int)blockIdx.y >= nsplit) return;
  const int s0 = (first_split + (int)blockIdx.y) * split_keys;
  const int klo = s0 > lo ? s0 : lo, khi = s0 + split_keys < ctx ? s0 + split_keys : ctx;   // never empty
  const int* table = a.block_table + (size_t)seq * a.table_stride;
  const int shift = a.page_shift, mask = (1 << shift) - 1;
  const int group = a.nh / a.nkv, tiles = (group + 15) / 16;
  const int kvh = blockIdx.x / tiles, tile = blockIdx.x % tiles;
  const int head0 = kvh * group + tile * 16;
  const int heads = group - tile * 16 < 16 ? group - tile * 16 : 16;
  const int my_head = head0 + (r < heads ? r : heads - 1);
  const int my_vh = a.value_head(my_head);
  const int vh0 = a.value_head(head0);
  const int units = 4 * (a.value_head(head0 + heads - 1) - vh0 + 1);

  // queries as they are up to kd and zeros from there on: what the keys' loads bring beyond kd does not matter
  bf16x8 qf[KS];
  const bf16* qrow = a.q + ((size_t)row * a.nh + my_head) * a.kd;
#pragma unroll
  for (int ks = 0; ks < KS; ++ks) {
    const int at = 32 * ks + 8 * g;
    const bf16x8 x = *reinterpret_cast<const bf16x8*>(qrow + (at < a.kd ? at : 0));
    qf[ks] = at < a.kd ? x : zero8();
  }
  f32x4 o[OT], l{0.f, 0.f, 0.f, 0.f};
#pragma unroll
  for (int t = 0; t < OT; ++t) o[t] = f32x4{0.f, 0.f, 0.f, 0.f};
  float ref = -INFINITY;                              // the column's largest score so far, the same in every wavefront
  const float c = a.sm.c;
  for (int b0 = s0; b0 < khi; b0 += kSharedBlock) {
    if (b0 + kSharedBlock <= klo) continue;
    const int step0 = b0 + 32 * (wave / 2), tt = wave % 2;
    // row r of the tile is key 8 (r / 4) + 4 tt + r % 4 of its 32
    int key = step0 + 8 * (r / 4) + 4 * tt + (r % 4);
    key = key < klo ? klo : (key >= khi ? khi - 1 : key);
    const bf16* krow = a.kc + ((((size_t)table[key >> shift] * a.nkv + kvh) << shift) + (key & mask)) * a.kd;
    bf16x8 kf[KS];
#pragma unroll
    for (int ks = 0; ks < KS; ++ks) {
      const int at = 32 * ks + 8 * g;
      kf[ks] = *reinterpret_cast<const bf16x8*>(krow + (at < a.kd ? at : 0));
    }
    // the eight keys 8g .. of unit u's 32, of its value head: one 16-byte piece (pages hold eight keys or more)
    auto load_values = [&](int u, bf16x8* va) {
      int ck = b0 + 32 * (u % 4) + 8 * g;
      if (ck + 7 < klo) ck = klo & ~7;
      if (ck >= khi) ck = (khi - 1) & ~7;
      const bf16* v = a.vc + ((((size_t)table[ck >> shift] * a.nv + vh0 + u / 4) * a.vd) << shift) + (ck & mask);
#pragma unroll
      for (int t = 0; t < OT; ++t) {
        const int d = 16 * t + r < a.vd ? 16 * t + r : a.vd - 1;      // rows past the value's width are not written out
        va[t] = *reinterpret_cast<const bf16x8*>(v + ((size_t)d << shift));
      }
    };
    const int u0 = wave < units ? wave : units - 1, u1 = wave + kSharedWaves < units ? wave + kSharedWaves : units - 1;
    bf16x8 va0[OT], va1[OT];
    load_values(u0, va0);
    load_values(u1, va1);
    f32x4 acc{0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int ks = 0; ks < KS; ++ks) acc = mfma16(kf[ks], qf[ks], acc);
    float s[4], mx = -INFINITY;
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const int k = step0 + 8 * g + 4 * tt + i;
      s[i] = (k >= klo && k < khi) ? acc[i] : -INFINITY;
      mx = fmaxf(mx, s[i]);
    }
    mx = xor_max16_32(mx);
    if (g == 0) lds_max[wave][r] = mx;
    __syncthreads();
    float m_new = ref;
#pragma unroll
    for (int w = 0; w < kSharedWaves; ++w) m_new = fmaxf(m_new, lds_max[w][r]);   // finite: a block that is worked on has a visible key
    const float alpha = ref == -INFINITY ? 1.0f : __builtin_amdgcn_exp2f((ref - m_new) * c);   // the first block rescales nothing
    ref = m_new;
    bf16x4 p4;
#pragma unroll
    for (int i = 0; i < 4; ++i) p4[i] = (bf16)__builtin_amdgcn_exp2f((s[i] - m_new) * c);
    *reinterpret_cast<bf16x4*>(&lds_p[wave / 2][r][8 * g + 4 * tt]) = p4;
    __syncthreads();
#pragma unroll
    for (int t = 0; t < OT; ++t)
#pragma unroll
      for (int i = 0; i < 4; ++i) o[t][i] *= alpha;
#pragma unroll
    for (int i = 0; i < 4; ++i) l[i] *= alpha;
    if (wave < 4) l = mfma16(ones8(), *reinterpret_cast<const bf16x8*>(&lds_p[wave][r][8 * g]), l);
    auto add_unit = [&](int u, const bf16x8* va) {
      const bf16x8 pb = *reinterpret_cast<const bf16x8*>(&lds_p[u % 4][r][8 * g]);
      bf16x8 pm;   // the probabilities of the heads that read the unit's value head
#pragma unroll
      for (int i = 0; i < 8; ++i) pm[i] = my_vh == vh0 + u / 4 ? pb[i] : (bf16)0.f;
#pragma unroll
      for (int t = 0; t < OT; ++t) o[t] = mfma16(va[t], pm, o[t]);
    };
    if (wave < units) add_unit(u0, va0);
    if (wave + kSharedWaves < units) add_unit(u1, va1);
    for (int u = wave + 2 * kSharedWaves; u < units; u += kSharedWaves) {
      load_values(u, va0);
      add_unit(u, va0);
    }
    __syncthreads();                                  // the probabilities have been read
  }
  const int ostride = a.vd + 1;
  if (wave < 4 && g == 0) lds_l[wave][r] = l[0];
#pragma unroll
  for (int t = 0; t < OT; ++t)
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const int d = 16 * t + 4 * g + i;
      if (d < a.vd) lds_o[((size_t)wave * 16 + r) * ostride + d] = o[t][i];
    }
  if (wave == 0 && g == 0) lds_max[0][r] = ref;
  __syncthreads();
  for (int e = tid; e < heads * a.vd; e += kSharedWaves * kWave) {
    const int j = e / a.vd, d = e % a.vd;
    float ov = 0.f;
#pragma unroll
    for (int v = 0; v < kSharedWaves; ++v) ov += lds_o[((size_t)v * 16 + j) * ostride + d];   // in the order of the wavefronts
    const float lv = (lds_l[0][j] + lds_l[1][j]) + (lds_l[2][j] + lds_l[3][j]);
    const float mm = lds_max[0][j] * c;               // the exponent's reference
    const int h = head0 + j;
    if (nsplit == 1) {
      a.out[(size_t)row * a.out_stride + (size_t)h * a.vd + d] = (bf16)a.gated(ov / (lv + a.sm.sink_term(h, mm)), row, h, d);
    } else {
      const size_t slot = ((size_t)blockIdx.z * a.nh + h) * max_splits + blockIdx.y;
      part_o[slot * a.vd + d] = ov;
      if (d == 0) {
        part_ml[slot * 2] = mm;
        part_ml[slot * 2 + 1] = lv;
      }
    }
  }
}

// Grid (heads, sequences); a thread a value dimension.
__global__ __launch_bounds__(256) void attn_shared_merge_kernel(WideArgs a, const float* __restrict__ part_o,
                                                               const float* __restrict__ part_ml, int split_keys, int max_splits) {
  const int h = blockIdx.x;
  const int seq = a.seq_ids ? a.seq_ids[blockIdx.y] : (int)blockIdx.y;
  const int ctx = a.context_lens[seq];
  const int pos = ctx - 1;
  const int lo = first_visible(pos, a.window, a.chunk);
  const int nsplit = (ctx + split_keys - 1) / split_keys - lo / split_keys;
  if (nsplit == 1) return;                            // written by the first kernel
  const size_t base = ((size_t)blockIdx.y * a.nh + h) * max_splits;
  const int lane = threadIdx.x % kWave, d = threadIdx.x;
  float mm = -INFINITY;
  for (int s = lane; s < nsplit; s += kWave) mm = fmaxf(mm, part_ml[(base + s) * 2]);
  mm = wave_max(mm);
  float o = 0.f, l = 0.f;
  constexpr int kBatch = 8;
  for (int b = 0; b < nsplit; b += kBatch) {          // in the order of the splits, a batch asked for together
    float po[kBatch], pm[kBatch], pl[kBatch];
#pragma unroll
    for (int i = 0; i < kBatch; ++i) {
      const int s = b + i < nsplit ? b + i : nsplit - 1;
      po[i] = d < a.vd ? part_o[(base + s) * a.vd + d] : 0.f;
      pm[i] = part_ml[(base + s) * 2];
      pl[i] = part_ml[(base + s) * 2 + 1];
    }
#pragma unroll
    for (int i = 0; i < kBatch; ++i)
      if (b + i < nsplit) {
        const float f = exp2f(pm[i] - mm);
        o += po[i] * f;
        l += pl[i] * f;
      }
  }
  const size_t row = a.cu_q[seq];
  if (d < a.vd) a.out[row * a.out_stride + (size_t)h * a.vd + d] = (bf16)a.gated(o / (l + a.sm.sink_term(h, mm)), row, h, d);
}

template <int KDM, int VDM, int QT, int NBUF>
static int launch_wide(hipStream_t st, const WideArgs& a, int nseq, int max_q_len) {
  typedef WideLds<KDM, VDM, QT, NBUF> L;
  static const hipError_t allowed = hipFuncSetAttribute(reinterpret_cast<const void*>(&attn_wide_kernel<KDM, VDM, QT, NBUF>),
                                                        hipFuncAttributeMaxDynamicSharedMemorySize, L::kBytes);
  if (allowed != hipSuccess) return pa::fail("attn_wide: %d bytes of LDS refused: %s", L::kBytes, hipGetErrorString(allowed));
  dim3 grid(a.nh, (max_q_len + 64 * QT - 1) / (64 * QT), nseq);
  hipLaunchKernelGGL((attn_wide_kernel<KDM, VDM, QT, NBUF>), grid, dim3(kWideThreads), L::kBytes, st, a);
  return check_launch("attn_wide");
}

template <int KDM, int VDM>
static int launch_shared(hipStream_t st, const WideArgs& a, float* work, int nseq, int split_keys, int max_splits) {
  const size_t lds = (size_t)kSharedWaves * 16 * (a.vd + 1) * sizeof(float);
  static const hipError_t allowed = hipFuncSetAttribute(reinterpret_cast<const void*>(&attn_shared_kernel<KDM, VDM>),
                                                        hipFuncAttributeMaxDynamicSharedMemorySize,
                                                        kSharedWaves * 16 * (VDM + 1) * (int)sizeof(float));
  if (allowed != hipSuccess) return pa::fail("attn_shared: %zu bytes of LDS refused: %s", lds, hipGetErrorString(allowed));
  float* part_ml = work;
  float* part_o = work + (size_t)nseq * a.nh * max_splits * 2;
  hipLaunchKernelGGL((attn_shared_kernel<KDM, VDM>), dim3(a.nkv * ((a.nh / a.nkv + 15) / 16), max_splits, nseq), dim3(kSharedWaves * kWave), lds, st, a,
                     part_o, part_ml, split_keys, max_splits);
  if (int rc = check_launch("attn_shared")) return rc;
  if (max_splits == 1) return 0;
  hipLaunchKernelGGL(attn_shared_merge_kernel, dim3(a.nh, nseq), dim3((a.vd + kWave - 1) / kWave * kWave), 0, st, a, part_o, part_ml,
                     split_keys, max_splits);
  return check_launch("attn_shared_merge");
}

}  // namespace pa

using namespace pa;

extern "C" int pa_attn_wide_supports(int kd, int vd, int page_size) {
  return kd > 0 && kd <= 512 && kd % 8 == 0 && vd > 0 && vd <= 256 && vd % 4 == 0 && page_size >= 8 && (page_size & (page_size - 1)) == 0;
}

static int wide_check(const char* what, int nseq, int nh, int nkv, int nv, int kd, int vd, int page_size, int table_stride, int window,
                      float scale, long out_stride, const void* q, const void* kc, const void* vc, const void* out) {
  PA_REQUIRE(pa_attn_wide_supports(kd, vd, page_size), "%s: keys of %d, values of %d or pages of %d are not taken", what, kd, vd, page_size);
  PA_REQUIRE(nseq > 0 && nh > 0 && nkv > 0 && nv > 0 && nh % nkv == 0 && (nv <= nkv ? nkv % nv == 0 : nh % nv == 0),
             "%s: %d sequences, %d query heads over %d key and %d value heads", what, nseq, nh, nkv, nv);
  PA_REQUIRE(table_stride > 0 && window >= 0 && scale > 0.f, "%s: table stride %d, window %d, scale %g", what, table_stride, window, (double)scale);
  PA_REQUIRE(out_stride >= (long)nh * vd && out_stride % 4 == 0, "%s: an output stride of %ld for %d heads of %d", what, out_stride, nh, vd);
  PA_REQUIRE(((uintptr_t)q & 15) == 0 && ((uintptr_t)kc & 15) == 0 && ((uintptr_t)vc & 15) == 0 && ((uintptr_t)out & 7) == 0,
             "%s: operands are not aligned", what);
  return 0;
}

extern "C" int pa_attn_wide(void* stream, const void* q, const void* kc, const void* vc, const int* block_table, int table_stride,
                            const int* seq_ids, const int* cu_q, const int* context_lens, void* out, long out_stride, int nseq,
                            int max_q_len, int nh, int nkv, int nv, int kd, int vd, int page_size, int window, float scale,
                            const float* sink, int chunk, const void* gate, long gate_stride) {
  if (nseq == 0 || max_q_len == 0) return 0;
  if (int rc = wide_check("attn_wide", nseq, nh, nkv, nv, kd, vd, page_size, table_stride, window, scale, out_stride, q, kc, vc, out)) return rc;
  PA_REQUIRE(chunk >= 0 && (!gate || gate_stride >= (long)nh * vd), "attn_wide: chunks of %d places or a gate of %ld columns", chunk, gate_stride);
  PA_REQUIRE(max_q_len > 0 && nseq <= 65535 && (max_q_len + 63) / 64 <= 65535, "attn_wide: portions of %d tokens", max_q_len);
  WideArgs a{(const bf16*)q, (const bf16*)kc, (const bf16*)vc, block_table, table_stride, seq_ids, cu_q, context_lens, (bf16*)out,
             (size_t)out_stride, nh, nkv, nv, kd, vd, __builtin_ctz(page_size), window, score_map(scale, 0.f, sink), chunk,
             (const bf16*)gate, (size_t)gate_stride};
  hipStream_t st = (hipStream_t)stream;
  if (vd <= 64) {
    if (kd <= 64) return launch_wide<64, 64, 2, 2>(st, a, nseq, max_q_len);
    if (kd <= 128) return launch_wide<128, 64, 2, 2>(st, a, nseq, max_q_len);
    if (kd <= 256) return launch_wide<256, 64, 2, 2>(st, a, nseq, max_q_len);
  }
  if (vd <= 128) {
    if (kd <= 64) return launch_wide<64, 128, 2, 2>(st, a, nseq, max_q_len);
    if (kd <= 128) return launch_wide<128, 128, 2, 2>(st, a, nseq, max_q_len);
    if (kd <= 192) return launch_wide<192, 128, 2, 2>(st, a, nseq, max_q_len);
    if (kd <= 256) return launch_wide<256, 128, 2, 2>(st, a, nseq, max_q_len);
    return launch_wide<512, 128, 1, 1>(st, a, nseq, max_q_len);
  }
  if (kd <= 256) return launch_wide<256, 256, 1, 1>(st, a, nseq, max_q_len);
  return launch_wide<512, 256, 1, 1>(st, a, nseq, max_q_len);
}

// 32-bit words of workspace
extern "C" long pa_attn_shared_workspace(int nseq, int nh, int vd, int max_splits) {
  return max_splits > 1 ? (long)nseq * nh * max_splits * (vd + 2L) : 1;
}

extern "C" int pa_attn_shared(void* stream, const void* q, const void* kc, const void* vc, const int* block_table, int table_stride,
                              const int* seq_ids, const int* cu_q, const int* context_lens, void* out, long out_stride, float* work,
                              int nseq, int nh, int nkv, int nv, int kd, int vd, int page_size, int window, float scale, const float* sink,
                              int split_keys, int max_splits, int chunk, const void* gate, long gate_stride) {
  if (nseq == 0) return 0;
  if (int rc = wide_check("attn_shared", nseq, nh, nkv, nv, kd, vd, page_size, table_stride, window, scale, out_stride, q, kc, vc, out)) return rc;
  PA_REQUIRE(chunk >= 0 && (!gate || gate_stride >= (long)nh * vd), "attn_shared: chunks of %d places or a gate of %ld columns", chunk, gate_stride);
  PA_REQUIRE(split_keys > 0 && split_keys % kSharedBlock == 0 && max_splits > 0 && max_splits <= 65535 && nseq <= 65535 && work,
             "attn_shared: splits of %d keys, %d at most", split_keys, max_splits);
  WideArgs a{(const bf16*)q, (const bf16*)kc, (const bf16*)vc, block_table, table_stride, seq_ids, cu_q, context_lens, (bf16*)out,
             (size_t)out_stride, nh, nkv, nv, kd, vd, __builtin_ctz(page_size), window, score_map(scale, 0.f, sink), chunk,
             (const bf16*)gate, (size_t)gate_stride};
  hipStream_t st = (hipStream_t)stream;
  if (vd <= 128) {
    if (kd <= 128) return launch_shared<128, 128>(st, a, work, nseq, split_keys, max_splits);
    if (kd <= 256) return launch_shared<256, 128>(st, a, work, nseq, split_keys, max_splits);
    return launch_shared<512, 128>(st, a, work, nseq, split_keys, max_splits);
  }
  if (kd <= 256) return launch_shared<256, 256>(st, a, work, nseq, split_keys, max_splits);
  return launch_shared<512, 256>(st, a, work, nseq, split_keys, max_splits);
}
