// The tile both attention libraries walk over the paged cache on the matrix cores (bf16, gfx950), and the flash kernel
// made of it.
//
// Both kernels compute S^T = K . Q^T and O^T = V^T . P with
// v_mfma_f32_16x16x32_bf16, whose operands want, per lane, 8 consecutive
// elements of the contraction dimension:
//   A (16 x 32): lane l holds A[l % 16][8 * (l / 16) .. + 8]
//   B (32 x 16): lane l holds B[8 * (l / 16) .. + 8][l % 16]
//   D (16 x 16): lane l holds D[4 * (l / 16) + r][l % 16], r = 0..3
// K pages [Hkv][D / 8][page][8] give A = 8-element pieces of K rows straight from
// memory (contraction over d; the pieces of consecutive keys are contiguous, so
// a quad of lanes reads 64 contiguous bytes); V pages [Hkv][D][page] (transposed)
// give A = V^T rows straight from memory (contraction over keys). K and V are
// not staged through LDS.
//
// A block of 32 keys is scored by two MFMA chains (a = 0, 1). Row i of chain a
// is key  kb + 8 * (i / 4) + 4 * a + (i % 4),  so lane group g = l / 16 ends up
// with the scores of keys kb + 8 g .. kb + 8 g + 7 in its eight result
// registers: exactly the B operand of the P.V product, with no shuffle.
// A query (a column, l % 16) keeps its running maximum, sum and output column in
// the same lanes through both products.
//
// Options of the flash kernel (KIND other than PLAIN; dinfer_attn_flash_ext, which serves single rows as well): the first
// keep_first keys stay visible behind the window (one more short run of key blocks, walked by wave 0); a sink a head joins
// the softmax's denominator when the waves' parts are combined; 2^(-slope_exp (h + 1) / H) times the distance is taken off
// the scores (in raw score units, before the maximum); the scores are capped, C tanh(s / C), and a query sees only the keys
// of its own chunk of positions (a lower bound a row, like a window's); the output is multiplied by out_scale; or (SIGMOID)
// the weights are sigmoids of the scores plus a bias a head, and nothing is normalised.
#pragma once
#include "common.cuh"

namespace dinfer {
namespace {

constexpr float LOG2E = 1.4426950408889634f;

__device__ __forceinline__ bf16x8 zero8() {
  bf16x8 z;
#pragma unroll
  for (int i = 0; i < 8; ++i) z[i] = (bf16)0.f;
  return z;
}

__device__ __forceinline__ int lane_of() { return threadIdx.x & 63; }

// 2^x by the hardware instruction alone: results below 2^-126 become 0, which a softmax weight may
__device__ __forceinline__ float exp2_raw(float x) { return __builtin_amdgcn_exp2f(x); }

__device__ __forceinline__ f32x4 mfma16(bf16x8 a, bf16x8 b, f32x4 c) {
  return __builtin_amdgcn_mfma_f32_16x16x32_bf16(a, b, c, 0, 0, 0);
}

// Block-table entries of 64 consecutive pages of one request, one per lane; a lane gets the
// entry it needs by a cross-lane read, so no key block waits for a table load of its own.
// P2: the page size is a power of two (shifts and masks instead of divisions).
template <bool P2>
struct Pages {
  const int32_t* bt;
  int max_blocks, base, reg, ps, ps_shift;

  __device__ __forceinline__ void init(const int32_t* table, int max_blocks_, int page_size, int first_key) {
    bt = table;
    max_blocks = max_blocks_;
    ps = page_size;
    ps_shift = P2 ? __builtin_ctz(page_size) : 0;
    fetch(page_of(first_key));
  }
  __device__ __forceinline__ int page_of(int key) const { return P2 ? key >> ps_shift : key / ps; }
  __device__ __forceinline__ int offset_of(int key) const { return P2 ? key & (ps - 1) : key % ps; }
  __device__ __forceinline__ void fetch(int first_page) {
    base = first_page;
    const int i = base + (int)(threadIdx.x & 63);
    reg = i < max_blocks ? bt[i] : 0;
  }
  // kb is wave-uniform and only grows; afterwards the pages of keys [kb, kb + 32) are on board
  __device__ __forceinline__ void ensure(int kb) {
    if (page_of(kb + 31) - base >= 64) fetch(page_of(kb));
  }
  // every lane of the wave must call this (it is a cross-lane operation)
  __device__ __forceinline__ int get(int page) const { return __shfl(reg, page - base, 64); }
};

// 16 bytes of cache pages; stream: past the caches (the bytes are used once)
template <bool STREAM>
__device__ __forceinline__ bf16x8 ld16(const bf16* p) {
  if constexpr (STREAM)
    return __builtin_nontemporal_load((const bf16x8*)p);
  else
    return *(const bf16x8*)p;
}

template <int DT, int DV>
struct Frags {
  static constexpr int KS = (DT + 1) / 2;
  bf16x8 k[2][KS];
  bf16x8 v[DV];
};

// NT column tiles (queries, or the heads of a group) against the keys of one request, 32 at a time.
//   qf[t][ks]   B operands of the score product, the whole head in registers
//   col_lo/hi   per column tile and lane: the column's visible keys are [col_lo, col_hi)
//   k_lo, k_hi  the keys this wave may touch at all (held pages, written slots)
// load() issues the loads of one block, compute() consumes them; walk() keeps the next block's
// loads in flight while the current one is computed.
//
// KIND: PLAIN softmax; OPTIONS softmax with options; SIGMOID the options' weights without a softmax: p = sigmoid(scale s +
// bias), nothing normalised over the keys (no running maximum, no sum). DV: 16-wide steps of a value head (DT: of a key).
enum : int { PLAIN = 0, OPTIONS = 1, SIGMOID = 2 };

template <int DT, int NT, bool P2, int KIND = PLAIN, int DV = DT>
struct Tile {
  static constexpr int KS = (DT + 1) / 2;  // 32-wide steps over the head dimension
  static constexpr bool EXT = KIND != PLAIN;
  using F = Frags<DT, DV>;
  float bias_log2e = 0.f;  // SIGMOID: the head's bias in base-2 units
  int keep_first = 0;      // EXT: keys below this stay visible whatever col_lo says
  float slope_raw = 0.f;   // EXT: taken off a raw score per key of distance (the slope divided by the scale)
  float cap = 0.f, cap_in = 0.f;   // OPTIONS: scores become cap tanh(.), cap_in = 2 log2(e) scale / cap (0: no cap)
  static constexpr float LAZY = 6.f;       // weights up to 2^6 before the reference follows the maximum
  f32x4 o[NT][DV];
  float m[NT], l[NT];
  Pages<P2> pages;
  const bf16* kc;
  const bf16* vc;
  int hk, Hkv, k_lo, k_hi;
  int page_stride, head_off;      // elements from key page to key page, and from the page's start to this kv head
  int v_page_stride, v_head_off;  // the same for value pages
  float scale_log2e;

  __device__ __forceinline__ void init(const bf16* kc_, const bf16* vc_, const int32_t* bt, int max_blocks, int hk_,
                                       int Hkv_, int ps, int k_lo_, int k_hi_, float scale_log2e_) {
    kc = kc_; vc = vc_; hk = hk_; Hkv = Hkv_; k_lo = k_lo_; k_hi = k_hi_; scale_log2e = scale_log2e_;
    page_stride = Hkv_ * ps * DT * 16;  // the host checks that this fits 31 bits
    head_off = hk_ * ps * DT * 16;
    v_page_stride = Hkv_ * ps * DV * 16;
    v_head_off = hk_ * ps * DV * 16;
    pages.init(bt, max_blocks, ps, k_lo_ & ~31);
#pragma unroll
    for (int t = 0; t < NT; ++t) {
      m[t] = -INFINITY;
      l[t] = 0.f;
#pragma unroll
      for (int d = 0; d < DV; ++d) o[t][d] = f32x4{0.f, 0.f, 0.f, 0.f};
    }
  }

  // Loads are unconditional: a key outside [k_lo, k_hi) is replaced by the nearest key inside, which
  // lies in a page the request holds, so straight-line code with all loads in flight at once. What
  // was loaded for such a key never counts: its score is masked, and accumulate() zeroes its value.
  // CLAMP = false: the block lies wholly inside [k_lo, k_hi), so no key needs replacing.
  // STREAM: K and V are read with non-temporal loads (a step's keys exceed the caches and each byte is used once).
  template <bool CLAMP, bool STREAM>
  __device__ __forceinline__ void load_k(F& f, int kb) {
    constexpr int D = DT * 16;
    const int lane = threadIdx.x & 63, i16 = lane & 15, g4 = lane >> 4;
    const int last = k_hi - 1;
    // K rows of this lane: keys kg_row + (i16 & 3) and + 4: one aligned group of 8, so one page (page size % 8 == 0)
    int key0 = kb + 8 * (i16 >> 2) + (i16 & 3), key1 = key0 + 4;
    if (CLAMP) {
      key0 = key0 < k_lo ? k_lo : (key0 > last ? last : key0);
      key1 = key1 < k_lo ? k_lo : (key1 > last ? last : key1);
    }
    const int pg0 = pages.get(pages.page_of(key0));
    const int pg1 = CLAMP ? pages.get(pages.page_of(key1)) : pg0;  // clamping may move the two into different pages
    // K pages are [Hkv][D / 8][page][8]: the 16-byte pieces of consecutive keys lie next to each other,
    // so the four lanes of a quad (four consecutive keys, one piece index) read 64 contiguous bytes
    const bf16* kr0 = kc + ((int64_t)pg0 * page_stride + (head_off + pages.offset_of(key0) * 8));
    const bf16* kr1 = CLAMP ? kc + ((int64_t)pg1 * page_stride + (head_off + pages.offset_of(key1) * 8)) : kr0 + 32;
    const int piece = pages.ps * 8;
#pragma unroll
    for (int ks = 0; ks < KS; ++ks) {
      int c = ks * 4 + g4;
      const bool dv = c * 8 < D;  // D % 32 == 16: the upper half of the last step is padding
      if (!dv) c = 0;
      f.k[0][ks] = ld16<STREAM>(kr0 + c * piece);
      f.k[1][ks] = ld16<STREAM>(kr1 + c * piece);
      if (DT % 2 == 1 && ks == KS - 1 && !dv) f.k[0][ks] = f.k[1][ks] = zero8();
    }
  }

  template <bool CLAMP, bool STREAM>
  __device__ __forceinline__ void load_v(F& f, int kb) {
    const int lane = threadIdx.x & 63, i16 = lane & 15, g4 = lane >> 4;
    const int ps = pages.ps;
    // V^T rows of this lane: d = 16 dt + i16, keys kg .. kg + 7 (one page)
    int kg = kb + 8 * g4;
    if (CLAMP) {
      const int g_lo = k_lo & ~7, g_hi = (k_hi - 1) & ~7;
      kg = kg < g_lo ? g_lo : (kg > g_hi ? g_hi : kg);
    }
    const int pgv = pages.get(pages.page_of(kg));
    const bf16* vrow = vc + ((int64_t)pgv * v_page_stride + (v_head_off + i16 * ps + pages.offset_of(kg)));
#pragma unroll
    for (int d = 0; d < DV; ++d) f.v[d] = ld16<STREAM>(vrow + d * 16 * ps);
  }

  template <bool CLAMP, bool STREAM>
  __device__ __forceinline__ void load(F& f, int kb) {
    pages.ensure(kb);
    load_k<CLAMP, STREAM>(f, kb);
    load_v<CLAMP, STREAM>(f, kb);
  }

  // S^T of one block: s[t][a] holds, for column i16 of tile t, the keys kb + 8 g4 + 4 a + {0..3}
  __device__ __forceinline__ void scores(const F& f, const bf16x8 (&qf)[NT][KS], f32x4 (&s)[NT][2]) {
#pragma unroll
    for (int t = 0; t < NT; ++t) s[t][0] = s[t][1] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int ks = 0; ks < KS; ++ks)
#pragma unroll
      for (int t = 0; t < NT; ++t) {
        s[t][0] = mfma16(f.k[0][ks], qf[t][ks], s[t][0]);
        s[t][1] = mfma16(f.k[1][ks], qf[t][ks], s[t][1]);
      }
  }

  // Online softmax per column; this lane holds keys kb + 8 g4 + {0..7} of column i16. Returns the
  // weights as the B operand of the second product.
  // MASK: some key of the block is invisible to some column, or lies outside [k_lo, k_hi)
  template <bool MASK>
  __device__ __forceinline__ void softmax(const f32x4 (&s)[NT][2], bf16x8 (&pf)[NT], int kb, const int (&col_lo)[NT],
                                          const int (&col_hi)[NT]) {
    const int kg = kb + 8 * ((threadIdx.x & 63) >> 4);
#pragma unroll
    for (int t = 0; t < NT; ++t) {
      // raw scores; the running maximum m is kept in raw units too, and the scale is folded into
      // one fused multiply-add per score: p = 2^(c s - c m), c = scale * log2(e) > 0
      float x[8];
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        x[r] = s[t][0][r];
        x[4 + r] = s[t][1][r];
      }
      if constexpr (KIND == OPTIONS) {
        if (cap_in != 0.f) {     // (uniform) tanh y = 1 - 2 / (1 + e^2y); what follows takes scores in units of one
#pragma unroll
          for (int e = 0; e < 8; ++e) x[e] = fmaf(-2.f * cap, __builtin_amdgcn_rcpf(1.f + exp2_raw(cap_in * x[e])), cap);
        }
      }
      if (EXT) {
        const float far = (float)(col_hi[t] - 1 - kg);   // the distance of the lane's first key from the column's position
#pragma unroll
        for (int e = 0; e < 8; ++e) x[e] = fmaf(-slope_raw, far - (float)e, x[e]);
      }
      if (MASK) {
#pragma unroll
        for (int e = 0; e < 8; ++e) {
          const int key = kg + e;
          if (EXT) {
            // (a kept key below the window may lie in a block of this run outside [k_lo, k_hi): its run comes later)
            if ((key < col_lo[t] && key >= keep_first) || key >= col_hi[t] || key < k_lo || key >= k_hi) x[e] = -INFINITY;
          } else if (key < col_lo[t] || key >= col_hi[t]) {
            x[e] = -INFINITY;
          }
        }
      }
      if constexpr (KIND == SIGMOID) {
#pragma unroll
        for (int e = 0; e < 8; ++e)      // (a masked score is -inf: 1 / (1 + inf) = 0)
          pf[t][e] = (bf16)__builtin_amdgcn_rcpf(1.f + exp2_raw(-fmaf(x[e], scale_log2e, bias_log2e)));
        continue;
      }
      float mx = x[0];
#pragma unroll
      for (int e = 1; e < 8; ++e) mx = fmaxf(mx, x[e]);
      mx = fmaxf(mx, __shfl_xor(mx, 16, 64));
      mx = fmaxf(mx, __shfl_xor(mx, 32, 64));
      // m is the reference the weights are taken against, not the maximum itself: it follows the maximum only
      // when that has risen by more than LAZY (in base-2 units) for some column of the wave (a uniform branch),
      // so weights stay below 2^LAZY and the output is rescaled rarely. Counted on random scores: among the
      // columns of a tile some maximum rises in most blocks, and every rise used to cost a multiplication of
      // the whole output tile. The sums and the final division use the same reference: the result is the same.
      if (__any((mx - m[t]) * scale_log2e > LAZY)) {  // m = -inf: any visible key moves it
        const float m_new = fmaxf(m[t], mx);
        const float alpha = m_new == m[t] ? 1.f : exp2_raw((m[t] - m_new) * scale_log2e);  // m = -inf: 0
        l[t] *= alpha;
#pragma unroll
        for (int d = 0; d < DV; ++d) o[t][d] *= alpha;
        m[t] = m_new;
      }
      const float mc = (m[t] == -INFINITY ? 0.f : m[t]) * scale_log2e;  // nothing visible yet: everything stays zero
      float ps_ = 0.f;
#pragma unroll
      for (int e = 0; e < 8; ++e) {
        const float p = exp2_raw(fmaf(x[e], scale_log2e, -mc));
        ps_ += p;
        pf[t][e] = (bf16)p;
      }
      l[t] += ps_;  // partial over this lane's keys; lane groups are summed at the end
    }
  }

  // O^T += V^T . P
  template <bool MASK>
  __device__ __forceinline__ void accumulate(const F& f, const bf16x8 (&pf)[NT], int kb) {
    const int kg = kb + 8 * ((threadIdx.x & 63) >> 4);
#pragma unroll
    for (int d = 0; d < DV; ++d) {
      bf16x8 vf = f.v[d];
      if (MASK) {
        // a stale slot may hold anything; its weight is 0, but 0 * inf would poison the sum
#pragma unroll
        for (int e = 0; e < 8; ++e)
          if (kg + e < k_lo || kg + e >= k_hi) vf[e] = (bf16)0.f;
      }
#pragma unroll
      for (int t = 0; t < NT; ++t) o[t][d] = mfma16(vf, pf[t], o[t][d]);
    }
  }

  template <bool MASK>
  __device__ __forceinline__ void compute(const F& f, const bf16x8 (&qf)[NT][KS], int kb,
                                          const int (&col_lo)[NT], const int (&col_hi)[NT]) {
    f32x4 s[NT][2];
    bf16x8 pf[NT];
    scores(f, qf, s);
    softmax<MASK>(s, pf, kb, col_lo, col_hi);
    accumulate<MASK>(f, pf, kb);
  }

  // All key blocks of [k_lo, k_hi); mask(kb) says whether block kb needs per-key masking.
  // TWO_BODIES: blocks that need no masking run a body without it (more code, fewer instructions
  // per block); otherwise every block runs the masking body.
  // A block's loads are issued right before its use and other waves hide the latency: reading a
  // block ahead was measured and does not pay (neither with a second set of registers nor by
  // refilling each fragment as soon as its last reader has issued; the split-K kernel with a second set at 8 to 64
  // requests of 2k and 4k keys, one wave a SIMD: within 1 % either way, 5.6 to 5.9 TB/s with it and without).
  // hook(kb, last): called before block kb's loads are issued; `last` says that kb is the wave's last block. The wave
  // that brings the row's own key issues that key's loads a block early there and stores it before the last block.
  template <bool TWO_BODIES, bool STREAM, class MaskFn, class Hook>
  __device__ __forceinline__ void walk(const bf16x8 (&qf)[NT][KS], const int (&col_lo)[NT], const int (&col_hi)[NT],
                                       MaskFn mask, Hook hook) {
    F f;
#pragma nounroll
    for (int kb = k_lo & ~31; kb < k_hi; kb += 32) {
      hook(kb, kb + 32 >= k_hi);
      if (!TWO_BODIES || mask(kb)) {
        load<true, STREAM>(f, kb);
        compute<true>(f, qf, kb, col_lo, col_hi);
      } else {
        load<false, STREAM>(f, kb);
        compute<false>(f, qf, kb, col_lo, col_hi);
      }
    }
  }
  template <bool TWO_BODIES, class MaskFn>
  __device__ __forceinline__ void walk(const bf16x8 (&qf)[NT][KS], const int (&col_lo)[NT], const int (&col_hi)[NT],
                                       MaskFn mask) {
    walk<TWO_BODIES, false>(qf, col_lo, col_hi, mask, [](int, bool) {});
  }

  // total of l over the four lane groups of a column
  __device__ __forceinline__ float sum_l(int t) const {
    float v = l[t];
    v += __shfl_xor(v, 16, 64);
    v += __shfl_xor(v, 32, 64);
    return v;
  }
};

// Flash kernel. A workgroup owns QT x 16 query rows of one head; its four waves share the rows and
// deal the key blocks among themselves in four contiguous runs, each wave keeping its own running
// (maximum, sum, output); at the end waves 1..3 hand theirs to wave 0 through LDS, which combines
// them and stores the rows. So every key block is read by one wave only, and a long row tile (many
// keys under a causal mask) is four short pieces of work instead of one long one: with a few
// thousand workgroups of unequal length issued longest first, the chip stays evenly busy.
// Measured on MI355X at head size 128 (one 2,048-token prompt, 32 heads): 122 us for the former
// one-wave-per-tile kernel, where the longest tile set the time.
struct FlashExt {
  int keep_first;       // with a window: keys below this stay visible
  const float* sinks;   // [H] float or null
  float slope_exp;      // 0: no distance bias
  float out_scale;
  float scale;          // the score scale itself (scale_log2e / log2(e)); with a cap: 1, the scale is in cap_in
  const float* biases;  // SIGMOID: [H] float, added to the scores
  float cap, cap_in;    // softly capped scores (cap_in 0: none)
  int chunk;            // > 0: keys of the row's own chunk of positions only
};

template <int DT, int QT, bool P2, int KIND = PLAIN, int DV = DT>
__global__ void __launch_bounds__(256) __attribute__((amdgpu_waves_per_eu(2, 8))) attn_flash_kernel(
    const bf16* __restrict__ q, int64_t ld_q, bf16* __restrict__ out, int64_t ld_out, const bf16* __restrict__ kc,
    const bf16* __restrict__ vc, const int32_t* __restrict__ block_table, int64_t max_blocks,
    const int32_t* __restrict__ cu_seqlens, const int32_t* __restrict__ seq_lens, int tiles_x, float scale_log2e,
    int window, int H, int Hkv, int ps, int skip_single, FlashExt ext = FlashExt{}) {
  constexpr bool EXT = KIND != PLAIN;
  constexpr int D = DT * 16;
  constexpr int KS = (DT + 1) / 2;
  constexpr int QW = 16 * QT;  // query rows per workgroup
  // what waves 1..3 hand to wave 0 (dynamic: three row tiles of head size 128 need more than the 64 KB a kernel
  // may declare): part_o[3][QT][DV][64] of f32x4, then part_m and part_l [3][QT][64] of float
  extern __shared__ __attribute__((aligned(16))) char flash_smem[];
  f32x4* const part_o_ = (f32x4*)flash_smem;
  float* const part_m_ = (float*)(flash_smem + sizeof(f32x4) * 3 * QT * DV * 64);
  float* const part_l_ = part_m_ + 3 * QT * 64;
  auto part_o = [&](int r, int t, int d) -> f32x4& { return part_o_[((r * QT + t) * DV + d) * 64 + lane_of()]; };
  auto part_m = [&](int r, int t) -> float& { return part_m_[(r * QT + t) * 64 + lane_of()]; };
  auto part_l = [&](int r, int t) -> float& { return part_l_[(r * QT + t) * 64 + lane_of()]; };
  // Block order: the head index runs fastest and visits kv heads round-robin, so that the
  // workgroups an XCD receives (linear id modulo 8) share kv heads, and with them the L2 lines
  // of K and V. Late query tiles (most keys) are issued first.
  const int L = blockIdx.x;
  const int e = L % H, rest = L / H;
  const int tile = tiles_x - 1 - rest % tiles_x, b = rest / tiles_x;
  const int G = H / Hkv;
  const int hk = e % Hkv, h = hk * G + e / Hkv;
  const int q_begin = cu_seqlens[b];
  const int q_len = cu_seqlens[b + 1] - q_begin;
  const int hist = seq_lens[b] - q_len;
  const int wave = threadIdx.x >> 6, lane = threadIdx.x & 63, i16 = lane & 15, g4 = lane >> 4;
  const int q0 = tile * QW;
  if (q0 >= q_len) return;                // the whole workgroup: nobody is left waiting at the barrier below
  if (skip_single && q_len == 1) return;  // single rows go to the split-K kernel
  const int32_t* bt = block_table + (int64_t)b * max_blocks;

  // the first key (but for kept ones) that the row at a position sees
  auto low_of = [&](int pos) {
    int lo = window > 0 ? (pos - window + 1 > 0 ? pos - window + 1 : 0) : 0;
    if constexpr (EXT) {
      if (ext.chunk > 0) lo = max(lo, pos - pos % ext.chunk);
    }
    return lo;
  };
  bf16x8 qf[QT][KS];
  int col_lo[QT], col_hi[QT];
#pragma unroll
  for (int t = 0; t < QT; ++t) {
    const int row = q0 + t * 16 + i16;
    const int rc = row < q_len ? row : q_len - 1;  // rows past the end compute something harmless, never stored
    const bf16* qp = q + (int64_t)(q_begin + rc) * ld_q + (int64_t)h * D;
#pragma unroll
    for (int ks = 0; ks < KS; ++ks) {
      const int d = ks * 32 + g4 * 8;
      qf[t][ks] = d < D ? *(const bf16x8*)(qp + d) : zero8();
    }
    const int pos = hist + rc;
    col_hi[t] = pos + 1;
    col_lo[t] = low_of(pos);
  }
  // the keys any row of the tile sees, and this wave's run of 32-key blocks among them
  const int p_first = hist + q0;
  const int p_last = hist + (q0 + QW < q_len ? q0 + QW : q_len) - 1;
  const int all_hi = p_last + 1;
  const int all_lo = low_of(p_first), last_lo = low_of(p_last);
  const int blk_first = all_lo >> 5, blk_end = (all_hi + 31) >> 5;
  const int per = (blk_end - blk_first + 3) >> 2;
  const int blk0 = blk_first + wave * per;
  const int blk1 = blk0 + per < blk_end ? blk0 + per : blk_end;
  const int k_lo = blk0 * 32 > all_lo ? blk0 * 32 : all_lo;
  const int k_hi = blk1 * 32 < all_hi ? blk1 * 32 : all_hi;

  Tile<DT, QT, P2, KIND, DV> tl;
  tl.init(kc, vc, bt, (int)max_blocks, hk, Hkv, ps, k_lo, k_hi, scale_log2e);
  if constexpr (EXT) {
    tl.keep_first = window > 0 || ext.chunk > 0 ? ext.keep_first : 0;
    tl.cap = ext.cap;
    tl.cap_in = ext.cap_in;
    tl.slope_raw = ext.slope_exp != 0.f ? exp2f(-ext.slope_exp * (float)(h + 1) / (float)H) / ext.scale : 0.f;
    if constexpr (KIND == SIGMOID) tl.bias_log2e = ext.biases[h] * LOG2E;
  }
  tl.template walk<true>(qf, col_lo, col_hi, [&](int kb) {
    return kb + 31 > p_first || kb < all_lo || kb < last_lo || (EXT && kb + 32 > k_hi);
  });
  if constexpr (EXT) {
    // the kept first keys that the window of the tile's first row has passed: one more run, every block masked
    const int kept = tl.keep_first < all_lo ? tl.keep_first : all_lo;
    if (wave == 0 && kept > 0) {
      tl.k_lo = 0;
      tl.k_hi = kept;
      tl.pages.init(bt, (int)max_blocks, ps, 0);
      tl.template walk<false>(qf, col_lo, col_hi, [](int) { return true; });
    }
  }

  if (wave > 0) {
#pragma unroll
    for (int t = 0; t < QT; ++t) {
      part_m(wave - 1, t) = tl.m[t];
      part_l(wave - 1, t) = tl.l[t];
#pragma unroll
      for (int d = 0; d < DV; ++d) part_o(wave - 1, t, d) = tl.o[t][d];
    }
  }
  __syncthreads();
  if (wave > 0) return;
#pragma unroll
  for (int t = 0; t < QT; ++t) {
    // every wave keeps a lane's share in the same places, so the parts combine lane by lane:
    // o = sum_r 2^(c (m_r - M)) o_r, likewise l (still a partial over the lane's keys)
    float inv;
    if constexpr (KIND == SIGMOID) {      // weights against no reference: the parts simply add up
#pragma unroll
      for (int r = 0; r < 3; ++r)
#pragma unroll
        for (int d = 0; d < DV; ++d) tl.o[t][d] += part_o(r, t, d);
      inv = ext.out_scale;
    } else {
      float mr[3], M = tl.m[t];
#pragma unroll
      for (int r = 0; r < 3; ++r) {
        mr[r] = part_m(r, t);
        M = fmaxf(M, mr[r]);
      }
      const float mc = (M == -INFINITY ? 0.f : M) * scale_log2e;
      const float a0 = exp2_raw(fmaf(tl.m[t], scale_log2e, -mc));  // an empty part has m = -inf: weight 0
      float lsum = tl.l[t] * a0;
#pragma unroll
      for (int d = 0; d < DV; ++d) tl.o[t][d] *= a0;
#pragma unroll
      for (int r = 0; r < 3; ++r) {
        const float ar = exp2_raw(fmaf(mr[r], scale_log2e, -mc));
        lsum += part_l(r, t) * ar;
#pragma unroll
        for (int d = 0; d < DV; ++d) tl.o[t][d] += part_o(r, t, d) * ar;
      }
      tl.l[t] = lsum;
      float lt = tl.sum_l(t);
      if constexpr (EXT) {
        float shrink = ext.out_scale;
        if (ext.sinks) {  // one more term of the denominator, 2^(sink log2(e) - mc) against the parts' reference
          const float d = ext.sinks[h] * LOG2E - mc;
          if (d > 30.f) {  // a sink far above every score: the sums shrink instead of the term growing
            const float f = exp2_raw(-d);
            lt = lt * f + 1.f;
            shrink *= f;
          } else {
            lt += exp2_raw(d);
          }
        }
        inv = lt > 0.f ? shrink / lt : 0.f;
      } else {
        inv = lt > 0.f ? 1.f / lt : 0.f;
      }
    }
    const int row = q0 + t * 16 + i16;
    if (row < q_len) {
      bf16* op = out + (int64_t)(q_begin + row) * ld_out + (int64_t)h * (DV * 16) + 4 * g4;
#pragma unroll
      for (int d = 0; d < DV; ++d) {
        bf16x4 r;
#pragma unroll
        for (int k = 0; k < 4; ++k) r[k] = (bf16)(tl.o[t][d][k] * inv);
        *(bf16x4*)(op + d * 16) = r;
      }
    }
  }
}

}  // namespace
}  // namespace dinfer
