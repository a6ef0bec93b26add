// Per-head q/k RMSNorm, rotary position encoding and the K/V cache write in
// one pass over a step's fused projection output.
//
//   qkv [T, ld]:  q heads at column q_off (H x D), k heads at k_off (Hkv x D),
//                 v heads at v_off (Hkv x D).
//   q, k:  y = x * rsqrt(mean(x^2) + eps) * (w + w_offset)   (skipped when the
//          gain pointer is null), then rotation of the first `rot` dims by the
//          angles of the token's position, all in float, one rounding.
//          q is written back in place; k goes to the cache only, or, where no
//          slot mapping is given (nothing is cached), back in place like q.
//   v:     copied to the cache unchanged. Its heads may have a size of their own (v_dim); without value pages
//          (a layer whose values are its keys) nothing is copied.
//
// Cache pages (chosen for MFMA operand loads on gfx950: both operands of
// Q.K^T and P.V want 8 consecutive elements of the contraction dimension):
//   K page  [Hkv][D / 8][page][8]   the 8-element pieces of consecutive keys are contiguous
//   V page  [Hkv][D][page]   transposed: for one d, the page's keys are contiguous
// A token's slot is block * page + offset; a negative slot writes nothing.
//
// The table row of position p is [cos(p f_0..f_{rot/2-1}) | sin(...)], float.
// style 0 pairs (i, i + rot/2) ("neox"), style 1 pairs (2i, 2i+1).
//
// Reference behaviour: crates/kernels/cuda/qkv_post.cu:26-91 (order norm ->
// rotation -> one rounding; v untouched; k written after norm and rotation),
// crates/layers/src/nn.rs:152-185 (table layout).
#include "common.cuh"

using namespace dinfer;

namespace {

constexpr int MAX_D = 512;
constexpr int WAVES = 4;

// Values mixed with another row's: v <- (1 - share) v + share first[t], `first` [T, ld] in the step's dtype, its kv heads
// side by side as v's are (null: v stays as it is).
struct ValueMix {
  const void* first;
  int64_t ld;
  float share;
};
template <class S>
__device__ __forceinline__ float mixed_value(float v, const ValueMix& mix, int64_t t, int c) {
  return __builtin_fmaf(mix.share, to_f32(((const S*)mix.first)[t * mix.ld + c]), (1.f - mix.share) * v);
}

__device__ __forceinline__ bf16x8 zero8() {
  bf16x8 z;
#pragma unroll
  for (int i = 0; i < 8; ++i) z[i] = (bf16)0.f;
  return z;
}

template <class S>
__global__ void __launch_bounds__(WAVES * 64) qkv_post_kernel(
    S* __restrict__ qkv, int64_t ld, int64_t q_off, int64_t k_off, int64_t v_off, const void* __restrict__ wq,
    const void* __restrict__ wk, int wf32, float eps, float w_offset, const int32_t* __restrict__ pos,
    const float* __restrict__ cos_sin, int rot, int style, S* __restrict__ k_cache, S* __restrict__ v_cache,
    const int64_t* __restrict__ slots, int H, int Hkv, int D, int page, int Dv, const float* __restrict__ bias,
    float temp_coef, int temp_every, const float* __restrict__ head_scale, ValueMix mix) {
  __shared__ float xs[WAVES][MAX_D];
  const int64_t t = blockIdx.x;
  const int wave = threadIdx.x >> 6, lane = threadIdx.x & 63;
  const int item = blockIdx.y * WAVES + wave;
  const bool live = item < H + 2 * Hkv;
  const bool is_v = live && item >= H + Hkv;
  const bool is_qk = live && !is_v;
  const bool is_q = live && item < H;
  S* row = qkv + t * ld;
  const int64_t slot = slots ? slots[t] : -1;
  const int64_t blk = slot >= 0 ? slot / page : 0;
  const int off = slot >= 0 ? (int)(slot % page) : 0;

  if (is_v && slot >= 0 && v_cache) {  // a v head: cache copy only
    const int hk = item - H - Hkv;
    const S* vs = row + v_off + (int64_t)hk * Dv;
    S* vd = v_cache + ((blk * Hkv + hk) * (int64_t)Dv) * page + off;
    if (bias || mix.first) {
      const float* vb = bias ? bias + (int64_t)(H + Hkv) * D + (int64_t)hk * Dv : nullptr;
      for (int d = lane; d < Dv; d += 64) {
        float v = to_f32(vs[d]) + (vb ? vb[d] : 0.f);
        if (mix.first) v = mixed_value<S>(v, mix, t, hk * Dv + d);
        vd[(int64_t)d * page] = from_f32<S>(v);
      }
    } else {
      for (int d = lane; d < Dv; d += 64) vd[(int64_t)d * page] = vs[d];
    }
  }

  const int hk = item - H;
  S* base = is_q ? row + q_off + (int64_t)item * D : row + k_off + (int64_t)hk * D;
  const void* w = is_q ? wq : wk;
  float* x = xs[wave];

  if (is_qk) {
    float ss = 0.f;
    const float* hb = bias ? bias + (int64_t)item * D : nullptr;   // q heads, then k heads
    for (int d = lane; d < D; d += 64) {
      float v = to_f32(base[d]);
      if (hb) v += hb[d];
      x[d] = v;
      ss += v * v;
    }
    if (w) {
      ss = wave_sum(ss);
      float inv = 1.f / sqrtf(ss / (float)D + eps);
      // a query grows with its position: 1 + coef ln(floor((p + 1) / every) + 1)
      if (is_q && temp_every > 0) inv *= 1.f + temp_coef * logf((float)((pos[t] + 1) / temp_every) + 1.f);
      // a temperature a query head: the head's scores are multiplied by it, so its query is
      if (is_q && head_scale) inv *= head_scale[item];
      // each lane rescales only the entries it wrote itself
      for (int d = lane; d < D; d += 64) x[d] = x[d] * inv * (ld_param<S>(w, d, wf32) + w_offset);
    }
  }
  __syncthreads();  // the rotation reads partners that other lanes wrote
  if (!is_qk) return;

  // (a head size that is no multiple of 8 fills its last 8-entry piece in part)
  S* kd = (!is_q && slot >= 0) ? k_cache + (blk * Hkv + hk) * (int64_t)page * ((D + 7) & ~7) : nullptr;  // the head's page
  const float* cs = cos_sin ? cos_sin + (int64_t)pos[t] * rot : nullptr;
  const int half = rot / 2;
  for (int d = lane; d < D; d += 64) {
    float y = x[d];
    if (cs && d < rot) {
      int i;         // index of the frequency
      float other;   // the partner in the pair
      bool first;    // whether d is the first element of its pair
      if (style == 0) {
        first = d < half;
        i = first ? d : d - half;
        other = x[first ? d + half : d - half];
      } else {
        first = (d & 1) == 0;
        i = d >> 1;
        other = x[d ^ 1];
      }
      const float c = cs[i], s = cs[half + i];
      y = first ? y * c - other * s : y * c + other * s;
    }
    const S r = from_f32<S>(y);
    if (is_q || !slots) base[d] = r;  // without a slot mapping nothing goes to the cache and k is written back like q
    if (kd) kd[k_page_offset((int)off, d, page)] = r;
  }
}

// The common case (pairs (i, i + D/2), the whole head rotated): both elements of a pair live in one
// lane, so there is no exchange through LDS and no barrier. A wave takes IPW heads of one token and
// issues every load of all of them (values, gains, angles) before the first use; fewer, fatter waves
// also keep the kernel off the wave-launch limit. NP pairs per lane cover D <= 128 * NP.
constexpr int IPW = 4;  // head items per wave

template <class S, int NP>
__global__ void __launch_bounds__(WAVES * 64) qkv_post_neox_kernel(
    S* __restrict__ qkv, int64_t ld, int64_t q_off, int64_t k_off, int64_t v_off, const void* __restrict__ wq,
    const void* __restrict__ wk, int wf32, float eps, float w_offset, const int32_t* __restrict__ pos,
    const float* __restrict__ cos_sin, S* __restrict__ k_cache, S* __restrict__ v_cache,
    const int64_t* __restrict__ slots, int H, int Hkv, int D, int page) {
  const int64_t t = blockIdx.x;
  const int wave = threadIdx.x >> 6, lane = threadIdx.x & 63;
  const int item0 = (blockIdx.y * WAVES + wave) * IPW;
  const int items = H + 2 * Hkv;
  if (item0 >= items) return;
  S* row = qkv + t * ld;
  const int64_t slot = slots ? slots[t] : -1;
  const int64_t blk = slot >= 0 ? slot / page : 0;
  const int off = slot >= 0 ? (int)(slot % page) : 0;
  const int half = D / 2;
  const float* cs = cos_sin ? cos_sin + (int64_t)pos[t] * D : nullptr;

  float x1[IPW][NP], x2[IPW][NP];
  float g1q[NP], g2q[NP], g1k[NP], g2k[NP], c[NP], sn[NP];
#pragma unroll
  for (int p = 0; p < NP; ++p) {
    const int i = lane + 64 * p;
    const bool ok = i < half;
    g1q[p] = (ok && wq) ? ld_param<S>(wq, i, wf32) + w_offset : 1.f;
    g2q[p] = (ok && wq) ? ld_param<S>(wq, i + half, wf32) + w_offset : 1.f;
    g1k[p] = (ok && wk) ? ld_param<S>(wk, i, wf32) + w_offset : 1.f;
    g2k[p] = (ok && wk) ? ld_param<S>(wk, i + half, wf32) + w_offset : 1.f;
    c[p] = (ok && cs) ? cs[i] : 1.f;
    sn[p] = (ok && cs) ? cs[half + i] : 0.f;
  }
#pragma unroll
  for (int u = 0; u < IPW; ++u) {
    const int item = item0 + u;
    // q heads, then k heads, then v heads lie one after the other in the row when the offsets say so;
    // in general each kind has its own offset
    const S* src = item < H ? row + q_off + (int64_t)item * D
                 : item < H + Hkv ? row + k_off + (int64_t)(item - H) * D
                                  : row + v_off + (int64_t)(item - H - Hkv) * D;
#pragma unroll
    for (int p = 0; p < NP; ++p) {
      const int i = lane + 64 * p;
      const bool ok = i < half && item < items;
      x1[u][p] = ok ? to_f32(src[i]) : 0.f;
      x2[u][p] = ok ? to_f32(src[i + half]) : 0.f;
    }
  }
#pragma unroll
  for (int u = 0; u < IPW; ++u) {
    const int item = item0 + u;
    if (item >= items) break;
    if (item >= H + Hkv) {  // a v head: cache copy only
      if (slot < 0) continue;
      const int hk = item - H - Hkv;
      S* vd = v_cache + ((blk * Hkv + hk) * (int64_t)D) * page + off;
#pragma unroll
      for (int p = 0; p < NP; ++p) {
        const int i = lane + 64 * p;
        if (i < half) {
          vd[(int64_t)i * page] = from_f32<S>(x1[u][p]);  // the value came from S: the round trip is exact
          vd[(int64_t)(i + half) * page] = from_f32<S>(x2[u][p]);
        }
      }
      continue;
    }
    const bool is_q = item < H;
    const bool normed = is_q ? wq != nullptr : wk != nullptr;
    float inv = 1.f;
    if (normed) {
      float ss = 0.f;
#pragma unroll
      for (int p = 0; p < NP; ++p) ss += x1[u][p] * x1[u][p] + x2[u][p] * x2[u][p];
      ss = wave_sum(ss);
      inv = 1.f / sqrtf(ss / (float)D + eps);
    }
    const int hk = item - H;
    S* base = is_q ? row + q_off + (int64_t)item * D : slots ? nullptr : row + k_off + (int64_t)hk * D;
    S* kd = (!is_q && slot >= 0) ? k_cache + (blk * Hkv + hk) * (int64_t)page * D : nullptr;  // the head's page
#pragma unroll
    for (int p = 0; p < NP; ++p) {
      const int i = lane + 64 * p;
      if (i < half) {
        const float y1 = normed ? x1[u][p] * inv * (is_q ? g1q[p] : g1k[p]) : x1[u][p];
        const float y2 = normed ? x2[u][p] * inv * (is_q ? g2q[p] : g2k[p]) : x2[u][p];
        const S r1 = from_f32<S>(y1 * c[p] - y2 * sn[p]), r2 = from_f32<S>(y2 * c[p] + y1 * sn[p]);
        if (base) {
          base[i] = r1;
          base[i + half] = r2;
        }
        if (kd) {
          kd[k_page_offset((int)off, i, page)] = r1;
          kd[k_page_offset((int)off, i + half, page)] = r2;
        }
      }
    }
  }
}

// V into its transposed pages for many tokens: one wave takes 8 consecutive tokens of one kv head.
// When their slots are 8 consecutive slots starting at a multiple of 8 (a prompt portion that starts
// on such a boundary), a lane gathers two dims of the 8 tokens and stores them as two 16-byte rows
// of V^T; otherwise it falls back to one 2-byte store per element.
// (group: which run of 8 * WAVES tokens the workgroup takes.)
__device__ __forceinline__ void v_write_transposed(const bf16* __restrict__ qkv, int64_t ld, int64_t v_off,
                                                   bf16* __restrict__ v_cache, const int64_t* __restrict__ slots, int T,
                                                   int Hkv, int D, int page, int group, int hk,
                                                   const float* __restrict__ vb = nullptr, ValueMix mix = ValueMix{}) {
  const int wave = threadIdx.x >> 6, lane = threadIdx.x & 63;
  const int t0 = (group * WAVES + wave) * 8;
  if (t0 >= T) return;
  const int n = T - t0 < 8 ? T - t0 : 8;
  const int64_t s0 = slots[t0];
  bool aligned = n == 8 && s0 >= 0 && (s0 & 7) == 0;
  for (int j = 1; j < n && aligned; ++j) aligned = slots[t0 + j] == s0 + j;
  const bf16* src = qkv + (int64_t)t0 * ld + v_off + (int64_t)hk * D;
  for (int d2 = lane; d2 < D / 2; d2 += 64) {
    bf16x2 v[8];
#pragma unroll
    for (int j = 0; j < 8; ++j)
      if (j < n) v[j] = *(const bf16x2*)(src + (int64_t)j * ld + 2 * d2);
    if (vb) {  // the head's bias (float), added as the kernels that take one value at a time add it
      const float b0 = vb[2 * d2], b1 = vb[2 * d2 + 1];
#pragma unroll
      for (int j = 0; j < 8; ++j)
        if (j < n) {
          v[j][0] = (bf16)((float)v[j][0] + b0);
          v[j][1] = (bf16)((float)v[j][1] + b1);
        }
    }
    if (mix.first) {
#pragma unroll
      for (int j = 0; j < 8; ++j)
        if (j < n) {
          v[j][0] = (bf16)mixed_value<bf16>((float)v[j][0], mix, t0 + j, hk * D + 2 * d2);
          v[j][1] = (bf16)mixed_value<bf16>((float)v[j][1], mix, t0 + j, hk * D + 2 * d2 + 1);
        }
    }
    if (aligned) {
      const int64_t blk = s0 / page;
      const int off = (int)(s0 % page);
      bf16* vd = v_cache + ((blk * Hkv + hk) * (int64_t)D + 2 * d2) * page + off;
      bf16x8 a, b;
#pragma unroll
      for (int j = 0; j < 8; ++j) {
        a[j] = v[j][0];
        b[j] = v[j][1];
      }
      *(bf16x8*)vd = a;
      *(bf16x8*)(vd + page) = b;
    } else {
#pragma unroll
      for (int j = 0; j < 8; ++j) {
        if (j >= n) break;
        const int64_t sl = slots[t0 + j];
        if (sl < 0) continue;
        bf16* vd = v_cache + (((sl / page) * Hkv + hk) * (int64_t)D + 2 * d2) * page + sl % page;
        vd[0] = v[j][0];
        vd[page] = v[j][1];
      }
    }
  }
}

// bf16, whole-head neox rotation, D in {64, 128, 256}: LPH = D / 8 lanes share a head, each with 8
// consecutive dims in one 16-byte load; the partner of a pair sits LPH / 2 lanes away and comes by a
// cross-lane read. A wave covers 64 / LPH heads of one token per instruction, an order of magnitude
// fewer memory instructions than 2-byte accesses.
// gather_v > 0: V is not written by the heads' lanes; the workgroups from blockIdx.x = `tokens` on (gather_v of them,
// one per kv head and run of 8 * WAVES tokens) gather it into its transposed pages, in the same launch (a kernel of
// its own for that cost a prefill layer 5.7 us, a step of prompt portions beside decoding requests 7.8).
template <int LPH>
__global__ void __launch_bounds__(WAVES * 64) qkv_post_vec_kernel(
    bf16* __restrict__ qkv, int64_t ld, int64_t q_off, int64_t k_off, int64_t v_off, const void* __restrict__ wq,
    const void* __restrict__ wk, int wf32, float eps, float w_offset, const int32_t* __restrict__ pos,
    const float* __restrict__ cos_sin, bf16* __restrict__ k_cache, bf16* __restrict__ v_cache,
    const int64_t* __restrict__ slots, int H, int Hkv, int page, int tokens, int gather_v,
    const float* __restrict__ bias, float temp_coef, int temp_every, const float* __restrict__ head_scale, ValueMix mix) {
  constexpr int D = LPH * 8, HALF = D / 2, HPW = 64 / LPH;  // heads per wave
  if ((int)blockIdx.x >= tokens) {
    const int j = (int)blockIdx.x - tokens;
    if (blockIdx.y == 0)
      v_write_transposed(qkv, ld, v_off, v_cache, slots, tokens, Hkv, D, page, j / Hkv, j % Hkv,
                         bias ? bias + (int64_t)(H + Hkv + j % Hkv) * D : nullptr, mix);
    return;
  }
  const bool skip_v = gather_v > 0;
  const int64_t t = blockIdx.x;
  const int wave = threadIdx.x >> 6, lane = threadIdx.x & 63;
  const int sub = lane / LPH, l = lane % LPH;  // which head of the wave, which 8 dims of it
  const int items = H + 2 * Hkv;
  // The workgroups of a token (gridDim.y of them) take its heads in rounds of gridDim.y * WAVES * HPW; a lane keeps
  // its 8 dims from round to round, so the angles of those dims are fetched once (with one workgroup a token, which
  // is how many tokens are launched, a lane serves three heads of the 8B sizes with one fetch: the angles are four
  // times the bytes of the head's own 8 values).
  const int per_round = gridDim.y * WAVES * HPW;
  const int first_item = (blockIdx.y * WAVES + wave) * HPW + sub;
  bf16* row = qkv + t * ld;
  const int64_t slot = slots ? slots[t] : -1;
  const int64_t blk = slot >= 0 ? slot / page : 0;
  const int off = slot >= 0 ? (int)(slot % page) : 0;
  const int d0 = 8 * l;
  auto source = [&](int item) {
    return item < H ? row + q_off + (int64_t)item * D
                    : item < H + Hkv ? row + k_off + (int64_t)(item - H) * D : row + v_off + (int64_t)(item - H - Hkv) * D;
  };
  // angles of this lane's dims: the pair index of dim d is d mod D/2
  float c[8], sn[8];
  const int pi = d0 % HALF;
  if (cos_sin) {
    const float* cs = cos_sin + (int64_t)pos[t] * D;
    const f32x4 c0 = *(const f32x4*)(cs + pi), c1 = *(const f32x4*)(cs + pi + 4);
    const f32x4 s0 = *(const f32x4*)(cs + HALF + pi), s1 = *(const f32x4*)(cs + HALF + pi + 4);
#pragma unroll
    for (int e = 0; e < 4; ++e) { c[e] = c0[e]; c[4 + e] = c1[e]; sn[e] = s0[e]; sn[4 + e] = s1[e]; }
  } else {
#pragma unroll
    for (int e = 0; e < 8; ++e) { c[e] = 1.f; sn[e] = 0.f; }
  }
  // (a wave's lanes leave the loop together: the cross-lane steps below need all of them)
  const int wave_first = (blockIdx.y * WAVES + wave) * HPW;
  bf16x8 xv = zero8();
  if (first_item < items) xv = *(const bf16x8*)(source(first_item) + d0);
  // (bias: float [q heads | k heads | v heads], a head of D each here: entry item * D + d of any item; asked for with the
  // values it is added to, a round ahead)
  f32x4 bn0 = {0.f, 0.f, 0.f, 0.f}, bn1 = {0.f, 0.f, 0.f, 0.f};
  if (bias && first_item < items) {
    bn0 = *(const f32x4*)(bias + (int64_t)first_item * D + d0);
    bn1 = *(const f32x4*)(bias + (int64_t)first_item * D + d0 + 4);
  }
  for (int base = 0; wave_first + base < items; base += per_round) {
    const int item = first_item + base;
    const bool live = item < items;
    const bool is_v = live && item >= H + Hkv, is_q = live && item < H, is_k = live && !is_q && !is_v;
    bf16* src = live ? source(item) : row;
    const bf16x8 xc = xv;
    // the next round's values are on their way while this round is computed
    xv = zero8();
    const f32x4 b0 = bn0, b1 = bn1;
    if (item + per_round < items) {
      xv = *(const bf16x8*)(source(item + per_round) + d0);
      if (bias) {
        bn0 = *(const f32x4*)(bias + (int64_t)(item + per_round) * D + d0);
        bn1 = *(const f32x4*)(bias + (int64_t)(item + per_round) * D + d0 + 4);
      }
    }
    float x[8], ss = 0.f;
#pragma unroll
    for (int e = 0; e < 8; ++e) x[e] = (float)xc[e];
    if (bias && live) {
#pragma unroll
      for (int e = 0; e < 4; ++e) { x[e] += b0[e]; x[4 + e] += b1[e]; }
    }
    if (is_v) {
      if (slot >= 0 && !skip_v) {
        if (mix.first) {
          const bf16x8 f = *(const bf16x8*)((const bf16*)mix.first + t * mix.ld + (int64_t)(item - H - Hkv) * D + d0);
#pragma unroll
          for (int e = 0; e < 8; ++e) x[e] = __builtin_fmaf(mix.share, (float)f[e], (1.f - mix.share) * x[e]);
        }
        bf16* vd = v_cache + ((blk * Hkv + (item - H - Hkv)) * (int64_t)D + d0) * page + off;
#pragma unroll
        for (int e = 0; e < 8; ++e) vd[(int64_t)e * page] = (bf16)x[e];
      }
    }
    const bool qk = is_q || is_k;
    const void* w = is_q ? wq : wk;
    float g[8];
    if (qk && w) {
      if (wf32) {
        const f32x4 a = *(const f32x4*)((const float*)w + d0), b = *(const f32x4*)((const float*)w + d0 + 4);
#pragma unroll
        for (int e = 0; e < 4; ++e) { g[e] = a[e] + w_offset; g[4 + e] = b[e] + w_offset; }
      } else {
        const bf16x8 gv = *(const bf16x8*)((const bf16*)w + d0);
#pragma unroll
        for (int e = 0; e < 8; ++e) g[e] = (float)gv[e] + w_offset;
      }
    } else {
#pragma unroll
      for (int e = 0; e < 8; ++e) g[e] = 1.f;
    }
#pragma unroll
    for (int e = 0; e < 8; ++e) ss = add_square(ss, x[e]);
    // every lane takes part in the cross-lane steps, whatever its head is
#pragma unroll
    for (int o = LPH / 2; o > 0; o >>= 1) ss += __shfl_xor(ss, o, 64);
    float inv = (qk && w) ? 1.f / sqrtf(ss / (float)D + eps) : 1.f;
    // a query grows with its position: 1 + coef ln(floor((p + 1) / every) + 1)
    if (is_q && w && temp_every > 0) inv *= 1.f + temp_coef * logf((float)((pos[t] + 1) / temp_every) + 1.f);
    if (is_q && w && head_scale) inv *= head_scale[item];
    float y[8], other[8];
#pragma unroll
    for (int e = 0; e < 8; ++e) y[e] = (qk && w) ? x[e] * inv * g[e] : x[e];
#pragma unroll
    for (int e = 0; e < 8; ++e) other[e] = __shfl_xor(y[e], LPH / 2, 64);
    if (!qk) continue;
    const bool first = l < LPH / 2;  // this lane holds the first elements of its pairs
    bf16x8 r;
#pragma unroll
    for (int e = 0; e < 8; ++e)
      r[e] = (bf16)(first ? rotated_first(y[e], other[e], c[e], sn[e]) : rotated_second(other[e], y[e], c[e], sn[e]));
    if (is_q || !slots) {
      *(bf16x8*)(src + d0) = r;
    } else if (slot >= 0) {
      *(bf16x8*)(k_cache + (blk * Hkv + (item - H)) * (int64_t)page * D + k_page_offset((int)off, d0, page)) = r;
    }
  }
}

// Norms over the whole projection: all q heads of a token share one root mean square, all k heads another (gains
// [H D] and [Hkv D], float), before the rotation.
//
// Any sizes and types: a workgroup takes a token, the row waits in LDS as floats between the sums and the rotation, which
// reads a pair's other element there.
template <class S>
__global__ void __launch_bounds__(256) qkv_row_post_kernel(
    S* __restrict__ qkv, int64_t ld, int64_t q_off, int64_t k_off, int64_t v_off, const float* __restrict__ wq,
    const float* __restrict__ wk, float eps, const int32_t* __restrict__ pos, const float* __restrict__ cos_sin, int rot,
    int style, S* __restrict__ k_cache, S* __restrict__ v_cache, const int64_t* __restrict__ slots, int H, int Hkv, int D,
    int page, int Dv, const float* __restrict__ bias, ValueMix mix) {
  extern __shared__ __attribute__((aligned(16))) float row_smem[];
  __shared__ float red[16];
  const int64_t t = blockIdx.x;
  S* row = qkv + t * ld;
  const int64_t slot = slots ? slots[t] : -1;
  const int64_t blk = slot >= 0 ? slot / page : 0;
  const int off = slot >= 0 ? (int)(slot % page) : 0;
  const int nq = H * D, n = nq + Hkv * D;
  float sq = 0.f, sk = 0.f;
  for (int i = threadIdx.x; i < n; i += 256) {
    float v = to_f32(i < nq ? row[q_off + i] : row[k_off + (i - nq)]);
    if (bias) v += bias[i];
    row_smem[i] = v;
    if (i < nq) sq = add_square(sq, v);
    else sk = add_square(sk, v);
  }
  // (the barriers inside also publish the row)
  const float fq = 1.f / sqrtf(block_sum(sq, red) / (float)nq + eps);
  const float fk = 1.f / sqrtf(block_sum(sk, red) / (float)(n - nq) + eps);
  const float* cs = cos_sin ? cos_sin + (int64_t)pos[t] * rot : nullptr;
  const int half = rot / 2, Dp = (D + 7) & ~7;
  for (int i = threadIdx.x; i < n; i += 256) {
    const bool is_q = i < nq;
    const int e0 = is_q ? i : i - nq, hd = e0 / D, d = e0 - hd * D;
    const float* w = is_q ? wq : wk;
    const float f = is_q ? fq : fk;
    float y = row_smem[i] * f * w[e0];
    if (cs && d < rot) {
      const bool first = style == 0 ? d < half : (d & 1) == 0;
      const int pi = style == 0 ? (first ? d : d - half) : d >> 1;
      const int step = style == 0 ? half : 1, other = first ? step : -step;
      const float o = row_smem[i + other] * f * w[e0 + other];
      y = first ? rotated_first(y, o, cs[pi], cs[half + pi]) : rotated_second(o, y, cs[pi], cs[half + pi]);
    }
    const S r = from_f32<S>(y);
    if (is_q) row[q_off + e0] = r;
    else if (!slots) row[k_off + e0] = r;
    else if (slot >= 0) k_cache[(blk * Hkv + hd) * (int64_t)page * Dp + k_page_offset(off, d, page)] = r;
  }
  if (slot < 0 || !v_cache) return;
  for (int i = threadIdx.x; i < Hkv * Dv; i += 256) {
    float v = to_f32(row[v_off + i]);
    if (bias) v += bias[n + i];
    if (mix.first) v = mixed_value<S>(v, mix, t, i);
    v_cache[(blk * Hkv * Dv + i) * (int64_t)page + off] = from_f32<S>(v);
  }
}

// bf16 rows of whole 16-byte pieces that no boundary of a head, of its rotated part or (style 0) of that part's halves cuts:
// a thread owns one piece of 8 entries (ITERS of them) of q | k and keeps its bias and gains in registers for the per_block
// tokens its workgroup goes through, one after the other with the next one's piece on its way. Pairs (2i, 2i + 1) lie in a
// piece; for pairs (i, i + rot/2) the row passes through LDS. gather_v as in qkv_post_vec_kernel: then the workgroups from
// blockIdx.x = `blocks` on write V (8 * WAVES tokens of a kv head each, by their first WAVES waves).
template <int ITERS>
__global__ void __launch_bounds__(1024) qkv_row_post_vec_kernel(
    bf16* __restrict__ qkv, int64_t ld, int64_t q_off, int64_t k_off, int64_t v_off, const float* __restrict__ wq,
    const float* __restrict__ wk, float eps, const int32_t* __restrict__ pos, const float* __restrict__ cos_sin, int rot,
    int style, bf16* __restrict__ k_cache, bf16* __restrict__ v_cache, const int64_t* __restrict__ slots, int H, int Hkv,
    int D, int page, int Dv, const float* __restrict__ bias, int tokens, int per_block, int blocks, int gather_v,
    ValueMix mix) {
  extern __shared__ __attribute__((aligned(16))) float row_smem[];   // style 0: the normed row
  __shared__ float red[2][2][16];                                    // two sums a wave, two tokens in turn
  if ((int)blockIdx.x >= blocks) {
    const int j = (int)blockIdx.x - blocks;
    if (threadIdx.x < WAVES * 64)
      v_write_transposed(qkv, ld, v_off, v_cache, slots, tokens, Hkv, Dv, page, j / Hkv, j % Hkv,
                         bias ? bias + (int64_t)(H + Hkv) * D + (int64_t)(j % Hkv) * Dv : nullptr, mix);
    return;
  }
  const int nq = H * D, n = nq + Hkv * D, half = rot / 2, threads = blockDim.x;
  const int wave = threadIdx.x >> 6, lane = threadIdx.x & 63, waves = threads >> 6;
  int at[ITERS], d0[ITERS];
  float g[ITERS][8], bs[ITERS][8];
  bf16x8 x[ITERS];
  const int first_t = blockIdx.x * per_block, last_t = first_t + per_block < tokens ? first_t + per_block : tokens;
  auto source = [&](int t, int i) { return qkv + (int64_t)t * ld + (i < nq ? q_off + i : k_off + (i - nq)); };
#pragma unroll
  for (int it = 0; it < ITERS; ++it) {
    const int i = 8 * (it * threads + threadIdx.x);
    at[it] = i < n ? i : -1;
    d0[it] = 0;
#pragma unroll
    for (int e = 0; e < 8; ++e) g[it][e] = bs[it][e] = 0.f;
    x[it] = zero8();
    if (i >= n) continue;
    const int e0 = i < nq ? i : i - nq;
    d0[it] = e0 % D;
    x[it] = *(const bf16x8*)source(first_t, i);
    const float* w = (i < nq ? wq : wk) + e0;
    const f32x4 a = *(const f32x4*)w, b = *(const f32x4*)(w + 4);
#pragma unroll
    for (int e = 0; e < 4; ++e) { g[it][e] = a[e]; g[it][4 + e] = b[e]; }
    if (bias) {
      const f32x4 c = *(const f32x4*)(bias + i), d = *(const f32x4*)(bias + i + 4);
#pragma unroll
      for (int e = 0; e < 4; ++e) { bs[it][e] = c[e]; bs[it][4 + e] = d[e]; }
    }
  }
  for (int t = first_t; t < last_t; ++t) {
    float v[ITERS][8], c[ITERS][8], sn[ITERS][8];
    float sq = 0.f, sk = 0.f;
    const int64_t slot = slots ? slots[t] : -1;
    const float* cs = cos_sin ? cos_sin + (int64_t)pos[t] * rot : nullptr;
#pragma unroll
    for (int it = 0; it < ITERS; ++it) {
      if (at[it] < 0) continue;
#pragma unroll
      for (int e = 0; e < 8; ++e) {
        v[it][e] = (float)x[it][e] + bs[it][e];
        if (at[it] < nq) sq = add_square(sq, v[it][e]);
        else sk = add_square(sk, v[it][e]);
      }
      if (cs && d0[it] < rot) {      // style 1: four pairs a piece; style 0: eight, of one half
        const int pi = style ? d0[it] / 2 : d0[it] < half ? d0[it] : d0[it] - half;
        const f32x4 c0 = *(const f32x4*)(cs + pi), s0 = *(const f32x4*)(cs + half + pi);
#pragma unroll
        for (int e = 0; e < 4; ++e) { c[it][e] = c0[e]; sn[it][e] = s0[e]; }
        if (!style) {
          const f32x4 c1 = *(const f32x4*)(cs + pi + 4), s1 = *(const f32x4*)(cs + half + pi + 4);
#pragma unroll
          for (int e = 0; e < 4; ++e) { c[it][4 + e] = c1[e]; sn[it][4 + e] = s1[e]; }
        }
      }
      if (t + 1 < last_t) x[it] = *(const bf16x8*)source(t + 1, at[it]);
    }
    sq = wave_sum(sq);
    sk = wave_sum(sk);
    float (&rd)[2][16] = red[(t - first_t) & 1];
    if (lane == 0) { rd[0][wave] = sq; rd[1][wave] = sk; }
    __syncthreads();
    sq = sk = 0.f;
    for (int w = 0; w < waves; ++w) { sq += rd[0][w]; sk += rd[1][w]; }      // a fixed order: the same in every thread
    const float fq = 1.f / sqrtf(sq / (float)nq + eps), fk = 1.f / sqrtf(sk / (float)(n - nq) + eps);
#pragma unroll
    for (int it = 0; it < ITERS; ++it) {
      if (at[it] < 0) continue;
      const float f = at[it] < nq ? fq : fk;
#pragma unroll
      for (int e = 0; e < 8; ++e) v[it][e] = v[it][e] * f * g[it][e];
      if (cs && !style) {
        f32x4 a, b;
#pragma unroll
        for (int e = 0; e < 4; ++e) { a[e] = v[it][e]; b[e] = v[it][4 + e]; }
        *(f32x4*)(row_smem + at[it]) = a;
        *(f32x4*)(row_smem + at[it] + 4) = b;
      }
    }
    if (cs && !style) __syncthreads();
    const int64_t blk = slot >= 0 ? slot / page : 0;
    const int off = slot >= 0 ? (int)(slot % page) : 0;
#pragma unroll
    for (int it = 0; it < ITERS; ++it) {
      if (at[it] < 0) continue;
      if (cs && d0[it] < rot) {
        if (style) {
#pragma unroll
          for (int e = 0; e < 4; ++e) {
            const float u = v[it][2 * e], w = v[it][2 * e + 1];
            v[it][2 * e] = rotated_first(u, w, c[it][e], sn[it][e]);
            v[it][2 * e + 1] = rotated_second(u, w, c[it][e], sn[it][e]);
          }
        } else {
          const bool first = d0[it] < half;
          const float* o = row_smem + at[it] + (first ? half : -half);
          const f32x4 o0 = *(const f32x4*)o, o1 = *(const f32x4*)(o + 4);
#pragma unroll
          for (int e = 0; e < 8; ++e) {
            const float other = e < 4 ? o0[e & 3] : o1[e & 3];
            v[it][e] = first ? rotated_first(v[it][e], other, c[it][e], sn[it][e]) : rotated_second(other, v[it][e], c[it][e], sn[it][e]);
          }
        }
      }
      bf16x8 r;
#pragma unroll
      for (int e = 0; e < 8; ++e) r[e] = (bf16)v[it][e];
      if (at[it] < nq || !slots) {
        *(bf16x8*)source(t, at[it]) = r;
      } else if (slot >= 0) {
        const int hd = (at[it] - nq) / D;
        *(bf16x8*)(k_cache + (blk * Hkv + hd) * (int64_t)page * D + k_page_offset(off, d0[it], page)) = r;
      }
    }
    if (cs && !style) __syncthreads();      // the row has been read before the next token's is written
    if (slot >= 0 && v_cache && gather_v == 0) {
      const bf16* vr = qkv + (int64_t)t * ld + v_off;
      for (int i = threadIdx.x; i < Hkv * Dv; i += threads) {
        float y = (float)vr[i];
        if (bias) y += bias[n + i];
        if (mix.first) y = mixed_value<bf16>(y, mix, t, i);
        v_cache[(blk * Hkv * Dv + i) * (int64_t)page + off] = (bf16)y;
      }
    }
  }
}

}  // namespace

// qkv_post with norms over the whole projection: q_gain [heads head_dim], k_gain [kv_heads head_dim], float. Everything
// else as there. kv_heads 0: queries alone (a layer that reads another one's keys); nothing is written to the cache.
extern "C" int dinfer_qkv_row_post(int dtype, void* qkv, int64_t tokens, int64_t ld, int64_t q_off, int64_t k_off,
                                   int64_t v_off, const float* q_gain, const float* k_gain, float eps,
                                   const int32_t* positions, const float* cos_sin, int rotary_dim, int style, void* k_cache,
                                   void* v_cache, const int64_t* slot_mapping, int heads, int kv_heads, int head_dim,
                                   int page_size, int token_runs, int v_dim, const float* bias, const void* v_first,
                                   int64_t ld_v_first, float v_share, hipStream_t stream) {
  if (v_dim <= 0) v_dim = head_dim;
  if (tokens <= 0) return OK;
  if (heads <= 0 || kv_heads < 0 || head_dim <= 0 || page_size <= 0 || tokens > 0x7fffffff || !q_gain ||
      (kv_heads > 0 && !k_gain) || (kv_heads == 0 && slot_mapping))
    return ERR_BAD_SHAPE;
  if (cos_sin && (rotary_dim <= 0 || rotary_dim > head_dim || rotary_dim % 2 != 0)) return ERR_BAD_SHAPE;
  if (style != 0 && style != 1) return ERR_UNSUPPORTED;
  const int64_t n = (int64_t)(heads + kv_heads) * head_dim;
  if (n > 32768) return ERR_UNSUPPORTED;      // (128 KB of LDS)
  const size_t lds = (size_t)n * sizeof(float);
  const ValueMix mix{v_first, ld_v_first, v_share};
  const int rot = cos_sin ? rotary_dim : 0;
  const bool vec = dtype == DT_BF16 && head_dim % 8 == 0 && rot % (style == 0 ? 16 : 8) == 0 && ld % 8 == 0 && q_off % 8 == 0 &&
                   k_off % 8 == 0 && v_off % 2 == 0 && v_dim % 2 == 0 && n <= 8 * 1024 * 2 && ((uintptr_t)qkv % 16) == 0 &&
                   ((uintptr_t)k_cache % 16) == 0 && ((uintptr_t)q_gain % 16) == 0 && ((uintptr_t)k_gain % 16) == 0 &&
                   ((uintptr_t)bias % 16) == 0 && ((uintptr_t)cos_sin % 16) == 0;
  if (vec) {
    const int64_t pieces = n / 8;
    const int iters = (int)((pieces + 1023) / 1024);
    int threads = (int)((pieces + iters - 1) / iters);
    threads = (threads + 63) / 64 * 64;
    const bool gather = slot_mapping && v_cache && token_runs && tokens >= 64 && page_size % 8 == 0 &&
                        ((uintptr_t)v_cache % 16) == 0;
    if (gather && threads < WAVES * 64) threads = WAVES * 64;
    const int64_t gather_v = gather ? (tokens + 8 * WAVES - 1) / (8 * WAVES) * kv_heads : 0;
    // many tokens: a workgroup takes several, so that gains and biases are fetched once for them
    const int per = tokens >= 1024 ? 4 : tokens >= 512 ? 2 : 1;
    const int64_t blocks = (tokens + per - 1) / per;
    if (blocks + gather_v > 0x7fffffff) return ERR_BAD_SHAPE;
    const size_t rows = rot && style == 0 ? lds : 0;
    auto kernel = iters == 1 ? qkv_row_post_vec_kernel<1> : qkv_row_post_vec_kernel<2>;
    if (rows > 65536 - 512 && hipFuncSetAttribute((const void*)kernel, hipFuncAttributeMaxDynamicSharedMemorySize, (int)rows) != hipSuccess)
      return ERR_LAUNCH;
    kernel<<<(unsigned)(blocks + gather_v), threads, rows, stream>>>(
        (bf16*)qkv, ld, q_off, k_off, v_off, q_gain, k_gain, eps, positions, cos_sin, rot, style, (bf16*)k_cache, (bf16*)v_cache,
        slot_mapping, heads, kv_heads, head_dim, page_size, v_dim, bias, (int)tokens, per, (int)blocks, (int)gather_v, mix);
    return launch_status();
  }
  DINFER_DISPATCH_DTYPE(dtype, {
    auto kernel = qkv_row_post_kernel<S>;
    if (lds > 65536 - 64 && hipFuncSetAttribute((const void*)kernel, hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds) != hipSuccess)
      return ERR_LAUNCH;
    kernel<<<(unsigned)tokens, 256, lds, stream>>>((S*)qkv, ld, q_off, k_off, v_off, q_gain, k_gain, eps, positions, cos_sin, rot,
                                                   style, (S*)k_cache, (S*)v_cache, slot_mapping, heads, kv_heads, head_dim,
                                                   page_size, v_dim, bias, mix);
  });
  return launch_status();
}

extern "C" int dinfer_qkv_post(int dtype, void* qkv, int64_t tokens, int64_t ld, int64_t q_off, int64_t k_off,
                               int64_t v_off, const void* q_gain, const void* k_gain, int w_f32, float eps,
                               float w_offset, const int32_t* positions, const float* cos_sin, int rotary_dim,
                               int style, void* k_cache, void* v_cache, const int64_t* slot_mapping, int heads,
                               int kv_heads, int head_dim, int page_size, int token_runs, int v_dim,
                               const float* bias, float temp_coef, int temp_every, const float* head_scale,
                               const void* v_first, int64_t ld_v_first, float v_share, hipStream_t stream) {
  // v_first (may be null): [tokens, ld_v_first] in the step's dtype, kv heads of v_dim side by side; the cached values are
  // (1 - v_share) v + v_share v_first.
  // head_scale (may be null): float [heads], q of head h is multiplied by head_scale[h] with the norm (gains needed).
  // bias (may be null): float [q heads | k heads | v heads], added to the product's output before anything else.
  // temp_every > 0: q is multiplied by 1 + temp_coef ln(floor((p + 1) / temp_every) + 1) with the norm (gains needed).
  // v_dim: the size of a value head, 0 for head_dim. v_cache may be null beside a k_cache (values are not stored).
  if (v_dim <= 0) v_dim = head_dim;
  // token_runs: the tokens come in runs of consecutive positions of a request (prompt portions), so
  // that gathering 8 tokens' values into 16-byte rows of the transposed V pages pays
  if (tokens <= 0) return OK;
  if (heads <= 0 || kv_heads <= 0 || head_dim <= 0 || page_size <= 0 || tokens > 0x7fffffff) return ERR_BAD_SHAPE;
  if (head_dim > MAX_D) return ERR_UNSUPPORTED;
  if (cos_sin && (rotary_dim <= 0 || rotary_dim > head_dim || rotary_dim % 2 != 0)) return ERR_BAD_SHAPE;
  if (style != 0 && style != 1) return ERR_UNSUPPORTED;
  if ((q_gain == nullptr) != (k_gain == nullptr)) return ERR_BAD_SHAPE;
  const int items = heads + 2 * kv_heads;
  const dim3 grid((unsigned)tokens, (unsigned)((items + WAVES - 1) / WAVES));
  if ((temp_every > 0 || head_scale) && !q_gain) return ERR_UNSUPPORTED;
  const bool whole_head_neox = style == 0 && head_dim % 8 == 0 && (!cos_sin || rotary_dim == head_dim) &&
                               v_dim == head_dim && (v_cache || !slot_mapping);
  const ValueMix mix{v_first, ld_v_first, v_share};
  const bool plain_head = !bias && temp_every <= 0 && !head_scale && !v_first;   // what the kernels of 2-byte accesses for whole heads take
  const bool vec_ok = dtype == DT_BF16 && (head_dim == 64 || head_dim == 128 || head_dim == 256) && ld % 8 == 0 &&
                      q_off % 8 == 0 && k_off % 8 == 0 && v_off % 8 == 0 && ((uintptr_t)qkv % 16) == 0 &&
                      ((uintptr_t)q_gain % 16) == 0 && ((uintptr_t)k_gain % 16) == 0 && ((uintptr_t)cos_sin % 16) == 0 &&
                      ((uintptr_t)k_cache % 16) == 0 && ((uintptr_t)bias % 16) == 0 &&
                      (!v_first || (((uintptr_t)v_first % 16) == 0 && ld_v_first % 8 == 0));
  if (whole_head_neox && vec_ok) {
    const int lph = head_dim / 8, hpw = 64 / lph;
    // many tokens fill the chip with one workgroup each; few tokens spread their heads over several
    // many tokens: V goes to its transposed pages through workgroups that gather it (16-byte stores)
    const bool gather = slot_mapping && token_runs && tokens >= 64 && page_size % 8 == 0 && ((uintptr_t)v_cache % 16) == 0;
    const int64_t gather_v = gather ? (tokens + 8 * WAVES - 1) / (8 * WAVES) * kv_heads : 0;
    if (tokens + gather_v > 0x7fffffff) return ERR_BAD_SHAPE;
    const dim3 vgrid((unsigned)(tokens + gather_v),
                     tokens >= 512 ? 1u : (unsigned)((items + WAVES * hpw - 1) / (WAVES * hpw)));
#define DINFER_QKV_VEC(LPH_)                                                                                          \
  qkv_post_vec_kernel<LPH_><<<vgrid, WAVES * 64, 0, stream>>>(                                                         \
      (bf16*)qkv, ld, q_off, k_off, v_off, q_gain, k_gain, w_f32, eps, w_offset, positions, cos_sin, (bf16*)k_cache, \
      (bf16*)v_cache, slot_mapping, heads, kv_heads, page_size, (int)tokens, (int)gather_v, bias, temp_coef,       \
      temp_every, head_scale, mix)
    if (lph == 8) DINFER_QKV_VEC(8);
    else if (lph == 16) DINFER_QKV_VEC(16);
    else DINFER_QKV_VEC(32);
#undef DINFER_QKV_VEC
    return launch_status();
  }
  if (whole_head_neox && plain_head) {
    const dim3 grid((unsigned)tokens, (unsigned)((items + WAVES * IPW - 1) / (WAVES * IPW)));
    DINFER_DISPATCH_DTYPE(dtype, {
      if (head_dim <= 128)
        qkv_post_neox_kernel<S, 1><<<grid, WAVES * 64, 0, stream>>>(
            (S*)qkv, ld, q_off, k_off, v_off, q_gain, k_gain, w_f32, eps, w_offset, positions, cos_sin, (S*)k_cache,
            (S*)v_cache, slot_mapping, heads, kv_heads, head_dim, page_size);
      else if (head_dim <= 256)
        qkv_post_neox_kernel<S, 2><<<grid, WAVES * 64, 0, stream>>>(
            (S*)qkv, ld, q_off, k_off, v_off, q_gain, k_gain, w_f32, eps, w_offset, positions, cos_sin, (S*)k_cache,
            (S*)v_cache, slot_mapping, heads, kv_heads, head_dim, page_size);
      else
        qkv_post_neox_kernel<S, 4><<<grid, WAVES * 64, 0, stream>>>(
            (S*)qkv, ld, q_off, k_off, v_off, q_gain, k_gain, w_f32, eps, w_offset, positions, cos_sin, (S*)k_cache,
            (S*)v_cache, slot_mapping, heads, kv_heads, head_dim, page_size);
    });
    return launch_status();
  }
  DINFER_DISPATCH_DTYPE(dtype, {
    qkv_post_kernel<S><<<grid, WAVES * 64, 0, stream>>>((S*)qkv, ld, q_off, k_off, v_off, q_gain, k_gain, w_f32, eps,
                                                        w_offset, positions, cos_sin, rotary_dim, style, (S*)k_cache,
                                                        (S*)v_cache, slot_mapping, heads, kv_heads, head_dim,
                                                        page_size, v_dim, bias, temp_coef, temp_every,
                                                        head_scale, mix);
  });
  return launch_status();
}
