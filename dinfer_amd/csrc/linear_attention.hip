// Gated linear attention: per request and head one matrix S [D, V] in float whose every row (a key channel) decays by a
// factor of its own,
//
//   per token:   S <- diag(a_t) S + k_t v_t^T;   o_t = S^T (q_t * q_scale)
//
//   channel_decay   a = sigmoid(z)^(1 / tau), z = W2 low + bias: a thread a channel, `low` (the step's inner projection)
//                   of up to 8 tokens in LDS, so a column of W2 is read once per 8 tokens; float out
//   recurrence      q, k and v are read as the projections left them, a in float. A request, a head and 8 CPT columns of
//                   S a workgroup: the 32 lanes of half a wave share CPT columns and own a strip of their rows; 16
//                   tokens' operands wait in LDS while the next 16 are on their way in registers
//
// The step is a linear map of S, so where a step's portions are too few to fill the chip they are cut into chunks of CL
// tokens that run side by side:
//   chunks pass     what every chunk makes of S = 0, and the product of its decays (the portion's last chunk: nothing)
//   scan            chunk by chunk, every entry of S by itself: a chunk's note becomes the S it starts from
//   recurrence      as above, a chunk a workgroup, from that S; the portion's last chunk stores the request's state
// With FIXED one constant decay a head takes the place of the decays a channel and token (lightning attention); then q, k
// and v may pass a silu on their way in.
// Chunks are counted from the portion's start. S is stored transposed, [slot][head][V][D]. A request whose step starts at
// position 0 starts from S = 0, whatever its slot held.
#include "common.cuh"

using namespace dinfer;

namespace {

constexpr int CH = 16;          // tokens whose operands wait in LDS
constexpr int CL = 128;         // tokens of a chunk (a multiple of CH)
constexpr int LOW_TOKENS = 8;
constexpr int MAX_LOW = 512;
constexpr float LOG2E = 1.4426950408889634f;

template <class S, int TT>
__global__ void __launch_bounds__(256) channel_decay_kernel(const S* __restrict__ proj, int64_t ld, int64_t low_off, int low,
                                                            const float* __restrict__ w2t, const float* __restrict__ bias,
                                                            float inv_tau, float* __restrict__ out, int64_t ld_out, int C,
                                                            int tokens) {
  __shared__ float lows[TT][MAX_LOW];
  const int t0 = blockIdx.y * TT, c = blockIdx.x * 256 + threadIdx.x;
  const int nt = tokens - t0 < TT ? tokens - t0 : TT;
  for (int i = threadIdx.x; i < TT * low; i += 256) {
    const int t = i / low, r = i - t * low;
    lows[t][r] = t < nt ? to_f32(proj[(int64_t)(t0 + t) * ld + low_off + r]) : 0.f;
  }
  __syncthreads();
  if (c >= C) return;
  float z[TT];
  const float b = bias[c];
#pragma unroll
  for (int t = 0; t < TT; ++t) z[t] = b;
#pragma unroll 4
  for (int r = 0; r < low; ++r) {
    const float w = w2t[(int64_t)r * C + c];
#pragma unroll
    for (int t = 0; t < TT; ++t) z[t] = __builtin_fmaf(w, lows[t][r], z[t]);
  }
#pragma unroll
  for (int t = 0; t < TT; ++t) {
    // log2 sigmoid(z) = min(y, 0) - log2(1 + 2^-|y|), y = z log2(e); the logarithm of one and next to nothing as the
    // first terms of its series, or the slow decays would lose what sets them apart from one
    const float y = z[t] * LOG2E, e = __builtin_amdgcn_exp2f(-fabsf(y));
    const float l = e < 0.0078125f ? LOG2E * e * (1.f - e * (0.5f - e * (1.f / 3.f))) : __builtin_amdgcn_logf(1.f + e);
    if (t < nt) out[(int64_t)(t0 + t) * ld_out + c] = __builtin_amdgcn_exp2f((fminf(y, 0.f) - l) * inv_tau);
  }
}

// A lane's value plus that of the lane a DPP pattern pairs it with (full-rate vector instructions, no LDS).
template <int CTRL>
__device__ __forceinline__ float dpp_add(float v) {
  return v + __builtin_bit_cast(float, __builtin_amdgcn_update_dpp(0, __builtin_bit_cast(int, v), CTRL, 0xf, 0xf, true));
}
// The sum over 32 lanes (two DPP rows of 16), in every lane of them.
__device__ __forceinline__ float half_wave_sum(float v) {
  v = dpp_add<0xB1>(v);    // quad_perm [1, 0, 3, 2]
  v = dpp_add<0x4E>(v);    // quad_perm [2, 3, 0, 1]
  v = dpp_add<0x141>(v);   // row_half_mirror
  v = dpp_add<0x140>(v);   // row_mirror
  return v + __shfl_xor(v, 16, WAVE);
}

// 8 consecutive operands of a token as they lie in memory
template <class O> struct Piece;
template <> struct Piece<bf16> {
  bf16x8 v;
  __device__ __forceinline__ void load(const bf16* p) { v = *(const bf16x8*)p; }
  __device__ __forceinline__ void zero() {
#pragma unroll
    for (int i = 0; i < 8; ++i) v[i] = (bf16)0.f;
  }
  __device__ __forceinline__ void set(int i, bf16 x) { v[i] = x; }
  __device__ __forceinline__ float get(int i) const { return (float)v[i]; }
};
template <> struct Piece<float> {
  f32x4 a, b;
  __device__ __forceinline__ void load(const float* p) { a = *(const f32x4*)p; b = *(const f32x4*)(p + 4); }
  __device__ __forceinline__ void zero() { a = b = f32x4{0.f, 0.f, 0.f, 0.f}; }
  __device__ __forceinline__ void set(int i, float x) { if (i < 4) a[i] = x; else b[i - 4] = x; }
  __device__ __forceinline__ float get(int i) const { return i < 4 ? a[i] : b[i - 4]; }
};

template <class O>
struct Gla {
  const O* q; const O* k; const O* v; int64_t ld;     // heads side by side from these columns of a row
  const float* decay; int64_t ldd;                    // [T, H D]
  float q_scale;
  float* state;                                       // [slots, H, V, D]
  float* notes; float* products;                      // [places, H, V, D], [places, H, D]
  const int32_t* slots; const int32_t* cu; const int32_t* seq_lens;
  float* out; int64_t ld_out;
  int H, D, V, cl, vec;                               // vec: pieces of 8 operands come by 16-byte loads
  const float* fixed;                                 // FIXED: [H], the head's decay
  int act;                                            // 1: q, k and v are silu of what lies in memory
};

// where a chunk's note lies: places of different requests never meet (floor(cu / CL) + request grows by at least the
// request's number of chunks)
__device__ __forceinline__ int64_t place_of(int t0, int b, int chunk) { return (int64_t)(t0 / CL) + b + chunk; }

// OUT: the recurrence itself; else the chunks pass. A thread owns RPT consecutive rows of CPT columns (D <= 32 RPT).
template <class O, int RPT, int CPT, bool OUT, bool FIXED>
__global__ void __launch_bounds__(256) gla_kernel(Gla<O> p) {
  constexpr int DP = 32 * RPT, COLS = 8 * CPT;
  __shared__ __attribute__((aligned(16))) float ks[CH][DP];
  __shared__ __attribute__((aligned(16))) float as[FIXED ? 1 : CH][DP];
  __shared__ __attribute__((aligned(16))) float qs[OUT ? CH : 1][DP];
  __shared__ __attribute__((aligned(16))) float vs[CH][COLS];
  // the request is the slowest index of the grid: the workgroups of one long request among many short ones then spread
  // over all XCDs
  const int blocks = (p.V + COLS - 1) / COLS;
  const int cb = blockIdx.x % blocks, h = blockIdx.x / blocks, chunk = blockIdx.y, b = blockIdx.z;
  const int tid = threadIdx.x, rg = tid & 31, cj = tid >> 5;
  const int D = p.D, V = p.V;
  const int r0 = p.cu[b], rows = p.cu[b + 1] - r0;
  const int64_t first = (int64_t)chunk * p.cl;
  if (first >= rows) return;
  const bool last = first + p.cl >= rows, single = rows <= p.cl;
  if (!OUT && last) return;
  const int t0 = r0 + (int)first, n = last ? rows - (int)first : p.cl;
  const int64_t place = single ? 0 : place_of(r0, b, chunk);
  const int64_t matrix = (int64_t)V * D;

  int col[CPT];
  float S[CPT][RPT];
  const bool quads = RPT % 4 == 0 && D % 4 == 0;
  const bool from_state = OUT && single && p.seq_lens[b] > rows;
  const float* init = nullptr;
  if (OUT) {
    if (!single) init = p.notes + (place * p.H + h) * matrix;
    else if (from_state) init = p.state + ((int64_t)p.slots[b] * p.H + h) * matrix;
  }
#pragma unroll
  for (int c = 0; c < CPT; ++c) {
    col[c] = cb * COLS + cj * CPT + c;
    const bool ok = init && col[c] < V;
    const float* sp = init + (int64_t)(ok ? col[c] : 0) * D + rg * RPT;
    if (quads) {
#pragma unroll
      for (int i = 0; i < RPT; i += 4) {
        f32x4 x = {0.f, 0.f, 0.f, 0.f};
        if (ok && rg * RPT + i < D) x = *(const f32x4*)(sp + i);
#pragma unroll
        for (int e = 0; e < 4; ++e)
          if (i + e < RPT) S[c][i + e] = x[e];
      }
    } else {
#pragma unroll
      for (int i = 0; i < RPT; ++i) S[c][i] = (ok && rg * RPT + i < D) ? sp[i] : 0.f;
    }
  }
  float prod[RPT];      // !OUT: the product of the chunk's decays (every column group has it)
#pragma unroll
  for (int i = 0; i < RPT; ++i) prod[i] = 1.f;

  // what a thread carries of the next 16 tokens: pieces of k, q and the decays, entries of v
  constexpr int PIECES = CH * DP / 8, NP = (PIECES + 255) / 256, NV = (CH * COLS + 255) / 256;
  Piece<O> pk[NP], pq[OUT ? NP : 1];
  Piece<float> pa[FIXED ? 1 : NP];
  const float head_decay = FIXED ? p.fixed[h] : 1.f;
  auto entry = [&](float x) { return p.act ? x / (1.f + expf(-x)) : x; };
  float pv[NV];
  auto piece = [&](auto& dst, const auto* src, bool in, int d) {
    if (!in) { dst.zero(); return; }
    if (p.vec) { dst.load(src); return; }
    dst.zero();
#pragma unroll
    for (int i = 0; i < 8; ++i)
      if (d + i < D) dst.set(i, src[i]);
  };
  auto fetch = [&](int ct) {
#pragma unroll
    for (int e = 0; e < NP; ++e) {
      const int idx = tid + e * 256;
      const int tok = idx / (DP / 8), d = (idx % (DP / 8)) * 8;
      const bool in = idx < PIECES && ct + tok < n && d < D;
      const int64_t t = t0 + ct + tok;
      piece(pk[e], p.k + t * p.ld + (int64_t)h * D + d, in, d);
      if constexpr (OUT) piece(pq[e], p.q + t * p.ld + (int64_t)h * D + d, in, d);
      if constexpr (!FIXED) piece(pa[e], p.decay + t * p.ldd + (int64_t)h * D + d, in, d);
    }
#pragma unroll
    for (int e = 0; e < NV; ++e) {
      const int idx = tid + e * 256;
      const int tok = idx / COLS, c = cb * COLS + idx % COLS;
      pv[e] = (idx < CH * COLS && ct + tok < n && c < V) ? entry(to_f32(p.v[(int64_t)(t0 + ct + tok) * p.ld + (int64_t)h * V + c])) : 0.f;
    }
  };
  auto put = [&](float* dst, const auto& src, float f, bool raw) {
    f32x4 a, b2;
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      a[i] = (raw ? src.get(i) : entry(src.get(i))) * f;
      b2[i] = (raw ? src.get(4 + i) : entry(src.get(4 + i))) * f;
    }
    *(f32x4*)dst = a;
    *(f32x4*)(dst + 4) = b2;
  };
  // one token: the state's update; with OUT the lane's share of its CPT outputs
  auto token = [&](int tok, float (&part)[CPT]) {
    float kk[RPT], aa[RPT], qq[RPT];
#pragma unroll
    for (int i = 0; i < RPT; ++i) {
      kk[i] = ks[tok][rg * RPT + i];
      aa[i] = FIXED ? head_decay : as[FIXED ? 0 : tok][rg * RPT + i];
      if constexpr (OUT) qq[i] = qs[tok][rg * RPT + i];
      else prod[i] *= aa[i];
    }
#pragma unroll
    for (int c = 0; c < CPT; ++c) {
      const float vt = vs[tok][cj * CPT + c];
      float o0 = 0.f, o1 = 0.f;   // two chains: a fixed order all the same
#pragma unroll
      for (int i = 0; i < RPT; ++i) {
        S[c][i] = __builtin_fmaf(kk[i], vt, aa[i] * S[c][i]);
        if constexpr (OUT) {
          if (i & 1) o1 = __builtin_fmaf(S[c][i], qq[i], o1);
          else o0 = __builtin_fmaf(S[c][i], qq[i], o0);
        }
      }
      part[c] = o0 + o1;
    }
  };
  fetch(0);
  for (int ct = 0; ct < n; ct += CH) {
    __syncthreads();  // the 16 tokens before have been consumed
#pragma unroll
    for (int e = 0; e < NP; ++e) {
      const int idx = tid + e * 256;
      if (idx < PIECES) {
        const int tok = idx / (DP / 8), d = (idx % (DP / 8)) * 8;
        put(&ks[tok][d], pk[e], 1.f, false);
        if constexpr (OUT) put(&qs[tok][d], pq[e], p.q_scale, false);
        if constexpr (!FIXED) put(&as[tok][d], pa[e], 1.f, true);
      }
    }
#pragma unroll
    for (int e = 0; e < NV; ++e) {
      const int idx = tid + e * 256;
      if (idx < CH * COLS) vs[idx / COLS][idx % COLS] = pv[e];
    }
    __syncthreads();
    if (ct + CH < n) fetch(ct + CH);  // in flight while these are worked through
    const int m = n - ct < CH ? n - ct : CH;
    // four tokens a round: only the state's update runs from token to token, the row sums meet the lanes together
    int t4 = 0;
    for (; t4 + 4 <= m; t4 += 4) {
      float part[4][CPT];
#pragma unroll
      for (int u = 0; u < 4; ++u) token(t4 + u, part[u]);
      if constexpr (OUT) {
#pragma unroll
        for (int u = 0; u < 4; ++u)
#pragma unroll
          for (int c = 0; c < CPT; ++c) part[u][c] = half_wave_sum(part[u][c]);
        if (rg < 4) {
#pragma unroll
          for (int c = 0; c < CPT; ++c) {
            const float o = rg == 0 ? part[0][c] : rg == 1 ? part[1][c] : rg == 2 ? part[2][c] : part[3][c];
            if (col[c] < V) p.out[(int64_t)(t0 + ct + t4 + rg) * p.ld_out + (int64_t)h * V + col[c]] = o;
          }
        }
      }
    }
    for (int tok = t4; tok < m; ++tok) {
      float part[CPT];
      token(tok, part);
      if constexpr (OUT) {
#pragma unroll
        for (int c = 0; c < CPT; ++c) {
          const float o = half_wave_sum(part[c]);
          if (rg == 0 && col[c] < V) p.out[(int64_t)(t0 + ct + tok) * p.ld_out + (int64_t)h * V + col[c]] = o;
        }
      }
    }
  }
  if (OUT && !last) return;
  float* to = OUT ? p.state + ((int64_t)p.slots[b] * p.H + h) * matrix : p.notes + (place * p.H + h) * matrix;
#pragma unroll
  for (int c = 0; c < CPT; ++c) {
    if (col[c] >= V) continue;
    float* sp = to + (int64_t)col[c] * D + rg * RPT;
    if (quads) {
#pragma unroll
      for (int i = 0; i < RPT; i += 4) {
        f32x4 x;
#pragma unroll
        for (int e = 0; e < 4; ++e) x[e] = S[c][i + e < RPT ? i + e : 0];
        if (rg * RPT + i < D) *(f32x4*)(sp + i) = x;
      }
    } else {
#pragma unroll
      for (int i = 0; i < RPT; ++i)
        if (rg * RPT + i < D) sp[i] = S[c][i];
    }
  }
  if (!OUT && cb == 0 && cj == 0) {
    float* pp = p.products + (place * p.H + h) * D + rg * RPT;
#pragma unroll
    for (int i = 0; i < RPT; ++i)
      if (rg * RPT + i < D) pp[i] = prod[i];
  }
}

// Every entry of S by itself: the notes of a request's chunks, in order, become the S each chunk starts from.
template <class O>
__global__ void __launch_bounds__(256) gla_scan_kernel(Gla<O> p) {
  const int b = blockIdx.z;
  const int r0 = p.cu[b], rows = p.cu[b + 1] - r0;
  if (rows <= p.cl) return;
  const int chunks = (rows + p.cl - 1) / p.cl;
  const int64_t per = (int64_t)p.H * p.V * p.D;
  const int64_t i = (int64_t)blockIdx.x * 256 + threadIdx.x;
  if (i >= per) return;
  const int d = (int)(i % p.D), h = (int)(i / ((int64_t)p.V * p.D));
  float s = p.seq_lens[b] > rows ? p.state[(int64_t)p.slots[b] * per + i] : 0.f;
  const int64_t base = place_of(r0, b, 0);
  float* note = p.notes + base * per + i;
  const float* prod = p.products + (base * p.H + h) * p.D + d;
  const int64_t pstep = (int64_t)p.H * p.D;
  int c = 0;
  for (; c + 4 < chunks; c += 4) {      // (the last chunk has no note of its own)
    float nb[4], na[4];
#pragma unroll
    for (int u = 0; u < 4; ++u) {
      nb[u] = note[(int64_t)(c + u) * per];
      na[u] = prod[(int64_t)(c + u) * pstep];
    }
#pragma unroll
    for (int u = 0; u < 4; ++u) {
      note[(int64_t)(c + u) * per] = s;
      s = __builtin_fmaf(na[u], s, nb[u]);
    }
  }
  for (; c < chunks; ++c) {
    const float nb = c + 1 < chunks ? note[(int64_t)c * per] : 0.f, na = c + 1 < chunks ? prod[(int64_t)c * pstep] : 1.f;
    note[(int64_t)c * per] = s;
    s = __builtin_fmaf(na, s, nb);
  }
}

template <class O, int RPT, bool FIXED>
void launch_gla(Gla<O> p, int64_t chunks, int num_reqs, bool wide, hipStream_t stream) {
  const auto grid = [&](int cols) { return dim3((unsigned)((p.V + cols - 1) / cols * p.H), (unsigned)chunks, (unsigned)num_reqs); };
  if (chunks > 1) {
    gla_kernel<O, RPT, 2, false, FIXED><<<grid(16), 256, 0, stream>>>(p);
    const int64_t per = (int64_t)p.H * p.V * p.D;
    gla_scan_kernel<O><<<dim3((unsigned)((per + 255) / 256), 1, (unsigned)num_reqs), 256, 0, stream>>>(p);
  }
  if (wide) gla_kernel<O, RPT, 2, true, FIXED><<<grid(16), 256, 0, stream>>>(p);
  else gla_kernel<O, RPT, 1, true, FIXED><<<grid(8), 256, 0, stream>>>(p);
}

template <class O, int RPT>
void pick_gla(const Gla<O>& p, int64_t chunks, int num_reqs, bool wide, hipStream_t stream) {
  if (p.fixed) launch_gla<O, RPT, true>(p, chunks, num_reqs, wide, stream);
  else launch_gla<O, RPT, false>(p, chunks, num_reqs, wide, stream);
}

}  // namespace

// Tokens of a chunk. A step that is cut into chunks needs tokens / chunk + requests + 1 notes of H V D floats and as many
// products of H D.
extern "C" int dinfer_gla_chunk() { return CL; }

// Whether a step with this many tokens, requests and rows in its longest portion is cut into chunks: where the work of
// the portions side by side would leave most of the chip idle while the longest runs.
extern "C" int dinfer_gla_cuts(int64_t tokens, int64_t max_rows, int num_reqs, int H, int V) {
  if (max_rows <= CL || num_reqs <= 0) return 0;
  const double at_once = (double)tokens / (double)max_rows * H * ((V + 7) / 8);     // workgroups busy on average
  return at_once < 2048. ? 1 : 0;
}

// proj [T, ld] in the step's dtype: the inner projection's `low` columns from low_off. w2t [low][C] float (transposed),
// bias [C] float. out [T, ld_out] float: sigmoid(w2 low + bias)^inv_tau.
extern "C" int dinfer_channel_decay(int dtype, const void* proj, int64_t ld, int64_t low_off, int low, const float* w2t,
                                    const float* bias, float inv_tau, float* out, int64_t ld_out, int64_t tokens, int64_t C,
                                    hipStream_t stream) {
  if (tokens <= 0) return OK;
  if (low <= 0 || C <= 0 || ld_out < C || tokens > 0x7fffffff || C > 0x7fffffff) return ERR_BAD_SHAPE;
  const int tt = tokens <= 64 ? 1 : LOW_TOKENS;
  const int64_t gy = (tokens + tt - 1) / tt;
  if (low > MAX_LOW || gy > 65535) return ERR_UNSUPPORTED;
  const dim3 grid((unsigned)((C + 255) / 256), (unsigned)gy);
  DINFER_DISPATCH_DTYPE(dtype, {
    if (tt == 1)
      channel_decay_kernel<S, 1><<<grid, 256, 0, stream>>>((const S*)proj, ld, low_off, low, w2t, bias, inv_tau, out, ld_out,
                                                           (int)C, (int)tokens);
    else
      channel_decay_kernel<S, LOW_TOKENS><<<grid, 256, 0, stream>>>((const S*)proj, ld, low_off, low, w2t, bias, inv_tau, out,
                                                                    ld_out, (int)C, (int)tokens);
  });
  return launch_status();
}

// q, k [T, H D], v [T, H V]: columns of rows of stride ld in the step's dtype; decay [T, ldd >= H D] float. state
// [slots, H, V, D] float; out [T, ld_out] float, head h at column h V. cut: the step runs in chunks (dinfer_gla_cuts),
// with notes [places, H, V, D] and products [places, H, D]. fixed [H] float in place of decay: one constant decay a head.
// act 1: q, k and v are the silu of what the operands hold.
extern "C" int dinfer_gla_recurrence(int dtype, const void* q, const void* k, const void* v, int64_t ld, const float* decay,
                                     int64_t ldd, float q_scale, float* state, float* notes, float* products,
                                     int64_t places, const int32_t* state_slots, const int32_t* cu_seqlens,
                                     const int32_t* seq_lens, float* out, int64_t ld_out, int num_reqs, int64_t tokens,
                                     int64_t max_rows, int cut, int H, int D, int V, const float* fixed, int act,
                                     hipStream_t stream) {
  if (num_reqs <= 0 || max_rows <= 0) return OK;
  if ((decay == nullptr) == (fixed == nullptr) || (act && !fixed)) return ERR_BAD_SHAPE;
  if (H <= 0 || D <= 0 || V <= 0 || num_reqs > 65535 || (decay && ldd < (int64_t)H * D) || ld_out < (int64_t)H * V || tokens > 0x7fffffff)
    return ERR_BAD_SHAPE;
  if (D > 256) return ERR_UNSUPPORTED;
  const int64_t chunks = cut ? (max_rows + CL - 1) / CL : 1;
  if (chunks > 65535) return ERR_UNSUPPORTED;
  if (chunks > 1 && (!notes || !products || places < tokens / CL + num_reqs + 1)) return ERR_WORKSPACE;
  DINFER_DISPATCH_DTYPE(dtype, {
    const size_t es = sizeof(S);
    const bool vec = D % 8 == 0 && ((int64_t)ld * es) % 16 == 0 && ldd % 4 == 0 && ((uintptr_t)q % 16) == 0 &&
                     ((uintptr_t)k % 16) == 0 && ((uintptr_t)decay % 16) == 0;
    Gla<S> p{(const S*)q, (const S*)k, (const S*)v, ld, decay, ldd, q_scale, state, notes, products, state_slots, cu_seqlens,
             seq_lens, out, ld_out, H, D, V, chunks > 1 ? CL : 0x40000000, vec ? 1 : 0, fixed, act};
    const bool wide = chunks > 1;
    if (D <= 32) pick_gla<S, 1>(p, chunks, num_reqs, wide, stream);
    else if (D <= 64) pick_gla<S, 2>(p, chunks, num_reqs, wide, stream);
    else if (D <= 128) pick_gla<S, 4>(p, chunks, num_reqs, wide, stream);
    else pick_gla<S, 8>(p, chunks, num_reqs, wide, stream);
  });
  return launch_status();
}
