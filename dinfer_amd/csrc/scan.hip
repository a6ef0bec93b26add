// Gated recurrences whose gates read the current token only ("minGRU"): every channel of a request carries one float S,
//
//   a_t = sigmoid(z_t + bz);   u = x_t + bx;   c_t = u + 1/2 where u >= 0, sigmoid(u) where u < 0
//   S <- (1 - a_t) S + a_t c_t;   out_t = S * silu(g_t)
//
// z, x and g come as the step's projections left them, everything after that is float. The step S -> (1 - a) S + a c is
// a linear map, so a portion is cut into chunks of CH tokens that run side by side, and a chunk into runs of WT tokens,
// one a wave of the workgroup that takes it, which meet in LDS:
//   min_gru_chunks   a chunk's map, the product of its (1 - a) and what it makes of S = 0 (only where some portion of the
//                    step is longer than a chunk; a portion's last chunk is not needed)
//   min_gru          folds the chunks before it, then the waves before, into a wave's first S, then goes token by token on
//                    gates that wait in registers; the wave of the portion's last token stores the request's state
// The first kernel's note of chunk 0 already holds the request's state, and a copy of the state itself, so no workgroup
// of the second reads the state another one writes. Chunks are counted from the portion's start. A request whose step
// starts at position 0 starts from S = 0, whatever its slot held.
#include "common.cuh"

using namespace dinfer;

namespace {

constexpr int WT = 8;           // tokens a wave goes through
constexpr int WAVES = 8;        // waves of a workgroup
constexpr int FEW = 4;          // portions up to this long take no chunks at all
constexpr int CH = WAVES * WT;  // tokens of a chunk: the waves of a workgroup, one after the other in time

// 1 / (1 + e^-x) by the hardware's exponential and reciprocal (a unit in the last place each)
__device__ __forceinline__ float sigmoid_f(float x) {
  return __builtin_amdgcn_rcpf(1.f + __builtin_amdgcn_exp2f(-1.4426950408889634f * x));
}

template <class S, int P>
struct Lane {      // P consecutive channels
  float v[P];
  __device__ __forceinline__ void load(const S* p) {
    if constexpr (P == 1) {
      v[0] = to_f32(p[0]);
    } else if constexpr (sizeof(S) == 2) {
      const bf16x2 t = *(const bf16x2*)p;
      v[0] = (float)t[0];
      v[1] = (float)t[1];
    } else {
      const f32x2 t = *(const f32x2*)p;
      v[0] = t[0];
      v[1] = t[1];
    }
  }
  __device__ __forceinline__ void store(S* p) const {
    if constexpr (P == 1) {
      p[0] = from_f32<S>(v[0]);
    } else if constexpr (sizeof(S) == 2) {
      bf16x2 t;
      t[0] = (bf16)v[0];
      t[1] = (bf16)v[1];
      *(bf16x2*)p = t;
    } else {
      f32x2 t = {v[0], v[1]};
      *(f32x2*)p = t;
    }
  }
};

struct Gru {
  const void* proj; int64_t ld, z_off, x_off, g_off;
  const float* bz; const float* bx;      // [N]
  float* state;                          // [slots, N]
  float* notes;                          // [places, 2, N]: a chunk's product of (1 - a), then its S from zero
  const int32_t* slots; const int32_t* cu; const int32_t* seq_lens;
  int N;
};

// where a chunk's note lies: places of different requests never meet (floor(cu / CH) + request grows by at least the
// request's number of chunks)
__device__ __forceinline__ int64_t place_of(int t0, int b, int chunk) { return (int64_t)(t0 / CH) + b + chunk; }

template <class S, int P>
__device__ __forceinline__ void gates(const Gru& p, const S* row, int c, const float (&bz)[P], const float (&bx)[P],
                                      float (&a)[P], float (&ac)[P]) {
  Lane<S, P> z, x;
  z.load(row + p.z_off + c);
  x.load(row + p.x_off + c);
#pragma unroll
  for (int e = 0; e < P; ++e) {
    a[e] = sigmoid_f(z.v[e] + bz[e]);
    const float u = x.v[e] + bx[e];
    ac[e] = a[e] * (u >= 0.f ? u + 0.5f : sigmoid_f(u));
  }
}

// A wave's tokens of a chunk: their gates go through every lane's registers at once, then the map they make of S,
// S -> m S + s. FULL: all WT of them; else the first n (the row `first` exists
// whatever n is), and the others change nothing (a = 0).
template <class S, int P, bool FULL>
__device__ __forceinline__ void wave_tokens(const Gru& p, int64_t first, int n, int c, const float (&bz)[P], const float (&bx)[P],
                                            float (&a)[WT][P], float (&ac)[WT][P], float (&m)[P], float (&s)[P]) {
  const S* row = (const S*)p.proj + first * p.ld;
#pragma unroll
  for (int t = 0; t < WT; ++t) {
    gates<S, P>(p, row + (FULL || t < n ? (int64_t)t * p.ld : 0), c, bz, bx, a[t], ac[t]);
    if (!FULL) {
#pragma unroll
      for (int e = 0; e < P; ++e) {
        a[t][e] = t < n ? a[t][e] : 0.f;
        ac[t][e] = t < n ? ac[t][e] : 0.f;
      }
    }
  }
#pragma unroll
  for (int e = 0; e < P; ++e) {
    m[e] = 1.f;
    s[e] = 0.f;
  }
#pragma unroll
  for (int t = 0; t < WT; ++t)
#pragma unroll
    for (int e = 0; e < P; ++e) {
      s[e] = __builtin_fmaf(1.f - a[t][e], s[e], ac[t][e]);
      m[e] *= 1.f - a[t][e];
    }
}

// A workgroup: 64 P channels and the CH tokens of a chunk, a wave WT of them.
template <class S, int P>
__global__ void __launch_bounds__(64 * WAVES) min_gru_chunks_kernel(Gru p) {
  __shared__ float ms[WAVES][2][64 * P];
  const int wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6), lane = threadIdx.x & 63;
  const int b = blockIdx.z, chunk = blockIdx.y, c = (blockIdx.x * 64 + lane) * P;
  const int t0 = p.cu[b], n = p.cu[b + 1] - t0;
  if ((chunk + 1) * CH >= n) return;      // the portion's last chunk has no followers (and so no note)
  const bool live = c < p.N;
  float bz[P], bx[P], m[P], s[P], a[WT][P], ac[WT][P];
  if (live) {
#pragma unroll
    for (int e = 0; e < P; ++e) {
      bz[e] = p.bz[c + e];
      bx[e] = p.bx[c + e];
    }
    wave_tokens<S, P, true>(p, t0 + chunk * CH + wave * WT, WT, c, bz, bx, a, ac, m, s);
#pragma unroll
    for (int e = 0; e < P; ++e) {
      ms[wave][0][lane * P + e] = m[e];
      ms[wave][1][lane * P + e] = s[e];
    }
  }
  __syncthreads();
  if (wave > 0 || !live) return;
  const bool has_state = chunk == 0 && p.seq_lens[b] > n;
  float* note = p.notes + place_of(t0, b, chunk) * 2 * p.N + c;
#pragma unroll
  for (int e = 0; e < P; ++e) {
    const float first = has_state ? p.state[(int64_t)p.slots[b] * p.N + c + e] : 0.f;
    float S0 = first, M = 1.f;
#pragma unroll
    for (int w = 0; w < WAVES; ++w) {
      S0 = __builtin_fmaf(ms[w][0][lane * P + e], S0, ms[w][1][lane * P + e]);
      M *= ms[w][0][lane * P + e];
    }
    note[e] = chunk == 0 ? first : M;      // (chunk 0: the state it started from)
    note[p.N + e] = S0;
  }
}

// One wave's part of min_gru; every wave of the workgroup comes here (there is a barrier inside).
template <class S, int P, bool FULL>
__device__ __forceinline__ void min_gru_wave(const Gru& p, S* __restrict__ out, int64_t ld_out, float (*ms)[2][64 * P], int b,
                                             int chunk, int t0, int n, int wave, int left) {
  const int lane = threadIdx.x & 63, c0 = (blockIdx.x * 64 + lane) * P;
  const bool live = c0 < p.N;
  const int c = live ? c0 : p.N - P;      // lanes past the last channel work on it too and store nothing
  const int64_t first = t0 + chunk * CH + wave * WT;
  float s[P], a[WT][P], ac[WT][P], g[WT][P], bz[P], bx[P], m[P], sw[P];
#pragma unroll
  for (int e = 0; e < P; ++e) {
    bz[e] = p.bz[c + e];
    bx[e] = p.bx[c + e];
  }
#pragma unroll
  for (int t = 0; t < WT; ++t) {
    Lane<S, P> x;
#pragma unroll
    for (int e = 0; e < P; ++e) x.v[e] = 0.f;
    if (FULL || t < left) x.load((const S*)p.proj + (first + t) * p.ld + p.g_off + c);
#pragma unroll
    for (int e = 0; e < P; ++e) g[t][e] = x.v[e];
  }
  wave_tokens<S, P, FULL>(p, left > 0 ? first : t0, left, c, bz, bx, a, ac, m, sw);
#pragma unroll
  for (int e = 0; e < P; ++e) {
    ms[wave][0][lane * P + e] = m[e];
    ms[wave][1][lane * P + e] = sw[e];
  }
  // the S the chunk starts from: the request's state, or what the chunks before make of it
  if (n <= CH) {
    const bool has_state = p.seq_lens[b] > n;
#pragma unroll
    for (int e = 0; e < P; ++e) s[e] = has_state ? p.state[(int64_t)p.slots[b] * p.N + c + e] : 0.f;
  } else {
    const float* note = p.notes + place_of(t0, b, 0) * 2 * p.N + c;
#pragma unroll
    for (int e = 0; e < P; ++e) s[e] = chunk == 0 ? note[e] : note[p.N + e];
#pragma unroll 8
    for (int j = 1; j < chunk; ++j) {
      const float* nj = note + (int64_t)j * 2 * p.N;
#pragma unroll
      for (int e = 0; e < P; ++e) s[e] = __builtin_fmaf(nj[e], s[e], nj[p.N + e]);
    }
  }
  __syncthreads();
  if (!live) return;
#pragma unroll
  for (int w = 0; w < WAVES - 1; ++w)
    if (w < wave) {
#pragma unroll
      for (int e = 0; e < P; ++e) s[e] = __builtin_fmaf(ms[w][0][lane * P + e], s[e], ms[w][1][lane * P + e]);
    }
#pragma unroll
  for (int t = 0; t < WT; ++t)
    if (FULL || t < left) {
      Lane<S, P> o;
#pragma unroll
      for (int e = 0; e < P; ++e) {
        s[e] = __builtin_fmaf(1.f - a[t][e], s[e], ac[t][e]);
        o.v[e] = s[e] * (g[t][e] * sigmoid_f(g[t][e]));
      }
      o.store(out + (first + t) * ld_out + c);
    }
  if (left > 0 && left <= WT && (chunk + 1) * CH >= n) {      // the wave with the portion's last token
#pragma unroll
    for (int e = 0; e < P; ++e) p.state[(int64_t)p.slots[b] * p.N + c + e] = s[e];
  }
}

template <class S, int P>
__global__ void __launch_bounds__(64 * WAVES) min_gru_kernel(Gru p, S* __restrict__ out, int64_t ld_out) {
  __shared__ float ms[WAVES][2][64 * P];
  const int wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6);
  const int b = blockIdx.z, chunk = blockIdx.y;
  const int t0 = p.cu[b], n = p.cu[b + 1] - t0;
  if (chunk * CH >= n) return;
  const int left = n - chunk * CH - wave * WT;      // tokens from this wave's first on (0 or less: it has none)
  if (n - chunk * CH >= CH) min_gru_wave<S, P, true>(p, out, ld_out, ms, b, chunk, t0, n, wave, left);
  else min_gru_wave<S, P, false>(p, out, ld_out, ms, b, chunk, t0, n, wave, left);
}

// Steps of single rows and portions of a few: a thread P channels of a request, token by token.
template <class S, int P>
__global__ void __launch_bounds__(64) min_gru_few_kernel(Gru p, S* __restrict__ out, int64_t ld_out) {
  const int b = blockIdx.y, c = (blockIdx.x * 64 + threadIdx.x) * P;
  if (c >= p.N) return;
  const int t0 = p.cu[b], n = p.cu[b + 1] - t0;
  const bool has_state = p.seq_lens[b] > n;
  float* state = p.state + (int64_t)p.slots[b] * p.N + c;
  float bz[P], bx[P], s[P];
#pragma unroll
  for (int e = 0; e < P; ++e) {
    bz[e] = p.bz[c + e];
    bx[e] = p.bx[c + e];
    s[e] = has_state ? state[e] : 0.f;
  }
  for (int t = 0; t < n; ++t) {
    const S* row = (const S*)p.proj + (int64_t)(t0 + t) * p.ld;
    float a[P], ac[P];
    Lane<S, P> g, o;
    g.load(row + p.g_off + c);
    gates<S, P>(p, row, c, bz, bx, a, ac);
#pragma unroll
    for (int e = 0; e < P; ++e) {
      s[e] = __builtin_fmaf(1.f - a[e], s[e], ac[e]);
      o.v[e] = s[e] * (g.v[e] * sigmoid_f(g.v[e]));
    }
    o.store(out + (int64_t)(t0 + t) * ld_out + c);
  }
#pragma unroll
  for (int e = 0; e < P; ++e) state[e] = s[e];
}

}  // namespace

// Rows of `notes` a step may need: tokens of the step / CH + requests + 1, each of 2 N floats.
extern "C" int dinfer_min_gru_chunk() { return CH; }

// proj [T, ld] in the step's dtype: N update-gate columns from z_off, N input columns from x_off, N output-gate columns
// from g_off; bz, bx [N] float. state [slots, N] float. out [T, ld_out] in the step's dtype. max_rows: the longest portion
// of the step. notes: float scratch of note_places * 2 N.
extern "C" int dinfer_min_gru(int dtype, const void* proj, int64_t ld, int64_t z_off, int64_t x_off, int64_t g_off,
                              const float* bz, const float* bx, float* state, float* notes, int64_t note_places,
                              const int32_t* state_slots, const int32_t* cu_seqlens, const int32_t* seq_lens, void* out,
                              int64_t ld_out, int num_reqs, int64_t tokens, int64_t max_rows, int64_t N,
                              hipStream_t stream) {
  if (num_reqs <= 0 || max_rows <= 0) return OK;
  if (N <= 0 || ld_out < N || num_reqs > 65535 || N > 0x3fffffff || tokens > 0x7fffffff)
    return ERR_BAD_SHAPE;
  const int64_t chunks = (max_rows + CH - 1) / CH;
  if (chunks > 65535) return ERR_UNSUPPORTED;
  if (chunks > 1 && (!notes || note_places < tokens / CH + num_reqs + 1)) return ERR_WORKSPACE;
  Gru p{proj, ld, z_off, x_off, g_off, bz, bx, state, notes, state_slots, cu_seqlens, seq_lens, (int)N};
  const int es = dtype == DT_F32 ? 4 : 2;
  const bool two = N % 2 == 0 && ld % 2 == 0 && z_off % 2 == 0 && x_off % 2 == 0 && g_off % 2 == 0 && ld_out % 2 == 0 &&
                   ((uintptr_t)proj % (2 * es)) == 0 && ((uintptr_t)out % (2 * es)) == 0;
  const int per = 64 * (two ? 2 : 1);
  const dim3 grid((unsigned)((N + per - 1) / per), (unsigned)chunks, (unsigned)num_reqs);
  DINFER_DISPATCH_DTYPE(dtype, {
    if (max_rows <= FEW) {
      const dim3 few((unsigned)((N + per - 1) / per), (unsigned)num_reqs);
      if (two) min_gru_few_kernel<S, 2><<<few, 64, 0, stream>>>(p, (S*)out, ld_out);
      else min_gru_few_kernel<S, 1><<<few, 64, 0, stream>>>(p, (S*)out, ld_out);
      return launch_status();
    }
    if (chunks > 1) {
      if (two) min_gru_chunks_kernel<S, 2><<<grid, 64 * WAVES, 0, stream>>>(p);
      else min_gru_chunks_kernel<S, 1><<<grid, 64 * WAVES, 0, stream>>>(p);
    }
    if (two) min_gru_kernel<S, 2><<<grid, 64 * WAVES, 0, stream>>>(p, (S*)out, ld_out);
    else min_gru_kernel<S, 1><<<grid, 64 * WAVES, 0, stream>>>(p, (S*)out, ld_out);
  });
  return launch_status();
}
