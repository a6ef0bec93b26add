// Gated recurrences whose gates read the current token only ("minGRU"): every channel of a request carries one float S,
//
//   a_t = sigmoid(z_t + bz);   u = x_t + bx;   c_t = u + 1/2 where u >= 0, sigmoid(u) where u < 0
//   S <- (1 - a_t) S + a_t c_t;   out_t = S * silu(g_t)
//
// z, x and g come as the step's projections left them, everything after that is float. The step S -> (1 - a) S + a c is
// a linear map, so a portion is cut into chunks of CH tokens that run side by side:
//   min_gru_chunks   a chunk a workgroup: the product of its (1 - a) and what it makes of S = 0 (only where some
//                    portion of the step is longer than a chunk; a portion's last chunk is not needed)
//   min_gru          a chunk a workgroup: folds the chunks before it into its first S, then goes token by token; the
//                    portion's last chunk stores the request's state
// The first kernel's note of chunk 0 already holds the request's state, and a copy of the state itself, so no workgroup
// of the second reads the state another one writes. Chunks are counted from the portion's start. A request whose step
// starts at position 0 starts from S = 0, whatever its slot held.
#include "common.cuh"

using namespace dinfer;

namespace {

constexpr int CH = 32;

__device__ __forceinline__ float sigmoid_f(float x) { return 1.f / (1.f + expf(-x)); }

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

template <class S, int P>
__global__ void __launch_bounds__(256) min_gru_chunks_kernel(Gru p) {
  const int b = blockIdx.z, chunk = blockIdx.y, c = (blockIdx.x * 256 + threadIdx.x) * P;
  const int t0 = p.cu[b], n = p.cu[b + 1] - t0;
  if ((chunk + 1) * CH >= n || c >= p.N) return;      // the portion's last chunk has no followers (and so no note)
  float bz[P], bx[P], m[P], s[P], first[P];
#pragma unroll
  for (int e = 0; e < P; ++e) {
    bz[e] = p.bz[c + e];
    bx[e] = p.bx[c + e];
    m[e] = 1.f;
    s[e] = 0.f;
    first[e] = 0.f;
  }
  const bool has_state = chunk == 0 && p.seq_lens[b] > n;
  if (has_state) {
#pragma unroll
    for (int e = 0; e < P; ++e) first[e] = s[e] = p.state[(int64_t)p.slots[b] * p.N + c + e];
  }
  const S* row = (const S*)p.proj + (int64_t)(t0 + chunk * CH) * p.ld;
#pragma unroll 8
  for (int t = 0; t < CH; ++t) {
    float a[P], ac[P];
    gates<S, P>(p, row + (int64_t)t * p.ld, c, bz, bx, a, ac);
#pragma unroll
    for (int e = 0; e < P; ++e) {
      s[e] = __builtin_fmaf(1.f - a[e], s[e], ac[e]);
      m[e] *= 1.f - a[e];
    }
  }
  float* note = p.notes + place_of(t0, b, chunk) * 2 * p.N + c;
#pragma unroll
  for (int e = 0; e < P; ++e) {
    note[e] = chunk == 0 ? first[e] : m[e];      // (chunk 0: the state it started from)
    note[p.N + e] = s[e];
  }
}

template <class S, int P>
__global__ void __launch_bounds__(256) min_gru_kernel(Gru p, S* __restrict__ out, int64_t ld_out) {
  const int b = blockIdx.z, chunk = blockIdx.y, c = (blockIdx.x * 256 + threadIdx.x) * P;
  const int t0 = p.cu[b], n = p.cu[b + 1] - t0;
  if (chunk * CH >= n || c >= p.N) return;
  float bz[P], bx[P], s[P];
#pragma unroll
  for (int e = 0; e < P; ++e) {
    bz[e] = p.bz[c + e];
    bx[e] = p.bx[c + e];
    s[e] = 0.f;
  }
  if (n <= CH) {
    if (p.seq_lens[b] > n) {
#pragma unroll
      for (int e = 0; e < P; ++e) s[e] = p.state[(int64_t)p.slots[b] * p.N + c + e];
    }
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
  const int first = t0 + chunk * CH, m = n - chunk * CH < CH ? n - chunk * CH : CH;
  auto token = [&](int t) {
    const S* row = (const S*)p.proj + (int64_t)(first + t) * p.ld;
    float a[P], ac[P];
    Lane<S, P> g, o;
    gates<S, P>(p, row, c, bz, bx, a, ac);
    g.load(row + p.g_off + c);
#pragma unroll
    for (int e = 0; e < P; ++e) {
      s[e] = __builtin_fmaf(1.f - a[e], s[e], ac[e]);
      o.v[e] = s[e] * (g.v[e] * sigmoid_f(g.v[e]));
    }
    o.store(out + (int64_t)(first + t) * ld_out + c);
  };
  if (m == CH) {
#pragma unroll 8
    for (int t = 0; t < CH; ++t) token(t);
  } else {
    for (int t = 0; t < m; ++t) token(t);
  }
  if ((chunk + 1) * CH >= n) {
#pragma unroll
    for (int e = 0; e < P; ++e) p.state[(int64_t)p.slots[b] * p.N + c + e] = s[e];
  }
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
  const int per = 256 * (two ? 2 : 1);
  const dim3 grid((unsigned)((N + per - 1) / per), (unsigned)chunks, (unsigned)num_reqs);
  DINFER_DISPATCH_DTYPE(dtype, {
    if (chunks > 1) {
      if (two) min_gru_chunks_kernel<S, 2><<<grid, 256, 0, stream>>>(p);
      else min_gru_chunks_kernel<S, 1><<<grid, 256, 0, stream>>>(p);
    }
    if (two) min_gru_kernel<S, 2><<<grid, 256, 0, stream>>>(p, (S*)out, ld_out);
    else min_gru_kernel<S, 1><<<grid, 256, 0, stream>>>(p, (S*)out, ld_out);
  });
  return launch_status();
}
