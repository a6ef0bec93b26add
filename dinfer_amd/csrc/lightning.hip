// Linear attention with a constant decay a head, over prompt portions on the matrix cores (bf16 operands, float state):
//
//   q, k, v <- silu of the projections (bf16);   per token:  S <- decay S + k v^T,  o_t = S^T q_t      (S [D, V] float)
//
// A portion is walked SUB = 64 tokens at a time. With i, j the places in such a block of n tokens and S what came before it:
//
//   O_i  = decay^(i+1) S^T q_i + sum_{j <= i} decay^(i-j) (q_i . k_j) v_j
//   S    <- decay^n S + sum_j k_j (decay^(n-1-j) v_j)^T
//
// The scores are float sums, weighted in float and rounded once, as operands of the product with the values (the way the
// attention kernels treat their weights). S and the decayed values are operands in two halves, bf16(x) and bf16(x - bf16(x)),
// so the products with them keep 16 bits of every entry and the state does not lose what a rounding would take from it token
// after token.
//
// A workgroup takes a head, 64 columns of S (16 a wave) and a chunk of a portion. v_mfma_f32_16x16x32_bf16: lane l holds row
// (first operand) or column (second) l % 16 and the 8 entries of the contraction of group g = l / 16; of the result, column
// l % 16 and rows 4 g .. + 3. Rows are numbered so that nothing crosses lanes between products:
//   scores   K Q^T: rows of the two key tiles of 32 tokens are numbered so that lane l ends up with the eight scores of keys
//            8 g .. 8 g + 7 against query l % 16: its first operand of the product with the values
//   state    K^T V: the same numbering of the channels, so the sums a lane keeps of two tiles of 16 channels are channels
//            8 g .. 8 g + 7 of column l % 16: its second operand of Q S (no trip through LDS, and 32 contiguous bytes of the
//            stored state, which is [slot][head][V][D])
// LDS holds a block's q and k by token, k and v by channel (the products that contract over tokens want consecutive tokens in
// a lane); a thread brings 4 x 8 (k) or 2 x 8 (v) entries and turns them on the way. The next block's pieces travel in
// registers while a block is multiplied.
//
// Portions too few to fill the chip are cut into chunks of CL tokens that run side by side: a first launch notes what every
// chunk makes of S = 0 (but the portion's last), a scan turns the notes into the S each chunk starts from, and the kernel runs
// over all chunks at once. Steps of single rows (and portions of a few) go through a kernel of their own, token by token: time is
// the time to read and write the states. A request whose step starts at position 0 starts from S = 0, whatever its slot held.
#include "common.cuh"

using namespace dinfer;

namespace {

constexpr int SUB = 64, LDT = SUB + 8;      // tokens of a block; row of the arrays by channel
constexpr int CL = 128;                     // tokens of a chunk (a multiple of SUB)
constexpr int VC = 64;                      // columns of S a workgroup
constexpr float LOG2E = 1.4426950408889634f;

__device__ __forceinline__ f32x4 mfma16(bf16x8 a, bf16x8 b, f32x4 c) {
  return __builtin_amdgcn_mfma_f32_16x16x32_bf16(a, b, c, 0, 0, 0);
}
__device__ __forceinline__ float exp2_of(float x) { return __builtin_amdgcn_exp2f(x); }
__device__ __forceinline__ bf16x8 silu8(bf16x8 x) {
  bf16x8 y;
#pragma unroll
  for (int e = 0; e < 8; ++e) {
    const float z = (float)x[e];
    y[e] = (bf16)(z * __builtin_amdgcn_rcpf(1.f + exp2_of(-LOG2E * z)));
  }
  return y;
}
__device__ __forceinline__ bf16x8 zero8() {
  bf16x8 z;
#pragma unroll
  for (int e = 0; e < 8; ++e) z[e] = (bf16)0.f;
  return z;
}

struct Args {
  const bf16* q; const bf16* k; const bf16* v; int64_t ld;     // heads side by side from these columns of a row
  const float* decay;                                          // [H]
  float* state;                                                // [slots, H, V, D]
  float* notes;                                                // [places, H, V, D]
  const int32_t* slots; const int32_t* cu; const int32_t* seq_lens;
  float* out; int64_t ld_out;
  int H, D, V, cl;
};

// where a chunk's note lies: places of different requests never meet (floor(cu / CL) + request grows by at least the
// request's number of chunks)
__device__ __forceinline__ int64_t place_of(int t0, int b, int chunk) { return (int64_t)(t0 / CL) + b + chunk; }

// KS: steps of 32 channels (D <= 32 KS). OUT: the whole rule; else a chunk's note.
template <int KS, bool OUT>
__global__ void __launch_bounds__(256, KS <= 4 ? 2 : 1) lightning_kernel(Args p) {
  constexpr int DP = 32 * KS, LDK = DP + 8;
  extern __shared__ __attribute__((aligned(16))) bf16 smem[];
  bf16* Kt = smem;                       // [DP][LDT]: k by channel
  bf16* Vt = Kt + DP * LDT;              // [VC][LDT]: v by column
  bf16* Ks = Vt + VC * LDT;              // [SUB][LDK]: k by token   (OUT)
  bf16* Qs = Ks + SUB * LDK;             // [SUB][LDK]: q by token   (OUT)
  const int blocks = (p.V + VC - 1) / VC;
  const int cb = blockIdx.x % blocks, h = blockIdx.x / blocks, chunk = blockIdx.y, b = blockIdx.z;
  const int D = p.D, V = p.V;
  const int r0 = p.cu[b], rows = p.cu[b + 1] - r0;
  const int64_t first = (int64_t)chunk * p.cl;
  if (first >= rows) return;
  const bool last = first + p.cl >= rows, single = rows <= p.cl;
  if (!OUT && last) return;
  const int t0 = r0 + (int)first, count = last ? rows - (int)first : p.cl;
  const int tid = threadIdx.x, wave = tid >> 6, lane = tid & 63, i16 = lane & 15, g = lane >> 4;
  const int64_t matrix = (int64_t)V * D;
  const int64_t place = single ? 0 : place_of(r0, b, chunk);
  const int col = cb * VC + wave * 16 + i16;      // this lane's column of S
  const bool col_ok = col < V;
  const bool wave_on = cb * VC + wave * 16 < V;   // (the others bring pieces and meet the barriers)
  const float l2 = log2f(p.decay[h]);

  // S: channels 32 ks + 8 g + 4 t + r of this lane's column in s[ks][t][r]
  f32x4 s[KS][2];
  {
    const float* init = nullptr;
    if (OUT) {
      if (!single) init = p.notes + (place * p.H + h) * matrix;
      else if (p.seq_lens[b] > rows) init = p.state + ((int64_t)p.slots[b] * p.H + h) * matrix;
    }
#pragma unroll
    for (int ks = 0; ks < KS; ++ks)
#pragma unroll
      for (int t = 0; t < 2; ++t) {
        const int d = 32 * ks + 8 * g + 4 * t;
        s[ks][t] = (init && col_ok && d < D) ? *(const f32x4*)(init + (int64_t)col * D + d) : f32x4{0.f, 0.f, 0.f, 0.f};
      }
  }
  // weights of the scores: decay^(i - j) of query i16 and keys 8 g + e, the query's tile 0, 16 or 32 tokens on
  float w0[8], w16[8], w32[8], up[4];
  const float d16 = exp2_of(16.f * l2);
  if constexpr (OUT) {
#pragma unroll
    for (int e = 0; e < 8; ++e) {
      const int far = i16 - 8 * g - e;
      w0[e] = far >= 0 ? exp2_of(l2 * (float)far) : 0.f;
      w16[e] = far + 16 >= 0 ? exp2_of(l2 * (float)(far + 16)) : 0.f;
      w32[e] = exp2_of(l2 * (float)(far + 32));
    }
#pragma unroll
    for (int r = 0; r < 4; ++r) up[r] = exp2_of(l2 * (float)(4 * g + r + 1));
  }

  // pieces on their way: q 8 entries each, k four tokens of 8 channels, v two tokens of 8 columns
  constexpr int NQ = OUT ? (SUB * DP / 8 + 255) / 256 : 1, NK = (SUB / 4 * DP / 8 + 255) / 256;
  bf16x8 pq[NQ], pk[NK][4], pv[2];
  auto fetch = [&](int ct) {
#pragma unroll
    for (int u = 0; u < NK; ++u) {
      const int idx = u * 256 + tid, quad = idx & 15, d = (idx >> 4) * 8;
#pragma unroll
      for (int e = 0; e < 4; ++e) {
        const int tok = ct + 4 * quad + e;
        pk[u][e] = (d < D && tok < count) ? *(const bf16x8*)(p.k + (int64_t)(t0 + tok) * p.ld + (int64_t)h * D + d) : zero8();
      }
    }
    {
      const int pair = tid & 31, c = cb * VC + (tid >> 5) * 8;
#pragma unroll
      for (int e = 0; e < 2; ++e) {
        const int tok = ct + 2 * pair + e;
        pv[e] = (c < V && tok < count) ? *(const bf16x8*)(p.v + (int64_t)(t0 + tok) * p.ld + (int64_t)h * V + c) : zero8();
      }
    }
    if constexpr (OUT) {
#pragma unroll
      for (int u = 0; u < NQ; ++u) {
        const int idx = u * 256 + tid, row = idx / (DP / 8), d = (idx % (DP / 8)) * 8;
        pq[u] = (row < SUB && d < D && ct + row < count)
                    ? *(const bf16x8*)(p.q + (int64_t)(t0 + ct + row) * p.ld + (int64_t)h * D + d) : zero8();
      }
    }
  };
  auto put = [&]() {
#pragma unroll
    for (int u = 0; u < NK; ++u) {
      const int idx = u * 256 + tid, quad = idx & 15, d = (idx >> 4) * 8;
      if (d < DP) {
        bf16x8 x[4];
#pragma unroll
        for (int e = 0; e < 4; ++e) {
          x[e] = silu8(pk[u][e]);
          if constexpr (OUT) *(bf16x8*)(Ks + (4 * quad + e) * LDK + d) = x[e];
        }
#pragma unroll
        for (int c = 0; c < 8; ++c) {
          bf16x4 y;
#pragma unroll
          for (int e = 0; e < 4; ++e) y[e] = x[e][c];
          *(bf16x4*)(Kt + (d + c) * LDT + 4 * quad) = y;
        }
      }
    }
    {
      const int pair = tid & 31, c0 = (tid >> 5) * 8;
      const bf16x8 x = silu8(pv[0]), y = silu8(pv[1]);
#pragma unroll
      for (int c = 0; c < 8; ++c) {
        bf16x2 z;
        z[0] = x[c];
        z[1] = y[c];
        *(bf16x2*)(Vt + (c0 + c) * LDT + 2 * pair) = z;
      }
    }
    if constexpr (OUT) {
#pragma unroll
      for (int u = 0; u < NQ; ++u) {
        const int idx = u * 256 + tid, row = idx / (DP / 8), d = (idx % (DP / 8)) * 8;
        if (row < SUB) *(bf16x8*)(Qs + row * LDK + d) = silu8(pq[u]);
      }
    }
  };

  const int krow = 8 * (i16 >> 2) + (i16 & 3);     // row of tile t -> entry krow + 4 t of its 32
  fetch(0);
  for (int ct = 0; ct < count; ct += SUB) {
    __syncthreads();      // the block before has been read
    put();
    __syncthreads();
    if (ct + SUB < count) fetch(ct + SUB);
    if (!wave_on) continue;
    const int n = count - ct < SUB ? count - ct : SUB;
    bf16x8 vf[2];
#pragma unroll
    for (int u = 0; u < 2; ++u) vf[u] = *(const bf16x8*)(Vt + (wave * 16 + i16) * LDT + 32 * u + 8 * g);

    if constexpr (OUT) {
      f32x4 o[4];
      // what came before the block: Q S in two halves of S
#pragma unroll
      for (int it = 0; it < 4; ++it) o[it] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int ks = 0; ks < KS; ++ks) {
        bf16x8 hi, lo;
#pragma unroll
        for (int e = 0; e < 8; ++e) {
          const float x = s[ks][e >> 2][e & 3];
          hi[e] = (bf16)x;
          lo[e] = (bf16)(x - (float)hi[e]);
        }
#pragma unroll
        for (int it = 0; it < 4; ++it)
          if (16 * it < n) {
            const bf16x8 qf = *(const bf16x8*)(Qs + (16 * it + i16) * LDK + 32 * ks + 8 * g);
            o[it] = mfma16(qf, hi, o[it]);
            o[it] = mfma16(qf, lo, o[it]);
          }
      }
      float step = 1.f;
#pragma unroll
      for (int it = 0; it < 4; ++it) {
#pragma unroll
        for (int r = 0; r < 4; ++r) o[it][r] *= up[r] * step;
        step *= d16;
      }
      // the block's own tokens, 32 keys at a time
#pragma unroll
      for (int jb = 0; jb < 2; ++jb) {
        if (32 * jb < n) {
          f32x4 sc[4][2];
#pragma unroll
          for (int it = 2 * jb; it < 4; ++it) sc[it][0] = sc[it][1] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
          for (int ks = 0; ks < KS; ++ks) {
            bf16x8 kf[2];
#pragma unroll
            for (int t = 0; t < 2; ++t) kf[t] = *(const bf16x8*)(Ks + (32 * jb + krow + 4 * t) * LDK + 32 * ks + 8 * g);
#pragma unroll
            for (int it = 2 * jb; it < 4; ++it)
              if (16 * it < n) {
                const bf16x8 qf = *(const bf16x8*)(Qs + (16 * it + i16) * LDK + 32 * ks + 8 * g);
#pragma unroll
                for (int t = 0; t < 2; ++t) sc[it][t] = mfma16(kf[t], qf, sc[it][t]);
              }
          }
#pragma unroll
          for (int it = 2 * jb; it < 4; ++it)
            if (16 * it < n) {
              const int on = it - 2 * jb;      // how many tiles of 16 the queries lie behind the first key
              bf16x8 pf;
#pragma unroll
              for (int e = 0; e < 8; ++e) {
                const float w = on == 0 ? w0[e] : on == 1 ? w16[e] : on == 2 ? w32[e] : w32[e] * d16;
                pf[e] = (bf16)(sc[it][e >> 2][e & 3] * w);
              }
              o[it] = mfma16(pf, vf[jb], o[it]);
            }
        }
      }
#pragma unroll
      for (int it = 0; it < 4; ++it)
#pragma unroll
        for (int r = 0; r < 4; ++r) {
          const int i = 16 * it + 4 * g + r;
          if (i < n && col_ok) p.out[(int64_t)(t0 + ct + i) * p.ld_out + (int64_t)h * V + col] = o[it][r];
        }
    }
    // the state behind the block
    const float keep = exp2_of(l2 * (float)n);
#pragma unroll
    for (int ks = 0; ks < KS; ++ks)
#pragma unroll
      for (int t = 0; t < 2; ++t) s[ks][t] *= keep;
#pragma unroll
    for (int u = 0; u < 2; ++u) {
      if (32 * u < n) {
        bf16x8 hi, lo;
#pragma unroll
        for (int e = 0; e < 8; ++e) {
          const int left = n - 1 - (32 * u + 8 * g + e);     // (tokens beyond the block's end are zeros)
          const float x = (float)vf[u][e] * exp2_of(l2 * (float)(left > 0 ? left : 0));
          hi[e] = (bf16)x;
          lo[e] = (bf16)(x - (float)hi[e]);
        }
#pragma unroll
        for (int ks = 0; ks < KS; ++ks)
#pragma unroll
          for (int t = 0; t < 2; ++t) {
            const bf16x8 kf = *(const bf16x8*)(Kt + (32 * ks + krow + 4 * t) * LDT + 32 * u + 8 * g);
            s[ks][t] = mfma16(kf, hi, s[ks][t]);
            s[ks][t] = mfma16(kf, lo, s[ks][t]);
          }
      }
    }
  }
  if ((OUT && !last) || !col_ok) return;
  float* to = (OUT ? p.state + ((int64_t)p.slots[b] * p.H + h) * matrix : p.notes + (place * p.H + h) * matrix) + (int64_t)col * D;
#pragma unroll
  for (int ks = 0; ks < KS; ++ks)
#pragma unroll
    for (int t = 0; t < 2; ++t) {
      const int d = 32 * ks + 8 * g + 4 * t;
      if (d < D) *(f32x4*)(to + d) = s[ks][t];
    }
}

// Four entries of S by themselves: the notes of a request's chunks, in order, become the S each chunk starts from.
__global__ void __launch_bounds__(256) lightning_scan_kernel(Args p) {
  const int b = blockIdx.z;
  const int r0 = p.cu[b], rows = p.cu[b + 1] - r0;
  if (rows <= p.cl) return;
  const int chunks = (rows + p.cl - 1) / p.cl;
  const int64_t per = (int64_t)p.H * p.V * p.D;
  const int64_t i = ((int64_t)blockIdx.x * 256 + threadIdx.x) * 4;
  if (i >= per) return;
  const int h = (int)(i / ((int64_t)p.V * p.D));
  const float a = exp2_of(log2f(p.decay[h]) * (float)p.cl);
  f32x4 s = {0.f, 0.f, 0.f, 0.f};
  if (p.seq_lens[b] > rows) s = *(const f32x4*)(p.state + (int64_t)p.slots[b] * per + i);
  float* note = p.notes + place_of(r0, b, 0) * per + i;
  int c = 0;
  for (; c + 4 < chunks; c += 4) {      // (the last chunk has no note of its own)
    f32x4 n[4];
#pragma unroll
    for (int u = 0; u < 4; ++u) n[u] = *(const f32x4*)(note + (int64_t)(c + u) * per);
#pragma unroll
    for (int u = 0; u < 4; ++u) {
      *(f32x4*)(note + (int64_t)(c + u) * per) = s;
      s = a * s + n[u];
    }
  }
  for (; c < chunks; ++c) {
    f32x4 n = {0.f, 0.f, 0.f, 0.f};
    if (c + 1 < chunks) n = *(const f32x4*)(note + (int64_t)c * per);
    *(f32x4*)(note + (int64_t)c * per) = s;
    s = a * s + n;
  }
}

// Portions of a few rows. LPC lanes share a column of S, 4 channels each (D <= 4 LPC, a multiple of 4), and own COLS columns,
// whose strips they read at once, keep through the portion's tokens and write back.
constexpr int COLS = 4;

__device__ __forceinline__ float silu_exact(float z) { return z / (1.f + expf(-z)); }

// A lane's value plus that of the lane a DPP pattern pairs it with (full-rate vector instructions, no LDS).
template <int CTRL>
__device__ __forceinline__ float dpp_add(float v) {
  return v + __builtin_bit_cast(float, __builtin_amdgcn_update_dpp(0, __builtin_bit_cast(int, v), CTRL, 0xf, 0xf, true));
}
// The sum over LPC lanes, in every lane of them.
template <int LPC>
__device__ __forceinline__ float lanes_sum(float v) {
  v = dpp_add<0xB1>(v);                            // quad_perm [1, 0, 3, 2]
  v = dpp_add<0x4E>(v);                            // quad_perm [2, 3, 0, 1]
  v = dpp_add<0x141>(v);                           // row_half_mirror
  if constexpr (LPC >= 16) v = dpp_add<0x140>(v);  // row_mirror
  if constexpr (LPC >= 32) v += __shfl_xor(v, 16, WAVE);
  if constexpr (LPC >= 64) v += __shfl_xor(v, 32, WAVE);
  return v;
}

template <class O>
struct Few {
  const O* q; const O* k; const O* v; int64_t ld;
  const float* decay; float* state;
  const int32_t* slots; const int32_t* cu; const int32_t* seq_lens;
  float* out; int64_t ld_out;
  int H, D, V;
};

template <class O, int LPC>
__global__ void __launch_bounds__(256) lightning_few_kernel(Few<O> p) {
  constexpr int TEAMS = 256 / LPC;                 // teams of LPC lanes; team t owns columns t, t + TEAMS, ...
  const int blocks = (p.V + TEAMS * COLS - 1) / (TEAMS * COLS);
  const int cb = blockIdx.x % blocks, h = blockIdx.x / blocks, b = blockIdx.y;
  const int D = p.D, V = p.V;
  const int t0 = p.cu[b], n = p.cu[b + 1] - t0;
  if (n <= 0) return;
  const int lane = threadIdx.x % LPC, team = threadIdx.x / LPC;
  const int d = 4 * lane, c0 = cb * TEAMS * COLS + team;
  const bool on = d < D;
  const float a = p.decay[h];
  float* st = p.state + ((int64_t)p.slots[b] * p.H + h) * V * D + (on ? d : 0);
  f32x4 s[COLS];
  const bool from_state = p.seq_lens[b] > n;
#pragma unroll
  for (int c = 0; c < COLS; ++c) {
    const int col = c0 + c * TEAMS;
    s[c] = from_state && on && col < V ? *(const f32x4*)(st + (int64_t)col * D) : f32x4{0.f, 0.f, 0.f, 0.f};
  }
  for (int t = t0; t < t0 + n; ++t) {
    float q[4], k[4], v[COLS];
#pragma unroll
    for (int e = 0; e < 4; ++e) {
      q[e] = on ? silu_exact(to_f32(p.q[(int64_t)t * p.ld + (int64_t)h * D + d + e])) : 0.f;
      k[e] = on ? silu_exact(to_f32(p.k[(int64_t)t * p.ld + (int64_t)h * D + d + e])) : 0.f;
    }
#pragma unroll
    for (int c = 0; c < COLS; ++c) {
      const int col = c0 + c * TEAMS;
      v[c] = col < V ? silu_exact(to_f32(p.v[(int64_t)t * p.ld + (int64_t)h * V + col])) : 0.f;
    }
    float o[COLS];
#pragma unroll
    for (int c = 0; c < COLS; ++c) {
      o[c] = 0.f;
#pragma unroll
      for (int e = 0; e < 4; ++e) {
        s[c][e] = __builtin_fmaf(k[e], v[c], a * s[c][e]);
        o[c] = __builtin_fmaf(s[c][e], q[e], o[c]);
      }
    }
#pragma unroll
    for (int c = 0; c < COLS; ++c) o[c] = lanes_sum<LPC>(o[c]);
    if (lane < COLS) {
      const int col = c0 + lane * TEAMS;
      const float y = lane == 0 ? o[0] : lane == 1 ? o[1] : lane == 2 ? o[2] : o[3];
      if (col < V) p.out[(int64_t)t * p.ld_out + (int64_t)h * V + col] = y;
    }
  }
#pragma unroll
  for (int c = 0; c < COLS; ++c) {
    const int col = c0 + c * TEAMS;
    if (on && col < V) *(f32x4*)(st + (int64_t)col * D) = s[c];
  }
}

template <class O, int LPC>
void launch_few(const Few<O>& p, int num_reqs, hipStream_t stream) {
  constexpr int per = 256 / LPC * COLS;
  lightning_few_kernel<O, LPC><<<dim3((unsigned)((p.V + per - 1) / per * p.H), (unsigned)num_reqs), 256, 0, stream>>>(p);
}

template <int KS>
int launch(const Args& p, int64_t chunks, int num_reqs, hipStream_t stream) {
  constexpr int DP = 32 * KS;
  constexpr size_t by_channel = (size_t)(DP + VC) * LDT * sizeof(bf16), by_token = (size_t)2 * SUB * (DP + 8) * sizeof(bf16);
  static bool sized = false;
  if (!sized) {      // (more than the 64 KB of LDS a launch may ask for without saying so)
    if (hipFuncSetAttribute((const void*)lightning_kernel<KS, true>, hipFuncAttributeMaxDynamicSharedMemorySize,
                            (int)(by_channel + by_token)) != hipSuccess)
      return ERR_LAUNCH;
    sized = true;
  }
  const dim3 grid((unsigned)((p.V + VC - 1) / VC * p.H), (unsigned)chunks, (unsigned)num_reqs);
  if (chunks > 1) {
    lightning_kernel<KS, false><<<grid, 256, by_channel, stream>>>(p);
    const int64_t quads = (int64_t)p.H * p.V * p.D / 4;
    lightning_scan_kernel<<<dim3((unsigned)((quads + 255) / 256), 1, (unsigned)num_reqs), 256, 0, stream>>>(p);
  }
  lightning_kernel<KS, true><<<grid, 256, by_channel + by_token, stream>>>(p);
  return launch_status();
}

}  // namespace

// Tokens of a chunk. A step that is cut into chunks needs tokens / chunk + requests + 1 notes of H V D floats.
extern "C" int dinfer_lightning_chunk() { return CL; }

// Whether the kernel takes these sizes (bf16 operands; ld: their row stride).
extern "C" int dinfer_lightning_supports(int D, int V, int64_t ld) {
  return D > 0 && D <= 256 && D % 8 == 0 && V > 0 && V % 8 == 0 && ld % 8 == 0 ? 1 : 0;
}

// Whether a step with this many tokens, requests and rows in its longest portion is cut into chunks: where the work of the
// portions side by side would leave most of the chip idle while the longest runs.
extern "C" int dinfer_lightning_cuts(int64_t tokens, int64_t max_rows, int num_reqs, int H, int V) {
  if (max_rows <= CL || num_reqs <= 0) return 0;
  const double at_once = (double)tokens / (double)max_rows * H * ((V + VC - 1) / VC);     // workgroups busy on average
  return at_once < 512. ? 1 : 0;
}

// q, k [T, H D], v [T, H V]: bf16 columns of rows of stride ld; decay [H] float in (0, 1]; state [slots, H, V, D] float; out
// [T, ld_out] float, head h at column h V. cut: the step runs in chunks, with notes [places, H, V, D].
extern "C" int dinfer_lightning(const void* q, const void* k, const void* v, int64_t ld, const float* decay, float* state,
                                float* notes, int64_t places, const int32_t* state_slots, const int32_t* cu_seqlens,
                                const int32_t* seq_lens, float* out, int64_t ld_out, int num_reqs, int64_t tokens,
                                int64_t max_rows, int cut, int H, int D, int V, hipStream_t stream) {
  if (num_reqs <= 0 || max_rows <= 0) return OK;
  if (H <= 0 || num_reqs > 65535 || ld_out < (int64_t)H * V || tokens > 0x7fffffff || ((uintptr_t)q % 16) ||
      ((uintptr_t)k % 16) || ((uintptr_t)v % 16) || ((uintptr_t)state % 16) || ((uintptr_t)notes % 16))
    return ERR_BAD_SHAPE;
  if (!dinfer_lightning_supports(D, V, ld)) return ERR_UNSUPPORTED;
  const int64_t chunks = cut ? (max_rows + CL - 1) / CL : 1;
  if (chunks > 65535) return ERR_UNSUPPORTED;
  if (chunks > 1 && (!notes || places < tokens / CL + num_reqs + 1)) return ERR_WORKSPACE;
  const Args p{(const bf16*)q, (const bf16*)k, (const bf16*)v, ld, decay, state, notes, state_slots, cu_seqlens, seq_lens, out,
               ld_out, H, D, V, chunks > 1 ? CL : 0x40000000};
  if (D <= 32) return launch<1>(p, chunks, num_reqs, stream);
  if (D <= 64) return launch<2>(p, chunks, num_reqs, stream);
  if (D <= 96) return launch<3>(p, chunks, num_reqs, stream);
  if (D <= 128) return launch<4>(p, chunks, num_reqs, stream);
  return launch<8>(p, chunks, num_reqs, stream);
}

// The same rule token by token, for portions of a few rows: q, k, v in the step's dtype, D a multiple of 4 up to 256.
extern "C" int dinfer_lightning_few(int dtype, const void* q, const void* k, const void* v, int64_t ld, const float* decay,
                                    float* state, const int32_t* state_slots, const int32_t* cu_seqlens, const int32_t* seq_lens,
                                    float* out, int64_t ld_out, int num_reqs, int H, int D, int V, hipStream_t stream) {
  if (num_reqs <= 0) return OK;
  if (H <= 0 || D <= 0 || V <= 0 || num_reqs > 65535 || ld_out < (int64_t)H * V || ((uintptr_t)state % 16)) return ERR_BAD_SHAPE;
  if (D > 256 || D % 4) return ERR_UNSUPPORTED;
  DINFER_DISPATCH_DTYPE(dtype, {
    const Few<S> p{(const S*)q, (const S*)k, (const S*)v, ld, decay, state, state_slots, cu_seqlens, seq_lens, out, ld_out, H, D, V};
    if (D <= 32) launch_few<S, 8>(p, num_reqs, stream);
    else if (D <= 64) launch_few<S, 16>(p, num_reqs, stream);
    else if (D <= 128) launch_few<S, 32>(p, num_reqs, stream);
    else launch_few<S, 64>(p, num_reqs, stream);
  });
  return launch_status();
}
