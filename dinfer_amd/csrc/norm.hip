// RMSNorm over the last dimension, one workgroup per row, with three optional
// fusions that each save one pass over the activations:
//   * residual add:  r = round(x + r) is written back, then the norm is taken
//     of the rounded r (the value the next layer will also read);
//   * row gather:    only the listed rows of x are normed (final norm before
//     the LM head);
//   * weight offset: y = x * inv * (w + offset), offset 0 for plain gains and
//     1 for gains stored around zero.
// ss, inv and all products are float; one rounding on store.
//
// Reference behaviour: crates/kernels/cuda/norm.cu:41-116,192-221 and
// rmsnorm_core.cuh:63-81 (inv = 1/sqrt(ss/n + eps), weight multiplies
// directly), norm.cu:69-85 (the add is rounded before it is normed).
#include "common.cuh"

using namespace dinfer;

namespace {

template <class S>
__global__ void __launch_bounds__(256) rmsnorm_kernel(const S* __restrict__ x, S* __restrict__ residual,
                                                      const int32_t* __restrict__ rows, const void* __restrict__ w,
                                                      int wf32, S* __restrict__ out, int64_t width, int64_t ld_x,
                                                      int64_t ld_res, float eps, float w_offset) {
  __shared__ float red[16];
  const int64_t r = blockIdx.x;
  const int64_t src = rows ? (int64_t)rows[r] : r;
  const S* xr = x + src * ld_x;
  S* rr = residual ? residual + src * ld_res : nullptr;
  S* o = out + r * width;
  float ss = 0.f;
  for (int64_t i = threadIdx.x; i < width; i += blockDim.x) {
    float v = to_f32(xr[i]);
    if (rr) {
      const S s = from_f32<S>(v + to_f32(rr[i]));
      rr[i] = s;
      v = to_f32(s);
    }
    ss += v * v;
  }
  ss = block_sum(ss, red);
  const float inv = 1.f / sqrtf(ss / (float)width + eps);
  const S* src2 = rr ? rr : xr;  // each thread re-reads only what it wrote itself
  for (int64_t i = threadIdx.x; i < width; i += blockDim.x)
    o[i] = from_f32<S>(to_f32(src2[i]) * inv * (ld_param<S>(w, i, wf32) + w_offset));
}

// bf16 rows whose width is a multiple of 8 and at most 256*8*ITERS: each
// thread keeps its 8-element pieces in registers between the two phases.
template <int ITERS>
__global__ void __launch_bounds__(256) rmsnorm_bf16x8_kernel(const bf16* __restrict__ x, bf16* __restrict__ residual,
                                                             const int32_t* __restrict__ rows,
                                                             const void* __restrict__ w, int wf32,
                                                             bf16* __restrict__ out, int64_t width, int64_t ld_x,
                                                             int64_t ld_res, float eps, float w_offset) {
  __shared__ float red[16];
  const int64_t r = blockIdx.x;
  const int64_t src = rows ? (int64_t)rows[r] : r;
  const bf16x8* xr = (const bf16x8*)(x + src * ld_x);
  bf16x8* rr = residual ? (bf16x8*)(residual + src * ld_res) : nullptr;
  bf16x8* o = (bf16x8*)(out + r * width);
  const int n8 = (int)(width / 8);
  float v[ITERS][8];
  float g[ITERS][8];  // the gains: loaded with the row, not after the sum (one memory round trip less)
  float ss = 0.f;
#pragma unroll
  for (int it = 0; it < ITERS; ++it) {
    const int i = it * 256 + threadIdx.x;
    if (i < n8) {
      const bf16x8 xv = xr[i];
      if (wf32) {
        const float* wp = (const float*)w + (int64_t)i * 8;
#pragma unroll
        for (int j = 0; j < 8; ++j) g[it][j] = wp[j] + w_offset;
      } else {
        const bf16x8 wv = ((const bf16x8*)w)[i];
#pragma unroll
        for (int j = 0; j < 8; ++j) g[it][j] = (float)wv[j] + w_offset;
      }
      if (rr) {
        const bf16x8 rv = rr[i];
        bf16x8 s;
#pragma unroll
        for (int j = 0; j < 8; ++j) {
          s[j] = (bf16)((float)xv[j] + (float)rv[j]);
          v[it][j] = (float)s[j];
        }
        rr[i] = s;
      } else {
#pragma unroll
        for (int j = 0; j < 8; ++j) v[it][j] = (float)xv[j];
      }
#pragma unroll
      for (int j = 0; j < 8; ++j) ss += v[it][j] * v[it][j];
    }
  }
  ss = block_sum(ss, red);
  const float inv = 1.f / sqrtf(ss / (float)width + eps);
#pragma unroll
  for (int it = 0; it < ITERS; ++it) {
    const int i = it * 256 + threadIdx.x;
    if (i < n8) {
      bf16x8 y;
#pragma unroll
      for (int j = 0; j < 8; ++j) y[j] = (bf16)(v[it][j] * inv * g[it][j]);
      o[i] = y;
    }
  }
}

// Layer norm with gain and bias over the last dimension: y = (x - mean) / sqrt(var + eps) * w + b, var the mean of the
// squared deviations (two passes over the row, which waits in LDS in float). The operands may differ in storage: the
// residual stream may be float where the branch added to it and the normed row are bf16. With a residual,
// r = round(x + r) is written back in the residual's own type first and normed as stored.
__device__ __forceinline__ float ld_any(const void* p, int64_t i, int dt) {
  return dt == DT_F32 ? ((const float*)p)[i] : (float)((const bf16*)p)[i];
}
__device__ __forceinline__ void st_any(void* p, int64_t i, int dt, float v) {
  if (dt == DT_F32) ((float*)p)[i] = v; else ((bf16*)p)[i] = (bf16)v;
}
__device__ __forceinline__ float round_any(float v, int dt) { return dt == DT_F32 ? v : (float)(bf16)v; }

__global__ void __launch_bounds__(256) layernorm_kernel(const void* __restrict__ x, int x_dt, void* __restrict__ residual,
                                                        int r_dt, const int32_t* __restrict__ rows,
                                                        const void* __restrict__ w, const void* __restrict__ b, int p_dt,
                                                        void* __restrict__ out, int o_dt, int64_t width, int64_t ld_x,
                                                        int64_t ld_res, float eps) {
  extern __shared__ float row[];
  __shared__ float red[16];
  const int64_t r = blockIdx.x;
  const int64_t src = rows ? (int64_t)rows[r] : r;
  float sum = 0.f;
  for (int64_t i = threadIdx.x; i < width; i += blockDim.x) {
    float v = ld_any(x, src * ld_x + i, x_dt);
    if (residual) {
      v = round_any(v + ld_any(residual, src * ld_res + i, r_dt), r_dt);
      st_any(residual, src * ld_res + i, r_dt, v);
    }
    row[i] = v;
    sum += v;
  }
  const float mean = block_sum(sum, red) / (float)width;
  float ss = 0.f;
  for (int64_t i = threadIdx.x; i < width; i += blockDim.x) {   // each thread re-reads what it wrote itself
    const float d = row[i] - mean;
    ss = add_square(ss, d);
  }
  const float inv = 1.f / sqrtf(block_sum(ss, red) / (float)width + eps);
  for (int64_t i = threadIdx.x; i < width; i += blockDim.x) {
    const float y = (row[i] - mean) * inv * ld_any(w, i, p_dt) + (b ? ld_any(b, i, p_dt) : 0.f);
    st_any(out, r * width + i, o_dt, y);
  }
}

// The same for widths that are multiples of 8 up to 256 * 8 * ITERS: a thread keeps its 8-entry pieces in registers
// between the passes (one read of the row, no LDS but for the two sums), and moves them 16 or 32 bytes at a time.
template <class SX, class SR, class SO, int ITERS>
__global__ void __launch_bounds__(256) layernorm_regs_kernel(const SX* __restrict__ x, SR* __restrict__ residual,
                                                             const int32_t* __restrict__ rows,
                                                             const float* __restrict__ w, const float* __restrict__ b,
                                                             SO* __restrict__ out, int64_t width, int64_t ld_x,
                                                             int64_t ld_res, float eps) {
  __shared__ float red[16];
  const int64_t r = blockIdx.x;
  const int64_t src = rows ? (int64_t)rows[r] : r;
  const SX* xr = x + src * ld_x;
  SR* rr = residual ? residual + src * ld_res : nullptr;
  const int n8 = (int)(width / 8);
  float v[ITERS][8];
  float sum = 0.f;
#pragma unroll
  for (int it = 0; it < ITERS; ++it) {
    const int i = it * 256 + threadIdx.x;
    if (i < n8) {
#pragma unroll
      for (int j = 0; j < 8; ++j) v[it][j] = to_f32(xr[(int64_t)i * 8 + j]);
      if (rr) {
#pragma unroll
        for (int j = 0; j < 8; ++j) {
          const SR s = from_f32<SR>(v[it][j] + to_f32(rr[(int64_t)i * 8 + j]));
          rr[(int64_t)i * 8 + j] = s;
          v[it][j] = to_f32(s);
        }
      }
#pragma unroll
      for (int j = 0; j < 8; ++j) sum += v[it][j];
    }
  }
  const float mean = block_sum(sum, red) / (float)width;
  float ss = 0.f;
#pragma unroll
  for (int it = 0; it < ITERS; ++it) {
    const int i = it * 256 + threadIdx.x;
    if (i < n8) {
#pragma unroll
      for (int j = 0; j < 8; ++j) ss = add_square(ss, v[it][j] - mean);
    }
  }
  const float inv = 1.f / sqrtf(block_sum(ss, red) / (float)width + eps);
  SO* o = out + r * width;
#pragma unroll
  for (int it = 0; it < ITERS; ++it) {
    const int i = it * 256 + threadIdx.x;
    if (i < n8) {
#pragma unroll
      for (int j = 0; j < 8; ++j) {
        const int64_t c = (int64_t)i * 8 + j;
        o[c] = from_f32<SO>((v[it][j] - mean) * inv * w[c] + (b ? b[c] : 0.f));
      }
    }
  }
}

template <class SX, class SR, class SO>
void launch_layernorm_regs(const void* x, void* residual, const int32_t* rows, const void* w, const void* b, void* out,
                           int64_t n_rows, int64_t width, int64_t ld_x, int64_t ld_res, float eps, hipStream_t stream) {
  const unsigned g = (unsigned)n_rows;
#define LN(IT)                                                                                                        \
  layernorm_regs_kernel<SX, SR, SO, IT><<<g, 256, 0, stream>>>((const SX*)x, (SR*)residual, rows, (const float*)w,    \
                                                               (const float*)b, (SO*)out, width, ld_x, ld_res, eps)
  if (width <= 256 * 8) LN(1);
  else if (width <= 256 * 8 * 2) LN(2);
  else LN(4);
#undef LN
}

inline bool aligned16(const void* p) { return ((uintptr_t)p % 16) == 0; }

}  // namespace

// x [*, width] with row stride ld_x; residual (may be null) has row stride
// ld_res and is updated in place; rows (may be null) lists the n_rows source
// rows; out is dense [n_rows, width]. w has `width` elements, float if w_f32.
extern "C" int dinfer_rmsnorm(int dtype, const void* x, void* residual, const int32_t* rows, const void* w, int w_f32,
                              void* out, int64_t n_rows, int64_t width, int64_t ld_x, int64_t ld_res, float eps,
                              float w_offset, hipStream_t stream) {
  if (n_rows <= 0) return OK;
  if (width <= 0 || ld_x < width || (residual && ld_res < width) || n_rows > 0x7fffffff) return ERR_BAD_SHAPE;
  if (dtype == DT_BF16) {
    const bool vec = width % 8 == 0 && ld_x % 8 == 0 && (!residual || ld_res % 8 == 0) && aligned16(x) &&
                     aligned16(out) && aligned16(w) && (!residual || aligned16(residual)) && width <= 256 * 8 * 4;
    const bf16* xp = (const bf16*)x;
    bf16* rp = (bf16*)residual;
    bf16* op = (bf16*)out;
    if (vec && width <= 256 * 8) {
      rmsnorm_bf16x8_kernel<1><<<(unsigned)n_rows, 256, 0, stream>>>(xp, rp, rows, w, w_f32, op, width, ld_x, ld_res,
                                                                     eps, w_offset);
    } else if (vec && width <= 256 * 8 * 2) {
      rmsnorm_bf16x8_kernel<2><<<(unsigned)n_rows, 256, 0, stream>>>(xp, rp, rows, w, w_f32, op, width, ld_x, ld_res,
                                                                     eps, w_offset);
    } else if (vec) {
      rmsnorm_bf16x8_kernel<4><<<(unsigned)n_rows, 256, 0, stream>>>(xp, rp, rows, w, w_f32, op, width, ld_x, ld_res,
                                                                     eps, w_offset);
    } else {
      rmsnorm_kernel<bf16><<<(unsigned)n_rows, 256, 0, stream>>>(xp, rp, rows, w, w_f32, op, width, ld_x, ld_res, eps,
                                                                 w_offset);
    }
  } else if (dtype == DT_F32) {
    rmsnorm_kernel<float><<<(unsigned)n_rows, 256, 0, stream>>>((const float*)x, (float*)residual, rows, w, 1,
                                                                (float*)out, width, ld_x, ld_res, eps, w_offset);
  } else {
    return ERR_BAD_DTYPE;
  }
  return launch_status();
}

// x, residual (may be null), w and b (b may be null) and out each with a dtype code of their own (w and b share one).
// out is dense [n_rows, width]. Width up to 16,384 (the row waits in LDS).
extern "C" int dinfer_layernorm(const void* x, int x_dtype, void* residual, int res_dtype, const int32_t* rows,
                                const void* w, const void* b, int param_dtype, void* out, int out_dtype, int64_t n_rows,
                                int64_t width, int64_t ld_x, int64_t ld_res, float eps, hipStream_t stream) {
  if (n_rows <= 0) return OK;
  if (width <= 0 || ld_x < width || (residual && ld_res < width) || n_rows > 0x7fffffff) return ERR_BAD_SHAPE;
  for (int dt : {x_dtype, res_dtype, param_dtype, out_dtype})
    if (dt != DT_F32 && dt != DT_BF16) return ERR_BAD_DTYPE;
  // the combinations the engine meets, with float parameters, rows in registers: a float stream normed into the
  // engine's type, alone or after a branch of the engine's type was added to it
  if (param_dtype == DT_F32 && width % 8 == 0 && width <= 256 * 8 * 4 && ld_x % 8 == 0 && (!residual || ld_res % 8 == 0)) {
    const bool res_f32 = !residual || res_dtype == DT_F32;
    if (x_dtype == DT_F32 && res_f32 && out_dtype == DT_BF16) {
      launch_layernorm_regs<float, float, bf16>(x, residual, rows, w, b, out, n_rows, width, ld_x, ld_res, eps, stream);
      return launch_status();
    }
    if (x_dtype == DT_BF16 && res_f32 && out_dtype == DT_BF16) {
      launch_layernorm_regs<bf16, float, bf16>(x, residual, rows, w, b, out, n_rows, width, ld_x, ld_res, eps, stream);
      return launch_status();
    }
    if (x_dtype == DT_F32 && res_f32 && out_dtype == DT_F32) {
      launch_layernorm_regs<float, float, float>(x, residual, rows, w, b, out, n_rows, width, ld_x, ld_res, eps, stream);
      return launch_status();
    }
  }
  if (width > 16384) return ERR_UNSUPPORTED;
  layernorm_kernel<<<(unsigned)n_rows, 256, (size_t)width * sizeof(float), stream>>>(
      x, x_dtype, residual, res_dtype, rows, w, b, param_dtype, out, out_dtype, width, ld_x, ld_res, eps);
  return launch_status();
}

// A residual stream between norms on both sides of every sublayer:
//   stream[s] += mult * branch[s] / sqrt(mean(branch[s]^2) + eps_b) * (wb + off_b)       (with a branch)
//   out[r]     = stream[s] / sqrt(mean(stream[s]^2) + eps) * (w + off)                   (with an out)
// s = rows[r] where rows are given (the model's last norm, on the rows whose logits are wanted), else r. Branch,
// stream, gains and out each have a storage type of their own (a float stream beside bf16 branches and outputs);
// sums, divisions and the addition are float, each stored value is rounded once. The row waits in LDS.
namespace {

__global__ void __launch_bounds__(256) rmsnorm_stream_kernel(const void* __restrict__ branch, int b_dt, int64_t ld_b,
                                                             const void* __restrict__ wb, float eps_b, float off_b,
                                                             float mult, void* __restrict__ stream, int s_dt,
                                                             int64_t ld_s, const int32_t* __restrict__ rows,
                                                             const void* __restrict__ w, int p_dt,
                                                             void* __restrict__ out, int o_dt, float eps, float off,
                                                             int64_t width) {
  extern __shared__ float row[];
  __shared__ float red[16];
  const int64_t r = blockIdx.x;
  const int64_t s = rows ? (int64_t)rows[r] : r;
  float ss = 0.f;
  if (branch) {
    for (int64_t i = threadIdx.x; i < width; i += blockDim.x) {
      const float v = ld_any(branch, s * ld_b + i, b_dt);
      row[i] = v;
      ss = add_square(ss, v);
    }
    const float inv_b = 1.f / sqrtf(block_sum(ss, red) / (float)width + eps_b);
    ss = 0.f;
    for (int64_t i = threadIdx.x; i < width; i += blockDim.x) {   // each thread re-reads what it wrote itself
      const float y = row[i] * inv_b * (ld_any(wb, i, p_dt) + off_b);
      const float x = round_any(__builtin_fmaf(mult, y, ld_any(stream, s * ld_s + i, s_dt)), s_dt);
      st_any(stream, s * ld_s + i, s_dt, x);
      row[i] = x;
      ss = add_square(ss, x);
    }
  } else {
    for (int64_t i = threadIdx.x; i < width; i += blockDim.x) {
      const float x = ld_any(stream, s * ld_s + i, s_dt);
      row[i] = x;
      ss = add_square(ss, x);
    }
  }
  if (!out) return;
  const float inv = 1.f / sqrtf(block_sum(ss, red) / (float)width + eps);
  for (int64_t i = threadIdx.x; i < width; i += blockDim.x)
    st_any(out, r * width + i, o_dt, row[i] * inv * (ld_any(w, i, p_dt) + off));
}

// The same for the combination the engine meets (float stream, float gains, branch and out of one type), widths that
// are multiples of 8 up to 256 * 8 * ITERS: a thread keeps its 8-entry pieces in registers from the first read to the
// last store and moves them 16 or 32 bytes at a time; the gains are asked for with the row, not after the sums.
template <class SB, int ITERS>
__global__ void __launch_bounds__(256) rmsnorm_stream_regs_kernel(const SB* __restrict__ branch, int64_t ld_b,
                                                                  const float* __restrict__ wb, float eps_b, float off_b,
                                                                  float mult, float* __restrict__ stream, int64_t ld_s,
                                                                  const int32_t* __restrict__ rows,
                                                                  const float* __restrict__ w, SB* __restrict__ out,
                                                                  float eps, float off, int64_t width) {
  __shared__ float red[16];
  const int64_t r = blockIdx.x;
  const int64_t s = rows ? (int64_t)rows[r] : r;
  const int n8 = (int)(width / 8);
  float x[ITERS][8], g[ITERS][8], y[ITERS][8];
  float ss = 0.f;
#pragma unroll
  for (int it = 0; it < ITERS; ++it) {
    const int i = it * 256 + threadIdx.x;
    if (i < n8) {
      const int64_t c = (int64_t)i * 8;
      const f32x4 s0 = *(const f32x4*)(stream + s * ld_s + c), s1 = *(const f32x4*)(stream + s * ld_s + c + 4);
#pragma unroll
      for (int j = 0; j < 4; ++j) {
        x[it][j] = s0[j];
        x[it][4 + j] = s1[j];
      }
      if (out) {
        const f32x4 g0 = *(const f32x4*)(w + c), g1 = *(const f32x4*)(w + c + 4);
#pragma unroll
        for (int j = 0; j < 4; ++j) {
          g[it][j] = g0[j] + off;
          g[it][4 + j] = g1[j] + off;
        }
      }
      if (branch) {
        const f32x4 b0 = *(const f32x4*)(wb + c), b1 = *(const f32x4*)(wb + c + 4);
        float bv[8];
        if constexpr (sizeof(SB) == 2) {
          const bf16x8 p = *(const bf16x8*)(branch + s * ld_b + c);
#pragma unroll
          for (int j = 0; j < 8; ++j) bv[j] = (float)p[j];
        } else {
#pragma unroll
          for (int j = 0; j < 8; ++j) bv[j] = to_f32(branch[s * ld_b + c + j]);
        }
#pragma unroll
        for (int j = 0; j < 8; ++j) {
          const float v = bv[j];
          y[it][j] = v * ((j < 4 ? b0[j] : b1[j - 4]) + off_b);
          ss = add_square(ss, v);
        }
      }
    }
  }
  if (branch) {
    const float inv_b = 1.f / sqrtf(block_sum(ss, red) / (float)width + eps_b);
#pragma unroll
    for (int it = 0; it < ITERS; ++it) {
      const int i = it * 256 + threadIdx.x;
      if (i < n8) {
        const int64_t c = (int64_t)i * 8;
        f32x4 s0, s1;
#pragma unroll
        for (int j = 0; j < 8; ++j) {
          x[it][j] = __builtin_fmaf(mult, y[it][j] * inv_b, x[it][j]);
          if (j < 4) s0[j] = x[it][j]; else s1[j - 4] = x[it][j];
        }
        *(f32x4*)(stream + s * ld_s + c) = s0;
        *(f32x4*)(stream + s * ld_s + c + 4) = s1;
      }
    }
  }
  if (!out) return;
  ss = 0.f;
#pragma unroll
  for (int it = 0; it < ITERS; ++it) {
    const int i = it * 256 + threadIdx.x;
    if (i < n8) {
#pragma unroll
      for (int j = 0; j < 8; ++j) ss = add_square(ss, x[it][j]);
    }
  }
  const float inv = 1.f / sqrtf(block_sum(ss, red) / (float)width + eps);
#pragma unroll
  for (int it = 0; it < ITERS; ++it) {
    const int i = it * 256 + threadIdx.x;
    if (i < n8) {
      SB* o = out + r * width + (int64_t)i * 8;
      if constexpr (sizeof(SB) == 2) {
        bf16x8 p;
#pragma unroll
        for (int j = 0; j < 8; ++j) p[j] = (bf16)(x[it][j] * inv * g[it][j]);
        *(bf16x8*)o = p;
      } else {
#pragma unroll
        for (int j = 0; j < 8; ++j) o[j] = from_f32<SB>(x[it][j] * inv * g[it][j]);
      }
    }
  }
}

template <class SB>
void launch_stream_regs(const void* branch, int64_t ld_b, const void* wb, float eps_b, float off_b, float mult, void* stream_,
                        int64_t ld_s, const int32_t* rows, const void* w, void* out, float eps, float off, int64_t n_rows,
                        int64_t width, hipStream_t stream) {
#define SN(IT)                                                                                                       \
  rmsnorm_stream_regs_kernel<SB, IT><<<(unsigned)n_rows, 256, 0, stream>>>(                                          \
      (const SB*)branch, ld_b, (const float*)wb, eps_b, off_b, mult, (float*)stream_, ld_s, rows, (const float*)w, \
      (SB*)out, eps, off, width)
  if (width <= 256 * 8) SN(1);
  else if (width <= 256 * 8 * 2) SN(2);
  else SN(4);
#undef SN
}

}  // namespace

// branch (may be null) [*, ld_b]; stream [*, ld_s], updated in place where a branch is given; out (may be null) dense
// [n_rows, width]; wb and w share the storage type param_dtype. Width up to 16,384.
extern "C" int dinfer_rmsnorm_stream(const void* branch, int branch_dtype, int64_t ld_b, const void* wb, float eps_b,
                                     float off_b, float mult, void* stream_, int stream_dtype, int64_t ld_s,
                                     const int32_t* rows, const void* w, int param_dtype, void* out, int out_dtype,
                                     float eps, float off, int64_t n_rows, int64_t width, hipStream_t stream) {
  if (n_rows <= 0) return OK;
  if (width <= 0 || ld_s < width || (branch && (ld_b < width || !wb)) || (out && !w) || (!branch && !out) ||
      n_rows > 0x7fffffff)
    return ERR_BAD_SHAPE;
  for (int dt : {branch_dtype, stream_dtype, param_dtype, out_dtype})
    if (dt != DT_F32 && dt != DT_BF16) return ERR_BAD_DTYPE;
  // a float stream with float gains, branch and out of one type, rows of whole 16-byte pieces: rows in registers
  const int io_dtype = branch ? branch_dtype : out_dtype;
  if (stream_dtype == DT_F32 && param_dtype == DT_F32 && (!branch || !out || branch_dtype == out_dtype) &&
      width % 8 == 0 && width <= 256 * 8 * 4 && ld_s % 4 == 0 && (!branch || ld_b % 8 == 0) && aligned16(stream_) &&
      (!branch || (aligned16(branch) && aligned16(wb))) && (!out || (aligned16(out) && aligned16(w)))) {
    if (io_dtype == DT_BF16)
      launch_stream_regs<bf16>(branch, ld_b, wb, eps_b, off_b, mult, stream_, ld_s, rows, w, out, eps, off, n_rows, width, stream);
    else
      launch_stream_regs<float>(branch, ld_b, wb, eps_b, off_b, mult, stream_, ld_s, rows, w, out, eps, off, n_rows, width, stream);
    return launch_status();
  }
  if (width > 16384) return ERR_UNSUPPORTED;
  rmsnorm_stream_kernel<<<(unsigned)n_rows, 256, (size_t)width * sizeof(float), stream>>>(
      branch, branch_dtype, ld_b, wb, eps_b, off_b, mult, stream_, stream_dtype, ld_s, rows, w, param_dtype, out,
      out_dtype, eps, off, width);
  return launch_status();
}

// ---- norms in groups, and branches that are normed before they are summed -----------------------------------------
// group_rmsnorm: a row of `width` columns in `groups` equal consecutive parts, each divided by its own root mean square:
//   stream[s] = round(stream[s] + x[s])                                                   (with a stream)
//   out[r, c] = v[c] / sqrt(mean over c's part of v^2 + eps) * w[c],   v = stream[s] (or x[s])
// joined_norms: M branches side by side in a row, each normed over its own `width` columns and then summed:
//   y[c] = scale * sum_m (b_m[c] + bias_m[c]) / sqrt(mean (b_m + bias_m)^2 + eps_m) * w_m[c]
//   out[r] = y,   or, with a stream:   stream[r] += y;   out[r] = group norm of stream[r]
// Both keep the sums in float and round every stored value once.
namespace {

constexpr int MAX_GROUPS = 1024;
constexpr int MAX_BRANCHES = 4;

// inv[g] = 1 / sqrt(mean of part g of row[] + eps): a wave takes every fourth part. row and inv lie in LDS; the caller
// has written row and not yet met a barrier.
__device__ __forceinline__ void group_inverses(const float* row, float* inv, int width, int groups, float eps) {
  const int part = width / groups, wave = threadIdx.x >> 6, lane = threadIdx.x & 63;
  __syncthreads();
  for (int g = wave; g < groups; g += (int)(blockDim.x >> 6)) {
    float ss = 0.f;
    for (int i = lane; i < part; i += 64) ss = add_square(ss, row[g * part + i]);
    ss = wave_sum(ss);
    if (lane == 0) inv[g] = 1.f / sqrtf(ss / (float)part + eps);
  }
  __syncthreads();
}

__global__ void __launch_bounds__(256) group_rmsnorm_kernel(const void* __restrict__ x, int x_dt, int64_t ld_x,
                                                            void* __restrict__ stream, int s_dt, int64_t ld_s,
                                                            const int32_t* __restrict__ rows, const float* __restrict__ w,
                                                            void* __restrict__ out, int o_dt, float eps, int width,
                                                            int groups) {
  extern __shared__ float row[];
  float* inv = row + width;
  const int64_t r = blockIdx.x;
  const int64_t s = rows ? (int64_t)rows[r] : r;
  for (int i = threadIdx.x; i < width; i += blockDim.x) {
    float v = ld_any(x, s * ld_x + i, x_dt);
    if (stream) {
      v = round_any(v + ld_any(stream, s * ld_s + i, s_dt), s_dt);
      st_any(stream, s * ld_s + i, s_dt, v);
    }
    row[i] = v;
  }
  group_inverses(row, inv, width, groups, eps);
  const int part = width / groups;
  for (int i = threadIdx.x; i < width; i += blockDim.x) st_any(out, r * width + i, o_dt, row[i] * inv[i / part] * w[i]);
}

// 8 consecutive values of a row of either type, as floats
__device__ __forceinline__ void load8(const bf16* p, float (&v)[8]) {
  const bf16x8 t = *(const bf16x8*)p;
#pragma unroll
  for (int j = 0; j < 8; ++j) v[j] = (float)t[j];
}
__device__ __forceinline__ void load8(const float* p, float (&v)[8]) {
  const f32x4 a = *(const f32x4*)p, b = *(const f32x4*)(p + 4);
#pragma unroll
  for (int j = 0; j < 4; ++j) { v[j] = a[j]; v[4 + j] = b[j]; }
}
__device__ __forceinline__ void store8(bf16* p, const float (&v)[8]) {
  bf16x8 t;
#pragma unroll
  for (int j = 0; j < 8; ++j) t[j] = (bf16)v[j];
  *(bf16x8*)p = t;
}
__device__ __forceinline__ void store8(float* p, const float (&v)[8]) {
  f32x4 a, b;
#pragma unroll
  for (int j = 0; j < 4; ++j) { a[j] = v[j]; b[j] = v[4 + j]; }
  *(f32x4*)p = a;
  *(f32x4*)(p + 4) = b;
}

// The end both register kernels share: the row's pieces v (a thread's it-th piece is number it * 256 + thread), parts of
// whole pieces. sums: [256 * ITERS] in LDS.
template <class SO, int ITERS>
__device__ __forceinline__ void group_norm_pieces(const float (&v)[ITERS][8], const float* __restrict__ w, SO* __restrict__ out,
                                                  int n8, int groups, float eps, float* sums, float* inv) {
  float g[ITERS][8];
#pragma unroll
  for (int it = 0; it < ITERS; ++it) {
    const int i = it * 256 + threadIdx.x;
    if (i < n8) {
      load8(w + (int64_t)i * 8, g[it]);
      float ss = 0.f;
#pragma unroll
      for (int j = 0; j < 8; ++j) ss = add_square(ss, v[it][j]);
      sums[i] = ss;
    }
  }
  const int part = n8 / groups, wave = threadIdx.x >> 6, lane = threadIdx.x & 63;
  __syncthreads();
  for (int q = wave; q < groups; q += 4) {
    float ss = 0.f;
    for (int i = lane; i < part; i += 64) ss += sums[q * part + i];
    ss = wave_sum(ss);
    if (lane == 0) inv[q] = 1.f / sqrtf(ss / (float)(part * 8) + eps);
  }
  __syncthreads();
#pragma unroll
  for (int it = 0; it < ITERS; ++it) {
    const int i = it * 256 + threadIdx.x;
    if (i < n8) {
      const float f = inv[i / part];
      float y[8];
#pragma unroll
      for (int j = 0; j < 8; ++j) y[j] = v[it][j] * f * g[it][j];
      store8(out + (int64_t)i * 8, y);
    }
  }
}

// The combinations the engine meets: a row in registers from the first read to the last store, 16 or 32 bytes a move.
template <class SX, class SO, int ITERS>
__global__ void __launch_bounds__(256) group_rmsnorm_regs_kernel(const SX* __restrict__ x, int64_t ld_x,
                                                                 float* __restrict__ stream, int64_t ld_s,
                                                                 const int32_t* __restrict__ rows,
                                                                 const float* __restrict__ w, SO* __restrict__ out,
                                                                 float eps, int width, int groups) {
  __shared__ float sums[256 * ITERS];
  __shared__ float inv[MAX_GROUPS];
  const int64_t r = blockIdx.x;
  const int64_t s = rows ? (int64_t)rows[r] : r;
  const int n8 = width / 8;
  float v[ITERS][8];
#pragma unroll
  for (int it = 0; it < ITERS; ++it) {
    const int i = it * 256 + threadIdx.x;
    if (i < n8) {
      load8(x + s * ld_x + (int64_t)i * 8, v[it]);
      if (stream) {
        float t[8];
        load8(stream + s * ld_s + (int64_t)i * 8, t);
#pragma unroll
        for (int j = 0; j < 8; ++j) v[it][j] += t[j];
        store8(stream + s * ld_s + (int64_t)i * 8, v[it]);
      }
    }
  }
  group_norm_pieces<SO, ITERS>(v, w, out + r * width, n8, groups, eps, sums, inv);
}

struct Branches {
  const float* w;      // [M][width]
  const float* bias;   // [M][width] or null
  float eps[MAX_BRANCHES];
  int m;
  int64_t stride;      // columns from one branch to the next
  float scale;
};

template <class S>
__global__ void __launch_bounds__(256) joined_norms_kernel(const S* __restrict__ x, int64_t ld_x, Branches br,
                                                           float* __restrict__ stream, int64_t ld_s,
                                                           const float* __restrict__ w, S* __restrict__ out, float eps,
                                                           int width, int groups) {
  extern __shared__ float row[];      // [width] sums, [groups] inverses
  __shared__ float red[16];
  float* inv = row + width;
  const int64_t r = blockIdx.x;
  for (int m = 0; m < br.m; ++m) {
    const S* b = x + r * ld_x + m * br.stride;
    const float* bias = br.bias ? br.bias + (int64_t)m * width : nullptr;
    float ss = 0.f;
    for (int i = threadIdx.x; i < width; i += blockDim.x) ss = add_square(ss, to_f32(b[i]) + (bias ? bias[i] : 0.f));
    const float f = 1.f / sqrtf(block_sum(ss, red) / (float)width + br.eps[m]);
    for (int i = threadIdx.x; i < width; i += blockDim.x) {      // (each thread re-reads what it wrote itself)
      const float y = (to_f32(b[i]) + (bias ? bias[i] : 0.f)) * f * br.w[(int64_t)m * width + i];
      row[i] = m ? row[i] + y : y;
    }
  }
  if (!stream) {
    for (int i = threadIdx.x; i < width; i += blockDim.x) out[r * width + i] = from_f32<S>(row[i] * br.scale);
    return;
  }
  for (int i = threadIdx.x; i < width; i += blockDim.x) {
    const float v = __builtin_fmaf(row[i], br.scale, stream[r * ld_s + i]);
    stream[r * ld_s + i] = v;
    row[i] = v;
  }
  if (!out) return;
  group_inverses(row, inv, width, groups, eps);
  const int part = width / groups;
  for (int i = threadIdx.x; i < width; i += blockDim.x) out[r * width + i] = from_f32<S>(row[i] * inv[i / part] * w[i]);
}

template <class S, int ITERS>
__global__ void __launch_bounds__(256) joined_norms_regs_kernel(const S* __restrict__ x, int64_t ld_x, Branches br,
                                                                float* __restrict__ stream, int64_t ld_s,
                                                                const float* __restrict__ w, S* __restrict__ out,
                                                                float eps, int width, int groups) {
  __shared__ float sums[256 * ITERS];
  __shared__ float inv[MAX_GROUPS];
  __shared__ float red[16];
  const int64_t r = blockIdx.x;
  const int n8 = width / 8;
  float v[ITERS][8], t[ITERS][8];
#pragma unroll
  for (int it = 0; it < ITERS; ++it) {      // asked for before the branches' sums are awaited
    const int i = it * 256 + threadIdx.x;
#pragma unroll
    for (int j = 0; j < 8; ++j) { v[it][j] = 0.f; t[it][j] = 0.f; }
    if (stream && i < n8) load8(stream + r * ld_s + (int64_t)i * 8, t[it]);
  }
  for (int m = 0; m < br.m; ++m) {
    float b[ITERS][8];
    float ss = 0.f;
#pragma unroll
    for (int it = 0; it < ITERS; ++it) {
      const int i = it * 256 + threadIdx.x;
      if (i < n8) {
        load8(x + r * ld_x + m * br.stride + (int64_t)i * 8, b[it]);
        if (br.bias) {
          float c[8];
          load8(br.bias + (int64_t)m * width + (int64_t)i * 8, c);
#pragma unroll
          for (int j = 0; j < 8; ++j) b[it][j] += c[j];
        }
#pragma unroll
        for (int j = 0; j < 8; ++j) ss = add_square(ss, b[it][j]);
      }
    }
    const float f = 1.f / sqrtf(block_sum(ss, red) / (float)width + br.eps[m]);
#pragma unroll
    for (int it = 0; it < ITERS; ++it) {
      const int i = it * 256 + threadIdx.x;
      if (i < n8) {
        float c[8];
        load8(br.w + (int64_t)m * width + (int64_t)i * 8, c);
#pragma unroll
        for (int j = 0; j < 8; ++j) v[it][j] += b[it][j] * f * c[j];
      }
    }
  }
#pragma unroll
  for (int it = 0; it < ITERS; ++it) {
    const int i = it * 256 + threadIdx.x;
#pragma unroll
    for (int j = 0; j < 8; ++j) v[it][j] = __builtin_fmaf(v[it][j], br.scale, t[it][j]);
    if (i < n8) {
      if (stream) store8(stream + r * ld_s + (int64_t)i * 8, v[it]);
      else store8(out + r * width + (int64_t)i * 8, v[it]);
    }
  }
  if (!stream || !out) return;
  group_norm_pieces<S, ITERS>(v, w, out + r * width, n8, groups, eps, sums, inv);
}

template <class SX, class SO>
void launch_group_regs(const void* x, int64_t ld_x, void* stream_, int64_t ld_s, const int32_t* rows, const float* w, void* out,
                       float eps, int64_t n_rows, int width, int groups, hipStream_t stream) {
#define GN(IT)                                                                                                        \
  group_rmsnorm_regs_kernel<SX, SO, IT><<<(unsigned)n_rows, 256, 0, stream>>>((const SX*)x, ld_x, (float*)stream_, ld_s, \
                                                                              rows, w, (SO*)out, eps, width, groups)
  if (width <= 256 * 8) GN(1);
  else if (width <= 256 * 8 * 2) GN(2);
  else GN(4);
#undef GN
}

template <class S>
void launch_joined_regs(const void* x, int64_t ld_x, const Branches& br, void* stream_, int64_t ld_s, const float* w,
                        void* out, float eps, int64_t n_rows, int width, int groups, hipStream_t stream) {
#define JN(IT)                                                                                                       \
  joined_norms_regs_kernel<S, IT><<<(unsigned)n_rows, 256, 0, stream>>>((const S*)x, ld_x, br, (float*)stream_, ld_s, w, \
                                                                        (S*)out, eps, width, groups)
  if (width <= 256 * 8) JN(1);
  else if (width <= 256 * 8 * 2) JN(2);
  else JN(4);
#undef JN
}

}  // namespace

// x [*, ld_x]; stream (may be null) [*, ld_s], updated in place; rows (may be null) lists the source rows; w [width]
// float; out dense [n_rows, width]. Width up to 16,384, `groups` a divisor of it.
extern "C" int dinfer_group_rmsnorm(const void* x, int x_dtype, int64_t ld_x, void* stream_, int stream_dtype, int64_t ld_s,
                                    const int32_t* rows, const float* w, void* out, int out_dtype, float eps,
                                    int64_t n_rows, int64_t width, int groups, hipStream_t stream) {
  if (n_rows <= 0) return OK;
  if (width <= 0 || ld_x < width || (stream_ && ld_s < width) || !w || !out || groups <= 0 || width % groups ||
      n_rows > 0x7fffffff)
    return ERR_BAD_SHAPE;
  for (int dt : {x_dtype, stream_dtype, out_dtype})
    if (dt != DT_F32 && dt != DT_BF16) return ERR_BAD_DTYPE;
  if (width > 16384 || groups > MAX_GROUPS) return ERR_UNSUPPORTED;
  if ((!stream_ || stream_dtype == DT_F32) && width % 8 == 0 && (width / groups) % 8 == 0 && width <= 256 * 8 * 4 &&
      ld_x % 8 == 0 && (!stream_ || (ld_s % 4 == 0 && aligned16(stream_))) && aligned16(x) && aligned16(w) && aligned16(out)) {
    if (x_dtype == DT_F32 && out_dtype == DT_F32)
      launch_group_regs<float, float>(x, ld_x, stream_, ld_s, rows, w, out, eps, n_rows, (int)width, groups, stream);
    else if (x_dtype == DT_F32)
      launch_group_regs<float, bf16>(x, ld_x, stream_, ld_s, rows, w, out, eps, n_rows, (int)width, groups, stream);
    else if (out_dtype == DT_F32)
      launch_group_regs<bf16, float>(x, ld_x, stream_, ld_s, rows, w, out, eps, n_rows, (int)width, groups, stream);
    else
      launch_group_regs<bf16, bf16>(x, ld_x, stream_, ld_s, rows, w, out, eps, n_rows, (int)width, groups, stream);
    return launch_status();
  }
  // (16,384 columns and their parts' inverses: up to 68 KB of LDS, more than a launch may ask for without saying so)
  const size_t lds = (size_t)(width + groups) * sizeof(float);
  if (lds > 65536 && hipFuncSetAttribute((const void*)group_rmsnorm_kernel, hipFuncAttributeMaxDynamicSharedMemorySize,
                                         (int)lds) != hipSuccess)
    return ERR_LAUNCH;
  group_rmsnorm_kernel<<<(unsigned)n_rows, 256, lds, stream>>>(
      x, x_dtype, ld_x, stream_, stream_dtype, ld_s, rows, w, out, out_dtype, eps, (int)width, groups);
  return launch_status();
}

// x [*, ld_x] holds `branches` rows of `width` side by side, `branch_stride` columns apart, in the step's dtype like out; bw and bias (bias may be null)
// [branches][width] float. stream (may be null) [*, ld_s] float: then it takes the sum, and out (may be null) its group
// norm by w; without a stream out takes the sum. Width up to 16,384.
extern "C" int dinfer_joined_norms(int dtype, const void* x, int64_t ld_x, int branches, int64_t branch_stride, const float* bw, const float* bias,
                                   const float* branch_eps, float scale, float* stream_, int64_t ld_s, const float* w,
                                   void* out, float eps, int64_t n_rows, int64_t width, int groups, hipStream_t stream) {
  if (n_rows <= 0) return OK;
  if (width <= 0 || branches <= 0 || branch_stride < width || ld_x < branch_stride * (branches - 1) + width || (stream_ && ld_s < width) || !bw || !branch_eps ||
      (!stream_ && !out) || (stream_ && out && !w) || groups <= 0 || width % groups || n_rows > 0x7fffffff)
    return ERR_BAD_SHAPE;
  if (dtype != DT_F32 && dtype != DT_BF16) return ERR_BAD_DTYPE;
  if (width > 16384 || groups > MAX_GROUPS || branches > MAX_BRANCHES) return ERR_UNSUPPORTED;
  Branches br{};
  br.w = bw; br.bias = bias; br.m = branches; br.stride = branch_stride; br.scale = scale;
  for (int m = 0; m < branches; ++m) br.eps[m] = branch_eps[m];      // (a host array)
  if (width % 8 == 0 && (width / groups) % 8 == 0 && width <= 256 * 8 * 4 && ld_x % 8 == 0 && branch_stride % 8 == 0 &&
      aligned16(x) && aligned16(bw) &&
      (!bias || aligned16(bias)) && (!stream_ || (ld_s % 4 == 0 && aligned16(stream_))) && (!out || aligned16(out)) &&
      (!w || aligned16(w))) {
    if (dtype == DT_BF16) launch_joined_regs<bf16>(x, ld_x, br, stream_, ld_s, w, out, eps, n_rows, (int)width, groups, stream);
    else launch_joined_regs<float>(x, ld_x, br, stream_, ld_s, w, out, eps, n_rows, (int)width, groups, stream);
    return launch_status();
  }
  const size_t lds = (size_t)(width + groups) * sizeof(float);
  DINFER_DISPATCH_DTYPE(dtype, {
    if (lds > 65536 && hipFuncSetAttribute((const void*)joined_norms_kernel<S>, hipFuncAttributeMaxDynamicSharedMemorySize,
                                           (int)lds) != hipSuccess)
      return ERR_LAUNCH;
    joined_norms_kernel<S><<<(unsigned)n_rows, 256, lds, stream>>>((const S*)x, ld_x, br, stream_, ld_s, w, (S*)out, eps,
                                                                  (int)width, groups);
  });
  return launch_status();
}

// ---- a branch normed on its way into the stream -----------------------------------------------------------------
//   stream[r] += (branch[r] - mean) / sqrt(var + eps) * w + b        (with a branch; var the mean of the squared deviations)
//   out[r]     = stream[r]                                           (with an out: the stream in out's storage type)
// for blocks whose sublayers read the stream itself and whose norms act on what the sublayers give.
namespace {

__global__ void __launch_bounds__(256) layernorm_add_kernel(const void* __restrict__ branch, int b_dt, int64_t ld_b,
                                                            const float* __restrict__ w, const float* __restrict__ bias,
                                                            float eps, void* __restrict__ stream, int s_dt, int64_t ld_s,
                                                            void* __restrict__ out, int o_dt, int64_t width) {
  extern __shared__ float row[];
  __shared__ float red[16];
  const int64_t r = blockIdx.x;
  float mean = 0.f, inv = 0.f;
  if (branch) {
    float sum = 0.f, ss = 0.f;
    for (int64_t i = threadIdx.x; i < width; i += blockDim.x) {
      row[i] = ld_any(branch, r * ld_b + i, b_dt);
      sum += row[i];
    }
    mean = block_sum(sum, red) / (float)width;
    for (int64_t i = threadIdx.x; i < width; i += blockDim.x) ss = add_square(ss, row[i] - mean);   // (what it wrote itself)
    inv = 1.f / sqrtf(block_sum(ss, red) / (float)width + eps);
  }
  for (int64_t i = threadIdx.x; i < width; i += blockDim.x) {
    float x = ld_any(stream, r * ld_s + i, s_dt);
    if (branch) {
      x = round_any(x + ((row[i] - mean) * inv * w[i] + (bias ? bias[i] : 0.f)), s_dt);
      st_any(stream, r * ld_s + i, s_dt, x);
    }
    if (out) st_any(out, r * width + i, o_dt, x);
  }
}

// The same for a float stream and widths that are multiples of 8 up to 256 * 8 * ITERS: rows in registers, 16 or 32 bytes
// at a time, the stream and the gains asked for with the branch.
template <class S, int ITERS>
__global__ void __launch_bounds__(256) layernorm_add_regs_kernel(const S* __restrict__ branch, int64_t ld_b,
                                                                 const float* __restrict__ w, const float* __restrict__ bias,
                                                                 float eps, float* __restrict__ stream, int64_t ld_s,
                                                                 S* __restrict__ out, int64_t width) {
  __shared__ float red[16];
  const int64_t r = blockIdx.x;
  const int n8 = (int)(width / 8);
  float v[ITERS][8], x[ITERS][8], g[ITERS][8];
  float sum = 0.f, ss = 0.f;
#pragma unroll
  for (int it = 0; it < ITERS; ++it) {
    const int i = it * 256 + threadIdx.x;
    if (i < n8) {
      load8(branch + r * ld_b + (int64_t)i * 8, v[it]);
      load8(stream + r * ld_s + (int64_t)i * 8, x[it]);
      load8(w + (int64_t)i * 8, g[it]);
#pragma unroll
      for (int j = 0; j < 8; ++j) sum += v[it][j];
    }
  }
  const float mean = block_sum(sum, red) / (float)width;
#pragma unroll
  for (int it = 0; it < ITERS; ++it) {
    const int i = it * 256 + threadIdx.x;
    if (i < n8) {
#pragma unroll
      for (int j = 0; j < 8; ++j) ss = add_square(ss, v[it][j] - mean);
    }
  }
  const float inv = 1.f / sqrtf(block_sum(ss, red) / (float)width + eps);
#pragma unroll
  for (int it = 0; it < ITERS; ++it) {
    const int i = it * 256 + threadIdx.x;
    if (i < n8) {
      float b[8];
      if (bias) load8(bias + (int64_t)i * 8, b);
#pragma unroll
      for (int j = 0; j < 8; ++j) x[it][j] += (v[it][j] - mean) * inv * g[it][j] + (bias ? b[j] : 0.f);
      store8(stream + r * ld_s + (int64_t)i * 8, x[it]);
      if (out) store8(out + r * width + (int64_t)i * 8, x[it]);
    }
  }
}

template <class S>
void launch_add_regs(const void* branch, int64_t ld_b, const float* w, const float* bias, float eps, void* stream_, int64_t ld_s,
                     void* out, int64_t n_rows, int64_t width, hipStream_t stream) {
#define LA(IT)                                                                                                          \
  layernorm_add_regs_kernel<S, IT><<<(unsigned)n_rows, 256, 0, stream>>>((const S*)branch, ld_b, w, bias, eps, (float*)stream_, \
                                                                         ld_s, (S*)out, width)
  if (width <= 256 * 8) LA(1);
  else if (width <= 256 * 8 * 2) LA(2);
  else LA(4);
#undef LA
}

}  // namespace

// branch (may be null) [*, ld_b]; stream [*, ld_s], updated in place where a branch is given; out (may be null) dense
// [n_rows, width]; w and bias (bias may be null) float. Width up to 16,384.
extern "C" int dinfer_layernorm_add(const void* branch, int branch_dtype, int64_t ld_b, const float* w, const float* bias,
                                    float eps, void* stream_, int stream_dtype, int64_t ld_s, void* out, int out_dtype,
                                    int64_t n_rows, int64_t width, hipStream_t stream) {
  if (n_rows <= 0) return OK;
  if (width <= 0 || !stream_ || ld_s < width || (branch && (ld_b < width || !w)) || (!branch && !out) || n_rows > 0x7fffffff)
    return ERR_BAD_SHAPE;
  for (int dt : {branch_dtype, stream_dtype, out_dtype})
    if (dt != DT_F32 && dt != DT_BF16) return ERR_BAD_DTYPE;
  if (branch && stream_dtype == DT_F32 && (!out || out_dtype == branch_dtype) && width % 8 == 0 && width <= 256 * 8 * 4 &&
      ld_s % 4 == 0 && ld_b % 8 == 0 && aligned16(stream_) && aligned16(branch) && aligned16(w) && aligned16(bias) &&
      aligned16(out)) {
    if (branch_dtype == DT_BF16) launch_add_regs<bf16>(branch, ld_b, w, bias, eps, stream_, ld_s, out, n_rows, width, stream);
    else launch_add_regs<float>(branch, ld_b, w, bias, eps, stream_, ld_s, out, n_rows, width, stream);
    return launch_status();
  }
  if (width > 16384) return ERR_UNSUPPORTED;
  layernorm_add_kernel<<<(unsigned)n_rows, 256, (size_t)width * sizeof(float), stream>>>(
      branch, branch_dtype, ld_b, w, bias, eps, stream_, stream_dtype, ld_s, out, out_dtype, width);
  return launch_status();
}
