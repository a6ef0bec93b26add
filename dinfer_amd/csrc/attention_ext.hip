// The flash kernel with options (attention_tile.cuh), for prompt portions and single rows alike: bf16, softmax weights
// with options or sigmoid weights, value heads of the keys' size or of another.
//
// Sizes: key heads of 32, 48, 64, 96, 128 or 256 with values of the same size, pages of any multiple of 8; any pair of 32,
// 48, 64, 96 and 128, and sigmoid weights at all, with pages of a power of two. Anything else is refused (the caller then
// uses the plain kernel).
#include "attention_tile.cuh"

using namespace dinfer;

namespace {

inline bool aligned16(const void* p) { return ((uintptr_t)p % 16) == 0; }

struct Args {
  const bf16* q; int64_t ld_q;
  bf16* out; int64_t ld_out;
  const bf16* kc; const bf16* vc;
  const int32_t* bt; int64_t max_blocks;
  const int32_t* cu; const int32_t* sl;
  int num_reqs, max_q_len, window, H, Hkv, ps;
  FlashExt ext;
};

template <int DT, int DV, int KIND, int QT>
int launch_rows(const Args& p, hipStream_t stream) {
  const int tiles = (p.max_q_len + 16 * QT - 1) / (16 * QT);
  const int64_t blocks = (int64_t)tiles * p.H * p.num_reqs;
  if (blocks > 0x7fffffff) return ERR_UNSUPPORTED;
  // page sizes that are no powers of two: only where keys and values are of one size, under a softmax
  constexpr bool ANY_PAGE = KIND == OPTIONS && DT == DV;
  auto kernel = attn_flash_kernel<DT, QT, true, KIND, DV>;
  if constexpr (ANY_PAGE) {
    if (p.ps & (p.ps - 1)) kernel = attn_flash_kernel<DT, QT, false, KIND, DV>;
  } else if (p.ps & (p.ps - 1)) {
    return ERR_UNSUPPORTED;
  }
  const size_t lds = (size_t)3 * QT * 64 * (sizeof(f32x4) * DV + 2 * sizeof(float));
  // (more than the 64 KB of LDS a launch may ask for without saying so)
  if (lds > 65536 && hipFuncSetAttribute((const void*)kernel, hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds) != hipSuccess)
    return ERR_LAUNCH;
  kernel<<<(unsigned)blocks, 256, lds, stream>>>(p.q, p.ld_q, p.out, p.ld_out, p.kc, p.vc, p.bt, p.max_blocks, p.cu, p.sl, tiles,
                                                p.ext.scale * LOG2E, p.window, p.H, p.Hkv, p.ps, 0, p.ext);
  return launch_status();
}

// Rows a workgroup takes: 48 at heads of 128 where the rows make several rounds of workgroups over the chip (rows of at
// most two tiles a request never fill the third), 32 where portions are longer than one tile, else 16.
template <int DT, int DV, int KIND>
int launch(const Args& p, hipStream_t stream) {
  if constexpr (DT == 8 && DV == 8) {
    if (p.max_q_len > 32 && (int64_t)((p.max_q_len + 47) / 48) * p.H * p.num_reqs >= 2000) return launch_rows<DT, DV, KIND, 3>(p, stream);
  }
  if constexpr (DT <= 8 && DV <= 8) {
    if (p.max_q_len > 16) return launch_rows<DT, DV, KIND, 2>(p, stream);
  }
  return launch_rows<DT, DV, KIND, 1>(p, stream);
}

template <int DT, int KIND>
int launch_values(int v_dim, const Args& p, hipStream_t stream) {
  switch (v_dim) {
    case 32: return launch<DT, 2, KIND>(p, stream);
    case 48: return launch<DT, 3, KIND>(p, stream);
    case 64: return launch<DT, 4, KIND>(p, stream);
    case 96: return launch<DT, 6, KIND>(p, stream);
    case 128: return launch<DT, 8, KIND>(p, stream);
    default: return ERR_UNSUPPORTED;
  }
}

template <int KIND>
int launch_keys(int head_dim, int v_dim, const Args& p, hipStream_t stream) {
  switch (head_dim) {
    case 32: return launch_values<2, KIND>(v_dim, p, stream);
    case 48: return launch_values<3, KIND>(v_dim, p, stream);
    case 64: return launch_values<4, KIND>(v_dim, p, stream);
    case 96: return launch_values<6, KIND>(v_dim, p, stream);
    case 128: return launch_values<8, KIND>(v_dim, p, stream);
    case 256: return v_dim == 256 ? launch<16, 16, KIND>(p, stream) : ERR_UNSUPPORTED;
    default: return ERR_UNSUPPORTED;
  }
}

inline bool listed(int d) { return d == 32 || d == 48 || d == 64 || d == 96 || d == 128; }

}  // namespace

// 1 if dinfer_attn_flash_ext takes this geometry (sigmoid: with sigmoid weights), else 0.
extern "C" int dinfer_attn_flash_ext_supports(int head_dim, int v_dim, int page_size, int heads, int kv_heads, int sigmoid) {
  if (!(listed(head_dim) && listed(v_dim)) && !(head_dim == 256 && v_dim == 256)) return 0;
  if (!(page_size > 0 && page_size % 8 == 0 && kv_heads > 0 && heads % kv_heads == 0)) return 0;
  if ((page_size & (page_size - 1)) && (sigmoid || head_dim != v_dim)) return 0;
  // the kernels keep the elements of one page (all kv heads) in 32-bit arithmetic
  const int wider = head_dim > v_dim ? head_dim : v_dim;
  return (int64_t)kv_heads * page_size * wider < (int64_t)1 << 30 ? 1 : 0;
}

// Keys below keep_first stay visible behind the window; sinks [heads] float (or null) join the denominator; slope_exp E
// takes 2^(-E (h + 1) / heads) times the distance off the scores; the output is multiplied by out_scale. v_dim: the size of
// a value head (0: head_dim); out holds head h at column h v_dim. sigmoid_bias (or null): [heads] float, the weights are
// sigmoid(score + bias), not normalised (no sinks then). softcap C > 0: the scores are C tanh(scale q . k / C) (softmax
// weights only); chunk N > 0: a row sees the keys of its own chunk of N positions only (counted from 0).
extern "C" int dinfer_attn_flash_ext(const void* q, int64_t ld_q, void* out, int64_t ld_out, const void* k_cache,
                                     const void* v_cache, const int32_t* block_table, int64_t max_blocks,
                                     const int32_t* cu_seqlens, const int32_t* seq_lens, int num_reqs, int max_q_len,
                                     float scale, int window, int keep_first, const float* sinks, float slope_exp,
                                     float out_scale, int heads, int kv_heads, int head_dim, int v_dim, int page_size,
                                     const float* sigmoid_bias, float softcap, int chunk, hipStream_t stream) {
  if (num_reqs <= 0 || max_q_len <= 0) return OK;
  if (v_dim <= 0) v_dim = head_dim;
  if (!dinfer_attn_flash_ext_supports(head_dim, v_dim, page_size, heads, kv_heads, sigmoid_bias ? 1 : 0) || (sigmoid_bias && (sinks || softcap > 0.f)))
    return ERR_UNSUPPORTED;
  if (window < 0 || keep_first < 0 || chunk < 0 || !(softcap >= 0.f) || !(scale > 0.f) || max_blocks <= 0 || ld_q % 8 || ld_out % 4 || !aligned16(q) ||
      !aligned16(k_cache) || !aligned16(v_cache) || ((uintptr_t)out % 8))
    return ERR_BAD_SHAPE;
  const Args p{(const bf16*)q, ld_q, (bf16*)out, ld_out, (const bf16*)k_cache, (const bf16*)v_cache, block_table, max_blocks,
               cu_seqlens, seq_lens, num_reqs, max_q_len, window, heads, kv_heads, page_size,
               FlashExt{keep_first, sinks, slope_exp, out_scale, softcap > 0.f ? 1.f : scale, sigmoid_bias, softcap,
                        softcap > 0.f ? 2.f * LOG2E * scale / softcap : 0.f, chunk}};
  return sigmoid_bias ? launch_keys<SIGMOID>(head_dim, v_dim, p, stream) : launch_keys<OPTIONS>(head_dim, v_dim, p, stream);
}
