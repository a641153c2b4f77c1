// HGRN2 linear attention (e2h_seq_hgrn2): S = diag(f) S + (1 - f) v^T per head, o = S^T q, RMS norm over the head.
//
// Token-by-token form: one workgroup per (sequence, head) keeps the head's whole state in registers (a thread owns four value
// columns and every RG-th row), reads it once and writes it once per call.
#include "e2h_seq_common.h"

namespace e2h {
namespace {

constexpr int kMaxDim = 256;

struct Gate {
  float f, k;  // forget gate and what is written, 1 - f, each without cancellation
};
__device__ __forceinline__ Gate hgrn_gate(float z, float low) {
  const float up = 1.0f - low;
  return Gate{low + up * sigmoid_f32(z), up * sigmoid_f32(-z)};
}

template <typename T, int BLOCK, int RPT>
__global__ __launch_bounds__(BLOCK) void hgrn2_tokens_kernel(const e2h_hgrn2_args a, int cp) {
  __shared__ float sh_q[kMaxDim], sh_f[kMaxDim], sh_k[kMaxDim];
  __shared__ __attribute__((aligned(16))) float sh_v[kMaxDim];
  __shared__ __attribute__((aligned(16))) f32x4_t part[BLOCK];
  const int D = static_cast<int>(a.dim), DV = static_cast<int>(a.vdim), seqlen = static_cast<int>(a.seqlen);
  const int b = blockIdx.x / static_cast<int>(a.heads), h = blockIdx.x % static_cast<int>(a.heads);
  const int cg = threadIdx.x & (cp - 1), rg = threadIdx.x / cp, RG = BLOCK / cp;
  const bool col_ok = cg * 4 < DV;
  const int64_t pos0 = a.input_pos[0], first = a.first ? a.first[b] : 0;
  float *st = a.state + (static_cast<size_t>(b) * a.heads + h) * D * DV;
  f32x4_t s[RPT];
#pragma unroll
  for (int i = 0; i < RPT; ++i) {
    const int r = rg + RG * i;
    s[i] = f32x4_t{0.f, 0.f, 0.f, 0.f};
    if (pos0 > 0 && col_ok && r < D) s[i] = load4(st + static_cast<size_t>(r) * DV + cg * 4);
  }
  const T *proj = static_cast<const T *>(a.proj);
  for (int t = 0; t < seqlen; ++t) {
    const size_t row = static_cast<size_t>(b) * seqlen + t;
    const T *src = proj + row * a.ld;
    const bool live = pos0 + t >= first;
    for (int i = threadIdx.x; i < D; i += BLOCK) {
      const int ch = h * D + i;
      const Gate g = hgrn_gate(to_f32(src[a.f_off + ch]) + a.f_bias[ch], a.lower[ch]);
      sh_q[i] = silu_f32(to_f32(src[a.q_off + ch]));
      sh_f[i] = live ? g.f : 1.f;
      sh_k[i] = live ? g.k : 0.f;
    }
    for (int i = threadIdx.x; i < DV; i += BLOCK) sh_v[i] = to_f32(src[a.v_off + static_cast<int64_t>(h) * DV + i]);
    __syncthreads();
    f32x4_t acc = {0.f, 0.f, 0.f, 0.f};
    f32x4_t v = {0.f, 0.f, 0.f, 0.f};
    if (col_ok) v = load4(sh_v + cg * 4);
#pragma unroll
    for (int i = 0; i < RPT; ++i) {
      const int r = rg + RG * i;
      if (r < D) {
        const float f = sh_f[r], k = sh_k[r], q = sh_q[r];
#pragma unroll
        for (int e = 0; e < 4; ++e) {
          s[i][e] = __builtin_fmaf(k, v[e], f * s[i][e]);
          acc[e] = __builtin_fmaf(q, s[i][e], acc[e]);
        }
      }
    }
    part[threadIdx.x] = acc;
    __syncthreads();
    if (threadIdx.x < 64) {  // all column groups of the head lie in wave 0
      f32x4_t o = {0.f, 0.f, 0.f, 0.f};
      if (threadIdx.x < cp && col_ok)
        for (int g = 0; g < RG; ++g) o += part[g * cp + threadIdx.x];
      const float ss = wave_add(o[0] * o[0] + o[1] * o[1] + o[2] * o[2] + o[3] * o[3]);
      const float inv = a.out_scale / sqrtf(ss / static_cast<float>(DV) + a.eps);
      if (threadIdx.x < cp && col_ok) {
        T *dst = static_cast<T *>(a.out) + row * a.ld_out + a.out_off + static_cast<int64_t>(h) * DV + cg * 4;
#pragma unroll
        for (int e = 0; e < 4; ++e) dst[e] = from_f32<T>(o[e] * inv * a.norm_weight[cg * 4 + e]);
      }
    }
  }
#pragma unroll
  for (int i = 0; i < RPT; ++i) {
    const int r = rg + RG * i;
    if (col_ok && r < D) store4(st + static_cast<size_t>(r) * DV + cg * 4, s[i]);
  }
}

template <typename T>
void launch_tokens(const e2h_hgrn2_args &a, hipStream_t s) {
  int cp = 1;
  while (cp * 4 < a.vdim) cp *= 2;
  const dim3 grid(static_cast<unsigned>(a.batch * a.heads));
  const int64_t need = (a.dim * cp + 255) / 256;  // rows per thread with 256 threads
  if (need <= 4) hipLaunchKernelGGL((hgrn2_tokens_kernel<T, 256, 4>), grid, dim3(256), 0, s, a, cp);
  else if (need <= 16) hipLaunchKernelGGL((hgrn2_tokens_kernel<T, 256, 16>), grid, dim3(256), 0, s, a, cp);
  else hipLaunchKernelGGL((hgrn2_tokens_kernel<T, 1024, 16>), grid, dim3(1024), 0, s, a, cp);
}

}  // namespace
}  // namespace e2h

using namespace e2h;

extern "C" int64_t e2h_seq_hgrn2_scratch_bytes(const e2h_hgrn2_args *a) { return a ? 0 : E2H_ERR_NULL_POINTER; }

extern "C" int e2h_seq_hgrn2(const e2h_hgrn2_args *a, void *stream) {
  if (!a || !a->proj || !a->f_bias || !a->lower || !a->norm_weight || !a->state || !a->input_pos || !a->out) return E2H_ERR_NULL_POINTER;
  if (a->dtype != E2H_SEQ_BF16 && a->dtype != E2H_SEQ_F32) return E2H_ERR_BAD_SHAPE;
  if (a->batch < 1 || a->seqlen < 1 || a->heads < 1 || a->dim < 1 || a->dim > kMaxDim || a->vdim < 4 || a->vdim % 4 != 0 || a->vdim > kMaxDim)
    return E2H_ERR_BAD_SHAPE;
  if (a->q_off < 0 || a->f_off < 0 || a->v_off < 0 || a->out_off < 0 || a->q_off + a->heads * a->dim > a->ld || a->f_off + a->heads * a->dim > a->ld ||
      a->v_off + a->heads * a->vdim > a->ld || a->out_off + a->heads * a->vdim > a->ld_out || a->batch * a->heads > INT32_MAX ||
      a->seqlen > INT32_MAX / 2)
    return E2H_ERR_BAD_SHAPE;
  if (!aligned16(a->state)) return E2H_ERR_MISALIGNED;
  if (a->dtype == E2H_SEQ_BF16) launch_tokens<bf16_t>(*a, static_cast<hipStream_t>(stream));
  else launch_tokens<float>(*a, static_cast<hipStream_t>(stream));
  return launch_status();
}
