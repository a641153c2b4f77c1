// Gated delta rule with short convolutions (e2h_seq_delta).  Per head: S = g S, u = beta (v - S^T k), S = S + k u^T, o = S^T q,
// then RMS norm over the head and a silu gate.
//
// delta_tokens_kernel: one workgroup per (sequence, head) with the head's state in registers.  For a single token it runs the
// convolutions, the unit norms and the gates itself; for more tokens delta_prepare_kernel has put them into scratch memory.
#include "e2h_seq_common.h"

namespace e2h {
namespace {

constexpr int kMaxDim = 256;
constexpr float kUnitEps = 1e-6f;

struct Prepared {
  float *q, *k;   // [rows, kv_heads, dim] unit vectors, q scaled
  float *v;       // [rows, heads, vdim]
  float *beta;    // [rows, heads]
  float *log_g;   // [rows, heads] logarithm of the decay
};

// causal convolution of one channel ending at token t (position pos0 + t), then silu
template <typename T>
__device__ __forceinline__ float conv_silu(const e2h_delta_args &a, size_t row0, int b, int t, int64_t pos0, int64_t first, int64_t col, int ch,
                                           int channels) {
  const T *proj = static_cast<const T *>(a.proj), *tail = static_cast<const T *>(a.tail_in);
  const float *w = a.conv + static_cast<size_t>(ch) * a.taps;
  float acc = 0.f;
  for (int j = 0; j < a.taps; ++j) {
    const int s = t - a.taps + 1 + j;
    const int64_t pos = pos0 + s;
    float x = 0.f;
    if (pos >= first && pos >= 0) x = s >= 0 ? to_f32(proj[(row0 + s) * a.ld + col]) : to_f32(tail[(static_cast<size_t>(b) * a.taps + pos % a.taps) * channels + ch]);
    acc = __builtin_fmaf(w[j], x, acc);
  }
  return silu_f32(acc);
}

__device__ __forceinline__ float delta_log_decay(float a_proj, float a_log, float dt_bias) { return -expf(a_log) * softplus_f32(a_proj + dt_bias); }

// one wave per (token, unit): unit = a query head, a key head, a value head, or (the last one) the per-head gates
template <typename T>
__global__ __launch_bounds__(256) void delta_prepare_kernel(const e2h_delta_args a, Prepared o) {
  const int lane = threadIdx.x & 63;
  const int kvh = static_cast<int>(a.kv_heads), H = static_cast<int>(a.heads), D = static_cast<int>(a.dim), DV = static_cast<int>(a.vdim);
  const int units = 2 * kvh + H + 1, seqlen = static_cast<int>(a.seqlen);
  const int64_t item = static_cast<int64_t>(blockIdx.x) * 4 + (threadIdx.x >> 6);
  const int64_t row = item / units;
  if (row >= a.batch * a.seqlen) return;  // whole waves; no barrier below
  const int u = static_cast<int>(item % units);
  const int b = static_cast<int>(row / seqlen), t = static_cast<int>(row % seqlen);
  const size_t row0 = static_cast<size_t>(b) * seqlen;
  const int64_t pos0 = a.input_pos[0], first = a.first ? a.first[b] : 0;
  const int channels = 2 * kvh * D + H * DV;
  const T *proj = static_cast<const T *>(a.proj);
  if (u == units - 1) {
    for (int h = lane; h < H; h += 64) {
      const bool live = pos0 + t >= first;
      o.beta[row * H + h] = live ? sigmoid_f32(to_f32(proj[row * a.ld + a.b_off + h])) : 0.f;
      o.log_g[row * H + h] = live ? delta_log_decay(to_f32(proj[row * a.ld + a.a_off + h]), a.a_log[h], a.dt_bias[h]) : 0.f;
    }
    return;
  }
  const bool is_q = u < kvh, is_k = !is_q && u < 2 * kvh;
  const int head = is_q ? u : is_k ? u - kvh : u - 2 * kvh;
  const int n = is_q || is_k ? D : DV;
  const int ch0 = is_q ? head * D : is_k ? (kvh + head) * D : 2 * kvh * D + head * DV;
  const int64_t col0 = is_q ? a.q_off + static_cast<int64_t>(head) * D : is_k ? a.k_off + static_cast<int64_t>(head) * D : a.v_off + static_cast<int64_t>(head) * DV;
  float x[kMaxDim / 64], ss = 0.f;
#pragma unroll
  for (int i = 0; i < kMaxDim / 64; ++i) {
    const int d = i * 64 + lane;
    x[i] = d < n ? conv_silu<T>(a, row0, b, t, pos0, first, col0 + d, ch0 + d, channels) : 0.f;
    ss = __builtin_fmaf(x[i], x[i], ss);
  }
  float scale = 1.f;
  if (is_q || is_k) {
    scale = 1.0f / sqrtf(wave_add(ss) + kUnitEps);
    if (is_q) scale /= sqrtf(static_cast<float>(D));
  }
  float *dst = is_q ? o.q + (row * kvh + head) * D : is_k ? o.k + (row * kvh + head) * D : o.v + (row * H + head) * DV;
#pragma unroll
  for (int i = 0; i < kMaxDim / 64; ++i) {
    const int d = i * 64 + lane;
    if (d < n) dst[d] = x[i] * scale;
  }
  // the last taps - 1 convolution inputs of the call; those from before it (a call shorter than the convolution) are carried over
  if (a.taps > 1 && t >= seqlen - (a.taps - 1)) {
    T *tail = static_cast<T *>(a.tail_out) + static_cast<size_t>(b) * a.taps * channels;
    for (int d = lane; d < n; d += 64) tail[((pos0 + t) % a.taps) * channels + ch0 + d] = proj[row * a.ld + col0 + d];
  }
  if (a.taps > 1 && t == 0) {
    const T *src = static_cast<const T *>(a.tail_in) + static_cast<size_t>(b) * a.taps * channels;
    T *tail = static_cast<T *>(a.tail_out) + static_cast<size_t>(b) * a.taps * channels;
    for (int s = seqlen - (a.taps - 1); s < 0; ++s) {
      if (pos0 + s < 0) continue;
      for (int d = lane; d < n; d += 64) tail[((pos0 + s) % a.taps) * channels + ch0 + d] = src[((pos0 + s) % a.taps) * channels + ch0 + d];
    }
  }
}

// RMS norm over the head, norm weight and silu gate of one head's read-out; four columns per lane of wave 0
template <typename T>
__device__ __forceinline__ void gated_norm_store(const e2h_delta_args &a, size_t row, int h, int cg, bool mine, f32x4_t o) {
  const int DV = static_cast<int>(a.vdim);
  const float ss = wave_add(mine ? o[0] * o[0] + o[1] * o[1] + o[2] * o[2] + o[3] * o[3] : 0.f);
  const float inv = a.out_scale / sqrtf(ss / static_cast<float>(DV) + a.eps);
  if (mine) {
    const T *gate = static_cast<const T *>(a.proj) + row * a.ld + a.g_off + static_cast<int64_t>(h) * DV + cg * 4;
    T *dst = static_cast<T *>(a.out) + row * a.ld_out + a.out_off + static_cast<int64_t>(h) * DV + cg * 4;
#pragma unroll
    for (int e = 0; e < 4; ++e) dst[e] = from_f32<T>(o[e] * inv * a.norm_weight[cg * 4 + e] * silu_f32(to_f32(gate[e])));
  }
}

template <typename T, int BLOCK, int RPT, bool ONE>
__global__ __launch_bounds__(BLOCK) void delta_tokens_kernel(const e2h_delta_args a, Prepared p, int cp) {
  __shared__ float sh_q[kMaxDim], sh_k[kMaxDim], sh_red[BLOCK / 64 * 2];
  __shared__ __attribute__((aligned(16))) float sh_v[kMaxDim], sh_u[kMaxDim];
  __shared__ __attribute__((aligned(16))) f32x4_t part_k[BLOCK], part_q[BLOCK];
  const int D = static_cast<int>(a.dim), DV = static_cast<int>(a.vdim), seqlen = ONE ? 1 : static_cast<int>(a.seqlen);
  const int H = static_cast<int>(a.heads), kvh = static_cast<int>(a.kv_heads);
  const int b = blockIdx.x / H, h = blockIdx.x % H, hk = h / (H / kvh);
  const int cg = threadIdx.x & (cp - 1), rg = threadIdx.x / cp, RG = BLOCK / cp;
  const bool col_ok = cg * 4 < DV;
  const int64_t pos0 = a.input_pos[0], first = a.first ? a.first[b] : 0;
  float *st = a.state + (static_cast<size_t>(b) * H + h) * D * DV;
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
    float g, beta;
    if (ONE) {
      const int channels = 2 * kvh * D + H * DV;
      float qs = 0.f, ks = 0.f;
      const bool owner = h % (H / kvh) == 0;  // of the shared query/key head's ring slot; nobody reads that slot in this call
      T *slot = static_cast<T *>(a.tail_out) + (static_cast<size_t>(b) * a.taps + (pos0 > 0 ? pos0 % a.taps : 0)) * channels;
      for (int i = threadIdx.x; i < D; i += BLOCK) {
        const int qc = hk * D + i, kc = (kvh + hk) * D + i;
        const float q = conv_silu<T>(a, row, b, 0, pos0, first, a.q_off + qc, qc, channels);
        const float k = conv_silu<T>(a, row, b, 0, pos0, first, a.k_off + hk * D + i, kc, channels);
        sh_q[i] = q;
        sh_k[i] = k;
        qs = __builtin_fmaf(q, q, qs);
        ks = __builtin_fmaf(k, k, ks);
        if (owner && a.taps > 1) {
          slot[qc] = proj[row * a.ld + a.q_off + qc];
          slot[kc] = proj[row * a.ld + a.k_off + hk * D + i];
        }
      }
      for (int i = threadIdx.x; i < DV; i += BLOCK) {
        const int vc = h * DV + i, ch = 2 * kvh * D + vc;
        sh_v[i] = conv_silu<T>(a, row, b, 0, pos0, first, a.v_off + vc, ch, channels);
        if (a.taps > 1) slot[ch] = proj[row * a.ld + a.v_off + vc];
      }
      qs = wave_add(qs);
      ks = wave_add(ks);
      if ((threadIdx.x & 63) == 0) {
        sh_red[(threadIdx.x >> 6) * 2] = qs;
        sh_red[(threadIdx.x >> 6) * 2 + 1] = ks;
      }
      __syncthreads();
      qs = ks = 0.f;
#pragma unroll
      for (int w = 0; w < BLOCK / 64; ++w) {
        qs += sh_red[2 * w];
        ks += sh_red[2 * w + 1];
      }
      qs = 1.0f / (sqrtf(qs + kUnitEps) * sqrtf(static_cast<float>(D)));
      ks = 1.0f / sqrtf(ks + kUnitEps);
      for (int i = threadIdx.x; i < D; i += BLOCK) {
        sh_q[i] *= qs;
        sh_k[i] *= ks;
      }
      const bool live = pos0 >= first;
      g = live ? expf(delta_log_decay(to_f32(proj[row * a.ld + a.a_off + h]), a.a_log[h], a.dt_bias[h])) : 1.f;
      beta = live ? sigmoid_f32(to_f32(proj[row * a.ld + a.b_off + h])) : 0.f;
    } else {
      for (int i = threadIdx.x; i < D; i += BLOCK) {
        sh_q[i] = p.q[(row * kvh + hk) * D + i];
        sh_k[i] = p.k[(row * kvh + hk) * D + i];
      }
      for (int i = threadIdx.x; i < DV; i += BLOCK) sh_v[i] = p.v[(row * H + h) * DV + i];
      g = expf(p.log_g[row * H + h]);
      beta = p.beta[row * H + h];
    }
    __syncthreads();
    // both read-outs of the decayed state in one pass: (S + k u^T)^T q = S^T q + (k . q) u
    f32x4_t ak = {0.f, 0.f, 0.f, 0.f}, aq = ak;
#pragma unroll
    for (int i = 0; i < RPT; ++i) {
      const int r = rg + RG * i;
      if (r < D) {
        const float k = sh_k[r], q = sh_q[r];
#pragma unroll
        for (int e = 0; e < 4; ++e) {
          s[i][e] *= g;
          ak[e] = __builtin_fmaf(k, s[i][e], ak[e]);
          aq[e] = __builtin_fmaf(q, s[i][e], aq[e]);
        }
      }
    }
    part_k[threadIdx.x] = ak;
    part_q[threadIdx.x] = aq;
    __syncthreads();
    if (threadIdx.x < 64) {  // all column groups of the head lie in wave 0
      float kq = 0.f;
      for (int i = threadIdx.x; i < D; i += 64) kq = __builtin_fmaf(sh_k[i], sh_q[i], kq);
      kq = wave_add(kq);
      const bool mine = threadIdx.x < cp && col_ok;
      f32x4_t o = {0.f, 0.f, 0.f, 0.f};
      if (mine) {
        f32x4_t u = o;
        for (int j = 0; j < RG; ++j) {
          u += part_k[j * cp + threadIdx.x];
          o += part_q[j * cp + threadIdx.x];
        }
        u = (load4(sh_v + cg * 4) - u) * beta;
        store4(sh_u + cg * 4, u);
        o += u * kq;
      }
      gated_norm_store<T>(a, row, h, cg, mine, o);
    }
    __syncthreads();
    if (col_ok) {
      const f32x4_t u = load4(sh_u + cg * 4);
#pragma unroll
      for (int i = 0; i < RPT; ++i) {
        const int r = rg + RG * i;
        if (r < D) {
          const float k = sh_k[r];
#pragma unroll
          for (int e = 0; e < 4; ++e) s[i][e] = __builtin_fmaf(k, u[e], s[i][e]);
        }
      }
    }
    if (!ONE) __syncthreads();  // k and u are read before the next token replaces them
  }
#pragma unroll
  for (int i = 0; i < RPT; ++i) {
    const int r = rg + RG * i;
    if (col_ok && r < D) store4(st + static_cast<size_t>(r) * DV + cg * 4, s[i]);
  }
}

template <typename T, bool ONE>
void launch_tokens(const e2h_delta_args &a, const Prepared &p, hipStream_t s) {
  int cp = 1;
  while (cp * 4 < a.vdim) cp *= 2;
  const dim3 grid(static_cast<unsigned>(a.batch * a.heads));
  const int64_t need = (a.dim * cp + 255) / 256;  // rows per thread with 256 threads
  if (need <= 4) hipLaunchKernelGGL((delta_tokens_kernel<T, 256, 4, ONE>), grid, dim3(256), 0, s, a, p, cp);
  else if (need <= 16) hipLaunchKernelGGL((delta_tokens_kernel<T, 256, 16, ONE>), grid, dim3(256), 0, s, a, p, cp);
  else hipLaunchKernelGGL((delta_tokens_kernel<T, 1024, 16, ONE>), grid, dim3(1024), 0, s, a, p, cp);
}

int64_t round256(int64_t n) { return (n + 255) / 256 * 256; }

// scratch layout; returns its size in bytes
int64_t carve(const e2h_delta_args &a, Prepared *p) {
  if (a.seqlen == 1) return 0;
  const int64_t rows = a.batch * a.seqlen;
  const int64_t qk = round256(rows * a.kv_heads * a.dim * 4), v = round256(rows * a.heads * a.vdim * 4), g = round256(rows * a.heads * 4);
  if (p) {
    uint8_t *base = static_cast<uint8_t *>(a.scratch);
    p->q = reinterpret_cast<float *>(base);
    p->k = reinterpret_cast<float *>(base + qk);
    p->v = reinterpret_cast<float *>(base + 2 * qk);
    p->beta = reinterpret_cast<float *>(base + 2 * qk + v);
    p->log_g = reinterpret_cast<float *>(base + 2 * qk + v + g);
  }
  return 2 * qk + v + 2 * g;
}

template <typename T>
int launch_delta(const e2h_delta_args &a, hipStream_t s) {
  Prepared p = {};
  if (a.seqlen == 1) {
    launch_tokens<T, true>(a, p, s);
    return launch_status();
  }
  carve(a, &p);
  const int64_t items = a.batch * a.seqlen * (2 * a.kv_heads + a.heads + 1);
  hipLaunchKernelGGL(delta_prepare_kernel<T>, dim3(static_cast<unsigned>((items + 3) / 4)), dim3(256), 0, s, a, p);
  launch_tokens<T, false>(a, p, s);
  return launch_status();
}

bool shape_ok(const e2h_delta_args &a) {
  if (a.dtype != E2H_SEQ_BF16 && a.dtype != E2H_SEQ_F32) return false;
  if (a.batch < 1 || a.seqlen < 1 || a.heads < 1 || a.kv_heads < 1 || a.heads % a.kv_heads != 0 || a.dim < 1 || a.dim > kMaxDim || a.vdim < 4 ||
      a.vdim % 4 != 0 || a.vdim > kMaxDim || a.taps < 1 || a.taps > 64 || a.seqlen > INT32_MAX / 2)
    return false;
  if (a.q_off < 0 || a.k_off < 0 || a.v_off < 0 || a.b_off < 0 || a.a_off < 0 || a.g_off < 0 || a.out_off < 0) return false;
  if (a.q_off + a.kv_heads * a.dim > a.ld || a.k_off + a.kv_heads * a.dim > a.ld || a.v_off + a.heads * a.vdim > a.ld || a.b_off + a.heads > a.ld ||
      a.a_off + a.heads > a.ld || a.g_off + a.heads * a.vdim > a.ld || a.out_off + a.heads * a.vdim > a.ld_out)
    return false;
  return a.batch * a.heads <= INT32_MAX && a.batch * a.seqlen * (2 * a.kv_heads + a.heads + 1) / 4 < INT32_MAX &&
         2 * a.kv_heads * a.dim + a.heads * a.vdim <= INT32_MAX;
}

}  // namespace
}  // namespace e2h

using namespace e2h;

extern "C" int64_t e2h_seq_delta_scratch_bytes(const e2h_delta_args *a) {
  if (!a) return E2H_ERR_NULL_POINTER;
  if (!shape_ok(*a)) return E2H_ERR_BAD_SHAPE;
  return carve(*a, nullptr);
}

extern "C" int e2h_seq_delta(const e2h_delta_args *a, void *stream) {
  if (!a || !a->proj || !a->conv || !a->a_log || !a->dt_bias || !a->norm_weight || !a->state || !a->input_pos || !a->out) return E2H_ERR_NULL_POINTER;
  if (!shape_ok(*a)) return E2H_ERR_BAD_SHAPE;
  if (a->taps > 1 && (!a->tail_in || !a->tail_out)) return E2H_ERR_NULL_POINTER;
  if (a->taps > 1 && a->seqlen > 1 && a->tail_in == a->tail_out) return E2H_ERR_BAD_SHAPE;
  if (!aligned16(a->state) || !aligned16(a->scratch)) return E2H_ERR_MISALIGNED;
  const int64_t need = carve(*a, nullptr);
  if (need > 0 && !a->scratch) return E2H_ERR_NULL_POINTER;
  if (need > a->scratch_bytes) return E2H_ERR_SCRATCH_TOO_SMALL;
  if (a->dtype == E2H_SEQ_BF16) return launch_delta<bf16_t>(*a, static_cast<hipStream_t>(stream));
  return launch_delta<float>(*a, static_cast<hipStream_t>(stream));
}
