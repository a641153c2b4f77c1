// Gated delta rule with short convolutions (e2h_seq_delta).  Per head: S = g S, u = beta (v - S^T k), S = S + k u^T, o = S^T q,
// then RMS norm over the head and a silu gate.
//
// delta_tokens_kernel: one workgroup per (sequence, head) with the head's state in registers.  For a single token it runs the
// convolutions, the unit norms and the gates itself; for more tokens delta_prepare_kernel has put them into scratch memory.
//
// Chunked form (many tokens), float32 matrix cores throughout.  Within a chunk of 64 tokens that starts from state S0, with
// G_t the decay from the chunk's start through token t,
//   u_t + sum_{s<t} beta_t (G_t / G_s) (k_t . k_s) u_s = beta_t (v_t - G_t S0^T k_t)
//   o_t = G_t S0^T q_t + sum_{s<=t} (G_t / G_s) (q_t . k_s) u_s,   S = G_end S0 + sum_s (G_end / G_s) k_s u_s^T
// 1. delta_chunk_kernel, parallel over chunks: T = (I + M)^-1 diag(beta) for the strictly lower triangular M above (the four
//    16 x 16 diagonal blocks by substitution, the others from products of blocks), and the masked, decayed products q k^T;
// 2. delta_scan_kernel, one workgroup per (sequence, head, 16 value columns), chunk after chunk: read-outs, u = T (v - G S0^T k),
//    outputs and the next state;
// 3. delta_gate_kernel: RMS norm over the head and the silu gate.
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

// The same for convolutions of up to four taps with everything in multiples of four channels: `cp` lanes (a power of two) hold
// one head's channels, four each, and walk kPrepareRun tokens with the previous inputs in registers.
constexpr int kPrepareRun = 8;

template <typename T>
__global__ __launch_bounds__(256) void delta_prepare4_kernel(const e2h_delta_args a, Prepared o, int cp, int runs) {
  const int kvh = static_cast<int>(a.kv_heads), H = static_cast<int>(a.heads), D = static_cast<int>(a.dim), DV = static_cast<int>(a.vdim);
  const int heads = 2 * kvh + H, per_wave = 64 / cp, groups = (heads + per_wave - 1) / per_wave, seqlen = static_cast<int>(a.seqlen), taps = a.taps;
  const int lane = threadIdx.x & 63;
  const int64_t item = static_cast<int64_t>(blockIdx.x) * 4 + (threadIdx.x >> 6);  // (sequence, run, group of heads)
  if (item >= a.batch * runs * groups) return;  // whole waves
  const int u = static_cast<int>(item % groups) * per_wave + lane / cp;
  const int64_t br = item / groups;
  const int b = static_cast<int>(br / runs), t_begin = static_cast<int>(br % runs) * kPrepareRun;
  const int t_end = t_begin + kPrepareRun < seqlen ? t_begin + kPrepareRun : seqlen;
  const bool is_q = u < kvh, is_k = !is_q && u < 2 * kvh;
  const int head = is_q ? u : is_k ? u - kvh : u - 2 * kvh, n = is_q || is_k ? D : DV, d = (lane & (cp - 1)) * 4;
  const bool mine = u < heads && d < n;
  const int ch = mine ? (is_q ? head * D : is_k ? (kvh + head) * D : 2 * kvh * D + head * DV) + d : 0;
  const int64_t col = mine ? (is_q ? a.q_off : is_k ? a.k_off : a.v_off) + static_cast<int64_t>(head) * n + d : a.q_off;
  const int64_t pos0 = a.input_pos[0], first = a.first ? a.first[b] : 0;
  const int channels = 2 * kvh * D + H * DV;
  const size_t row0 = static_cast<size_t>(b) * seqlen;
  const T *src = static_cast<const T *>(a.proj) + row0 * a.ld + col;
  const T *tail = static_cast<const T *>(a.tail_in) + static_cast<size_t>(b) * taps * channels + ch;
  const f32x4_t zero = {0.f, 0.f, 0.f, 0.f};
  f32x4_t w[4];  // shallower convolutions: zero weights in front
#pragma unroll
  for (int j = 0; j < 4; ++j) {
    w[j] = zero;
    const int jj = j - (4 - taps);
    if (jj >= 0) {
#pragma unroll
      for (int e = 0; e < 4; ++e) w[j][e] = a.conv[static_cast<size_t>(ch + e) * taps + jj];
    }
  }
  Quad<T> x[kPrepareRun + 3];
  bool there[kPrepareRun + 3];
#pragma unroll
  for (int i = 0; i < kPrepareRun + 3; ++i) {
    const int t = t_begin - 3 + i;
    const int64_t pos = pos0 + t;
    there[i] = pos >= first && pos >= 0 && t >= -(taps - 1);
    if (t >= 0) x[i] = load_quad(src + static_cast<int64_t>(t < seqlen ? t : seqlen - 1) * a.ld);
    else x[i] = load_quad(there[i] ? tail + (pos % taps) * channels : src);
  }
#pragma unroll
  for (int i = 0; i < kPrepareRun; ++i) {
    const int t = t_begin + i;
    if (t >= t_end) break;
    f32x4_t y = zero;
#pragma unroll
    for (int j = 0; j < 4; ++j)
      if (there[i + j]) {
        const f32x4_t v = x[i + j].f32();
#pragma unroll
        for (int e = 0; e < 4; ++e) y[e] = __builtin_fmaf(w[j][e], v[e], y[e]);
      }
    float ss = 0.f;
#pragma unroll
    for (int e = 0; e < 4; ++e) {
      y[e] = mine ? fast_silu(y[e]) : 0.f;
      ss = __builtin_fmaf(y[e], y[e], ss);
    }
    for (int off = 1; off < cp; off <<= 1) ss += __shfl_xor(ss, off);
    if (is_q || is_k) y *= is_q ? 1.0f / (sqrtf(ss + kUnitEps) * sqrtf(static_cast<float>(D))) : 1.0f / sqrtf(ss + kUnitEps);
    const size_t row = row0 + t;
    if (mine) store4(is_q ? o.q + (row * kvh + head) * D + d : is_k ? o.k + (row * kvh + head) * D + d : o.v + (row * H + head) * DV + d, y);
  }
  if (taps > 1 && t_end == seqlen && mine) {  // the last taps - 1 inputs, some of them carried over when the call is that short
    T *dst = static_cast<T *>(a.tail_out) + static_cast<size_t>(b) * taps * channels + ch;
#pragma unroll
    for (int i = 0; i < kPrepareRun + 3; ++i) {
      const int t = t_begin - 3 + i;
      if (t < t_end && t >= t_end - (taps - 1) && pos0 + t >= 0)
        *reinterpret_cast<decltype(x[i].raw) *>(dst + ((pos0 + t) % taps) * channels) = x[i].raw;
    }
  }
}

template <typename T>
__global__ __launch_bounds__(256) void delta_gates_kernel(const e2h_delta_args a, Prepared o) {
  const int H = static_cast<int>(a.heads);
  const int64_t i = static_cast<int64_t>(blockIdx.x) * 256 + threadIdx.x;
  if (i >= a.batch * a.seqlen * H) return;
  const int64_t row = i / H;
  const int h = static_cast<int>(i % H);
  const bool live = a.input_pos[0] + row % a.seqlen >= (a.first ? a.first[row / a.seqlen] : 0);
  const T *src = static_cast<const T *>(a.proj) + row * a.ld;
  o.beta[i] = live ? sigmoid_f32(to_f32(src[a.b_off + h])) : 0.f;
  o.log_g[i] = live ? delta_log_decay(to_f32(src[a.a_off + h]), a.a_log[h], a.dt_bias[h]) : 0.f;
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
    if (pos0 > 0 && col_ok && r < D) s[i] = load4_stream(st + static_cast<size_t>(r) * DV + cg * 4);
  }
  const T *proj = static_cast<const T *>(a.proj);
  for (int t = 0; t < seqlen; ++t) {
    const size_t row = static_cast<size_t>(b) * seqlen + t;
    float log_g, beta;
    if (ONE) {
      const int channels = 2 * kvh * D + H * DV;
      float qs = 0.f, ks = 0.f;
      const bool owner = h % (H / kvh) == 0;  // of the shared query/key head's ring slot; nobody reads that slot in this call
      const uint32_t taps = static_cast<uint32_t>(a.taps), at = static_cast<uint32_t>(pos0 > 0 ? pos0 : 0);
      T *slot = static_cast<T *>(a.tail_out) + (static_cast<size_t>(b) * a.taps + at % taps) * channels;
      size_t kept[3];  // ring rows of the three tokens before this one
      bool there[3];
#pragma unroll
      for (int j = 0; j < 3; ++j) {
        const int64_t pos = pos0 - 3 + j;
        there[j] = taps > 3u - j && pos >= first && pos >= 0;
        kept[j] = (static_cast<size_t>(b) * a.taps + (there[j] ? static_cast<uint32_t>(pos) % taps : 0u)) * channels;
      }
      for (int i = threadIdx.x; i < 2 * D + DV; i += BLOCK) {  // channels of q, k, v
        const bool is_q = i < D, is_k = !is_q && i < 2 * D;
        const int d = is_q ? i : is_k ? i - D : i - 2 * D;
        const int ch = is_q ? hk * D + d : is_k ? (kvh + hk) * D + d : 2 * kvh * D + h * DV + d;
        const int64_t c0 = is_q ? a.q_off + hk * D + d : is_k ? a.k_off + hk * D + d : a.v_off + static_cast<int64_t>(h) * DV + d;
        float y;
        if (taps <= 4) {  // everything in flight at once
          const T now = proj[row * a.ld + c0];
          const T *tail = static_cast<const T *>(a.tail_in);
          T x[3];
          float w[4];
#pragma unroll
          for (int j = 0; j < 3; ++j) x[j] = *(there[j] ? tail + kept[j] + ch : proj + row * a.ld + c0);
#pragma unroll
          for (int j = 0; j < 4; ++j) w[j] = a.conv[static_cast<size_t>(ch) * taps + (j + taps >= 4u ? j + taps - 4u : 0u)];
          y = w[3] * to_f32(now);
#pragma unroll
          for (int j = 0; j < 3; ++j) y = __builtin_fmaf(w[j], there[j] ? to_f32(x[j]) : 0.f, y);
          y = silu_f32(y);
          if (taps > 1 && (owner || !(is_q || is_k))) slot[ch] = now;
        } else {
          y = conv_silu<T>(a, row, b, 0, pos0, first, c0, ch, channels);
          if (owner || !(is_q || is_k)) slot[ch] = proj[row * a.ld + c0];
        }
        if (is_q) qs = __builtin_fmaf(y, y, qs);
        if (is_k) ks = __builtin_fmaf(y, y, ks);
        (is_q ? sh_q : is_k ? sh_k : sh_v)[d] = y;
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
      log_g = live ? delta_log_decay(to_f32(proj[row * a.ld + a.a_off + h]), a.a_log[h], a.dt_bias[h]) : 0.f;
      beta = live ? sigmoid_f32(to_f32(proj[row * a.ld + a.b_off + h])) : 0.f;
    } else {
      for (int i = threadIdx.x; i < D; i += BLOCK) {
        sh_q[i] = p.q[(row * kvh + hk) * D + i];
        sh_k[i] = p.k[(row * kvh + hk) * D + i];
      }
      for (int i = threadIdx.x; i < DV; i += BLOCK) sh_v[i] = p.v[(row * H + h) * DV + i];
      log_g = p.log_g[row * H + h];
      beta = p.beta[row * H + h];
    }
    __syncthreads();
    const Decay g = decay_of(expf(log_g), -expm1f(log_g));
    // both read-outs of the decayed state in one pass: (S + k u^T)^T q = S^T q + (k . q) u
    f32x4_t ak = {0.f, 0.f, 0.f, 0.f}, aq = ak;
#pragma unroll
    for (int i = 0; i < RPT; ++i) {
      const int r = rg + RG * i;
      if (r < D) {
        const float k = sh_k[r], q = sh_q[r];
#pragma unroll
        for (int e = 0; e < 4; ++e) {
          s[i][e] = decayed(g, s[i][e]);
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
    if (col_ok && r < D) store4_stream(st + static_cast<size_t>(r) * DV + cg * 4, s[i]);
  }
}

// ---- chunked form ----------------------------------------------------------------------------------------------------------
constexpr int kChunk = 64;

struct ChunkScratch {
  float *t;  // [batch * heads, chunks, 64, 64]
  float *p;  // [batch * heads, chunks, 64, 64]
  int chunks;
};

// four consecutive values of a row at column d; zero beyond the row's n values (n % 4 == 0) or when the row does not exist
__device__ __forceinline__ f32x4_t row4(const float *base, bool exists, int d, int n) {
  return exists && d < n ? load4(base + d) : f32x4_t{0.f, 0.f, 0.f, 0.f};
}

// step 1: 4 waves, one (sequence, head, chunk) each; wave w owns the token rows 16 w .. 16 w + 15
__global__ __launch_bounds__(256) void delta_chunk_kernel(const e2h_delta_args a, Prepared p, ChunkScratch cs) {
  constexpr int kRow = kChunk + 4;
  __shared__ __attribute__((aligned(16))) float sm[kChunk * kRow];  // M, then its blocks are replaced by the inverse's
  __shared__ __attribute__((aligned(16))) float si[kChunk * kRow];  // inverse
  __shared__ float sg[kChunk], sb[kChunk];
  const int D = static_cast<int>(a.dim), H = static_cast<int>(a.heads), kvh = static_cast<int>(a.kv_heads), seqlen = static_cast<int>(a.seqlen);
  const int chunk = blockIdx.x % cs.chunks, bh = blockIdx.x / cs.chunks;
  const int b = bh / H, h = bh % H, hk = h / (H / kvh);
  const int wave = threadIdx.x >> 6, c = threadIdx.x & 15, b4 = (threadIdx.x & 63) >> 4;
  const size_t row0 = static_cast<size_t>(b) * seqlen + static_cast<size_t>(chunk) * kChunk;
  const int live = seqlen - chunk * kChunk < kChunk ? seqlen - chunk * kChunk : kChunk;  // tokens past the end: beta 0, decay 1, q = k = 0
  if (threadIdx.x < 64) {
    const int t = threadIdx.x;
    float g = t < live ? p.log_g[(row0 + t) * H + h] : 0.f;
#pragma unroll
    for (int off = 1; off < 64; off <<= 1) {
      const float up = __shfl_up(g, off);
      if (t >= off) g += up;
    }
    sg[t] = g * kLog2e;
    sb[t] = t < live ? p.beta[(row0 + t) * H + h] : 0.f;
  }
  for (int i = threadIdx.x; i < kChunk * kRow; i += 256) si[i] = 0.f;
  // k k^T and q k^T for the column blocks up to this wave's
  f32x4_t kk[4], qk[4];
#pragma unroll
  for (int j = 0; j < 4; ++j) kk[j] = qk[j] = f32x4_t{0.f, 0.f, 0.f, 0.f};
  const size_t stride = static_cast<size_t>(kvh) * D;
  const float *kb = p.k + (row0 * kvh + hk) * D, *qb = p.q + (row0 * kvh + hk) * D;
  const int tr = 16 * wave + c;
  for (int d = 4 * b4; d < (D + 15) / 16 * 16; d += 16) {
    const f32x4_t ka = row4(kb + tr * stride, tr < live, d, D), qa = row4(qb + tr * stride, tr < live, d, D);
#pragma unroll
    for (int j = 0; j < 4; ++j) {
      if (j > wave) break;
      const f32x4_t kc = j == wave ? ka : row4(kb + (16 * j + c) * stride, 16 * j + c < live, d, D);
      kk[j] = mfma4(ka, kc, kk[j]);
      qk[j] = mfma4(qa, kc, qk[j]);
    }
  }
  __syncthreads();
  float *pt = cs.p + (static_cast<size_t>(bh) * cs.chunks + chunk) * kChunk * kChunk;
#pragma unroll
  for (int j = 0; j < 4; ++j) {
    if (j > wave) break;
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int t = 16 * wave + 4 * b4 + r, s = 16 * j + c;
      const float dec = s <= t ? __builtin_amdgcn_exp2f(sg[t] - sg[s]) : 0.f;
      sm[t * kRow + s] = s < t ? sb[t] * dec * kk[j][r] : 0.f;
      pt[t * kChunk + s] = dec * qk[j][r];
    }
  }
  __syncthreads();
  // inverse of the unit lower triangular diagonal blocks: wave w, lane c = column c of block w, substitution down the rows
  if (b4 == 0) {
    float x[16];
    const float *m = sm + (16 * wave) * kRow + 16 * wave;
#pragma unroll
    for (int t = 0; t < 16; ++t) {
      float v = t == c ? 1.f : 0.f;
#pragma unroll
      for (int s = 0; s < 16; ++s)
        if (s < t) v = __builtin_fmaf(-m[t * kRow + s], x[s], v);
      x[t] = v;
      si[(16 * wave + t) * kRow + 16 * wave + c] = v;
    }
  }
  __syncthreads();
  // blocks off the diagonal, by distance: I_ij = -I_ii sum_{j <= l < i} M_il I_lj
#pragma unroll
  for (int dist = 1; dist < 4; ++dist) {
    const int i = wave, j = wave - dist;
    f32x4_t acc = {0.f, 0.f, 0.f, 0.f};
    if (j >= 0) {
      for (int l = j; l < i; ++l) {
        f32x4_t bb;
#pragma unroll
        for (int r = 0; r < 4; ++r) bb[r] = si[(16 * l + 4 * b4 + r) * kRow + 16 * j + c];
        acc = mfma4(load4(sm + (16 * i + c) * kRow + 16 * l + 4 * b4), bb, acc);
      }
      const f32x4_t res = mfma4(load4(si + (16 * i + c) * kRow + 16 * i + 4 * b4), acc, f32x4_t{0.f, 0.f, 0.f, 0.f});
#pragma unroll
      for (int r = 0; r < 4; ++r) si[(16 * i + 4 * b4 + r) * kRow + 16 * j + c] = -res[r];
    }
    __syncthreads();
  }
  float *tt = cs.t + (static_cast<size_t>(bh) * cs.chunks + chunk) * kChunk * kChunk;
  for (int i = threadIdx.x; i < kChunk * kChunk; i += 256) {
    const int s = i & 63;
    tt[i] = si[(i >> 6) * kRow + s] * sb[s];
  }
}

// What one wave of the scan reads of a chunk: its 16 token rows of k, T and v, or of q and the decayed q k^T.  None of it
// depends on the state, so it is fetched a chunk ahead.
template <int DT>
struct ChunkRows {
  f32x4_t rows[DT], square[4], v;
  float log_g;
};

// step 2: DT = head dimension in tiles of 16.  Eight waves: wave w < 4 owns the token rows 16 w .. 16 w + 15 on the writing side
// (k, T, v: what u is made of), wave w + 4 the same rows on the reading side (q and the outputs); the state's row tiles w, w + 8
// are wave w's.  The state is kept twice: in accumulators by its owner, and in LDS, transposed, as the B operand of
// everybody's read-outs.  The keys go through LDS once to be read transposed in the state update.
// WHOLE: the head dimension fills its tiles, so no load needs a mask (rows past the end are read from the last token: their beta is
// 0, which keeps them out of u, and their outputs are not stored).
template <int DT, bool WHOLE>
__global__ __launch_bounds__(512) void delta_scan_kernel(const e2h_delta_args a, Prepared p, ChunkScratch cs, int v_blocks) {
  constexpr int DP = DT * 16, OWN = (DT + 7) / 8, kRow = DP + 4, kTok = 20;
  __shared__ __attribute__((aligned(16))) float st[16 * kRow];                         // state, [value column][row]
  __shared__ __attribute__((aligned(16))) float sk[kChunk * kRow];                     // keys, [token][channel]
  __shared__ __attribute__((aligned(16))) float sx[kChunk * kTok], su[kChunk * kTok];  // [token][value column]
  __shared__ float sg[2][kChunk];
  const int D = static_cast<int>(a.dim), DV = static_cast<int>(a.vdim), H = static_cast<int>(a.heads), kvh = static_cast<int>(a.kv_heads);
  const int seqlen = static_cast<int>(a.seqlen), bh_count = static_cast<int>(a.batch) * H;
  // the value blocks of one head read the same keys and queries: keep them on one die (workgroups go round robin over 8)
  int bh, vb;
  const int whole = bh_count / 8 * 8 * v_blocks;
  if (static_cast<int>(blockIdx.x) < whole) {
    const int die = blockIdx.x & 7, i = blockIdx.x >> 3;
    bh = (i / v_blocks) * 8 + die;
    vb = i % v_blocks;
  } else {
    bh = bh_count / 8 * 8 + (blockIdx.x - whole) / v_blocks;
    vb = (blockIdx.x - whole) % v_blocks;
  }
  const int b = bh / H, h = bh % H, hk = h / (H / kvh);
  const int wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6), c = threadIdx.x & 15, b4 = (threadIdx.x & 63) >> 4;
  const bool reader = wave >= 4;
  const int block = wave & 3;  // of 16 tokens
  const int col = vb * 16 + c;
  const bool col_ok = col < DV;
  float *state = a.state + static_cast<size_t>(bh) * D * DV;
  const bool carried = a.input_pos[0] > 0;
  f32x4_t s[OWN];
#pragma unroll
  for (int i = 0; i < OWN; ++i) {
    const int dt = wave + 8 * i;
    s[i] = f32x4_t{0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int d = dt * 16 + 4 * b4 + r;
      if (carried && d < D && col_ok) s[i][r] = state[static_cast<size_t>(d) * DV + col];
    }
    if (dt < DT) store4(st + c * kRow + dt * 16 + 4 * b4, s[i]);
  }
  const size_t stride = static_cast<size_t>(kvh) * D;
  const int tr = 16 * block + c;
  const size_t seq0 = static_cast<size_t>(b) * seqlen;
  const float *squares = (reader ? cs.p : cs.t) + static_cast<size_t>(bh) * cs.chunks * kChunk * kChunk;
  const float *vectors = reader ? p.q : p.k;

  auto fetch = [&](int chunk, ChunkRows<DT> &x) {
    const size_t row0 = seq0 + static_cast<size_t>(chunk) * kChunk;
    const int live = seqlen - chunk * kChunk < kChunk ? seqlen - chunk * kChunk : kChunk;
    const float *mine = vectors + ((row0 + (tr < live ? tr : live - 1)) * kvh + hk) * D;
#pragma unroll
    for (int dt = 0; dt < DT; ++dt) x.rows[dt] = WHOLE ? load4(mine + dt * 16 + 4 * b4) : row4(mine, true, dt * 16 + 4 * b4, D);
    const float *sq = squares + static_cast<size_t>(chunk) * kChunk * kChunk + tr * kChunk + 4 * b4;
#pragma unroll
    for (int j = 0; j < 4; ++j)
      if (j <= block) x.square[j] = load4(sq + 16 * j);
    if (!reader) {
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int t = 16 * block + 4 * b4 + r;
        x.v[r] = p.v[((row0 + (t < live ? t : live - 1)) * H + h) * DV + (col_ok ? col : 0)];
      }
    }
    if (wave == 0) x.log_g = p.log_g[(row0 + (static_cast<int>(threadIdx.x) < live ? threadIdx.x : live - 1)) * H + h];
  };

  ChunkRows<DT> cur, next;
  fetch(0, cur);
  for (int chunk = 0; chunk < cs.chunks; ++chunk) {
    const int live = seqlen - chunk * kChunk < kChunk ? seqlen - chunk * kChunk : kChunk;
    float *g = sg[chunk & 1];
    if (wave == 0) {
      float x = static_cast<int>(threadIdx.x) < live ? cur.log_g : 0.f;
#pragma unroll
      for (int off = 1; off < 64; off <<= 1) {
        const float up = __shfl_up(x, off);
        if (static_cast<int>(threadIdx.x) >= off) x += up;
      }
      g[threadIdx.x] = x * kLog2e;
    }
    if (!reader) {
#pragma unroll
      for (int dt = 0; dt < DT; ++dt) store4(sk + tr * kRow + dt * 16 + 4 * b4, cur.rows[dt]);
    }
    if (chunk + 1 < cs.chunks) fetch(chunk + 1, next);
    lds_barrier();  // state, keys and decays of this chunk are in LDS; the loads above stay in flight
    f32x4_t y = {0.f, 0.f, 0.f, 0.f}, gt;  // S0^T k or S0^T q, decayed to each token
#pragma unroll
    for (int dt = 0; dt < DT; ++dt) y = mfma4(cur.rows[dt], load4(st + c * kRow + dt * 16 + 4 * b4), y);
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      gt[r] = __builtin_amdgcn_exp2f(g[16 * block + 4 * b4 + r]);
      y[r] *= gt[r];
      if (!reader) sx[(16 * block + 4 * b4 + r) * kTok + c] = cur.v[r] - y[r];
    }
    lds_barrier();
    if (!reader) {
      f32x4_t u = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int j = 0; j < 4; ++j) {
        if (j > block) break;
        f32x4_t x;
#pragma unroll
        for (int r = 0; r < 4; ++r) x[r] = sx[(16 * j + 4 * b4 + r) * kTok + c];
        u = mfma4(cur.square[j], x, u);
      }
#pragma unroll
      for (int r = 0; r < 4; ++r) su[(16 * block + 4 * b4 + r) * kTok + c] = u[r];
    }
    lds_barrier();
    f32x4_t ub[4];
#pragma unroll
    for (int j = 0; j < 4; ++j) {
#pragma unroll
      for (int r = 0; r < 4; ++r) ub[j][r] = su[(16 * j + 4 * b4 + r) * kTok + c];
      if (reader && j <= block) y = mfma4(cur.square[j], ub[j], y);
    }
    if (reader) {
#pragma unroll
      for (int r = 0; r < 4; ++r) {  // over the values this workgroup has read
        const int t = 16 * block + 4 * b4 + r;
        if (t < live && col_ok) p.v[((seq0 + static_cast<size_t>(chunk) * kChunk + t) * H + h) * DV + col] = y[r];
      }
    }
    const float g_end = g[kChunk - 1], dec = __builtin_amdgcn_exp2f(g_end);
#pragma unroll
    for (int j = 0; j < 4; ++j)
#pragma unroll
      for (int r = 0; r < 4; ++r) ub[j][r] *= __builtin_amdgcn_exp2f(g_end - g[16 * j + 4 * b4 + r]);
#pragma unroll
    for (int i = 0; i < OWN; ++i) {
      if (wave + 8 * i >= DT) break;
#pragma unroll
      for (int r = 0; r < 4; ++r) s[i][r] *= dec;
#pragma unroll
      for (int j = 0; j < 4; ++j) {
        f32x4_t kt;
#pragma unroll
        for (int r = 0; r < 4; ++r) kt[r] = sk[(16 * j + 4 * b4 + r) * kRow + (wave + 8 * i) * 16 + c];
        s[i] = mfma4(kt, ub[j], s[i]);
      }
      store4(st + c * kRow + (wave + 8 * i) * 16 + 4 * b4, s[i]);
    }
    lds_barrier();  // the keys have been read; the next chunk's take their place
    cur = next;
  }
#pragma unroll
  for (int i = 0; i < OWN; ++i)
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int d = (wave + 8 * i) * 16 + 4 * b4 + r;
      if (d < D && col_ok) state[static_cast<size_t>(d) * DV + col] = s[i][r];
    }
}

// step 3: `cp` lanes per (token, head), four columns each; the read-outs stand where the values were
template <typename T>
__global__ __launch_bounds__(256) void delta_gate_kernel(const e2h_delta_args a, Prepared p, int cp) {
  const int64_t item = (static_cast<int64_t>(blockIdx.x) * 256 + threadIdx.x) / cp;
  const int d = static_cast<int>(threadIdx.x & (cp - 1)) * 4, DV = static_cast<int>(a.vdim), H = static_cast<int>(a.heads);
  const bool mine = d < DV && item < a.batch * a.seqlen * H;
  const int64_t row = mine ? item / H : 0;
  const int h = mine ? static_cast<int>(item % H) : 0, dc = mine ? d : 0;
  const f32x4_t o = load4(p.v + (row * H + h) * DV + dc), w = load4(a.norm_weight + dc);
  const f32x4_t gate = load4(static_cast<const T *>(a.proj) + row * a.ld + a.g_off + static_cast<int64_t>(h) * DV + dc);
  float ss = mine ? o[0] * o[0] + o[1] * o[1] + o[2] * o[2] + o[3] * o[3] : 0.f;
  for (int off = 1; off < cp; off <<= 1) ss += __shfl_xor(ss, off);
  const float inv = a.out_scale / sqrtf(ss / static_cast<float>(DV) + a.eps);
  if (!mine) return;
  f32x4_t y;
#pragma unroll
  for (int e = 0; e < 4; ++e) y[e] = o[e] * inv * w[e] * fast_silu(gate[e]);
  store4(static_cast<T *>(a.out) + row * a.ld_out + a.out_off + static_cast<int64_t>(h) * DV + d, y);
}

int lanes_for(int64_t values) {  // power of two, four values per lane
  int cp = 1;
  while (cp * 4 < values) cp *= 2;
  return cp;
}

// four channels per access everywhere
bool quads_ok(const e2h_delta_args &a) {
  return a.dim % 4 == 0 && a.ld % 4 == 0 && a.q_off % 4 == 0 && a.k_off % 4 == 0 && a.v_off % 4 == 0 && a.g_off % 4 == 0 && a.ld_out % 4 == 0 &&
         a.out_off % 4 == 0 && aligned16(a.proj) && aligned16(a.tail_in) && aligned16(a.tail_out) && aligned16(a.out) && aligned16(a.norm_weight);
}

bool use_chunks(const e2h_delta_args &a) {
  if (a.seqlen == 1 || seq_options().recurrence_form == 1 || !quads_ok(a)) return false;
  return seq_options().recurrence_form == 2 || a.seqlen >= 24;
}

template <int DT>
void launch_scan(const e2h_delta_args &a, const Prepared &p, const ChunkScratch &cs, hipStream_t s) {
  const int v_blocks = static_cast<int>((a.vdim + 15) / 16);
  const dim3 grid(static_cast<unsigned>(a.batch * a.heads * v_blocks)), block(512);
  if (a.dim == DT * 16) hipLaunchKernelGGL((delta_scan_kernel<DT, true>), grid, block, 0, s, a, p, cs, v_blocks);
  else hipLaunchKernelGGL((delta_scan_kernel<DT, false>), grid, block, 0, s, a, p, cs, v_blocks);
}

template <typename T>
void launch_chunks(const e2h_delta_args &a, const Prepared &p, const ChunkScratch &cs, hipStream_t s) {
  const dim3 grid(static_cast<unsigned>(a.batch * a.heads * cs.chunks)), block(256);
  hipLaunchKernelGGL(delta_chunk_kernel, grid, block, 0, s, a, p, cs);
  if (a.dim <= 64) launch_scan<4>(a, p, cs, s);
  else if (a.dim <= 128) launch_scan<8>(a, p, cs, s);
  else launch_scan<16>(a, p, cs, s);
  const int cp = lanes_for(a.vdim);
  hipLaunchKernelGGL(delta_gate_kernel<T>, dim3(static_cast<unsigned>((a.batch * a.seqlen * a.heads * cp + 255) / 256)), block, 0, s, a, p, cp);
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
int64_t carve(const e2h_delta_args &a, Prepared *p, ChunkScratch *cs) {
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
  const int64_t prepared = 2 * qk + v + 2 * g;
  if (!use_chunks(a)) return prepared;
  const int64_t chunks = (a.seqlen + kChunk - 1) / kChunk, squares = a.batch * a.heads * chunks * kChunk * kChunk * 4;
  if (cs) {
    cs->t = reinterpret_cast<float *>(static_cast<uint8_t *>(a.scratch) + prepared);
    cs->p = reinterpret_cast<float *>(static_cast<uint8_t *>(a.scratch) + prepared + squares);
    cs->chunks = static_cast<int>(chunks);
  }
  return prepared + 2 * squares;
}

template <typename T>
int launch_delta(const e2h_delta_args &a, hipStream_t s) {
  Prepared p = {};
  if (a.seqlen == 1) {
    launch_tokens<T, true>(a, p, s);
    return launch_status();
  }
  ChunkScratch cs = {};
  carve(a, &p, &cs);
  if (a.taps <= 4 && quads_ok(a)) {
    const int cp = lanes_for(a.dim > a.vdim ? a.dim : a.vdim), runs = static_cast<int>((a.seqlen + kPrepareRun - 1) / kPrepareRun);
    const int64_t waves = a.batch * runs * ((2 * a.kv_heads + a.heads + 64 / cp - 1) / (64 / cp));
    hipLaunchKernelGGL(delta_prepare4_kernel<T>, dim3(static_cast<unsigned>((waves + 3) / 4)), dim3(256), 0, s, a, p, cp, runs);
    hipLaunchKernelGGL(delta_gates_kernel<T>, dim3(static_cast<unsigned>((a.batch * a.seqlen * a.heads + 255) / 256)), dim3(256), 0, s, a, p);
  } else {
    const int64_t items = a.batch * a.seqlen * (2 * a.kv_heads + a.heads + 1);
    hipLaunchKernelGGL(delta_prepare_kernel<T>, dim3(static_cast<unsigned>((items + 3) / 4)), dim3(256), 0, s, a, p);
  }
  if (use_chunks(a)) launch_chunks<T>(a, p, cs, s);
  else launch_tokens<T, false>(a, p, s);
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
  return a.batch * a.heads * ((a.seqlen + kChunk - 1) / kChunk) <= INT32_MAX && a.batch * a.heads * ((a.vdim + 15) / 16) <= INT32_MAX &&
         a.batch * a.seqlen * (2 * a.kv_heads + a.heads + 1) / 4 < INT32_MAX &&
         2 * a.kv_heads * a.dim + a.heads * a.vdim <= INT32_MAX;
}

}  // namespace
}  // namespace e2h

using namespace e2h;

extern "C" int64_t e2h_seq_delta_scratch_bytes(const e2h_delta_args *a) {
  if (!a) return E2H_ERR_NULL_POINTER;
  if (!shape_ok(*a)) return E2H_ERR_BAD_SHAPE;
  return carve(*a, nullptr, nullptr);
}

extern "C" int e2h_seq_delta(const e2h_delta_args *a, void *stream) {
  if (!a || !a->proj || !a->conv || !a->a_log || !a->dt_bias || !a->norm_weight || !a->state || !a->input_pos || !a->out) return E2H_ERR_NULL_POINTER;
  if (!shape_ok(*a)) return E2H_ERR_BAD_SHAPE;
  if (a->taps > 1 && (!a->tail_in || !a->tail_out)) return E2H_ERR_NULL_POINTER;
  if (a->taps > 1 && a->seqlen > 1 && a->tail_in == a->tail_out) return E2H_ERR_BAD_SHAPE;
  if (!aligned16(a->state) || !aligned16(a->scratch)) return E2H_ERR_MISALIGNED;
  const int64_t need = carve(*a, nullptr, nullptr);
  if (need > 0 && !a->scratch) return E2H_ERR_NULL_POINTER;
  if (need > a->scratch_bytes) return E2H_ERR_SCRATCH_TOO_SMALL;
  if (a->dtype == E2H_SEQ_BF16) return launch_delta<bf16_t>(*a, static_cast<hipStream_t>(stream));
  return launch_delta<float>(*a, static_cast<hipStream_t>(stream));
}
