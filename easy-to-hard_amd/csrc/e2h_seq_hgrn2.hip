// HGRN2 linear attention (e2h_seq_hgrn2): S = diag(f) S + (1 - f) v^T per head, o = S^T q, RMS norm over the head.
//
// Token-by-token form: one workgroup per (sequence, head) keeps the head's whole state in registers (a thread owns four value
// columns and every RG-th row), reads it once and writes it once per call.
//
// Chunked form (many tokens), float32 matrix cores throughout (v_mfma_f32_16x16x4_f32): three launches,
//   1. per chunk: what the chunk adds to the state, and its total decay           (parallel over chunks)
//   2. per state element: the state at every chunk's start                         (a scan over chunks)
//   3. per chunk: from that state, blocks of 16 tokens one after the other: read-out of the state, products among the
//      block's own tokens, state update.
// The state lives in accumulator registers: element r of lane (b, c) is row 4 b + r, column c of a 16 x 16 tile, which is
// also the layout of the B operand when step r of a product over 16 rows takes rows {4 b + r}.
// Decays are kept as base-2 logarithms summed from the block's start.  Every factor used is a decay from an earlier to a
// later token, so no exponent is positive: for the products among the block's tokens, tokens t > s whose highest differing
// index bit is l are tied to the last token m of the lower half of their common 2^(l+1)-block, decay(s -> t) =
// decay(s -> m) decay(m -> t), one matrix product per l and one for t = s.
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
  __shared__ float sh_q[kMaxDim], sh_k[kMaxDim];
  __shared__ Decay sh_f[kMaxDim];
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
    if (pos0 > 0 && col_ok && r < D) s[i] = load4_stream(st + static_cast<size_t>(r) * DV + cg * 4);
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
      sh_f[i] = live ? decay_of(g.f, g.k) : Decay{0.f, 1.f};
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
        const Decay f = sh_f[r];
        const float k = sh_k[r], q = sh_q[r];
#pragma unroll
        for (int e = 0; e < 4; ++e) {
          s[i][e] = __builtin_fmaf(k, v[e], decayed(f, s[i][e]));
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
    if (col_ok && r < D) store4_stream(st + static_cast<size_t>(r) * DV + cg * 4, s[i]);
  }
}

// ---- chunked form ----------------------------------------------------------------------------------------------------------
constexpr int kBlockTokens = 16;
struct ChunkPlan {
  float *delta;  // [chunks, batch * heads, dim, vdim]: a chunk's contribution, then the state at its start
  float *decay;  // [chunks, batch * heads, dim]
  int chunks, tokens;  // tokens per chunk
};

// A block's projections on their way into LDS (rows of DP + 4 / VP + 4 floats).  `fetch` issues the loads, one block ahead of
// `commit`, which turns them into queries, keys and base-2 log decays summed over the block.  Tokens past the end and
// padding tokens become ones that leave the state alone.  NT threads; a thread's channels are the same in every block.
template <typename T, int DP, int VP, int NT, bool QUERIES>
struct BlockLoader {
  static constexpr int kQuads = kBlockTokens * DP / 4 / NT, kVQuads = kBlockTokens * VP / 4 / NT;
  static_assert(kQuads * NT * 4 == kBlockTokens * DP && kVQuads * NT * 4 == kBlockTokens * VP && NT % (DP / 4) == 0 && NT % (VP / 4) == 0);
  Quad<T> q[kQuads], f[kQuads], v[kVQuads];
  f32x4_t bias, low;
  const T *src;  // the sequence's first row
  int64_t ld;
  int d, vd, seqlen, dim, vdim;

  __device__ __forceinline__ BlockLoader(const e2h_hgrn2_args &a, size_t row0, int h) {
    d = static_cast<int>(threadIdx.x % (DP / 4)) * 4;
    vd = static_cast<int>(threadIdx.x % (VP / 4)) * 4;
    dim = static_cast<int>(a.dim);
    vdim = static_cast<int>(a.vdim);
    seqlen = static_cast<int>(a.seqlen);
    ld = a.ld;
    src = static_cast<const T *>(a.proj) + row0 * a.ld;
    const int ch = h * dim + (d < dim ? d : 0);
    bias = load4(a.f_bias + ch);
    low = load4(a.lower + ch);
    q_col = a.q_off + ch;
    f_col = a.f_off + ch;
    v_col = a.v_off + static_cast<int64_t>(h) * vdim + (vd < vdim ? vd : 0);
  }
  int64_t q_col, f_col, v_col;

  __device__ __forceinline__ void fetch(int t0) {
#pragma unroll
    for (int i = 0; i < kQuads; ++i) {
      const int t = t0 + static_cast<int>(threadIdx.x / (DP / 4)) + i * (NT / (DP / 4));
      const T *row = src + static_cast<int64_t>(t < seqlen ? t : seqlen - 1) * ld;
      if (QUERIES) q[i] = load_quad(row + q_col);
      f[i] = load_quad(row + f_col);
    }
#pragma unroll
    for (int i = 0; i < kVQuads; ++i) {
      const int t = t0 + static_cast<int>(threadIdx.x / (VP / 4)) + i * (NT / (VP / 4));
      v[i] = load_quad(src + static_cast<int64_t>(t < seqlen ? t : seqlen - 1) * ld + v_col);
    }
  }

  __device__ __forceinline__ void commit(int t0, int64_t pos0, int64_t first, float *sq, float *sk, float *sc, float *sv) {
    const f32x4_t zero = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int i = 0; i < kQuads; ++i) {
      const int t = static_cast<int>(threadIdx.x / (DP / 4)) + i * (NT / (DP / 4));
      const bool there = d < dim && t0 + t < seqlen, live = there && pos0 + t0 + t >= first;
      f32x4_t qv = zero, kv = zero, lg = zero;
      const f32x4_t fz = f[i].f32() + bias;
#pragma unroll
      for (int e = 0; e < 4; ++e) {
        const float up = 1.0f - low[e], sn = fast_sigmoid(-fz[e]);
        kv[e] = up * sn;
        lg[e] = log2_one_minus(kv[e], __builtin_fmaf(up, fast_sigmoid(fz[e]), low[e]));
      }
      if (QUERIES) {
        qv = q[i].f32();
#pragma unroll
        for (int e = 0; e < 4; ++e) qv[e] = fast_silu(qv[e]);
        store4(sq + t * (DP + 4) + d, there ? qv : zero);
      }
      store4(sk + t * (DP + 4) + d, live ? kv : zero);
      store4(sc + t * (DP + 4) + d, live ? lg : zero);
    }
#pragma unroll
    for (int i = 0; i < kVQuads; ++i) {
      const int t = static_cast<int>(threadIdx.x / (VP / 4)) + i * (NT / (VP / 4));
      store4(sv + t * (VP + 4) + vd, vd < vdim && t0 + t < seqlen ? v[i].f32() : zero);
    }
    __syncthreads();
    if (threadIdx.x < DP) {
      float c[kBlockTokens];
#pragma unroll
      for (int t = 0; t < kBlockTokens; ++t) c[t] = sc[t * (DP + 4) + threadIdx.x];
#pragma unroll
      for (int t = 1; t < kBlockTokens; ++t) c[t] += c[t - 1];
#pragma unroll
      for (int t = 0; t < kBlockTokens; ++t) sc[t * (DP + 4) + threadIdx.x] = c[t];
    }
    __syncthreads();
  }
};

// S = decay of the block * S + k~^T V, k~ the keys decayed to the block's end (in sk)
template <int DT, int VTW, int DP, int VP>
__device__ __forceinline__ void update_state(const float *sk, const float *sc, const float *sv, int vt0, f32x4_t (&s)[DT][VTW]) {
  const int c = threadIdx.x & 15, b4 = (threadIdx.x & 63) >> 4;
  f32x4_t vb[VTW];
#pragma unroll
  for (int v = 0; v < VTW; ++v)
#pragma unroll
    for (int r = 0; r < 4; ++r) vb[v][r] = sv[(4 * b4 + r) * (VP + 4) + (vt0 + v) * 16 + c];
#pragma unroll
  for (int dt = 0; dt < DT; ++dt) {
    f32x4_t ka;
    const f32x4_t e = load4(sc + (kBlockTokens - 1) * (DP + 4) + dt * 16 + 4 * b4);
#pragma unroll
    for (int r = 0; r < 4; ++r) ka[r] = sk[(4 * b4 + r) * (DP + 4) + dt * 16 + c];
    f32x4_t dec;
#pragma unroll
    for (int r = 0; r < 4; ++r) dec[r] = __builtin_amdgcn_exp2f(e[r]);
#pragma unroll
    for (int v = 0; v < VTW; ++v) {
#pragma unroll
      for (int r = 0; r < 4; ++r) s[dt][v][r] *= dec[r];
      s[dt][v] = mfma4(ka, vb[v], s[dt][v]);
    }
  }
}

// step 1
template <typename T, int DT, int VTW, int NW>
__global__ __launch_bounds__(64 * NW) void hgrn2_chunk_state_kernel(const e2h_hgrn2_args a, ChunkPlan plan) {
  constexpr int DP = DT * 16, VP = VTW * NW * 16, NT = 64 * NW;
  __shared__ __attribute__((aligned(16))) float sk[kBlockTokens * (DP + 4)], sc[kBlockTokens * (DP + 4)], sv[kBlockTokens * (VP + 4)];
  const int D = static_cast<int>(a.dim), DV = static_cast<int>(a.vdim);
  const int bh_count = static_cast<int>(a.batch * a.heads);
  const int bh = blockIdx.x % bh_count, chunk = blockIdx.x / bh_count;
  const int b = bh / static_cast<int>(a.heads), h = bh % static_cast<int>(a.heads);
  const int64_t pos0 = a.input_pos[0], first = a.first ? a.first[b] : 0;
  const size_t row0 = static_cast<size_t>(b) * a.seqlen;
  const int c = threadIdx.x & 15, b4 = (threadIdx.x & 63) >> 4, vt0 = (threadIdx.x >> 6) * VTW;
  f32x4_t s[DT][VTW];
#pragma unroll
  for (int dt = 0; dt < DT; ++dt)
#pragma unroll
    for (int v = 0; v < VTW; ++v) s[dt][v] = f32x4_t{0.f, 0.f, 0.f, 0.f};
  float total[(DP + NT - 1) / NT] = {};
  BlockLoader<T, DP, VP, NT, false> loader(a, row0, h);
  loader.fetch(chunk * plan.tokens);
  for (int t0 = chunk * plan.tokens; t0 < (chunk + 1) * plan.tokens; t0 += kBlockTokens) {  // all chunks but the last are whole
    loader.commit(t0, pos0, first, nullptr, sk, sc, sv);
    loader.fetch(t0 + kBlockTokens);
    for (int i = threadIdx.x; i < kBlockTokens * DP; i += NT) {
      const int t = i / DP, d = i % DP;
      sk[t * (DP + 4) + d] *= __builtin_amdgcn_exp2f(sc[(kBlockTokens - 1) * (DP + 4) + d] - sc[t * (DP + 4) + d]);
    }
#pragma unroll
    for (int i = 0; i < (DP + NT - 1) / NT; ++i)
      if (threadIdx.x + i * NT < DP) total[i] += sc[(kBlockTokens - 1) * (DP + 4) + threadIdx.x + i * NT];
    __syncthreads();
    update_state<DT, VTW, DP, VP>(sk, sc, sv, vt0, s);
    __syncthreads();
  }
  float *dst = plan.delta + (static_cast<size_t>(chunk) * bh_count + bh) * D * DV;
#pragma unroll
  for (int dt = 0; dt < DT; ++dt)
#pragma unroll
    for (int v = 0; v < VTW; ++v)
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int d = dt * 16 + 4 * b4 + r, col = (vt0 + v) * 16 + c;
        if (d < D && col < DV) dst[static_cast<size_t>(d) * DV + col] = s[dt][v][r];
      }
#pragma unroll
  for (int i = 0; i < (DP + NT - 1) / NT; ++i) {
    const int d = threadIdx.x + i * NT;
    if (d < D) plan.decay[(static_cast<size_t>(chunk) * bh_count + bh) * D + d] = __builtin_amdgcn_exp2f(total[i]);
  }
}

// step 2: four neighbouring value columns per thread
__global__ __launch_bounds__(256) void hgrn2_scan_kernel(const e2h_hgrn2_args a, ChunkPlan plan) {
  const int64_t quads = a.batch * a.heads * a.dim * a.vdim / 4;
  const int64_t i = static_cast<int64_t>(blockIdx.x) * 256 + threadIdx.x;
  if (i >= quads) return;
  const int64_t row = i * 4 / a.vdim, rows = a.batch * a.heads * a.dim;  // (sequence, head, channel)
  f32x4_t s = {0.f, 0.f, 0.f, 0.f};
  if (a.input_pos[0] > 0) s = load4(a.state + i * 4);
  f32x4_t d = load4(plan.delta + i * 4);
  float g = plan.decay[row];
  for (int c = 0; c < plan.chunks; ++c) {
    const f32x4_t d0 = d;
    const float g0 = g;
    if (c + 1 < plan.chunks) {
      d = load4(plan.delta + (static_cast<size_t>(c + 1) * quads + i) * 4);
      g = plan.decay[static_cast<size_t>(c + 1) * rows + row];
    }
    store4(plan.delta + (static_cast<size_t>(c) * quads + i) * 4, s);
#pragma unroll
    for (int e = 0; e < 4; ++e) s[e] = __builtin_fmaf(g0, s[e], d0[e]);
  }
  // the last chunk's own contribution comes from step 3, which starts from the state stored above
}

// step 3
template <typename T, int DT, int VTW, int NW>
__global__ __launch_bounds__(64 * NW) void hgrn2_chunk_output_kernel(const e2h_hgrn2_args a, ChunkPlan plan) {
  constexpr int DP = DT * 16, VP = VTW * NW * 16, NT = 64 * NW;
  constexpr int kLevels = 5;
  __shared__ __attribute__((aligned(16))) float sq[kBlockTokens * (DP + 4)], sk[kBlockTokens * (DP + 4)], sc[kBlockTokens * (DP + 4)];
  __shared__ __attribute__((aligned(16))) float sv[kBlockTokens * (VP + 4)], sqd[kBlockTokens * (DP + 4)];
  __shared__ __attribute__((aligned(16))) float sa[16 * 20], spart[NW][16 * 17], snorm[NW][16];
  const int D = static_cast<int>(a.dim), DV = static_cast<int>(a.vdim), seqlen = static_cast<int>(a.seqlen);
  const int bh_count = static_cast<int>(a.batch * a.heads);
  const int bh = blockIdx.x % bh_count, chunk = blockIdx.x / bh_count;
  const int b = bh / static_cast<int>(a.heads), h = bh % static_cast<int>(a.heads);
  const int64_t pos0 = a.input_pos[0], first = a.first ? a.first[b] : 0;
  const size_t row0 = static_cast<size_t>(b) * a.seqlen;
  const int wave = threadIdx.x >> 6, c = threadIdx.x & 15, b4 = (threadIdx.x & 63) >> 4, vt0 = wave * VTW;
  float *state = a.state + static_cast<size_t>(bh) * D * DV;
  const float *src = plan.chunks > 1 ? plan.delta + (static_cast<size_t>(chunk) * bh_count + bh) * D * DV : state;
  const bool empty = plan.chunks == 1 && pos0 <= 0;
  f32x4_t s[DT][VTW];
#pragma unroll
  for (int dt = 0; dt < DT; ++dt)
#pragma unroll
    for (int v = 0; v < VTW; ++v)
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int d = dt * 16 + 4 * b4 + r, col = (vt0 + v) * 16 + c;
        s[dt][v][r] = !empty && d < D && col < DV ? src[static_cast<size_t>(d) * DV + col] : 0.f;
      }
  float w[VTW];
#pragma unroll
  for (int v = 0; v < VTW; ++v) w[v] = (vt0 + v) * 16 + c < DV ? a.norm_weight[(vt0 + v) * 16 + c] * a.out_scale : 0.f;

  BlockLoader<T, DP, VP, NT, true> loader(a, row0, h);
  loader.fetch(chunk * plan.tokens);
  const int t_end = (chunk + 1) * plan.tokens < seqlen ? (chunk + 1) * plan.tokens : seqlen;
  for (int t0 = chunk * plan.tokens; t0 < t_end; t0 += kBlockTokens) {
    loader.commit(t0, pos0, first, sq, sk, sc, sv);
    loader.fetch(t0 + kBlockTokens);
    // products among the block's tokens: this wave's share of the channels, one accumulator per level
    f32x4_t lev[kLevels];
#pragma unroll
    for (int l = 0; l < kLevels; ++l) lev[l] = f32x4_t{0.f, 0.f, 0.f, 0.f};
    for (int dt = wave; dt < DT; dt += NW) {
      const int o = dt * 16 + 4 * b4;
      const f32x4_t q = load4(sq + c * (DP + 4) + o), k = load4(sk + c * (DP + 4) + o), cc = load4(sc + c * (DP + 4) + o);
      lev[0] = mfma4(q, k, lev[0]);
#pragma unroll
      for (int l = 0; l < 4; ++l) {
        const int m = (c & ~((2 << l) - 1)) + (1 << l) - 1;
        const f32x4_t cm = load4(sc + m * (DP + 4) + o);
        const bool upper = (c >> l) & 1;  // upper half: only its query factor is used; lower half: only its key factor
        f32x4_t f;
#pragma unroll
        for (int e = 0; e < 4; ++e) f[e] = __builtin_amdgcn_exp2f(upper ? cc[e] - cm[e] : cm[e] - cc[e]);
        lev[l + 1] = mfma4(q * f, k * f, lev[l + 1]);
      }
    }
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int t = 4 * b4 + r;  // row; column (earlier token) c
      float v = 0.f;
      if (t == c) v = lev[0][r];
#pragma unroll
      for (int l = 0; l < 4; ++l)
        if (t > c && ((t ^ c) >> l) == 1) v = lev[l + 1][r];
      spart[wave][t * 17 + c] = v;
    }
    for (int i = threadIdx.x; i < kBlockTokens * DP; i += NT) {
      const int t = i / DP, d = i % DP;
      sqd[t * (DP + 4) + d] = sq[t * (DP + 4) + d] * __builtin_amdgcn_exp2f(sc[t * (DP + 4) + d]);
    }
    __syncthreads();
    for (int i = threadIdx.x; i < kBlockTokens * DP; i += NT) {
      const int t = i / DP, d = i % DP;
      sk[t * (DP + 4) + d] *= __builtin_amdgcn_exp2f(sc[(kBlockTokens - 1) * (DP + 4) + d] - sc[t * (DP + 4) + d]);
    }
    if (threadIdx.x < 256) {
      const int t = threadIdx.x >> 4, u = threadIdx.x & 15;
      float v = 0.f;
#pragma unroll
      for (int x = 0; x < NW; ++x) v += spart[x][t * 17 + u];
      sa[t * 20 + u] = v;
    }
    __syncthreads();
    // read-out: q~ S + A V
    f32x4_t o[VTW];
#pragma unroll
    for (int v = 0; v < VTW; ++v) {
      f32x4_t vb;
#pragma unroll
      for (int r = 0; r < 4; ++r) vb[r] = sv[(4 * b4 + r) * (VP + 4) + (vt0 + v) * 16 + c];
      o[v] = mfma4(load4(sa + c * 20 + 4 * b4), vb, f32x4_t{0.f, 0.f, 0.f, 0.f});
    }
#pragma unroll
    for (int dt = 0; dt < DT; ++dt) {
      const f32x4_t q = load4(sqd + c * (DP + 4) + dt * 16 + 4 * b4);
#pragma unroll
      for (int v = 0; v < VTW; ++v) o[v] = mfma4(q, s[dt][v], o[v]);
    }
    update_state<DT, VTW, DP, VP>(sk, sc, sv, vt0, s);
    // RMS over the head's value columns, which are spread over lanes and waves
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      float ss = 0.f;
#pragma unroll
      for (int v = 0; v < VTW; ++v) ss = __builtin_fmaf(o[v][r], o[v][r], ss);
#pragma unroll
      for (int off = 1; off < 16; off <<= 1) ss += __shfl_xor(ss, off);
      if (c == 0) snorm[wave][4 * b4 + r] = ss;
    }
    __syncthreads();
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int t = 4 * b4 + r;
      float ss = 0.f;
#pragma unroll
      for (int x = 0; x < NW; ++x) ss += snorm[x][t];
      const float inv = 1.0f / sqrtf(ss / static_cast<float>(DV) + a.eps);
      if (t0 + t < seqlen) {
        const int64_t base = static_cast<int64_t>(row0 + t0 + t) * a.ld_out + a.out_off + static_cast<int64_t>(h) * DV;
#pragma unroll
        for (int v = 0; v < VTW; ++v) {
          const int col = (vt0 + v) * 16 + c;
          if (col < DV) {
            const float y = o[v][r] * inv * w[v];
            static_cast<T *>(a.out)[base + col] = from_f32<T>(y);
          }
        }
      }
    }
  }
  if (chunk == plan.chunks - 1) {  // no other workgroup of this head reads the state: with several chunks they start from step 2's copy
#pragma unroll
    for (int dt = 0; dt < DT; ++dt)
#pragma unroll
      for (int v = 0; v < VTW; ++v)
#pragma unroll
        for (int r = 0; r < 4; ++r) {
          const int d = dt * 16 + 4 * b4 + r, col = (vt0 + v) * 16 + c;
          if (d < D && col < DV) state[static_cast<size_t>(d) * DV + col] = s[dt][v][r];
        }
  }
}

// Tokens per chunk: whole blocks, enough chunks to fill the chip, and no more than that (every chunk boundary costs a state)
ChunkPlan plan_chunks(const e2h_hgrn2_args &a) {
  ChunkPlan p = {};
  int64_t tokens = seq_options().recurrence_chunk;
  if (!tokens) {
    tokens = a.batch * a.heads * a.seqlen / 1024 / kBlockTokens * kBlockTokens;
    tokens = tokens < 64 ? 64 : tokens > 512 ? 512 : tokens;
  }
  p.tokens = static_cast<int>(tokens);
  p.chunks = static_cast<int>((a.seqlen + tokens - 1) / tokens);
  return p;
}

bool use_chunks(const e2h_hgrn2_args &a) {
  if (seq_options().recurrence_form == 1) return false;
  if (a.dim % 4 != 0 || a.ld % 4 != 0 || a.q_off % 4 != 0 || a.f_off % 4 != 0 || a.v_off % 4 != 0) return false;  // four channels per load
  return seq_options().recurrence_form == 2 ? a.seqlen > 1 : a.seqlen >= 24;
}

int64_t delta_bytes(const e2h_hgrn2_args &a, const ChunkPlan &p) { return (p.chunks * a.batch * a.heads * a.dim * a.vdim * 4 + 255) / 256 * 256; }

int64_t chunk_scratch_bytes(const e2h_hgrn2_args &a) {
  if (!use_chunks(a)) return 0;
  const ChunkPlan p = plan_chunks(a);
  return p.chunks > 1 ? delta_bytes(a, p) + p.chunks * a.batch * a.heads * a.dim * 4 : 0;
}

template <typename T, int DT, int VTW, int NW>
void launch_chunks_sized(const e2h_hgrn2_args &a, const ChunkPlan &p, hipStream_t s) {
  const int64_t bh = a.batch * a.heads;
  if (p.chunks > 1) {
    hipLaunchKernelGGL((hgrn2_chunk_state_kernel<T, DT, VTW, NW>), dim3(static_cast<unsigned>(bh * (p.chunks - 1))), dim3(64 * NW), 0, s, a, p);
    hipLaunchKernelGGL(hgrn2_scan_kernel, dim3(static_cast<unsigned>((bh * a.dim * a.vdim / 4 + 255) / 256)), dim3(256), 0, s, a, p);
  }
  hipLaunchKernelGGL((hgrn2_chunk_output_kernel<T, DT, VTW, NW>), dim3(static_cast<unsigned>(bh * p.chunks)), dim3(64 * NW), 0, s, a, p);
}

template <typename T, int DT>
void launch_chunks_dim(const e2h_hgrn2_args &a, const ChunkPlan &p, hipStream_t s) {
  if (a.vdim <= 64) launch_chunks_sized<T, DT, 1, 4>(a, p, s);
  else if (a.vdim <= 128) launch_chunks_sized<T, DT, 2, 4>(a, p, s);
  else launch_chunks_sized<T, DT, (DT <= 4 ? 4 : 2), (DT <= 4 ? 4 : 8)>(a, p, s);
}

template <typename T>
void launch_chunks(const e2h_hgrn2_args &a, hipStream_t s) {
  ChunkPlan p = plan_chunks(a);
  if (p.chunks > 1) {
    p.delta = static_cast<float *>(a.scratch);
    p.decay = reinterpret_cast<float *>(static_cast<uint8_t *>(a.scratch) + delta_bytes(a, p));
  }
  if (a.dim <= 64) launch_chunks_dim<T, 4>(a, p, s);
  else if (a.dim <= 128) launch_chunks_dim<T, 8>(a, p, s);
  else launch_chunks_dim<T, 16>(a, p, s);
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

extern "C" int64_t e2h_seq_hgrn2_scratch_bytes(const e2h_hgrn2_args *a) {
  if (!a) return E2H_ERR_NULL_POINTER;
  if (a->batch < 1 || a->seqlen < 1 || a->heads < 1 || a->dim < 1 || a->vdim < 1) return E2H_ERR_BAD_SHAPE;
  return chunk_scratch_bytes(*a);
}

extern "C" int e2h_seq_hgrn2(const e2h_hgrn2_args *a, void *stream) {
  if (!a || !a->proj || !a->f_bias || !a->lower || !a->norm_weight || !a->state || !a->input_pos || !a->out) return E2H_ERR_NULL_POINTER;
  if (a->dtype != E2H_SEQ_BF16 && a->dtype != E2H_SEQ_F32) return E2H_ERR_BAD_SHAPE;
  if (a->batch < 1 || a->seqlen < 1 || a->heads < 1 || a->dim < 1 || a->dim > kMaxDim || a->vdim < 4 || a->vdim % 4 != 0 || a->vdim > kMaxDim)
    return E2H_ERR_BAD_SHAPE;
  if (a->q_off < 0 || a->f_off < 0 || a->v_off < 0 || a->out_off < 0 || a->q_off + a->heads * a->dim > a->ld || a->f_off + a->heads * a->dim > a->ld ||
      a->v_off + a->heads * a->vdim > a->ld || a->out_off + a->heads * a->vdim > a->ld_out || a->batch * a->heads > INT32_MAX ||
      a->seqlen > INT32_MAX / 2)
    return E2H_ERR_BAD_SHAPE;
  if (!aligned16(a->state) || !aligned16(a->scratch)) return E2H_ERR_MISALIGNED;
  if (use_chunks(*a)) {
    const ChunkPlan p = plan_chunks(*a);
    const int64_t need = chunk_scratch_bytes(*a);
    if (a->batch * a->heads * p.chunks > INT32_MAX || a->batch * a->heads * a->dim * a->vdim / 1024 > INT32_MAX - 1) return E2H_ERR_BAD_SHAPE;
    if (need > 0 && !a->scratch) return E2H_ERR_NULL_POINTER;
    if (need > a->scratch_bytes) return E2H_ERR_SCRATCH_TOO_SMALL;
    if (!aligned16(a->proj) || !aligned16(a->f_bias) || !aligned16(a->lower)) return E2H_ERR_MISALIGNED;
    if (a->dtype == E2H_SEQ_BF16) launch_chunks<bf16_t>(*a, static_cast<hipStream_t>(stream));
    else launch_chunks<float>(*a, static_cast<hipStream_t>(stream));
    return launch_status();
  }
  if (a->dtype == E2H_SEQ_BF16) launch_tokens<bf16_t>(*a, static_cast<hipStream_t>(stream));
  else launch_tokens<float>(*a, static_cast<hipStream_t>(stream));
  return launch_status();
}
