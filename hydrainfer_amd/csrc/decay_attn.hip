// decay_attn.hip — linear attention with a fixed decay per head: S <- d_h S + k v^T, o = S^T q, S [dim, vdim] per head and
// sequence, all of it in float.
//
// Portions of prompts (decay_chunk_kernel): because the decay does not depend on the token, a chunk of 32 tokens is four
// matrix products, which run on the matrix cores with float operands (v_mfma_f32_16x16x4_f32: nothing is rounded to a narrower
// type, so a chunk differs from 32 single steps by the order of float sums alone).  With n tokens i, j = 0 .. n - 1 and S the
// state before them:
//     P[i, j] = (q_i . k_j) d^(i - j) for j <= i,     o_i = d^(i + 1) S^T q_i + sum_j P[i, j] v_j,
//     S <- d^n S + sum_j d^(n - 1 - j) k_j v_j^T.
// The powers come from a table of every head (no quotient of powers appears: a small decay underflows to zero, not to
// 0 / 0).  A workgroup of four waves owns 32 value channels of one (sequence, head) and walks the portion; wave (r, c) owns
// tokens 16 r .. of the chunk for value channels 16 c .., and every other 16-row tile of the state for these channels.  An
// accumulator of the state, as the matrix core leaves it (rows 4 (lane / 16) + e, column lane % 16), is at the same time an
// operand of S^T q when the sum over key channels is taken in the order k = 16 tile + 4 (lane / 16) + e; so the state's tiles
// pass between waves through LDS lane by lane, 16 bytes each, and never change their layout.  The next chunk's rows are on
// their way into registers while a chunk is worked on.
//
// Single tokens (decay_step_kernel): a workgroup per (sequence, head) streams the state once, 16 bytes a lane, everything
// requested before the queries and keys are ready; it can rotate q and k on their way in and finish with the head's norm
// and gate, so that a decode step's mixer is this kernel between two matrix products.
#include "hx_common.h"
#include "mix_rows.h"
#include "../../include/hydra_mix.h"

namespace hxm {
int& last_hip_error();
int check_launch();
}  // namespace hxm

namespace {

using namespace hx;

constexpr int kChunk = HXM_DECAY_CHUNK;

template <typename A, bool SILU>
__device__ __forceinline__ float operand(float x) {
  if constexpr (SILU) return x * sigmoid_of<A>(x);
  else return x;
}
__device__ __forceinline__ float act_of(float x, int act, int dtype) {
  if (act != HXM_ACT_SILU) return x;
  return dtype == HX_F32 ? operand<F32, true>(x) : operand<BF16, true>(x);
}
__device__ __forceinline__ float load_elem(const void* p, int dtype, int64_t e) {
  return dtype == HX_F32 ? ((const float*)p)[e] : BF16::to_float(((const u16*)p)[e]);
}

// A chunk's rows of one operand, KP channels padded, on their way from global memory to LDS: thread `tid` of 256 holds KP / 32
// groups of four channels as they came, read from clamped addresses (no branch stands between two requests, and nothing is
// computed on them before store(), which puts zeros where a row or a channel does not exist).
template <typename A, bool VEC> struct Four;
template <> struct Four<F32, true> {
  f32x4 v;
  __device__ __forceinline__ void load(const float* row, int c, int K) { v = *reinterpret_cast<const f32x4*>(row + (c < K ? c : 0)); }
  __device__ __forceinline__ float get(int j) const { return v[j]; }
};
template <> struct Four<BF16, true> {
  u16x4 v;
  __device__ __forceinline__ void load(const u16* row, int c, int K) { v = *reinterpret_cast<const u16x4*>(row + (c < K ? c : 0)); }
  __device__ __forceinline__ float get(int j) const { return BF16::to_float(v[j]); }
};
template <typename A> struct Four<A, false> {
  typename A::storage v[4];
  __device__ __forceinline__ void load(const typename A::storage* row, int c, int K) {
#pragma unroll
    for (int j = 0; j < 4; ++j) v[j] = row[c + j < K ? c + j : 0];
  }
  __device__ __forceinline__ float get(int j) const { return A::to_float(v[j]); }
};

template <typename A, int KP, bool VEC>
struct ChunkRows {
  static constexpr int NI = KP / 32, PER = KP / 4;
  Four<A, VEC> r[NI];
  __device__ __forceinline__ void fetch(const void* base, int64_t stride, int64_t first, int K, int64_t t0, int n, int tid) {
#pragma unroll
    for (int i = 0; i < NI; ++i) {
      const int g = tid + i * 256, row = g / PER;
      r[i].load((const typename A::storage*)base + (t0 + (row < n ? row : n - 1)) * stride + first, g % PER * 4, K);
    }
  }
  template <bool SILU>
  __device__ __forceinline__ void store(float* lds, int K, int n, float scale, int tid) const {
#pragma unroll
    for (int i = 0; i < NI; ++i) {
      const int g = tid + i * 256, row = g / PER, c = g % PER * 4;
      f32x4 f;
#pragma unroll
      for (int j = 0; j < 4; ++j) f[j] = row < n && c + j < K ? operand<A, SILU>(r[i].get(j)) * scale : 0.f;
      *reinterpret_cast<f32x4*>(lds + row * (KP + 4) + c) = f;
    }
  }
};

template <int KP, typename Q, typename VT, bool SILU, bool VEC>
__global__ __launch_bounds__(256) void decay_chunk_kernel(hxm_decay_attn_args a) {
  constexpr int C = kChunk, RS = KP + 4, PS = C + 4, KT = KP / 16, OWN = KT / 2;
  __shared__ __attribute__((aligned(16))) float qs[C * RS], ks[C * RS], ps[C * PS];
  __shared__ f32x4 ss[KT * 2 * 64];        // the state's tiles, [tile][value half][lane]
  __shared__ float dp[C + 1];
  const int seq = blockIdx.x, head = blockIdx.y;
  // (the wave's number as a scalar: a matrix instruction ignores the lanes' mask, so what chooses its waves must be a branch)
  const int tid = threadIdx.x, wave = __builtin_amdgcn_readfirstlane(tid >> 6), lane = tid & 63;
  const int r = wave >> 1, c = wave & 1, g = lane >> 4, m = lane & 15;
  const int K = a.dim, V = a.vdim;
  const int col = (int)blockIdx.z * 32 + 16 * c + m;
  const bool col_ok = col < V;
  const int64_t t_begin = a.q_cu[seq], t_end = a.q_cu[seq + 1];
  if (t_end <= t_begin) return;
  float* slot = a.state + (int64_t)a.slots[seq] * a.slot_stride + (int64_t)head * K * V;
  const bool fresh = a.positions[t_begin] == 0;
  f32x4 S[OWN];                            // tile 2 o + r
#pragma unroll
  for (int o = 0; o < OWN; ++o) S[o] = f32x4{0.f, 0.f, 0.f, 0.f};
  if (!fresh) {                            // (clamped addresses: one request after the other, no branch between)
    const float* at = slot + (col_ok ? col : 0);
#pragma unroll
    for (int o = 0; o < OWN; ++o) {
#pragma unroll
      for (int e = 0; e < 4; ++e) {
        const int kk = 16 * (2 * o + r) + 4 * g + e;
        S[o][e] = at[(int64_t)(kk < K ? kk : 0) * V];
      }
    }
#pragma unroll
    for (int o = 0; o < OWN; ++o) {
#pragma unroll
      for (int e = 0; e < 4; ++e) S[o][e] = col_ok && 16 * (2 * o + r) + 4 * g + e < K ? S[o][e] : 0.f;
    }
  }
  for (int i = tid; i <= C; i += 256) dp[i] = a.decay_pow[(int64_t)head * (C + 1) + i];

  ChunkRows<Q, KP, VEC> rq, rk;
  typename VT::storage rv[8];              // the chunk's values as they came: tokens 16 s + 4 g + e at 4 s + e
  const typename VT::storage* vcol = (const typename VT::storage*)a.v + (int64_t)head * V + (col_ok ? col : 0);
  auto fetch = [&](int64_t t0) {
    const int n = (int)(t_end - t0 < C ? t_end - t0 : C);
    rq.fetch(a.q, a.q_stride, (int64_t)head * K, K, t0, n, tid);
    rk.fetch(a.k, a.k_stride, (int64_t)head * K, K, t0, n, tid);
#pragma unroll
    for (int i = 0; i < 8; ++i) {
      const int t = 16 * (i >> 2) + 4 * g + (i & 3);
      rv[i] = vcol[(t0 + (t < n ? t : n - 1)) * a.v_stride];
    }
  };
  fetch(t_begin);
  for (int64_t t0 = t_begin; t0 < t_end; t0 += C) {
    const int n = (int)(t_end - t0 < C ? t_end - t0 : C);
    rq.template store<SILU>(qs, K, n, 1.0f, tid);
    rk.template store<SILU>(ks, K, n, a.k_scale, tid);
#pragma unroll
    for (int o = 0; o < OWN; ++o) ss[((2 * o + r) * 2 + c) * 64 + lane] = S[o];
    float v[8];
#pragma unroll
    for (int i = 0; i < 8; ++i) {
      const int t = 16 * (i >> 2) + 4 * g + (i & 3);
      v[i] = t < n && col_ok ? operand<VT, SILU>(VT::to_float(rv[i])) : 0.f;
    }
    lds_barrier();                         // the chunk and the state stand in LDS
    if (t0 + C < t_end) fetch(t0 + C);
    if (wave < 3) {                        // P: three tiles (0, 0), (1, 0), (1, 1)
      const int ti = wave > 0, tj = wave > 1;
      f32x4 p0 = f32x4{0.f, 0.f, 0.f, 0.f}, p1 = p0;
#pragma unroll
      for (int kc = 0; kc < KT; ++kc) {
        const f32x4 x = *reinterpret_cast<const f32x4*>(qs + (16 * ti + m) * RS + 16 * kc + 4 * g);
        const f32x4 y = *reinterpret_cast<const f32x4*>(ks + (16 * tj + m) * RS + 16 * kc + 4 * g);
        p0 = __builtin_amdgcn_mfma_f32_16x16x4f32(x[0], y[0], p0, 0, 0, 0);
        p1 = __builtin_amdgcn_mfma_f32_16x16x4f32(x[1], y[1], p1, 0, 0, 0);
        p0 = __builtin_amdgcn_mfma_f32_16x16x4f32(x[2], y[2], p0, 0, 0, 0);
        p1 = __builtin_amdgcn_mfma_f32_16x16x4f32(x[3], y[3], p1, 0, 0, 0);
      }
#pragma unroll
      for (int e = 0; e < 4; ++e) {
        const int i = 16 * ti + 4 * g + e, j = 16 * tj + m;
        ps[i * PS + j] = j <= i ? (p0[e] + p1[e]) * dp[i - j] : 0.f;
      }
    }
    f32x4 o0 = f32x4{0.f, 0.f, 0.f, 0.f}, o1 = o0;
#pragma unroll
    for (int kt = 0; kt < KT; ++kt) {      // S^T q
      const f32x4 x = *reinterpret_cast<const f32x4*>(qs + (16 * r + m) * RS + 16 * kt + 4 * g);
      const f32x4 y = ss[(kt * 2 + c) * 64 + lane];
      o0 = __builtin_amdgcn_mfma_f32_16x16x4f32(x[0], y[0], o0, 0, 0, 0);
      o1 = __builtin_amdgcn_mfma_f32_16x16x4f32(x[1], y[1], o1, 0, 0, 0);
      o0 = __builtin_amdgcn_mfma_f32_16x16x4f32(x[2], y[2], o0, 0, 0, 0);
      o1 = __builtin_amdgcn_mfma_f32_16x16x4f32(x[3], y[3], o1, 0, 0, 0);
    }
#pragma unroll
    for (int e = 0; e < 4; ++e) o0[e] = (o0[e] + o1[e]) * dp[16 * r + 4 * g + e + 1];
    lds_barrier();                         // P stands; the state in LDS has been read
#pragma unroll
    for (int s = 0; s < 2; ++s) {          // P v (a wave of the first sixteen tokens: their own tile only)
      if (s <= r) {
        const f32x4 x = *reinterpret_cast<const f32x4*>(ps + (16 * r + m) * PS + 16 * s + 4 * g);
#pragma unroll
        for (int e = 0; e < 4; ++e) o0 = __builtin_amdgcn_mfma_f32_16x16x4f32(x[e], v[4 * s + e], o0, 0, 0, 0);
      }
    }
#pragma unroll
    for (int e = 0; e < 4; ++e) {
      const int i = 16 * r + 4 * g + e;
      if (i < n && col_ok) ((float*)a.out)[(t0 + i) * a.out_stride + (int64_t)head * V + col] = o0[e];
    }
#pragma unroll
    for (int i = 0; i < 8; ++i) {
      const int t = 16 * (i >> 2) + 4 * g + (i & 3);
      v[i] *= t < n ? dp[n - 1 - t] : 0.f;
    }
    const float dn = dp[n];
#pragma unroll
    for (int o = 0; o < OWN; ++o) {
#pragma unroll
      for (int e = 0; e < 4; ++e) S[o][e] *= dn;
    }
#pragma unroll
    for (int i = 0; i < 8; ++i) {          // k v^T
      const float* row = ks + (16 * (i >> 2) + 4 * g + (i & 3)) * RS + m;
#pragma unroll
      for (int o = 0; o < OWN; ++o) S[o] = __builtin_amdgcn_mfma_f32_16x16x4f32(row[16 * (2 * o + r)], v[i], S[o], 0, 0, 0);
    }
    lds_barrier();                         // the chunk has been read
  }
#pragma unroll
  for (int o = 0; o < OWN; ++o) {
#pragma unroll
    for (int e = 0; e < 4; ++e) {
      const int kk = 16 * (2 * o + r) + 4 * g + e;
      if (col_ok && kk < K) slot[(int64_t)kk * V + col] = S[o][e];
    }
  }
}

// VEC: value channels a lane moves at a time.  LDS: q | k [dim each], the head's result [vdim rounded up to VEC], partial sums
// [256 * VEC], and four floats.
template <typename A, int VEC>
__global__ __launch_bounds__(256) void decay_step_kernel(hxm_decay_attn_args a, int groups_log2) {
  constexpr int U = VEC == 4 ? 16 : 32;                   // state rows a lane holds at a time
  typedef float row_t __attribute__((ext_vector_type(VEC)));
  extern __shared__ __attribute__((aligned(16))) float lds[];
  const int seq = blockIdx.x, head = blockIdx.y, tid = threadIdx.x;
  const int64_t t = a.q_cu[seq];
  if (a.q_cu[seq + 1] <= t) return;
  const int K = a.dim, V = a.vdim, VV = (V + VEC - 1) / VEC * VEC;
  float* qs = lds;
  float* ks = lds + K;
  float* res = lds + (2 * K + 3) / 4 * 4;
  float* part = res + (VV + 3) / 4 * 4;
  float* red = part + 256 * VEC;
  const int p = a.positions[t];
  const bool fresh = p == 0;
  const float decay = a.decay_pow[(int64_t)head * (kChunk + 1) + 1];
  float* slot = a.state + (int64_t)a.slots[seq] * a.slot_stride + (int64_t)head * K * V;
  const int gcols = 1 << groups_log2, NG = 256 >> groups_log2;      // lanes side by side over value channels, rows dealt to NG groups
  const int cg = tid & (gcols - 1), rg = tid >> groups_log2;
  row_t S[U];
  auto load_rows = [&](int c, int r0) {
#pragma unroll
    for (int u = 0; u < U; ++u) {
      const int kk = r0 + u * NG;
      S[u] = row_t(0.f);
      if (!fresh && c < V && kk < K) S[u] = *reinterpret_cast<const row_t*>(slot + (int64_t)kk * V + c);
    }
  };
  load_rows(VEC * cg, rg);                                // on its way while q and k are made ready
  const int64_t qk = (int64_t)head * K;
  for (int i = tid; i < K; i += 256) {
    qs[i] = act_of(load_elem(a.q, a.qk_dtype, t * a.q_stride + qk + i), a.act, a.qk_dtype);
    ks[i] = act_of(load_elem(a.k, a.qk_dtype, t * a.k_stride + qk + i), a.act, a.qk_dtype) * a.k_scale;
  }
  if (a.inv_freq) {
    lds_barrier();
    const int half = a.rot_dims / 2;
    for (int i = tid; i < half; i += 256) {
      const double ang = (double)p * a.inv_freq[i];        // (reduced in double, as in the rotation kernel for rows)
      const double turns = rint(ang * 0.15915494309189535);
      float sn, cs;
      sincosf((float)fma(-turns, 2.4492935982947064e-16, fma(-turns, 6.283185307179586, ang)), &sn, &cs);
      const int i0 = a.layout == HXM_ROT_HALVES ? i : 2 * i, i1 = a.layout == HXM_ROT_HALVES ? i + half : i0 + 1;
      const float qu = qs[i0], qv = qs[i1], ku = ks[i0], kv = ks[i1];
      qs[i0] = qu * cs - qv * sn;
      qs[i1] = qv * cs + qu * sn;
      ks[i0] = ku * cs - kv * sn;
      ks[i1] = kv * cs + ku * sn;
    }
  }
  lds_barrier();
  for (int c0 = 0; c0 < V; c0 += VEC * gcols) {
    const int c = c0 + VEC * cg;
    float v[VEC];
    row_t o = row_t(0.f);
#pragma unroll
    for (int j = 0; j < VEC; ++j)
      v[j] = c + j < V ? act_of(load_elem(a.v, a.v_dtype, t * a.v_stride + (int64_t)head * V + c + j), a.act, a.v_dtype) : 0.f;
    for (int r0 = rg; r0 < K; r0 += U * NG) {
      if (c0 > 0 || r0 != rg) load_rows(c, r0);
#pragma unroll
      for (int u = 0; u < U; ++u) {
        const int kk = r0 + u * NG;
        if (kk < K && c < V) {
          const float kf = ks[kk], qf = qs[kk];
#pragma unroll
          for (int j = 0; j < VEC; ++j) {
            const float s = decay * S[u][j] + kf * v[j];
            S[u][j] = s;
            o[j] += s * qf;
          }
          *reinterpret_cast<row_t*>(slot + (int64_t)kk * V + c) = S[u];
        }
      }
    }
    *reinterpret_cast<row_t*>(part + VEC * tid) = o;
    lds_barrier();
    if (rg == 0 && c < V) {
      for (int x = 1; x < NG; ++x) o += *reinterpret_cast<const row_t*>(part + VEC * (tid + x * gcols));
      *reinterpret_cast<row_t*>(res + c) = o;
    }
    lds_barrier();
  }
  const int64_t at = t * a.out_stride + (int64_t)head * V;
  if (!a.finish) {
    for (int i = tid; i < V; i += 256) ((float*)a.out)[at + i] = res[i];
    return;
  }
  float ss[1] = {0.f};
  for (int i = tid; i < V; i += 256) ss[0] += res[i] * res[i];
  block_sums<1>(ss, red);
  const float inv = 1.0f / sqrtf(ss[0] / (float)V + a.eps);
  typedef typename A::storage T;
  for (int i = tid; i < V; i += 256) {
    float y = res[i] * inv;
    if (a.gate) y *= act_apply<A>(A::to_float(((const T*)a.gate)[t * a.gate_stride + (int64_t)head * V + i]), a.gate_act);
    ((T*)a.out)[at + i] = A::from_float(y);
  }
}

template <int KP, typename Q, typename VT, bool SILU>
void launch_width(const hxm_decay_attn_args& a, bool vec, hipStream_t s) {
  const dim3 grid((unsigned)a.n_seq, (unsigned)a.heads, (unsigned)((a.vdim + 31) / 32)), block(256);
  if (vec) decay_chunk_kernel<KP, Q, VT, SILU, true><<<grid, block, 0, s>>>(a);
  else decay_chunk_kernel<KP, Q, VT, SILU, false><<<grid, block, 0, s>>>(a);
}

template <typename Q, typename VT, bool SILU>
int launch_chunks(const hxm_decay_attn_args& a, hipStream_t s) {
  const uintptr_t four = a.qk_dtype == HX_F32 ? 16 : 8;    // four channels at a time where every row allows it
  const bool vec = a.dim % 4 == 0 && a.q_stride % 4 == 0 && a.k_stride % 4 == 0 && (uintptr_t)a.q % four == 0 && (uintptr_t)a.k % four == 0;
  if (a.dim <= 32) launch_width<32, Q, VT, SILU>(a, vec, s);
  else if (a.dim <= 64) launch_width<64, Q, VT, SILU>(a, vec, s);
  else if (a.dim <= 128) launch_width<128, Q, VT, SILU>(a, vec, s);
  else launch_width<256, Q, VT, SILU>(a, vec, s);
  return hxm::check_launch();
}

}  // namespace

extern "C" int hxm_decay_attention(const hxm_decay_attn_args* args, void* stream) {
  if (!args) return HX_ERR_NULL;
  const hxm_decay_attn_args& a = *args;
  if (a.n_tokens < 0 || a.n_seq < 0 || a.heads < 1 || a.dim < 1 || a.dim > 256 || a.vdim < 1 || a.vdim > 4096) return HX_ERR_SHAPE;
  if (a.n_tokens == 0 || a.n_seq == 0) return HX_OK;
  if (!a.out || !a.q || !a.k || !a.v || !a.decay_pow || !a.state || !a.slots || !a.q_cu || !a.positions) return HX_ERR_NULL;
  for (int d : {a.qk_dtype, a.v_dtype, a.dtype})
    if (d != HX_F32 && d != HX_BF16) return HX_ERR_DTYPE;
  const int64_t qk = (int64_t)a.heads * a.dim, hv = (int64_t)a.heads * a.vdim;
  if (a.q_stride < qk || a.k_stride < qk || a.v_stride < hv || a.out_stride < hv || (a.gate && a.gate_stride < hv)) return HX_ERR_STRIDE;
  if (a.inv_freq && (a.rot_dims < 2 || a.rot_dims % 2 || a.rot_dims > a.dim || (a.layout != HXM_ROT_HALVES && a.layout != HXM_ROT_INTERLEAVED)))
    return HX_ERR_SHAPE;
  if ((!a.single && (a.inv_freq || a.finish)) || (a.act != HXM_ACT_NONE && a.act != HXM_ACT_SILU)) return HX_ERR_UNSUPPORTED;
  if (a.single && a.n_tokens > a.n_seq) return HX_ERR_SHAPE;
  hipStream_t s = (hipStream_t)stream;
  const dim3 block(256);
  if (!a.single) {
    const bool silu = a.act == HXM_ACT_SILU;
    if (a.qk_dtype == HX_F32 && a.v_dtype == HX_F32) return silu ? launch_chunks<F32, F32, true>(a, s) : launch_chunks<F32, F32, false>(a, s);
    if (a.qk_dtype == HX_BF16 && a.v_dtype == HX_BF16) return silu ? launch_chunks<BF16, BF16, true>(a, s) : launch_chunks<BF16, BF16, false>(a, s);
    if (a.qk_dtype == HX_F32 && !silu) return launch_chunks<F32, BF16, false>(a, s);
    return HX_ERR_DTYPE;
  }
  const dim3 grid((unsigned)a.n_seq, (unsigned)a.heads);
  const bool vec = a.vdim % 4 == 0 && ((uintptr_t)a.state % 16) == 0 && a.slot_stride % 4 == 0;
  const int per = vec ? 4 : 1, cols = (a.vdim + per - 1) / per;
  int groups_log2 = 0;
  while ((1 << groups_log2) < cols && groups_log2 < 8) ++groups_log2;
  auto up4 = [](size_t n) { return (n + 3) / 4 * 4; };
  const size_t lds = (up4(2 * (size_t)a.dim) + up4((size_t)cols * per) + 256 * (size_t)per + 4) * sizeof(float);
  if (a.dtype == HX_F32) {
    if (vec) decay_step_kernel<F32, 4><<<grid, block, lds, s>>>(a, groups_log2);
    else decay_step_kernel<F32, 1><<<grid, block, lds, s>>>(a, groups_log2);
  } else {
    if (vec) decay_step_kernel<BF16, 4><<<grid, block, lds, s>>>(a, groups_log2);
    else decay_step_kernel<BF16, 1><<<grid, block, lds, s>>>(a, groups_log2);
  }
  return hxm::check_launch();
}
