// Matrix memory with exponential gates: what is its own of it. The recurrence itself, S <- keep S + write
// k [v | 1]^T, is a form of those in retention.hip (token by token) and statespace.hip (chunk by chunk).
//
// memory_gates: from the logits of a token's input and forget gates, i and f after their soft caps and the
// forget gate's log sigmoid, the running maximum of a sequence and head,
//     m_t = max(f_t + m_(t-1), i_t),
// and with it the logarithms of what the token keeps of the memory, f_t + m_(t-1) - m_t, and of what its
// write weighs, i_t - m_t, none of them above 0. One wave per sequence and head takes 64 tokens at a time:
// with F_t the sum of f over the tile up to t, m_t = F_t + max(m_before, max_(s <= t) (i_s - F_s)), two scans
// over the lanes, in float64 so that a sum of many strongly negative logarithms costs no digits.
//
// memory_out: the read-out over the larger of |n . q| and exp(-m), each head over its root mean square,
// times the weight of all heads and the output gate's sigmoid.
#include "common.h"
#include <math.h>

struct GatesArgs {
  const float* logits;     // [T, heads input | heads forget]
  const float* bias;       // [2 heads]
  float cap;
  float* top;              // [slots, heads] running maxima, brought up to date
  float* out;              // [T, 3, heads]: log keep, log write, m
  const int* cu_q; const int* state_slots;
  int heads;
};

// A block of W waves: a head each (W = 4, spans of up to 64 tokens), or one head whose tiles of 64 tokens
// the waves take side by side (W = 16): what a tile does to the maximum before it is one pair of numbers,
// m -> F + max(m, u) with the tile's sum and its largest i_s - F_s, so every wave finds the maximum before its
// own tile from the pairs of the tiles before, in their order. Spans of one token need no scan.
template <int W>
__global__ __launch_bounds__(64 * W) void memory_gates_kernel(GatesArgs a) {
  __shared__ double tile_sum[16], tile_max[16];
  constexpr bool SPREAD = W == 16;
  const int lane = threadIdx.x & 63, wave = uniform_wave_number(), seq = blockIdx.y;
  const int head = SPREAD ? blockIdx.x : blockIdx.x * W + wave;
  if (head >= a.heads) return;  // the whole wave; with one head a block, never
  const int t0 = a.cu_q[seq], t1 = a.cu_q[seq + 1];
  if (t0 >= t1) return;
  float* top = a.top + (size_t)a.state_slots[seq] * a.heads + head;
  const float bi = a.bias[head], bf = a.bias[a.heads + head];
  float m = *top;
  // the lane that has a tile's sum and maximum: lanes behind the last token carry them on
  const int last = t1 - t0 > 1 ? 63 : 0;
  for (int base = t0; base < t1; base += SPREAD ? 1024 : 64) {
    const int t = base + lane + (SPREAD ? 64 * wave : 0);
    const bool ok = t < t1;
    const float* row = a.logits + (size_t)min(t, t1 - 1) * 2 * a.heads;
    const float li = a.cap * tanhf((row[head] + bi) / a.cap), c = a.cap * tanhf((row[a.heads + head] + bf) / a.cap);
    const float lf = fminf(c, 0.f) - log1pf(expf(-fabsf(c)));
    double F = ok ? (double)lf : 0.0;
    double u = ok ? (double)li - F : -INFINITY;
    if (t1 - t0 > 1) {
#pragma unroll
      for (int o = 1; o < 64; o <<= 1) {
        const double before = __shfl_up(F, o, 64);
        if (lane >= o) F += before;
      }
      u = ok ? (double)li - F : -INFINITY;
#pragma unroll
      for (int o = 1; o < 64; o <<= 1) {
        const double before = __shfl_up(u, o, 64);
        if (lane >= o) u = fmax(u, before);
      }
    }
    float next = 0.f;  // the maximum behind these 1,024 tokens
    if (SPREAD) {
      if (lane == last) {
        tile_sum[wave] = F;
        tile_max[wave] = u;
      }
      __syncthreads();
      float run = m;
      for (int j = 0; j < 16; ++j) {
        if (j == wave) m = run;
        run = (float)(tile_sum[j] + fmax((double)run, tile_max[j]));
      }
      next = run;
    }
    const float mt = (float)(F + fmax((double)m, u));
    float mp = __shfl_up(mt, 1, 64);
    if (lane == 0) mp = m;
    if (ok) {
      float* o = a.out + (size_t)t * 3 * a.heads + head;
      o[0] = lf + mp - mt;
      o[a.heads] = li - mt;
      o[2 * a.heads] = mt;
    }
    m = SPREAD ? next : __shfl(mt, last, 64);
    if (SPREAD) __syncthreads();             // the pairs have been read
  }
  if (lane == 0 && (!SPREAD || wave == 0)) *top = m;
}

// max_span: the most tokens a sequence has in this step
extern "C" int qrt_memory_gates(const float* logits, const float* bias, float cap, float* top, float* out, const int* cu_q,
                                const int* state_slots, int heads, int num_tokens, int num_seqs, int max_span, hipStream_t stream) {
  QRT_CHECK(heads > 0 && cap > 0.f && num_tokens >= 0 && num_seqs >= 0 && num_seqs <= 65535, "memory_gates: bad sizes");
  if (num_tokens == 0 || num_seqs == 0) return 0;
  const GatesArgs a{logits, bias, cap, top, out, cu_q, state_slots, heads};
  if (max_span > 64) memory_gates_kernel<16><<<dim3(heads, num_seqs), 1024, 0, stream>>>(a);
  else memory_gates_kernel<4><<<dim3((heads + 3) / 4, num_seqs), 256, 0, stream>>>(a);
  QRT_LAUNCH_CHECK("memory_gates");
  return 0;
}

// one wave per (token, head); VEC neighbouring elements a lane and access
template <typename TG, typename TO, int VEC>
__global__ __launch_bounds__(256) void memory_out_kernel(const float* __restrict__ read, const float* __restrict__ norm_read,
                                                         const float* __restrict__ gates, const float* __restrict__ weight,
                                                         const TG* __restrict__ out_gate, long gate_stride, TO* __restrict__ out,
                                                         long items, int heads, int vdim, float eps, float q_scale) {
  typedef float fvec_t __attribute__((ext_vector_type(VEC)));
  typedef TG gvec_t __attribute__((ext_vector_type(VEC)));
  typedef TO ovec_t __attribute__((ext_vector_type(VEC)));
  constexpr int KEEP = 2;
  const int lane = threadIdx.x & 63;
  const long item = (long)blockIdx.x * 4 + (threadIdx.x >> 6);
  if (item >= items) return;
  const long t = item / heads;
  const int h = (int)(item - t * heads);
  const float* row = read + (size_t)item * vdim;
  const float* w = weight + (size_t)h * vdim;
  const TG* g = out_gate + (size_t)t * gate_stride + (size_t)h * vdim;
  const float nq = norm_read[item] * q_scale, m = gates[(size_t)(3 * t + 2) * heads + h];
  // everything a lane needs is asked for before the first use (heads of up to 64 * VEC * KEEP elements)
  fvec_t x[KEEP], wv[KEEP];
  gvec_t gv[KEEP];
  float ss = 0.f;
#pragma unroll
  for (int j = 0; j < KEEP; ++j) {
    const int c = min((lane + 64 * j) * VEC, vdim - VEC);
    x[j] = *(const fvec_t*)(row + c);
    wv[j] = *(const fvec_t*)(w + c);
    gv[j] = *(const gvec_t*)(g + c);
  }
#pragma unroll
  for (int j = 0; j < KEEP; ++j)
    if ((lane + 64 * j) * VEC < vdim)
#pragma unroll
      for (int e = 0; e < VEC; ++e) ss += x[j][e] * x[j][e];
  for (int c = (lane + 64 * KEEP) * VEC; c < vdim; c += 64 * VEC) {
    const fvec_t v = *(const fvec_t*)(row + c);
#pragma unroll
    for (int e = 0; e < VEC; ++e) ss += v[e] * v[e];
  }
  const float by = q_scale / (fmaxf(fabsf(nq), expf(-m)) + 1e-6f);
  const float inv = by / sqrtf(wave_sum(ss) * by * by / (float)vdim + eps);
  auto finish = [&](int c, const fvec_t& v, const fvec_t& ww, const gvec_t& gg) {
    ovec_t y;
#pragma unroll
    for (int e = 0; e < VEC; ++e) y[e] = from_f32<TO>(v[e] * inv * ww[e] / (1.0f + expf(-to_f32<TG>(gg[e]))));
    *(ovec_t*)(out + (size_t)item * vdim + c) = y;
  };
#pragma unroll
  for (int j = 0; j < KEEP; ++j)
    if ((lane + 64 * j) * VEC < vdim) finish((lane + 64 * j) * VEC, x[j], wv[j], gv[j]);
  for (int c = (lane + 64 * KEEP) * VEC; c < vdim; c += 64 * VEC)
    finish(c, *(const fvec_t*)(row + c), *(const fvec_t*)(w + c), *(const gvec_t*)(g + c));
}

extern "C" int qrt_memory_out(const float* read, const float* norm_read, const float* gates, const float* weight,
                              const void* out_gate, long gate_stride, int gate_dtype, void* out, int out_dtype, int num_tokens,
                              int heads, int vdim, float eps, float q_scale, hipStream_t stream) {
  QRT_CHECK(num_tokens >= 0 && heads > 0 && vdim > 0 && gate_stride >= (long)heads * vdim, "memory_out: bad sizes");
  if (num_tokens == 0) return 0;
  const long items = (long)num_tokens * heads;
  const dim3 grid((unsigned)((items + 3) / 4)), block(256);
  const bool pairs = vdim % 2 == 0 && gate_stride % 2 == 0 && (uintptr_t)out_gate % 8 == 0 && (uintptr_t)read % 8 == 0 &&
                     (uintptr_t)weight % 8 == 0 && (uintptr_t)out % 8 == 0;
#define GO(TG, TO)                                                                                                         \
  do {                                                                                                                     \
    if (pairs) memory_out_kernel<TG, TO, 2><<<grid, block, 0, stream>>>(read, norm_read, gates, weight, (const TG*)out_gate, \
                                                                       gate_stride, (TO*)out, items, heads, vdim, eps, q_scale); \
    else memory_out_kernel<TG, TO, 1><<<grid, block, 0, stream>>>(read, norm_read, gates, weight, (const TG*)out_gate,      \
                                                                  gate_stride, (TO*)out, items, heads, vdim, eps, q_scale); \
  } while (0)
  if (gate_dtype == QRT_F32 && out_dtype == QRT_F32) GO(float, float);
  else if (gate_dtype == QRT_BF16 && out_dtype == QRT_BF16) GO(bf16_t, bf16_t);
  else if (gate_dtype == QRT_F32 && out_dtype == QRT_BF16) GO(float, bf16_t);
  else return qrt_fail("memory_out: unknown dtypes %d %d", gate_dtype, out_dtype);
#undef GO
  QRT_LAUNCH_CHECK("memory_out");
  return 0;
}
