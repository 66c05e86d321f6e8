// The state-space recurrence over spans of many tokens, chunk by chunk on MFMA, for bfloat16 inputs.
//
//   D_t = softplus(step_t + bias), a_t = exp(-exp(a_log) D_t)
//   S <- a_t S + D_t x_t B_t^T;   y_t = S C_t + skip x_t            (S [P, N] per sequence and head)
//
// With l_t = sum of log a over the chunk up to and including t, a chunk of 64 tokens is three products:
//
//   y_t  = sum_{s <= t} [ exp(l_t - l_s) D_s (C_t . B_s) + skip (s = t) ] x_s  +  exp(l_t) S_0 C_t
//   S_64 = exp(l_63) S_0 + sum_s exp(l_63 - l_s) D_s x_s B_s^T
//
// x, B and C come in bfloat16 (the short convolution's output) and are exact as operands. What is
// float32 (the bracket, the state as an operand, the weighted x of the state's update) enters as three
// bfloat16 terms whose sum is the float32 value to 24 bits; sums are float32, and so are step sizes,
// logarithms of decays and exponentials. The exponents are differences l_t - l_s <= 0, so nothing
// overflows however fast a head forgets. The recurrence written out token by token is in retention.hip;
// the two differ by the rounding of float32 sums.
//
// A block of four waves owns one head of one sequence and 64 of its P channels, and walks the span's
// chunks in order with the state in registers: wave w holds channels 16 w .. 16 w + 15, S transposed as
// the accumulator tiles of the update (tile i: rows n = 16 i + 4 quad + r, column p = lane & 15), which
// read in pairs are also the operand of the product with C (two runs of four neighbouring n a lane; C
// is read from LDS in the same order). B is staged by rows for C . B and transposed for the update, x
// transposed; a thread turns 8 x 8 pieces round in registers on the way into LDS. The next chunk's
// global loads are in flight while a chunk is computed. The bracket is computed once for the block,
// 16 rows a wave, in the layout its product wants (the keys of two 16-row tiles permuted so that a lane
// ends up with eight neighbouring s for its t), and shared through LDS.
#include "common.h"
#include <math.h>

struct SpaceArgs {
  const bf16_t* xbc;         // [T, channels]: x heads | B groups | C groups
  int channels;
  const void* step; long step_stride; int step_code;   // [T, heads] step logits
  const float* step_bias; const float* a_log; const float* skip;  // [heads]
  float* state;              // [slots, heads, P, N]
  float* out;                // [T, heads, P]
  const int* cu_q; const int* state_slots;
  const int* seq_ids;        // the sequences of this launch; null: all of the step's
  int heads, groups, n, p;
};

constexpr int CHUNK = 64;
constexpr int TERMS = 3;
constexpr int TROW = CHUNK + 16;   // elements of a transposed row in LDS: 32 bytes modulo 64

__device__ __forceinline__ void split_terms(const float* v, bf16x8_t* out) {
#pragma unroll
  for (int e = 0; e < 8; ++e) {
    float r = v[e];
#pragma unroll
    for (int k = 0; k < TERMS; ++k) {
      const bf16_t t = (bf16_t)r;
      out[k][e] = t;
      r -= (float)t;
    }
  }
}

// KS steps of 32 state elements (N padded with zeros)
template <int KS>
__global__ __launch_bounds__(256) void state_space_chunk_kernel(SpaceArgs a) {
  constexpr int NP = 32 * KS, BROW = NP + 16;
  constexpr int B_TASKS = 32 * KS, TASKS = B_TASKS + 64;     // 8 x 8 pieces of B and of x
  constexpr int R = (TASKS + 255) / 256;
  extern __shared__ __attribute__((aligned(16))) bf16_t lds[];
  bf16_t* brow = lds;                      // [64][BROW]
  bf16_t* crow = brow + CHUNK * BROW;      // [64][BROW]
  bf16_t* bt = crow + CHUNK * BROW;        // [NP][TROW]
  bf16_t* xt = bt + NP * TROW;             // [64][TROW]
  bf16_t* pm = xt + CHUNK * TROW;          // [6][TERMS][64 lanes][8]
  float* dts = (float*)(pm + 6 * TERMS * 512);  // [64] step sizes
  float* acs = dts + CHUNK;                // [64] logarithms of the decay since the chunk's start

  const int tid = threadIdx.x, lane = tid & 63, wave = uniform_wave_number();
  const int r16 = lane & 15, quad = lane >> 4;
  const int head = blockIdx.x, p0 = blockIdx.y * 64;
  const int seq = a.seq_ids ? a.seq_ids[blockIdx.z] : blockIdx.z;
  const int t0 = a.cu_q[seq], t1 = a.cu_q[seq + 1];
  if (t1 <= t0) return;
  const int N = a.n, P = a.p, group = head / (a.heads / a.groups);
  const int x_col = head * P + p0, b_col = a.heads * P + group * N, c_col = b_col + a.groups * N;
  const float rate = expf(a.a_log[head]), bias = a.step_bias[head], skip = a.skip[head];
  const bool has_tile = p0 + 16 * wave < P;   // the same for the whole wave
  const int my_p = p0 + 16 * wave + r16;
  const bool p_ok = my_p < P;

  float* st = a.state + (((size_t)a.state_slots[seq] * a.heads + head) * P + (p_ok ? my_p : 0)) * N;
  f32x4_t S[2 * KS];
#pragma unroll
  for (int i = 0; i < 2 * KS; ++i) {
    const int nn = 16 * i + 4 * quad;    // N is a multiple of 8: four neighbours are in or out together
    S[i] = (p_ok && nn < N) ? *(const f32x4_t*)(st + nn) : (f32x4_t){0.f, 0.f, 0.f, 0.f};
  }

  bf16x8_t pre[R][8], pre_c[KS];
  float pre_step = 0.f;
  // piece `task`: of B (tokens 8 sg .., channels 8 cg ..) or of x
  auto where = [&](int task, int& sg, int& cg, bool& is_b, bool& ok) {
    is_b = task < B_TASKS;
    const int idx = is_b ? task : task - B_TASKS, per = is_b ? 4 * KS : 8;
    sg = idx / per;
    cg = idx - sg * per;
    ok = is_b ? 8 * cg < N : p0 + 8 * cg < P;
  };
  auto fetch = [&](int c0) {
#pragma unroll
    for (int r = 0; r < R; ++r) {
      const int task = tid + 256 * r;
      if (task < TASKS) {
        int sg, cg;
        bool is_b, ok;
        where(task, sg, cg, is_b, ok);
        const int col = (is_b ? b_col : x_col) + (ok ? 8 * cg : 0);
#pragma unroll
        for (int j = 0; j < 8; ++j)  // tokens after the span's last: the last one again, weighed by zero below
          pre[r][j] = *(const bf16x8_t*)(a.xbc + (size_t)min(c0 + 8 * sg + j, t1 - 1) * a.channels + col);
      }
    }
#pragma unroll
    for (int k = 0; k < KS; ++k) {
      const int piece = tid + 256 * k, row = piece / (4 * KS), cg = piece - row * (4 * KS);
      pre_c[k] = *(const bf16x8_t*)(a.xbc + (size_t)min(c0 + row, t1 - 1) * a.channels + c_col + (8 * cg < N ? 8 * cg : 0));
    }
    if (tid < CHUNK) {
      const size_t at = (size_t)min(c0 + tid, t1 - 1) * a.step_stride + head;
      pre_step = a.step_code == QRT_F32 ? ((const float*)a.step)[at] : (float)((const bf16_t*)a.step)[at];
    }
  };
  const bf16x8_t zero8 = __builtin_bit_cast(bf16x8_t, (u32x4_t){0, 0, 0, 0});
  auto put = [&](int c0) {
#pragma unroll
    for (int r = 0; r < R; ++r) {
      const int task = tid + 256 * r;
      if (task < TASKS) {
        int sg, cg;
        bool is_b, ok;
        where(task, sg, cg, is_b, ok);
#pragma unroll
        for (int j = 0; j < 8; ++j) {
          if (!ok) pre[r][j] = zero8;
          if (is_b) *(bf16x8_t*)(brow + (8 * sg + j) * BROW + 8 * cg) = pre[r][j];
        }
        bf16_t* dst = is_b ? bt : xt;
#pragma unroll
        for (int e = 0; e < 8; ++e) {
          bf16x8_t v;
#pragma unroll
          for (int j = 0; j < 8; ++j) v[j] = pre[r][j][e];
          *(bf16x8_t*)(dst + (8 * cg + e) * TROW + 8 * sg) = v;
        }
      }
    }
#pragma unroll
    for (int k = 0; k < KS; ++k) {
      const int piece = tid + 256 * k, row = piece / (4 * KS), cg = piece - row * (4 * KS);
      *(bf16x8_t*)(crow + row * BROW + 8 * cg) = 8 * cg < N ? pre_c[k] : zero8;
    }
    if (wave == 0) {
      const float z = pre_step + bias;
      const float d = c0 + lane < t1 ? (z > 20.f ? z : log1pf(expf(z))) : 0.f;
      float v = -rate * d;
#pragma unroll
      for (int o = 1; o < 64; o <<= 1) {
        const float u = __shfl_up(v, o, 64);
        if (lane >= o) v += u;
      }
      dts[lane] = d;
      acs[lane] = v;
    }
  };

  fetch(t0);
  for (int c0 = t0; c0 < t1; c0 += CHUNK) {
    put(c0);
    __syncthreads();
    if (c0 + CHUNK < t1) fetch(c0 + CHUNK);  // on its way while this chunk is computed
    {
      // the bracket: rows t = 16 wave + r16, keys 32 kb + 8 quad + e
      const int t = 16 * wave + r16;
      const float lt = acs[t];
      for (int kb = 0; kb <= (wave >> 1); ++kb) {
        f32x4_t sc[2];
#pragma unroll
        for (int s2 = 0; s2 < 2; ++s2) {
          sc[s2] = (f32x4_t){0.f, 0.f, 0.f, 0.f};
          const int key = 32 * kb + 8 * (r16 >> 2) + 4 * s2 + (r16 & 3);
#pragma unroll
          for (int j = 0; j < KS; ++j)
            sc[s2] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(*(const bf16x8_t*)(brow + key * BROW + 32 * j + 8 * quad),
                                                             *(const bf16x8_t*)(crow + t * BROW + 32 * j + 8 * quad), sc[s2], 0, 0, 0);
        }
        float m[8];
#pragma unroll
        for (int e = 0; e < 8; ++e) {
          const int s = 32 * kb + 8 * quad + e;
          const float w = s <= t ? expf(lt - acs[s]) * dts[s] : 0.f;
          m[e] = sc[e >> 2][e & 3] * w + (s == t ? skip : 0.f);
        }
        bf16x8_t terms[TERMS];
        split_terms(m, terms);
        const int combo = wave < 2 ? wave : 2 * wave - 2 + kb;
#pragma unroll
        for (int k = 0; k < TERMS; ++k) *(bf16x8_t*)(pm + ((combo * TERMS + k) * 64 + lane) * 8) = terms[k];
      }
    }
    __syncthreads();
    if (has_tile) {
      bf16x8_t sterm[KS][TERMS], xa[2];
#pragma unroll
      for (int j = 0; j < KS; ++j) {
        float v[8];
#pragma unroll
        for (int e = 0; e < 8; ++e) v[e] = S[2 * j + (e >> 2)][e & 3];
        split_terms(v, sterm[j]);
      }
#pragma unroll
      for (int kb = 0; kb < 2; ++kb) xa[kb] = *(const bf16x8_t*)(xt + (16 * wave + r16) * TROW + 32 * kb + 8 * quad);
#pragma unroll
      for (int t4 = 0; t4 < 4; ++t4) {
        f32x4_t own = {0.f, 0.f, 0.f, 0.f}, before[TERMS];
#pragma unroll
        for (int kb = 0; kb <= (t4 >> 1); ++kb) {
          const int combo = t4 < 2 ? t4 : 2 * t4 - 2 + kb;
#pragma unroll
          for (int k = 0; k < TERMS; ++k)
            own = __builtin_amdgcn_mfma_f32_16x16x32_bf16(xa[kb], *(const bf16x8_t*)(pm + ((combo * TERMS + k) * 64 + lane) * 8), own, 0, 0, 0);
        }
#pragma unroll
        for (int k = 0; k < TERMS; ++k) before[k] = (f32x4_t){0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int j = 0; j < KS; ++j) {
          const bf16_t* cp = crow + (16 * t4 + r16) * BROW + 32 * j + 4 * quad;
          const bf16x4_t lo = *(const bf16x4_t*)cp, hi = *(const bf16x4_t*)(cp + 16);
          const bf16x8_t cb = __builtin_shufflevector(lo, hi, 0, 1, 2, 3, 4, 5, 6, 7);
#pragma unroll
          for (int k = 0; k < TERMS; ++k) before[k] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(sterm[j][k], cb, before[k], 0, 0, 0);
        }
        const int tok = c0 + 16 * t4 + r16, p = p0 + 16 * wave + 4 * quad;
        const float since = expf(acs[16 * t4 + r16]);
        const f32x4_t y = own + since * (before[0] + (before[1] + before[2]));
        if (tok < t1 && p < P) *(f32x4_t*)(a.out + ((size_t)tok * a.heads + head) * P + p) = y;
      }
      const float last = acs[CHUNK - 1], whole = expf(last);
#pragma unroll
      for (int i = 0; i < 2 * KS; ++i) S[i] *= whole;
#pragma unroll
      for (int kb = 0; kb < 2; ++kb) {
        float v[8];
#pragma unroll
        for (int e = 0; e < 8; ++e) {
          const int s = 32 * kb + 8 * quad + e;
          v[e] = (float)xa[kb][e] * (dts[s] * expf(last - acs[s]));
        }
        bf16x8_t xw[TERMS];
        split_terms(v, xw);
#pragma unroll
        for (int i = 0; i < 2 * KS; ++i) {
          const bf16x8_t bn = *(const bf16x8_t*)(bt + (16 * i + r16) * TROW + 32 * kb + 8 * quad);
#pragma unroll
          for (int k = 0; k < TERMS; ++k) S[i] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(bn, xw[k], S[i], 0, 0, 0);
        }
      }
    }
    __syncthreads();  // the next chunk takes the same LDS
  }
  if (p_ok) {
#pragma unroll
    for (int i = 0; i < 2 * KS; ++i) {
      const int nn = 16 * i + 4 * quad;
      if (nn < N) *(f32x4_t*)(st + nn) = S[i];
    }
  }
}

template <int KS>
static int space_launch(const SpaceArgs& a, int num_seqs, hipStream_t stream) {
  constexpr int NP = 32 * KS, BROW = NP + 16;
  constexpr size_t smem = (size_t)(2 * CHUNK * BROW + NP * TROW + CHUNK * TROW + 6 * TERMS * 512) * sizeof(bf16_t) + 2 * CHUNK * sizeof(float);
  static_assert(smem <= 160 * 1024, "the chunk does not fit a compute unit's LDS");
  static bool allowed = smem <= 64 * 1024;  // once: not again inside every stream capture
  if (!allowed) {
    if (hipFuncSetAttribute((const void*)state_space_chunk_kernel<KS>, hipFuncAttributeMaxDynamicSharedMemorySize, (int)smem) != hipSuccess)
      return qrt_fail("state_space_chunks: cannot get %zu bytes of LDS", smem);
    allowed = true;
  }
  state_space_chunk_kernel<KS><<<dim3(a.heads, (a.p + 63) / 64, num_seqs), 256, smem, stream>>>(a);
  return 0;
}

// num_seqs: sequences of this launch (entries of seq_ids where it is given)
extern "C" int qrt_state_space_chunks(const SpaceArgs* args, int num_seqs, hipStream_t stream) {
  const SpaceArgs& a = *args;
  QRT_CHECK(a.heads > 0 && a.groups > 0 && a.heads % a.groups == 0, "state_space_chunks: %d heads in %d groups", a.heads, a.groups);
  QRT_CHECK(a.n >= 8 && a.n <= 256 && a.n % 8 == 0 && a.p >= 8 && a.p % 8 == 0,
            "state_space_chunks: a state of %d x %d (multiples of 8, the first up to 256)", a.n, a.p);
  QRT_CHECK(a.channels == a.heads * a.p + 2 * a.groups * a.n, "state_space_chunks: %d channels", a.channels);
  QRT_CHECK((uintptr_t)a.xbc % 16 == 0 && (uintptr_t)a.state % 16 == 0 && (uintptr_t)a.out % 16 == 0, "state_space_chunks: not aligned to 16 bytes");
  QRT_CHECK(a.step && a.step_bias && a.a_log && a.skip && a.step_stride >= a.heads, "state_space_chunks: no step logits, bias, rate or skip");
  QRT_CHECK(num_seqs >= 0 && num_seqs <= 65535, "state_space_chunks: %d sequences", num_seqs);
  if (num_seqs == 0) return 0;
  int rc;
  if (a.n <= 32) rc = space_launch<1>(a, num_seqs, stream);
  else if (a.n <= 64) rc = space_launch<2>(a, num_seqs, stream);
  else if (a.n <= 128) rc = space_launch<4>(a, num_seqs, stream);
  else rc = space_launch<8>(a, num_seqs, stream);
  if (rc != 0) return rc;
  QRT_LAUNCH_CHECK("state_space_chunks");
  return 0;
}
