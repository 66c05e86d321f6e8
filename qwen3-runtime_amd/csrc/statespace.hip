// The state-space and matrix-memory recurrences over spans of many tokens, chunk by chunk on MFMA, for bfloat16 inputs.
//
//   D_t = softplus(step_t + bias), a_t = exp(-exp(a_log) D_t)
//   S <- a_t S + D_t x_t B_t^T;   y_t = S C_t + skip x_t            (S [P, N] per sequence and head)
//
// With l_t = sum of log a (base 2 in the code) over the chunk up to and including t, a chunk of 64 tokens is three products:
//
//   y_t  = sum_{s <= t} [ exp(l_t - l_s) D_s (C_t . B_s) + skip (s = t) ] x_s  +  exp(l_t) S_0 C_t
//   S_64 = exp(l_63) S_0 + sum_s exp(l_63 - l_s) D_s x_s B_s^T
//
// x, B and C come in bfloat16 (the short convolution's output) and are exact as operands. What is
// float32 enters as a sum of bfloat16 terms: the weighted x of the state's update as three, which hold
// all 24 bits, so that the state is kept to float32; the bracket and the state as they are read out as two
// (17 bits; a read-out is gated, normed and rounded to 8). Sums are float32, and so are step sizes,
// logarithms of decays and exponentials. The exponents are differences l_t - l_s <= 0, so nothing
// overflows however fast a head forgets. The recurrence written out token by token is in retention.hip;
// the two differ by the rounding of float32 sums.
//
// Matrix memory (GATES) is the same recurrence with other names: values x, keys B, queries C (a head's
// own), no skip, and per token and head the logarithms of what it keeps of the state (in place of a's) and
// of what its write weighs (in place of D's). Its state has one more row, the sum of the weighted keys n; its
// read-out n . q is the brackets' sum over s plus what is left of n_0 . q, both of which the block has at
// hand, so the blocks of a head's first channels keep n in float32 beside their tiles, a thread an element.
//
// A block of four waves owns one head of one sequence and 64 of its P channels, and walks the span's
// chunks in order with the state in registers: wave w holds channels 16 w .. 16 w + 15, S transposed as
// the accumulator tiles of the update (tile i: rows n = 16 i + 4 quad + r, column p = lane & 15), which
// read in pairs are also the operand of the product with C (two runs of four neighbouring n a lane; C
// is read from LDS in the same order). B is staged by rows for C . B and transposed for the update, x
// transposed; for the transposed ones a thread turns 8 x 8 pieces round in registers on the way into LDS
// (neighbouring threads take neighbouring tokens, so that they write neighbouring pieces of a row). The next chunk's
// global loads are in flight while a chunk is computed. The bracket is computed once for the block,
// 16 rows a wave, in the layout its product wants (the keys of two 16-row tiles permuted so that a lane
// ends up with eight neighbouring s for its t), and shared through LDS.
#include "common.h"
#include <math.h>

struct SpaceArgs {
  const bf16_t* xbc;         // [T, channels]: x heads, B groups and C groups from the columns below on
  int channels;
  int x_first, b_first, c_first;
  const void* step; long step_stride; int step_code;   // [T, heads] step logits
  const float* step_bias; const float* a_log; const float* skip;  // [heads]
  float* state;              // [slots, heads, P, N]; GATES: [slots, heads, P + 1, N]
  float* out;                // [T, heads, P]
  const int* cu_q; const int* state_slots;
  const int* seq_ids;        // the sequences of this launch; null: all of the step's
  int heads, groups, n, p;
  const float* gates;        // [T, 3, heads]: log keep, log write (a third row is not read); null: step sizes
  float* last_out;           // [T, heads]: n . q (GATES)
};

constexpr int CHUNK = 64;
constexpr int READ_TERMS = 2, WRITE_TERMS = 3;  // bfloat16 terms of a float32 value in a read-out, in the state's update
constexpr int TROW = CHUNK + 16;   // elements of a transposed row in LDS: 32 bytes modulo 64

// v as a sum of COUNT bfloat16 terms, the last one rounded, those before cut off (8 bits each: what is
// left is exact, and three terms hold a float32's 24 bits). Two values' halves leave in one register.
template <int COUNT>
__device__ __forceinline__ void split_terms(const float* v, bf16x8_t* out) {
  float r[8];
#pragma unroll
  for (int e = 0; e < 8; ++e) r[e] = v[e];
#pragma unroll
  for (int k = 0; k < COUNT - 1; ++k) {
    u32x4_t bits;
#pragma unroll
    for (int e = 0; e < 4; ++e)  // the upper halves of two neighbours
      bits[e] = __builtin_amdgcn_perm(__float_as_uint(r[2 * e + 1]), __float_as_uint(r[2 * e]), 0x07060302u);
    out[k] = __builtin_bit_cast(bf16x8_t, bits);
#pragma unroll
    for (int e = 0; e < 8; ++e) r[e] -= __uint_as_float(__float_as_uint(r[e]) & 0xffff0000u);
  }
#pragma unroll
  for (int e = 0; e < 8; ++e) out[COUNT - 1][e] = (bf16_t)r[e];
}

// sum over the lanes up to and including this one (DPP: shifts within rows of 16, then the rows before)
__device__ __forceinline__ float wave_running_sum(float x) {
#define STEP_(ctrl, rows)                                                                                         \
  x += __builtin_bit_cast(float, __builtin_amdgcn_update_dpp(0, __builtin_bit_cast(int, x), ctrl, rows, 0xF, false))
  STEP_(0x111, 0xF);  // row_shr 1, 2, 4, 8: a lane without a source adds 0
  STEP_(0x112, 0xF);
  STEP_(0x114, 0xF);
  STEP_(0x118, 0xF);
  STEP_(0x142, 0xA);  // row_bcast 15 into rows 1 and 3
  STEP_(0x143, 0xC);  // row_bcast 31 into rows 2 and 3
#undef STEP_
  return x;
}

// KS steps of 32 state elements (N padded with zeros)
template <int KS, bool GATES>
__global__ __launch_bounds__(256, 1) void state_space_chunk_kernel(SpaceArgs a) {
  constexpr int NP = 32 * KS, BROW = NP + 16;
  constexpr int B_TASKS = 32 * KS, TASKS = B_TASKS + 64;     // 8 x 8 pieces of B and of x
  constexpr int R = (TASKS + 255) / 256;
  extern __shared__ __attribute__((aligned(16))) bf16_t lds[];
  bf16_t* brow = lds;                      // [64][BROW]
  bf16_t* crow = brow + CHUNK * BROW;      // [64][BROW]
  bf16_t* bt = crow + CHUNK * BROW;        // [NP][TROW]
  bf16_t* xt = bt + NP * TROW;             // [64][TROW]
  bf16_t* pm = xt + CHUNK * TROW;          // [6][READ_TERMS][64 lanes][8]
  float* dts = (float*)(pm + 6 * READ_TERMS * 512);  // [64] step sizes
  float* acs = dts + CHUNK;                // [64] base-2 logarithms of the decay since the chunk's start, the token's own included
  float* since = acs + CHUNK;              // [64] 2^acs: what is left of the state before the chunk
  float* left = since + CHUNK;             // [64] step size times what is left of the token's write at the chunk's end
  float* nvec = left + CHUNK;              // [NP] the sum of the weighted keys before the chunk (GATES)

  const int tid = threadIdx.x, lane = tid & 63, wave = uniform_wave_number();
  const int r16 = lane & 15, quad = lane >> 4;
  const int head = blockIdx.x, p0 = blockIdx.y * 64;
  const int seq = a.seq_ids ? a.seq_ids[blockIdx.z] : blockIdx.z;
  const int t0 = a.cu_q[seq], t1 = a.cu_q[seq + 1];
  if (t1 <= t0) return;
  const int N = a.n, P = a.p, group = head / (a.heads / a.groups);
  const int x_col = a.x_first + head * P + p0, b_col = a.b_first + group * N, c_col = a.c_first + group * N;
  const float rate = GATES ? 0.f : expf(a.a_log[head]) * 1.4426950408889634f, bias = GATES ? 0.f : a.step_bias[head];
  const float skip = GATES ? 0.f : a.skip[head];
  const int state_rows = GATES ? P + 1 : P;
  const bool has_n = GATES && blockIdx.y == 0;  // the same for the block
  const bool has_tile = p0 + 16 * wave < P;   // the same for the whole wave
  const int my_p = p0 + 16 * wave + r16;
  const bool p_ok = my_p < P;

  float* st = a.state + (((size_t)a.state_slots[seq] * a.heads + head) * state_rows + (p_ok ? my_p : 0)) * N;
  float* st_n = a.state + (((size_t)a.state_slots[seq] * a.heads + head) * state_rows + P) * N;  // GATES
  float own_n = 0.f;
  if (has_n) {
    if (tid < N) own_n = st_n[tid];
    if (tid < NP) nvec[tid] = own_n;
  }
  f32x4_t S[2 * KS];
#pragma unroll
  for (int i = 0; i < 2 * KS; ++i) {
    const int nn = 16 * i + 4 * quad;    // N is a multiple of 8: four neighbours are in or out together
    S[i] = (p_ok && nn < N) ? *(const f32x4_t*)(st + nn) : (f32x4_t){0.f, 0.f, 0.f, 0.f};
  }

  bf16x8_t pre[R][8], pre_b[KS], pre_c[KS];
  float pre_step = 0.f, pre_write = 0.f;
  const bool padded = N < NP || p0 + 64 > P;   // some pieces lie outside the state: zeros (the same for the block)
  // piece `task`: of B (tokens 8 sg .., channels 8 cg ..) or of x
  auto where = [&](int task, int& sg, int& cg, bool& is_b, bool& ok) {
    is_b = task < B_TASKS;
    const int idx = is_b ? task : task - B_TASKS;
    sg = idx & 7;
    cg = idx >> 3;
    ok = !padded || (is_b ? 8 * cg < N : p0 + 8 * cg < P);
  };
  // where a thread reads: element offsets from a chunk's first token, in a chunk of 64 whole tokens
  int at_piece[R], at_row[KS];
#pragma unroll
  for (int r = 0; r < R; ++r) {
    int sg, cg;
    bool is_b, ok;
    where(tid + 256 * r, sg, cg, is_b, ok);
    at_piece[r] = 8 * sg * a.channels + (is_b ? b_col : x_col) + (ok ? 8 * cg : 0);
  }
#pragma unroll
  for (int k = 0; k < KS; ++k) {
    const int piece = tid + 256 * k, row = piece / (4 * KS), cg = piece - row * (4 * KS);
    at_row[k] = row * a.channels + (8 * cg < N ? 8 * cg : 0);
  }
  auto fetch = [&](int c0) {
    const bf16_t* base = a.xbc + (size_t)c0 * a.channels;
    if (c0 + CHUNK <= t1) {
#pragma unroll
      for (int r = 0; r < R; ++r)
        if (tid + 256 * r < TASKS) {
#pragma unroll
          for (int j = 0; j < 8; ++j) pre[r][j] = *(const bf16x8_t*)(base + at_piece[r] + j * a.channels);
        }
#pragma unroll
      for (int k = 0; k < KS; ++k) {
        pre_b[k] = *(const bf16x8_t*)(base + at_row[k] + b_col);
        pre_c[k] = *(const bf16x8_t*)(base + at_row[k] + c_col);
      }
    } else {  // tokens after the span's last: the last one again, weighed by zero below
      const int last = t1 - 1 - c0;
#pragma unroll
      for (int r = 0; r < R; ++r)
        if (tid + 256 * r < TASKS) {
          const int sg = (tid + 256 * r < B_TASKS ? tid + 256 * r : tid + 256 * r - B_TASKS) & 7;
#pragma unroll
          for (int j = 0; j < 8; ++j)
            pre[r][j] = *(const bf16x8_t*)(base + at_piece[r] + (min(8 * sg + j, last) - 8 * sg) * a.channels);
        }
#pragma unroll
      for (int k = 0; k < KS; ++k) {
        const int row = (tid + 256 * k) / (4 * KS), back = (min(row, last) - row) * a.channels;
        pre_b[k] = *(const bf16x8_t*)(base + at_row[k] + back + b_col);
        pre_c[k] = *(const bf16x8_t*)(base + at_row[k] + back + c_col);
      }
    }
    if (GATES && tid < CHUNK) {
      const float* row = a.gates + (size_t)min(c0 + tid, t1 - 1) * 3 * a.heads + head;
      pre_step = row[0];
      pre_write = row[a.heads];
    }
    if (!GATES && tid < CHUNK) {
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
        for (int j = 0; j < 8; ++j)
          if (padded && !ok) pre[r][j] = zero8;
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
      if (padded && 8 * cg >= N) pre_b[k] = pre_c[k] = zero8;
      // row 32 kb + 16 s2 + 4 q + r of `brow` is token 32 kb + 8 q + 4 s2 + r: the 16 lanes of an operand
      // read 16 neighbouring rows
      const int brow_at = (row & 32) + ((row & 4) << 2) + ((row & 24) >> 1) + (row & 3);
      *(bf16x8_t*)(brow + brow_at * BROW + 8 * cg) = pre_b[k];
      *(bf16x8_t*)(crow + row * BROW + 8 * cg) = pre_c[k];
    }
    if (wave == 0) {
      float d, log_keep;  // what the token's write weighs; the base-2 logarithm of what it keeps of the state
      if (GATES) {
        d = c0 + lane < t1 ? expf(pre_write) : 0.f;
        log_keep = c0 + lane < t1 ? pre_step * 1.4426950408889634f : 0.f;
      } else {
        const float z = pre_step + bias;
        d = c0 + lane < t1 ? (z > 20.f ? z : log1pf(expf(z))) : 0.f;
        log_keep = -rate * d;
      }
      const float v = wave_running_sum(log_keep);
      dts[lane] = d;
      acs[lane] = v;
      since[lane] = __builtin_amdgcn_exp2f(v);
      left[lane] = d * __builtin_amdgcn_exp2f(__int_as_float(__builtin_amdgcn_readlane(__float_as_int(v), 63)) - v);
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
      float n_read = 0.f, row_sum = 0.f;  // this lane's share of n_0 . q_t and of the row's bracket
      for (int kb = 0; kb <= (wave >> 1); ++kb) {
        // everything the rows need from LDS is asked for before the first product
        bf16x8_t kk[2][KS], cc[KS];
        f32x4_t ls[2], dd[2];
#pragma unroll
        for (int j = 0; j < KS; ++j) {
          cc[j] = *(const bf16x8_t*)(crow + t * BROW + 32 * j + 8 * quad);
#pragma unroll
          for (int s2 = 0; s2 < 2; ++s2)
            kk[s2][j] = *(const bf16x8_t*)(brow + (32 * kb + 16 * s2 + r16) * BROW + 32 * j + 8 * quad);
        }
#pragma unroll
        for (int s2 = 0; s2 < 2; ++s2) {
          ls[s2] = *(const f32x4_t*)(acs + 32 * kb + 8 * quad + 4 * s2);
          dd[s2] = *(const f32x4_t*)(dts + 32 * kb + 8 * quad + 4 * s2);
        }
        if (has_n && kb == 0) {
#pragma unroll
          for (int j = 0; j < KS; ++j) {
            const f32x4_t n0 = *(const f32x4_t*)(nvec + 32 * j + 8 * quad), n1 = *(const f32x4_t*)(nvec + 32 * j + 8 * quad + 4);
#pragma unroll
            for (int e = 0; e < 4; ++e) {
              n_read = fmaf(n0[e], (float)cc[j][e], n_read);
              n_read = fmaf(n1[e], (float)cc[j][e + 4], n_read);
            }
          }
        }
        f32x4_t sc[2] = {{0.f, 0.f, 0.f, 0.f}, {0.f, 0.f, 0.f, 0.f}};
#pragma unroll
        for (int j = 0; j < KS; ++j)
#pragma unroll
          for (int s2 = 0; s2 < 2; ++s2) sc[s2] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(kk[s2][j], cc[j], sc[s2], 0, 0, 0);
        float m[8];
#pragma unroll
        for (int e = 0; e < 8; ++e) {
          const int s = 32 * kb + 8 * quad + e;
          // keys after the row's token: the exponent is held at 0 (so that nothing overflows) and the weight is 0
          const float w = __builtin_amdgcn_exp2f(fminf(lt - ls[e >> 2][e & 3], 0.f)) * dd[e >> 2][e & 3];
          m[e] = sc[e >> 2][e & 3] * (s <= t ? w : 0.f) + (!GATES && s == t ? skip : 0.f);
          if (GATES) row_sum += m[e];
        }
        bf16x8_t terms[READ_TERMS];
        split_terms<READ_TERMS>(m, terms);
        const int combo = wave < 2 ? wave : 2 * wave - 2 + kb;
#pragma unroll
        for (int k = 0; k < READ_TERMS; ++k) *(bf16x8_t*)(pm + ((combo * READ_TERMS + k) * 64 + lane) * 8) = terms[k];
      }
      if (has_n) {
        float q_n = fmaf(since[t], n_read, row_sum);
        q_n += __shfl_xor(q_n, 16, 64);
        q_n += __shfl_xor(q_n, 32, 64);
        if (quad == 0 && c0 + t < t1) a.last_out[(size_t)(c0 + t) * a.heads + head] = q_n;
      }
    }
    __syncthreads();
    if (has_n && tid < NP) {  // the sum of the weighted keys moves on: nobody reads nvec before the next barrier
      float acc = 0.f;
#pragma unroll
      for (int sg = 0; sg < CHUNK / 8; ++sg) {
        const bf16x8_t kv = *(const bf16x8_t*)(bt + tid * TROW + 8 * sg);
        const f32x4_t l0 = *(const f32x4_t*)(left + 8 * sg), l1 = *(const f32x4_t*)(left + 8 * sg + 4);
#pragma unroll
        for (int e = 0; e < 4; ++e) {
          acc = fmaf(l0[e], (float)kv[e], acc);
          acc = fmaf(l1[e], (float)kv[e + 4], acc);
        }
      }
      own_n = fmaf(since[CHUNK - 1], own_n, acc);
      nvec[tid] = own_n;
    }
    if (has_tile) {
      bf16x8_t sterm[KS][READ_TERMS], xa[2];
#pragma unroll
      for (int j = 0; j < KS; ++j) {
        float v[8];
#pragma unroll
        for (int e = 0; e < 8; ++e) v[e] = S[2 * j + (e >> 2)][e & 3];
        split_terms<READ_TERMS>(v, sterm[j]);
      }
#pragma unroll
      for (int kb = 0; kb < 2; ++kb) xa[kb] = *(const bf16x8_t*)(xt + (16 * wave + r16) * TROW + 32 * kb + 8 * quad);
      // the operands of a 16-row tile, asked for a tile ahead (where the registers allow it)
      constexpr bool AHEAD = KS <= 4;
      bf16x8_t pt[2][2 * READ_TERMS], ct[2][KS];
      auto ask = [&](int t4) {
#pragma unroll
        for (int kb = 0; kb <= (t4 >> 1); ++kb) {
          const int combo = t4 < 2 ? t4 : 2 * t4 - 2 + kb;
#pragma unroll
          for (int k = 0; k < READ_TERMS; ++k) pt[t4 & 1][kb * READ_TERMS + k] = *(const bf16x8_t*)(pm + ((combo * READ_TERMS + k) * 64 + lane) * 8);
        }
#pragma unroll
        for (int j = 0; j < KS; ++j) {
          const bf16_t* cp = crow + (16 * t4 + r16) * BROW + 32 * j + 4 * quad;
          const bf16x4_t lo = *(const bf16x4_t*)cp, hi = *(const bf16x4_t*)(cp + 16);
          ct[t4 & 1][j] = __builtin_shufflevector(lo, hi, 0, 1, 2, 3, 4, 5, 6, 7);
        }
      };
      f32x4_t lw[2][2];
      float gone[4];
#pragma unroll
      for (int kb = 0; kb < 2; ++kb)
#pragma unroll
        for (int h = 0; h < 2; ++h) lw[kb][h] = *(const f32x4_t*)(left + 32 * kb + 8 * quad + 4 * h);
#pragma unroll
      for (int t4 = 0; t4 < 4; ++t4) gone[t4] = since[16 * t4 + r16];
      const float whole = since[CHUNK - 1];
      if (AHEAD) ask(0);
#pragma unroll
      for (int t4 = 0; t4 < 4; ++t4) {
        if (!AHEAD) ask(t4);
        else if (t4 < 3) ask(t4 + 1);
        f32x4_t own = {0.f, 0.f, 0.f, 0.f}, before[READ_TERMS];
#pragma unroll
        for (int kb = 0; kb <= (t4 >> 1); ++kb)
#pragma unroll
          for (int k = 0; k < READ_TERMS; ++k) own = __builtin_amdgcn_mfma_f32_16x16x32_bf16(xa[kb], pt[t4 & 1][kb * READ_TERMS + k], own, 0, 0, 0);
#pragma unroll
        for (int k = 0; k < READ_TERMS; ++k) before[k] = (f32x4_t){0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int j = 0; j < KS; ++j)
#pragma unroll
          for (int k = 0; k < READ_TERMS; ++k)
            before[k] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(sterm[j][k], ct[t4 & 1][j], before[k], 0, 0, 0);
        const int tok = c0 + 16 * t4 + r16, p = p0 + 16 * wave + 4 * quad;
        const f32x4_t y = own + gone[t4] * (before[0] + before[1]);
        if (tok < t1 && p < P) *(f32x4_t*)(a.out + ((size_t)tok * a.heads + head) * P + p) = y;
      }
      bf16x8_t bn[2][2 * KS], xw[2][WRITE_TERMS];
#pragma unroll
      for (int kb = 0; kb < 2; ++kb)
#pragma unroll
        for (int i = 0; i < 2 * KS; ++i) bn[kb][i] = *(const bf16x8_t*)(bt + (16 * i + r16) * TROW + 32 * kb + 8 * quad);
#pragma unroll
      for (int kb = 0; kb < 2; ++kb) {
        float v[8];
#pragma unroll
        for (int e = 0; e < 8; ++e) v[e] = (float)xa[kb][e] * lw[kb][e >> 2][e & 3];
        split_terms<WRITE_TERMS>(v, xw[kb]);
      }
#pragma unroll
      for (int i = 0; i < 2 * KS; ++i) S[i] *= whole;
#pragma unroll
      for (int kb = 0; kb < 2; ++kb)
#pragma unroll
        for (int k = 0; k < WRITE_TERMS; ++k)
#pragma unroll
          for (int i = 0; i < 2 * KS; ++i) S[i] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(bn[kb][i], xw[kb][k], S[i], 0, 0, 0);
    }
    __syncthreads();  // the next chunk takes the same LDS
  }
  if (has_n && tid < N) st_n[tid] = own_n;
  if (p_ok) {
#pragma unroll
    for (int i = 0; i < 2 * KS; ++i) {
      const int nn = 16 * i + 4 * quad;
      if (nn < N) *(f32x4_t*)(st + nn) = S[i];
    }
  }
}

template <int KS, bool GATES>
static int space_launch(const SpaceArgs& a, int num_seqs, hipStream_t stream) {
  constexpr int NP = 32 * KS, BROW = NP + 16;
  constexpr size_t smem = (size_t)(2 * CHUNK * BROW + NP * TROW + CHUNK * TROW + 6 * READ_TERMS * 512) * sizeof(bf16_t) + (4 * CHUNK + (GATES ? NP : 0)) * sizeof(float);
  static_assert(smem <= 160 * 1024, "the chunk does not fit a compute unit's LDS");
  static bool allowed = smem <= 64 * 1024;  // once: not again inside every stream capture
  if (!allowed) {
    if (hipFuncSetAttribute((const void*)state_space_chunk_kernel<KS, GATES>, hipFuncAttributeMaxDynamicSharedMemorySize, (int)smem) != hipSuccess)
      return qrt_fail("state_space_chunks: cannot get %zu bytes of LDS", smem);
    allowed = true;
  }
  state_space_chunk_kernel<KS, GATES><<<dim3(a.heads, (a.p + 63) / 64, num_seqs), 256, smem, stream>>>(a);
  return 0;
}

// num_seqs: sequences of this launch (entries of seq_ids where it is given)
extern "C" int qrt_state_space_chunks(const SpaceArgs* args, int num_seqs, hipStream_t stream) {
  const SpaceArgs& a = *args;
  QRT_CHECK(a.heads > 0 && a.groups > 0 && a.heads % a.groups == 0, "state_space_chunks: %d heads in %d groups", a.heads, a.groups);
  QRT_CHECK(a.n >= 8 && a.n <= 256 && a.n % 8 == 0 && a.p >= 8 && a.p % 8 == 0,
            "state_space_chunks: a state of %d x %d (multiples of 8, the first up to 256)", a.n, a.p);
  QRT_CHECK(a.channels % 8 == 0 && a.x_first % 8 == 0 && a.b_first % 8 == 0 && a.c_first % 8 == 0 && a.x_first >= 0 &&
                a.b_first >= 0 && a.c_first >= 0 && a.x_first + a.heads * a.p <= a.channels &&
                a.b_first + a.groups * a.n <= a.channels && a.c_first + a.groups * a.n <= a.channels,
            "state_space_chunks: rows of %d channels, the three parts from %d, %d and %d on", a.channels, a.x_first, a.b_first, a.c_first);
  QRT_CHECK((uintptr_t)a.xbc % 16 == 0 && (uintptr_t)a.state % 16 == 0 && (uintptr_t)a.out % 16 == 0, "state_space_chunks: not aligned to 16 bytes");
  QRT_CHECK(a.gates ? a.last_out != nullptr : a.step && a.step_bias && a.a_log && a.skip && a.step_stride >= a.heads, "state_space_chunks: no step logits, bias, rate or skip");
  QRT_CHECK(num_seqs >= 0 && num_seqs <= 65535, "state_space_chunks: %d sequences", num_seqs);
  if (num_seqs == 0) return 0;
  int rc;
#define GO(KS) rc = a.gates ? space_launch<KS, true>(a, num_seqs, stream) : space_launch<KS, false>(a, num_seqs, stream)
  if (a.n <= 32) GO(1);
  else if (a.n <= 64) GO(2);
  else if (a.n <= 128) GO(4);
  else GO(8);
#undef GO
  if (rc != 0) return rc;
  QRT_LAUNCH_CHECK("state_space_chunks");
  return 0;
}
