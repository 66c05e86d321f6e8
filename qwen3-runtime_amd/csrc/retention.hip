// Recurrences of linear attention with one decay per head, float32.
//
//   S <- d S + k v^T;   o = S^T q                (S [dim, vdim] per sequence and head)
//
// Retention: d is a constant of the head. State-space form (STEP): a step size per token and head,
// D = softplus(logit + bias), makes both the decay d = exp(-exp(a_log) D) and the written value v = D x,
// the read-out has a skip, o = S^T q + skip x, and neighbouring heads share keys and queries (head h has
// those of h / share).
// Matrix memory (GATES): what a token keeps of the state and what its write weighs come per token and
// head as logarithms, and the state has one more column, whose value is always 1: the sum of the weighted
// keys, whose read-out goes to a place of its own.
//
// over each sequence's tokens of the step, from the state in the sequence's slot, which is left
// there for the next step: [slots, heads, vdim, dim], a value channel's column of S contiguous.
// q, k, v come as float32 [T, 2 heads dim + heads vdim] (queries, keys, values; rotated and
// scaled by whoever made them). A block of 256 threads owns 16 columns of one head's state for
// one sequence; 16 neighbouring lanes share a column, each holding its rows in registers four
// neighbours at a time (rows 4 (lane + 16 g) .. + 3 of group g), so that state, keys and queries
// move 16 bytes a lane and the sum over rows that a read-out needs ends in a DPP sum inside a row
// of 16 lanes. Tokens are staged through LDS 16 at a time; the next tile's global loads are in
// flight while a tile is walked, the walk has no global access and no branch between tokens, and
// the tile's read-outs leave together afterwards. The order of the float32 operations per token
// does not depend on how the tokens are cut into steps, tiles or batches.
#include "common.h"
#include <math.h>

struct RetentionArgs {
  const void* qkv;        // [T, channels] float32, or (STEP) bfloat16
  int channels, q_first, k_first, v_first;
  const float* decay;     // [heads]
  float* state;           // [slots, heads, vdim, dim]
  float* out;             // [T, heads, vdim]
  const int* cu_q; const int* state_slots;
  int heads, dim, vdim;
  int share;              // heads that have one key and query in common (1: each its own)
  const void* step; long step_stride; int step_code;   // [T, heads] step logits, float32 or bfloat16; null: retention
  const float* step_bias; const float* a_log; const float* skip;  // [heads]
  int qkv_code;
  const int* seq_ids;     // the sequences of this launch; null: all of the step's
  const float* gates;     // [T, 3, heads] (GATES): log keep, log write (a third row is not read here)
  float* last_out;        // [T, heads] (GATES): the read-out of the state's last column
};

constexpr int RT_CONSTANT = 0, RT_STEP = 1, RT_GATES = 2;  // where decays and writes come from

#define RT_COLS 16   // columns of the state per block

// the sum over the 16 lanes of a row (every lane gets it)
__device__ __forceinline__ float row16_sum(float x) {
  int v = __builtin_bit_cast(int, x);
  x += __builtin_bit_cast(float, __builtin_amdgcn_update_dpp(0, v, 0xB1, 0xF, 0xF, true));   // quad_perm [1,0,3,2]
  v = __builtin_bit_cast(int, x);
  x += __builtin_bit_cast(float, __builtin_amdgcn_update_dpp(0, v, 0x4E, 0xF, 0xF, true));   // quad_perm [2,3,0,1]
  v = __builtin_bit_cast(int, x);
  x += __builtin_bit_cast(float, __builtin_amdgcn_update_dpp(0, v, 0x141, 0xF, 0xF, true));  // row_half_mirror
  v = __builtin_bit_cast(int, x);
  x += __builtin_bit_cast(float, __builtin_amdgcn_update_dpp(0, v, 0x140, 0xF, 0xF, true));  // row_mirror
  return x;
}

// G groups of four rows a lane: heads of up to 64 G key elements (padded with zero rows). RT_TILE
// tokens a tile: 16 (8 for the widest heads: what fits 64 KB), or 4 for steps of single tokens,
// whose blocks then are all resident at once with a quarter of the LDS and of the loads.
template <int G, int RT_TILE, int MODE, typename TI>
__global__ __launch_bounds__(256) void retention_kernel(RetentionArgs a) {
  constexpr bool STEP = MODE == RT_STEP, GATES = MODE == RT_GATES, PER_TOKEN = STEP || GATES;
  constexpr int DP = 64 * G;                          // rows staged
  constexpr int NQK = 2 * RT_TILE * DP / 256;         // q and k elements a thread fetches per tile
  __shared__ __attribute__((aligned(16))) float qs[RT_TILE * DP];
  __shared__ __attribute__((aligned(16))) float ks[RT_TILE * DP];
  __shared__ float vs[RT_TILE * RT_COLS];
  __shared__ float os[RT_TILE * RT_COLS];
  __shared__ float ds[RT_TILE], steps[RT_TILE];  // a token's decay and what its value is multiplied by (PER_TOKEN)
  const int seq = a.seq_ids ? a.seq_ids[blockIdx.x] : blockIdx.x, head = blockIdx.y, col0 = blockIdx.z * RT_COLS;
  const int t0 = a.cu_q[seq], t1 = a.cu_q[seq + 1];
  if (t1 <= t0) return;
  const int dim = a.dim, vdim = a.vdim;
  const int cols = GATES ? vdim + 1 : vdim;  // columns of the state
  const TI* qkv = (const TI*)a.qkv;
  const int sub = threadIdx.x & 15, colg = threadIdx.x >> 4;  // lane within its column, column of the block
  const int col = col0 + colg;
  const bool col_ok = col < cols;
  const float decay = PER_TOKEN ? 0.f : a.decay[head];
  const float rate = STEP ? expf(a.a_log[head]) : 0.f, bias = STEP ? a.step_bias[head] : 0.f, skip = STEP ? a.skip[head] : 0.f;
  const int qk_head = head / a.share;
  float* st = a.state + (((size_t)a.state_slots[seq] * a.heads + head) * cols + min(col, cols - 1)) * dim;
  const bool vec = (dim & 3) == 0;  // a lane's four rows are 16 aligned bytes of the column
  float s[G][4];
#pragma unroll
  for (int g = 0; g < G; ++g) {
    const int d = 4 * (sub + 16 * g);
    if (vec && d < dim && col_ok) {
      const float4 x = *(const float4*)(st + d);
      s[g][0] = x.x; s[g][1] = x.y; s[g][2] = x.z; s[g][3] = x.w;
    } else {
#pragma unroll
      for (int j = 0; j < 4; ++j) s[g][j] = (d + j < dim && col_ok) ? st[d + j] : 0.f;
    }
  }
  // what this thread fetches of a tile: elements threadIdx.x + 256 i of q | k ([which][token][row]), one of v
  float pre[NQK], pre_v, pre_step = 0.f, pre_write = 0.f;
  auto fetch = [&](int base) {
    const int n = min(RT_TILE, t1 - base);
#pragma unroll
    for (int i = 0; i < NQK; ++i) {
      const int e = threadIdx.x + 256 * i;
      const int which = e / (RT_TILE * DP), tok = (e / DP) % RT_TILE, d = e % DP;
      const bool ok = tok < n && d < dim;
      const TI* row = qkv + (size_t)(base + min(tok, n - 1)) * a.channels + (which ? a.k_first : a.q_first) + qk_head * dim;
      pre[i] = ok ? to_f32<TI>(row[d]) : 0.f;
    }
    const int tok = min((int)threadIdx.x / RT_COLS, RT_TILE - 1), c = threadIdx.x % RT_COLS;
    if (STEP && (int)threadIdx.x < n) {
      const size_t at = (size_t)(base + threadIdx.x) * a.step_stride + head;
      pre_step = a.step_code == QRT_F32 ? ((const float*)a.step)[at] : (float)((const bf16_t*)a.step)[at];
    }
    if (GATES && (int)threadIdx.x < n) {
      const float* row = a.gates + (size_t)(base + threadIdx.x) * 3 * a.heads + head;
      pre_step = row[0];
      pre_write = row[a.heads];
    }
    pre_v = GATES && col0 + c == vdim ? 1.f : (tok < n && col0 + c < vdim) ? to_f32<TI>(qkv[(size_t)(base + tok) * a.channels + a.v_first + head * vdim + col0 + c]) : 0.f;
  };
  fetch(t0);
  for (int base = t0; base < t1; base += RT_TILE) {
    const int n = min(RT_TILE, t1 - base);
    __syncthreads();  // the tile before has been walked and its read-outs have left
#pragma unroll
    for (int i = 0; i < NQK; ++i) {
      const int e = threadIdx.x + 256 * i;
      if (e < RT_TILE * DP) qs[e] = pre[i];
      else ks[e - RT_TILE * DP] = pre[i];
    }
    if (threadIdx.x < RT_TILE * RT_COLS) vs[threadIdx.x] = pre_v;
    if (STEP && threadIdx.x < RT_TILE) {
      const float z = pre_step + bias;
      const float sp = z > 20.f ? z : log1pf(expf(z));
      steps[threadIdx.x] = sp;
      ds[threadIdx.x] = expf(-rate * sp);
    }
    if (GATES && threadIdx.x < RT_TILE) {
      ds[threadIdx.x] = expf(pre_step);
      steps[threadIdx.x] = expf(pre_write);
    }
    __syncthreads();
    if (base + RT_TILE < t1) fetch(base + RT_TILE);  // on its way during the walk
    auto token = [&](int i) {
      const float x = vs[i * RT_COLS + colg];
      const float d = PER_TOKEN ? ds[i] : decay, v = PER_TOKEN ? x * steps[i] : x;
      float acc = 0.f;
#pragma unroll
      for (int g = 0; g < G; ++g) {
        const float4 kd = *(const float4*)(ks + i * DP + 4 * (sub + 16 * g));
        const float4 qd = *(const float4*)(qs + i * DP + 4 * (sub + 16 * g));
        s[g][0] = fmaf(d, s[g][0], kd.x * v); acc = fmaf(s[g][0], qd.x, acc);
        s[g][1] = fmaf(d, s[g][1], kd.y * v); acc = fmaf(s[g][1], qd.y, acc);
        s[g][2] = fmaf(d, s[g][2], kd.z * v); acc = fmaf(s[g][2], qd.z, acc);
        s[g][3] = fmaf(d, s[g][3], kd.w * v); acc = fmaf(s[g][3], qd.w, acc);
      }
      acc = row16_sum(acc);
      if (STEP) acc = fmaf(skip, x, acc);
      if (sub == 0) os[i * RT_COLS + colg] = acc;
    };
    if (n == RT_TILE) {
#pragma unroll 4
      for (int i = 0; i < RT_TILE; ++i) token(i);
    } else {
      for (int i = 0; i < n; ++i) token(i);
    }
    __syncthreads();
    {  // the tile's read-outs: thread (token, column)
      const int tok = threadIdx.x / RT_COLS, c = threadIdx.x % RT_COLS;
      if (tok < n && tok < RT_TILE && col0 + c < vdim) a.out[((size_t)(base + tok) * a.heads + head) * vdim + col0 + c] = os[threadIdx.x];
      if (GATES && tok < n && tok < RT_TILE && col0 + c == vdim) a.last_out[(size_t)(base + tok) * a.heads + head] = os[threadIdx.x];
    }
  }
  if (col_ok) {
#pragma unroll
    for (int g = 0; g < G; ++g) {
      const int d = 4 * (sub + 16 * g);
      if (vec && d < dim) {
        *(float4*)(st + d) = make_float4(s[g][0], s[g][1], s[g][2], s[g][3]);
      } else {
#pragma unroll
        for (int j = 0; j < 4; ++j)
          if (d + j < dim) st[d + j] = s[g][j];
      }
    }
  }
}

extern "C" int qrt_retention(const RetentionArgs* args, int num_tokens, int num_seqs, int num_slots, hipStream_t stream) {
  RetentionArgs a = *args;
  QRT_CHECK(num_tokens >= 0 && num_seqs >= 0 && num_slots > 0, "retention: bad counts");
  QRT_CHECK(a.heads > 0 && a.heads <= 65535 && a.dim > 0 && a.dim <= 512 && a.vdim > 0, "retention: %d heads of %d x %d", a.heads, a.dim, a.vdim);
  if (a.share == 0) a.share = 1;
  QRT_CHECK(a.qkv_code == QRT_F32 || (a.qkv_code == QRT_BF16 && (a.step || a.gates)), "retention: unknown input type %d", a.qkv_code);
  QRT_CHECK(a.share > 0 && a.heads % a.share == 0, "retention: %d heads, %d of which share a key", a.heads, a.share);
  QRT_CHECK(a.channels >= 2 * (a.heads / a.share) * a.dim + a.heads * a.vdim, "retention: %d channels hold no q, k and v", a.channels);
  QRT_CHECK(!a.gates || (a.last_out && !a.step), "retention: gates without a place for the last column's read-out, or beside step logits");
  QRT_CHECK(a.gates ? true : a.step ? a.step_bias && a.a_log && a.skip && a.step_stride >= a.heads : a.decay != nullptr,
            "retention: neither constant decays nor step logits with their bias, rate and skip");
  if (num_tokens == 0 || num_seqs == 0) return 0;
  const dim3 grid(num_seqs, a.heads, (a.vdim + (a.gates ? 1 : 0) + RT_COLS - 1) / RT_COLS);
  const int groups = (a.dim + 63) / 64;
#define GO(G, TILE)                                                                 \
  do {                                                                              \
    if (a.gates && a.qkv_code == QRT_BF16) retention_kernel<G, TILE, RT_GATES, bf16_t><<<grid, 256, 0, stream>>>(a); \
    else if (a.gates) retention_kernel<G, TILE, RT_GATES, float><<<grid, 256, 0, stream>>>(a); \
    else if (a.step && a.qkv_code == QRT_BF16) retention_kernel<G, TILE, RT_STEP, bf16_t><<<grid, 256, 0, stream>>>(a); \
    else if (a.step) retention_kernel<G, TILE, RT_STEP, float><<<grid, 256, 0, stream>>>(a); \
    else retention_kernel<G, TILE, RT_CONSTANT, float><<<grid, 256, 0, stream>>>(a);      \
  } while (0)
  if (num_tokens <= 2 * num_seqs) {  // decoded tokens, mostly
    if (groups <= 1) GO(1, 4);
    else if (groups <= 2) GO(2, 4);
    else if (groups <= 4) GO(4, 4);
    else GO(8, 4);
  } else if (groups <= 1) GO(1, 16);
  else if (groups <= 2) GO(2, 16);
  else if (groups <= 4) GO(4, 16);
  else GO(8, 8);
#undef GO
  QRT_LAUNCH_CHECK("retention");
  return 0;
}
