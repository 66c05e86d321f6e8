// RMS norms in groups: a row is divided into `groups` equal parts of neighbouring elements, each part
// over its own root mean square (eps inside the root), the whole times one weight vector. float32.
//
// group_norm_update: a sub-layer's output joins the residual stream through such a norm, and the
// stream leaves as the next sub-layer reads it (as it is, or through a norm of its own).
// gated_group_norm: the read-out of a recurrence times silu(gate), then the norm.
//
// A block per row. `wpg` waves share a group and `slots` groups are worked on at once, by neighbouring
// waves, so that a group's sum of squares is a wave's sum (wpg = 1) or one exchange over a few floats
// of LDS. A lane takes VEC neighbouring elements at a time and keeps KEEP such pieces in registers (one in
// steps of few rows, which spread a group over as many waves as it has pieces for), all
// of them and the weights asked for before the first use; what a wider group has beyond them is read
// a second time. The order of the additions is fixed by the row's shape and the launch alone.
#include "common.h"
#include <math.h>

template <int VEC> struct VecOf {
  typedef float f __attribute__((ext_vector_type(VEC)));
  typedef bf16_t b __attribute__((ext_vector_type(VEC)));
};

struct GroupSource {  // a matrix (float32 or bfloat16), or float32 planes whose sum it is
  const void* p; int code; int planes; long plane_stride;
};

// PL: the number of planes where it is known when compiling (1: a matrix of either type), -1: any.
template <int VEC, int PL>
__device__ __forceinline__ typename VecOf<VEC>::f source_at(const GroupSource& y, size_t i) {
  typedef typename VecOf<VEC>::f fvec;
  typedef typename VecOf<VEC>::b bvec;
  fvec v;
  if (PL > 1) {
    fvec part[PL > 1 ? PL : 1];
#pragma unroll
    for (int k = 0; k < PL; ++k) part[k] = *(const fvec*)((const float*)y.p + (size_t)k * y.plane_stride + i);
    v = part[0];
#pragma unroll
    for (int k = 1; k < PL; ++k) v += part[k];
    return v;
  }
  if (y.code == QRT_BF16) {
    const bvec b = *(const bvec*)((const bf16_t*)y.p + i);
#pragma unroll
    for (int e = 0; e < VEC; ++e) v[e] = (float)b[e];
    return v;
  }
  const float* p = (const float*)y.p;
  v = *(const fvec*)(p + i);
  if (PL == 1 || y.planes == 1) return v;
  // up to eight planes asked for together (one that is not there: the first again, dropped), added in order
  fvec part[7];
#pragma unroll
  for (int k = 1; k < 8; ++k) part[k - 1] = *(const fvec*)(p + (size_t)(k < y.planes ? k : 0) * y.plane_stride + i);
#pragma unroll
  for (int k = 1; k < 8; ++k)
    if (k < y.planes) v += part[k - 1];
  for (int k = 8; k < y.planes; ++k) v += *(const fvec*)(p + (size_t)k * y.plane_stride + i);
  return v;
}

template <int VEC>
__device__ __forceinline__ float squares(const typename VecOf<VEC>::f& v) {
  float s = 0.f;
#pragma unroll
  for (int e = 0; e < VEC; ++e) s += v[e] * v[e];
  return s;
}

// The sum over the `wpg` waves of a group; every lane of them gets it. With several waves a group all
// waves of the block come here the same number of times (the launch makes as many slots as groups).
__device__ __forceinline__ float group_sum(float x, float* red, int slot, int wpg) {
  x = wave_sum(x);
  if (wpg == 1) return x;
  const int wave = threadIdx.x >> 6;
  __syncthreads();  // red may still be read for the sum before this one
  if ((threadIdx.x & 63) == 0) red[wave] = x;
  __syncthreads();
  x = 0.f;
  for (int i = 0; i < wpg; ++i) x += red[slot * wpg + i];
  return x;
}

template <int VEC, typename TO>
__device__ __forceinline__ void store_vec(TO* p, const typename VecOf<VEC>::f& v) {
  typedef TO ovec __attribute__((ext_vector_type(VEC)));
  ovec o;
#pragma unroll
  for (int e = 0; e < VEC; ++e) o[e] = from_f32<TO>(v[e]);
  *(ovec*)p = o;
}

// r = rows ? rows[b] : b
// x = residual[r] + (w_after ? y[r] / rms(y[r]) * w_after : y[r])   (y.p null: residual[r]); written back
// without `rows`;  out[b] = weight ? x / rms(x) * weight : x
template <typename TO, int VEC, int KEEP, int PL>
__global__ __launch_bounds__(1024) void group_norm_update_kernel(float* __restrict__ residual, GroupSource y,
                                                                 const float* __restrict__ w_after, float eps_after,
                                                                 const float* __restrict__ weight, float eps,
                                                                 const int* __restrict__ rows, TO* __restrict__ out,
                                                                 int hidden, int groups, int wpg, int slots) {
  typedef typename VecOf<VEC>::f fvec;
  __shared__ float red[16];
  const int wave = threadIdx.x >> 6, slot = wave / wpg;
  const int first = ((wave - slot * wpg) * 64 + (threadIdx.x & 63)) * VEC;  // this lane's first element of a group
  const int stride = wpg * 64 * VEC, size = hidden / groups;
  const size_t row = (size_t)(rows ? rows[blockIdx.x] : blockIdx.x) * hidden;
  const size_t orow = (size_t)blockIdx.x * hidden;
  const fvec zero = {};
  for (int g = slot; g < groups; g += slots) {
    const int base = g * size;
    fvec vx[KEEP], vy[KEEP], wa[KEEP], wn[KEEP];
#pragma unroll
    for (int j = 0; j < KEEP; ++j) {
      const int i = base + min(first + j * stride, size - VEC);  // beyond the group: some element of it, dropped below
      vx[j] = *(const fvec*)(residual + row + i);
      vy[j] = y.p ? source_at<VEC, PL>(y, row + i) : zero;
      wa[j] = w_after ? *(const fvec*)(w_after + i) : zero;
      wn[j] = weight ? *(const fvec*)(weight + i) : zero;
    }
    float iy = 1.0f;
    if (w_after) {
      float s = 0.f;
#pragma unroll
      for (int j = 0; j < KEEP; ++j)
        if (first + j * stride < size) s += squares<VEC>(vy[j]);
      for (int i = first + KEEP * stride; i < size; i += stride) s += squares<VEC>(source_at<VEC, PL>(y, row + base + i));
      iy = 1.0f / sqrtf(group_sum(s, red, slot, wpg) / (float)size + eps_after);
    }
    auto joined = [&](const fvec& x, const fvec& d, const fvec& w) -> fvec {
      if (!y.p) return x;
      return w_after ? x + d * iy * w : x + d;
    };
    const bool write_back = y.p && !rows;
    float s = 0.f;
#pragma unroll
    for (int j = 0; j < KEEP; ++j) {
      vx[j] = joined(vx[j], vy[j], wa[j]);
      if (first + j * stride < size) {
        s += squares<VEC>(vx[j]);
        if (write_back) *(fvec*)(residual + row + base + first + j * stride) = vx[j];
        if (!weight) store_vec<VEC, TO>(out + orow + base + first + j * stride, vx[j]);
      }
    }
    for (int i = base + first + KEEP * stride; i < base + size; i += stride) {
      const fvec x = joined(*(const fvec*)(residual + row + i), y.p ? source_at<VEC, PL>(y, row + i) : zero,
                            w_after ? *(const fvec*)(w_after + i) : zero);
      s += squares<VEC>(x);
      if (write_back) *(fvec*)(residual + row + i) = x;
      if (!weight) store_vec<VEC, TO>(out + orow + i, x);
    }
    if (!weight) continue;
    const float ix = 1.0f / sqrtf(group_sum(s, red, slot, wpg) / (float)size + eps);
#pragma unroll
    for (int j = 0; j < KEEP; ++j)
      if (first + j * stride < size) store_vec<VEC, TO>(out + orow + base + first + j * stride, vx[j] * ix * wn[j]);
    for (int i = base + first + KEEP * stride; i < base + size; i += stride) {
      fvec x = *(const fvec*)(residual + row + i);  // the sum already, where it was written back
      if (!write_back)
        x = joined(x, y.p ? source_at<VEC, PL>(y, row + i) : zero, w_after ? *(const fvec*)(w_after + i) : zero);
      store_vec<VEC, TO>(out + orow + i, x * ix * *(const fvec*)(weight + i));
    }
  }
}

// o [T, width] float32, gate rows `gate_stride` elements apart:
// v = o * silu(gate);  out = v / rms(v, per group) * weight
template <typename TG, typename TO, int VEC, int KEEP>
__global__ __launch_bounds__(1024) void gated_group_norm_kernel(const float* __restrict__ o, const TG* __restrict__ gate,
                                                                long gate_stride, const float* __restrict__ weight, float eps,
                                                                TO* __restrict__ out, int width, int groups, int wpg, int slots) {
  typedef typename VecOf<VEC>::f fvec;
  typedef TG gvec __attribute__((ext_vector_type(VEC)));
  __shared__ float red[16];
  const int wave = threadIdx.x >> 6, slot = wave / wpg;
  const int first = ((wave - slot * wpg) * 64 + (threadIdx.x & 63)) * VEC;
  const int stride = wpg * 64 * VEC, size = width / groups;
  const float* orow = o + (size_t)blockIdx.x * width;
  const TG* grow = gate + (size_t)blockIdx.x * gate_stride;
  TO* dst = out + (size_t)blockIdx.x * width;
  auto gated = [&](const fvec& v, const gvec& z) -> fvec {
    fvec r;
#pragma unroll
    for (int e = 0; e < VEC; ++e) {
      const float f = to_f32<TG>(z[e]);
      r[e] = v[e] * (f / (1.0f + expf(-f)));
    }
    return r;
  };
  for (int g = slot; g < groups; g += slots) {
    const int base = g * size;
    fvec v[KEEP], w[KEEP];
    gvec z[KEEP];
#pragma unroll
    for (int j = 0; j < KEEP; ++j) {
      const int i = base + min(first + j * stride, size - VEC);
      v[j] = *(const fvec*)(orow + i);
      z[j] = *(const gvec*)(grow + i);
      w[j] = *(const fvec*)(weight + i);
    }
    float s = 0.f;
#pragma unroll
    for (int j = 0; j < KEEP; ++j) {
      v[j] = gated(v[j], z[j]);
      if (first + j * stride < size) s += squares<VEC>(v[j]);
    }
    for (int i = base + first + KEEP * stride; i < base + size; i += stride)
      s += squares<VEC>(gated(*(const fvec*)(orow + i), *(const gvec*)(grow + i)));
    const float inv = 1.0f / sqrtf(group_sum(s, red, slot, wpg) / (float)size + eps);
#pragma unroll
    for (int j = 0; j < KEEP; ++j)
      if (first + j * stride < size) store_vec<VEC, TO>(dst + base + first + j * stride, v[j] * inv * w[j]);
    for (int i = base + first + KEEP * stride; i < base + size; i += stride)
      store_vec<VEC, TO>(dst + i, gated(*(const fvec*)(orow + i), *(const gvec*)(grow + i)) * inv * *(const fvec*)(weight + i));
  }
}

// Waves a group and groups at once. Few rows: as many waves as the row can use, for one round of
// latency; many rows: as few as hold a group's pieces in registers, so that more rows fit a compute unit.
static void group_launch_shape(int rows, int size, int groups, int vec, int* wpg, int* slots) {
  if (groups > 16) {
    *wpg = 1;
    *slots = 16;
    return;
  }
  const int most = 16 / groups;
  const int per_wave = 64 * vec;
  const int pieces = (size + per_wave - 1) / per_wave;   // waves for one piece a lane
  const int enough = (pieces + 3) / 4;                   // waves that keep the group in registers, four pieces a lane
  const int want = rows <= 256 ? pieces : enough;
  *wpg = want < 1 ? 1 : (want > most ? most : want);
  *slots = groups;
}

// pieces a lane keeps: one or two where that is all there is
static int group_keep(int size, int wpg, int vec) {
  const int wave_pieces = wpg * 64 * vec;
  return size <= wave_pieces ? 1 : size <= 2 * wave_pieces ? 2 : 4;
}

static bool lined_up(const void* p, size_t bytes) { return (uintptr_t)p % bytes == 0; }

extern "C" int qrt_group_norm_update(float* residual, const void* y, int y_code, int y_planes, long plane_stride,
                                     const float* w_after, float eps_after, const float* weight, float eps, const int* rows,
                                     void* out, int out_dtype, int num_out, int hidden, int groups, hipStream_t stream) {
  QRT_CHECK(num_out >= 0 && hidden > 0 && groups >= 1 && hidden % groups == 0, "group_norm_update: %d elements in %d groups", hidden, groups);
  QRT_CHECK(y || !w_after, "group_norm_update: a norm on an output that is not there");
  QRT_CHECK(!y || (y_planes >= 1 && (y_code == QRT_F32 || (y_code == QRT_BF16 && y_planes == 1))), "group_norm_update: planes are float32");
  QRT_CHECK(out_dtype == QRT_F32 || out_dtype == QRT_BF16, "group_norm_update: unknown dtype %d", out_dtype);
  if (num_out == 0) return 0;
  const GroupSource src{y, y_code, y ? y_planes : 1, plane_stride};
  const int size = hidden / groups;
  const bool vec4 = size % 4 == 0 && lined_up(residual, 16) && lined_up(y, 16) && lined_up(w_after, 16) && lined_up(weight, 16) &&
                    lined_up(out, 16) && plane_stride % 4 == 0;
  int wpg, slots;
  group_launch_shape(num_out, size, groups, vec4 ? 4 : 1, &wpg, &slots);
  const dim3 grid(num_out), block(64 * wpg * slots);
  const int keep = group_keep(size, wpg, vec4 ? 4 : 1), pl = y ? y_planes : 1;
#define GO(TO, VEC, KEEP, PL) group_norm_update_kernel<TO, VEC, KEEP, PL><<<grid, block, 0, stream>>>( \
    residual, src, w_after, eps_after, weight, eps, rows, (TO*)out, hidden, groups, wpg, slots)
#define PICK(TO)                              \
  do {                                        \
    if (!vec4) GO(TO, 1, 4, -1);              \
    else if (keep == 4 && pl == 1) GO(TO, 4, 4, 1); \
    else if (keep == 4) GO(TO, 4, 4, -1);     \
    else if (keep == 2 && pl == 1) GO(TO, 4, 2, 1); \
    else if (keep == 2 && pl == 2) GO(TO, 4, 2, 2); \
    else if (keep == 2) GO(TO, 4, 2, -1);     \
    else if (pl == 1) GO(TO, 4, 1, 1);        \
    else if (pl == 2) GO(TO, 4, 1, 2);        \
    else if (pl == 3) GO(TO, 4, 1, 3);        \
    else if (pl == 4) GO(TO, 4, 1, 4);        \
    else if (pl == 5) GO(TO, 4, 1, 5);        \
    else if (pl == 8) GO(TO, 4, 1, 8);        \
    else if (pl == 9) GO(TO, 4, 1, 9);        \
    else GO(TO, 4, 1, -1);                    \
  } while (0)
  if (out_dtype == QRT_F32) PICK(float);
  else PICK(bf16_t);
#undef PICK
#undef GO
  QRT_LAUNCH_CHECK("group_norm_update");
  return 0;
}

extern "C" int qrt_gated_group_norm(const float* o, const void* gate, long gate_stride, int gate_dtype, const float* weight,
                                    float eps, void* out, int out_dtype, int num_tokens, int width, int groups,
                                    hipStream_t stream) {
  QRT_CHECK(num_tokens >= 0 && width > 0 && groups >= 1 && width % groups == 0 && gate_stride >= width,
            "gated_group_norm: %d elements in %d groups, gate rows of %ld", width, groups, gate_stride);
  QRT_CHECK((gate_dtype == QRT_F32 && out_dtype == QRT_F32) || (gate_dtype == QRT_BF16 && out_dtype == QRT_BF16) ||
                (gate_dtype == QRT_F32 && out_dtype == QRT_BF16),
            "gated_group_norm: unknown dtypes %d %d", gate_dtype, out_dtype);
  if (num_tokens == 0) return 0;
  const int size = width / groups;
  const size_t gate_bytes = gate_dtype == QRT_F32 ? 16 : 8;
  const bool vec4 = size % 4 == 0 && gate_stride % 4 == 0 && lined_up(o, 16) && lined_up(gate, gate_bytes) && lined_up(weight, 16) && lined_up(out, 16);
  int wpg, slots;
  group_launch_shape(num_tokens, size, groups, vec4 ? 4 : 1, &wpg, &slots);
  const dim3 grid(num_tokens), block(64 * wpg * slots);
  const int keep = group_keep(size, wpg, vec4 ? 4 : 1);
#define GO(TG, TO, VEC, KEEP) gated_group_norm_kernel<TG, TO, VEC, KEEP><<<grid, block, 0, stream>>>( \
    o, (const TG*)gate, gate_stride, weight, eps, (TO*)out, width, groups, wpg, slots)
#define PICK(TG, TO) do { if (!vec4) GO(TG, TO, 1, 4); else if (keep == 4) GO(TG, TO, 4, 4); else if (keep == 2) GO(TG, TO, 4, 2); else GO(TG, TO, 4, 1); } while (0)
  if (gate_dtype == QRT_F32 && out_dtype == QRT_F32) PICK(float, float);
  else if (gate_dtype == QRT_BF16) PICK(bf16_t, bf16_t);
  else PICK(float, bf16_t);
#undef PICK
#undef GO
  QRT_LAUNCH_CHECK("gated_group_norm");
  return 0;
}
