// Kernels around attention through a cached latent: an RMS norm over a run of columns of a wider row, and a
// rotation by position of a part of every head's vector with a choice of pairing.  Both read 32-bit results of a
// product and write in the dtype of whatever reads them next, into a place of the caller's (a run of columns of a
// wider row), so that a norm, a rotation and the assembly of a cached row or of a query need no copies.
#include "common.h"

namespace {

// out[r, :] = src[r, :] / sqrt(mean(src[r, :]^2) + eps) * w; one workgroup a row
template <typename T>
__global__ __launch_bounds__(256) void rmsnorm_cols_kernel(const float* __restrict__ src, int lds_, const float* __restrict__ w,
                                                           float eps, T* __restrict__ out, int ldo, int n) {
  __shared__ float red[16];
  const float* s = src + (long long)blockIdx.x * lds_;
  T* o = out + (long long)blockIdx.x * ldo;
  float acc = 0.f;
  for (int i = threadIdx.x; i < n; i += 256) acc = fmaf(s[i], s[i], acc);
  const float inv = 1.f / sqrtf(block_sum(acc, red) / (float)n + eps);
  for (int i = threadIdx.x; i < n; i += 256) o[i] = from_f32<T>(s[i] * inv * w[i]);
}

// Row r, head h: the vector src[r, h * size .. + size) goes to out[r, h * ohs .. + size); its first `dims` entries
// are rotated by the angles row_pos[r] * freqs[j], in pairs (j, j + dims / 2) or (2 j, 2 j + 1): (u, v) ->
// (u c - v s, v c + u s) with c and s times `mag`; the rest pass.  Angles in double, reduced to [-pi, pi] before
// the 32-bit sine and cosine.
template <typename T>
__global__ __launch_bounds__(128) void rotary_kernel(const float* __restrict__ src, int lds_, T* __restrict__ out, int ldo,
                                                     int heads, int size, int ohs, int dims, int interleaved,
                                                     const double* __restrict__ freqs, float mag,
                                                     const int* __restrict__ row_pos) {
  extern __shared__ float cs[];  // cos[dims / 2], sin[dims / 2]
  const int r = blockIdx.x, half = dims / 2;
  const int p = row_pos[r];
  for (int j = threadIdx.x; j < half; j += blockDim.x) {
    const double a = (double)p * freqs[j];
    const double n = rint(a * 0.15915494309189533577);
    double rem = fma(-n, 6.283185307179586232, a);
    rem = fma(-n, 2.4492935982947064e-16, rem);
    float sn, c;
    sincosf((float)rem, &sn, &c);
    cs[j] = c * mag;
    cs[half + j] = sn * mag;
  }
  __syncthreads();
  const float* s = src + (long long)r * lds_;
  T* o = out + (long long)r * ldo;
  for (int e = threadIdx.x; e < heads * size; e += blockDim.x) {
    const int h = e / size, i = e - h * size;
    const float* v = s + h * size;
    float res;
    if (i >= dims) {
      res = v[i];
    } else {
      int j, mate;
      bool first;
      if (interleaved) j = i >> 1, first = !(i & 1), mate = i ^ 1;
      else first = i < half, j = first ? i : i - half, mate = first ? i + half : i - half;
      const float c = cs[j], sn = cs[half + j];
      res = first ? v[i] * c - v[mate] * sn : v[i] * c + v[mate] * sn;
    }
    o[h * ohs + i] = from_f32<T>(res);
  }
}

// Queries, keys and values of a step's rows, from the 32-bit result of their one product to what the attention
// kernel and the cache read.  src [rows, (H + G) D + G V]: H query heads, G key heads, G value heads.  Of every query
// and key head the first `dims` entries are rotated as in `rotary_kernel`; then, with norm_eps >= 0, the whole head
// is divided by its root mean square over D (eps inside the root); values pass.  gridDim.y workgroups a row share
// its heads and values out (one where the rows alone fill the chip); a wavefront takes a head at a time (its sum of
// squares is the wavefront's fixed tree, so it depends on the row alone, not on how the heads were shared out).
template <typename T>
__global__ __launch_bounds__(256) void rotary_qkv_kernel(const float* __restrict__ src, int lds_, T* __restrict__ q_out,
                                                         int ldq, T* __restrict__ k_out, int ldk, T* __restrict__ v_out,
                                                         int ldv, int H, int G, int D, int VW, int dims, int interleaved,
                                                         const double* __restrict__ freqs, float mag, float norm_eps,
                                                         const int* __restrict__ row_pos) {
  extern __shared__ float cs[];  // cos[dims / 2], sin[dims / 2]
  const int r = blockIdx.x, half = dims / 2;
  const int p = row_pos[r];
  for (int j = threadIdx.x; j < half; j += blockDim.x) {
    const double a = (double)p * freqs[j];
    const double n = rint(a * 0.15915494309189533577);
    double rem = fma(-n, 6.283185307179586232, a);
    rem = fma(-n, 2.4492935982947064e-16, rem);
    float sn, c;
    sincosf((float)rem, &sn, &c);
    cs[j] = c * mag;
    cs[half + j] = sn * mag;
  }
  __syncthreads();
  const float* s = src + (long long)r * lds_;
  const int wave = threadIdx.x >> 6, lane = threadIdx.x & 63, waves = blockDim.x >> 6;
  for (int h = blockIdx.y * waves + wave; h < H + G; h += waves * gridDim.y) {
    const float* v = s + h * D;
    T* o = h < H ? q_out + (long long)r * ldq + h * D : k_out + (long long)r * ldk + (h - H) * D;
    auto turned = [&](int i) -> float {
      if (i >= dims) return v[i];
      int j, mate;
      bool first;
      if (interleaved) j = i >> 1, first = !(i & 1), mate = i ^ 1;
      else first = i < half, j = first ? i : i - half, mate = first ? i + half : i - half;
      const float c = cs[j], sn = cs[half + j];
      return first ? v[i] * c - v[mate] * sn : v[i] * c + v[mate] * sn;
    };
    float inv = 1.f;
    if (norm_eps >= 0.f) {
      float ss = 0.f;
      for (int i = lane; i < D; i += 64) {
        const float t = turned(i);
        ss = fmaf(t, t, ss);
      }
      inv = 1.f / sqrtf(wave_sum(ss) / (float)D + norm_eps);
    }
    for (int i = lane; i < D; i += 64) o[i] = from_f32<T>(turned(i) * inv);
  }
  const float* vs = s + (H + G) * D;
  T* vo = v_out + (long long)r * ldv;
  for (int e = blockIdx.y * blockDim.x + threadIdx.x; e < VW; e += blockDim.x * gridDim.y) vo[e] = from_f32<T>(vs[e]);
}

// Queries, keys and values of a step's rows, from the 32-bit result of their one product to what the attention kernel
// reads and straight into the paged cache.  src [rows, H D + G D (+ G V)]; `bias` (a number a column, or null) is added
// first.  With `cs` (cos and sin of the row's angles, [rows][dims / 2][2]) the first `dims` entries of every query and key
// head are then rotated, pairs and magnitude as in `rotary_kernel` (units of a head only).  q and k are normed in units of `unit_q` and `unit_k` entries (a head each, or the whole row of
// all heads; units divided by their root mean square, eps inside the root, times a weight of the unit's size), values in
// units of a head without a weight (`norm_v`) or not at all; `v_from_k`: there are no value columns, the values are the
// keys as they are before rotation and norm.  k and v go to the row's position in the cache (K [block][G][BS][D],
// V [block][G][V][BS]); kcache null: q alone is wanted.  A wavefront takes a unit (WIDE: a workgroup), so a unit's sum of
// squares is one fixed tree whatever else is in the launch.
struct QkvUnits {
  int lds, ldq, H, G, D, V, unit_q, unit_k, norm_qk, norm_v, v_from_k;
  float eps;
  const float *bias, *wq, *wk;
  const int *row_pos, *row_seq, *seq_slot, *block_table;
  int bt_stride, BS;
  int unit_v;  // value entries a unit
  const float* cs;
  int dims, interleaved;
  float mag;
};

// Entry i of a head (v its value, `mate` what the entry of its pair holds) after the rotation.
__device__ inline float turned_entry(const QkvUnits& a, const float* cs, int i, float v, float mate) {
  const int half = a.dims >> 1, j = a.interleaved ? i >> 1 : i < half ? i : i - half;
  const bool first = a.interleaved ? !(i & 1) : i < half;
  const float c = cs[2 * j] * a.mag, s = cs[2 * j + 1] * a.mag;
  return first ? v * c - mate * s : v * c + mate * s;
}

__device__ inline int pair_mate(const QkvUnits& a, int i) {
  return a.interleaved ? i ^ 1 : i < (a.dims >> 1) ? i + (a.dims >> 1) : i - (a.dims >> 1);
}

template <typename T, bool WIDE>
__global__ __launch_bounds__(256) void qkv_norm_store_kernel(const float* __restrict__ src, T* __restrict__ q_out,
                                                             T* __restrict__ kcache, T* __restrict__ vcache, QkvUnits a) {
  __shared__ float red[16];
  const int r = blockIdx.x;
  const int i0 = WIDE ? threadIdx.x : threadIdx.x & 63;
  constexpr int STEP = WIDE ? 256 : 64;
  int u = WIDE ? (int)blockIdx.y : (int)blockIdx.y * 4 + (int)(threadIdx.x >> 6);
  const int QW = a.H * a.D, KW = a.G * a.D, VW = a.G * a.V, unit_v = a.unit_v;
  const int nq = QW / a.unit_q, nk = kcache != nullptr ? KW / a.unit_k : 0, nv = kcache != nullptr ? VW / unit_v : 0;
  if (u >= nq + nk + nv) return;  // (WIDE: the whole workgroup)
  const int which = u < nq ? 0 : u < nq + nk ? 1 : 2;
  int n, at, col;  // the unit's entries, its first entry among its kind, its first column in src
  const float* w = nullptr;
  bool norm = a.norm_qk != 0;
  if (which == 0) n = a.unit_q, at = u * n, col = at, w = a.wq;
  else if (which == 1) n = a.unit_k, at = (u - nq) * n, col = QW + at, w = a.wk;
  else n = unit_v, at = (u - nq - nk) * n, col = (a.v_from_k ? QW : QW + KW) + at, norm = a.norm_v != 0;
  const float* s = src + (long long)r * a.lds + col;
  const float* b = a.bias != nullptr ? a.bias + col : nullptr;
  const float* cs = a.cs != nullptr && which != 2 ? a.cs + (long long)r * a.dims : nullptr;
  auto entry = [&](int i) -> float {
    const float v = b != nullptr ? s[i] + b[i] : s[i];
    if (cs == nullptr || i >= a.dims) return v;
    const int m = pair_mate(a, i);
    return turned_entry(a, cs, i, v, b != nullptr ? s[m] + b[m] : s[m]);
  };
  float inv = 1.f;
  if (norm) {
    float ss = 0.f;
    for (int i = i0; i < n; i += STEP) {
      const float v = entry(i);
      ss = fmaf(v, v, ss);
    }
    inv = 1.f / sqrtf((WIDE ? block_sum(ss, red) : wave_sum(ss)) / (float)n + a.eps);
  }
  long long blk = 0;
  int off = 0;
  if (which != 0) {
    const int p = a.row_pos[r];
    blk = a.block_table[(long long)a.seq_slot[a.row_seq[r]] * a.bt_stride + p / a.BS];
    off = p % a.BS;
  }
  for (int i = i0; i < n; i += STEP) {
    float v = entry(i);
    if (norm) v *= inv;
    if (w != nullptr) v *= w[i];
    const int e = at + i;
    if (which == 0) {
      q_out[(long long)r * a.ldq + e] = from_f32<T>(v);
    } else if (which == 1) {
      const int g = e / a.D;
      kcache[((blk * a.G + g) * a.BS + off) * (long long)a.D + e - g * a.D] = from_f32<T>(v);
    } else {
      const int g = e / a.V;
      vcache[((blk * a.G + g) * (long long)a.V + e - g * a.V) * a.BS + off] = from_f32<T>(v);
    }
  }
}

// The same with a unit's entries in registers (a unit is read once), for units, head sizes and rows in fours: PER runs of
// four entries a thread.
template <typename T, bool WIDE, int PER>
__global__ __launch_bounds__(256) void qkv_norm_store4_kernel(const float* __restrict__ src, T* __restrict__ q_out,
                                                              T* __restrict__ kcache, T* __restrict__ vcache, QkvUnits a) {
  __shared__ float red[16];
  const int r = blockIdx.x;
  const int i0 = WIDE ? threadIdx.x : threadIdx.x & 63;
  constexpr int STEP = WIDE ? 256 : 64;
  const int u = WIDE ? (int)blockIdx.y : (int)blockIdx.y * 4 + (int)(threadIdx.x >> 6);
  const int QW = a.H * a.D, KW = a.G * a.D, VW = a.G * a.V, unit_v = a.unit_v;
  const int nq = QW / a.unit_q, nk = kcache != nullptr ? KW / a.unit_k : 0, nv = kcache != nullptr ? VW / unit_v : 0;
  if (u >= nq + nk + nv) return;  // (WIDE: the whole workgroup)
  const int which = u < nq ? 0 : u < nq + nk ? 1 : 2;
  int n, at, col;
  const float* w = nullptr;
  bool norm = a.norm_qk != 0;
  if (which == 0) n = a.unit_q, at = u * n, col = at, w = a.wq;
  else if (which == 1) n = a.unit_k, at = (u - nq) * n, col = QW + at, w = a.wk;
  else n = unit_v, at = (u - nq - nk) * n, col = (a.v_from_k ? QW : QW + KW) + at, norm = a.norm_v != 0;
  const float4* s = (const float4*)(src + (long long)r * a.lds + col);
  const float4* b = a.bias != nullptr ? (const float4*)(a.bias + col) : nullptr;
  const int quads = n / 4;
  float4 v[PER];
  float ss = 0.f;
#pragma unroll
  for (int j = 0; j < PER; ++j) {
    const int i = i0 + j * STEP;
    v[j] = i < quads ? s[i] : make_float4(0.f, 0.f, 0.f, 0.f);
    if (b != nullptr && i < quads) {
      const float4 add = b[i];
      v[j].x += add.x, v[j].y += add.y, v[j].z += add.z, v[j].w += add.w;
    }
  }
  if (a.cs != nullptr && which != 2) {
    const float* cs = a.cs + (long long)r * a.dims;
    const float* sf = (const float*)s;
    const float* bf = (const float*)b;
#pragma unroll
    for (int j = 0; j < PER; ++j) {
      const int e = 4 * (i0 + j * STEP);
      if (e >= n || e >= a.dims) continue;
      float* x = &v[j].x;
      float mate[4];
#pragma unroll
      for (int k = 0; k < 4; ++k) {
        if (a.interleaved) mate[k] = x[k ^ 1];
        else {
          const int m = e + k < a.dims ? pair_mate(a, e + k) : e;
          mate[k] = bf != nullptr ? sf[m] + bf[m] : sf[m];
        }
      }
#pragma unroll
      for (int k = 0; k < 4; ++k)
        if (e + k < a.dims) x[k] = turned_entry(a, cs, e + k, x[k], mate[k]);
    }
  }
  long long blk = 0;
  int off = 0;
  if (which != 0) {
    const int p = a.row_pos[r];
    blk = a.block_table[(long long)a.seq_slot[a.row_seq[r]] * a.bt_stride + p / a.BS];
    off = p % a.BS;
  }
  float inv = 1.f;
  if (norm) {
#pragma unroll
    for (int j = 0; j < PER; ++j)
      ss = fmaf(v[j].x, v[j].x, fmaf(v[j].y, v[j].y, fmaf(v[j].z, v[j].z, fmaf(v[j].w, v[j].w, ss))));
    inv = 1.f / sqrtf((WIDE ? block_sum(ss, red) : wave_sum(ss)) / (float)n + a.eps);
  }
#pragma unroll
  for (int j = 0; j < PER; ++j) {
    const int i = i0 + j * STEP;
    if (i >= quads) continue;
    float x0 = v[j].x * inv, x1 = v[j].y * inv, x2 = v[j].z * inv, x3 = v[j].w * inv;
    if (w != nullptr) {
      const float4 wv = ((const float4*)w)[i];
      x0 *= wv.x, x1 *= wv.y, x2 *= wv.z, x3 *= wv.w;
    }
    const int e = at + 4 * i;
    if (which == 2) {
      const int g = e / a.V;
      T* o = vcache + ((blk * a.G + g) * (long long)a.V + e - g * a.V) * a.BS + off;
      o[0] = from_f32<T>(x0), o[a.BS] = from_f32<T>(x1), o[2 * a.BS] = from_f32<T>(x2), o[3 * a.BS] = from_f32<T>(x3);
      continue;
    }
    const int g = e / a.D;
    T* o = which == 0 ? q_out + (long long)r * a.ldq + e : kcache + ((blk * a.G + g) * a.BS + off) * (long long)a.D + e - g * a.D;
    if constexpr (sizeof(T) == 4) {
      *(float4*)o = make_float4(x0, x1, x2, x3);
    } else {
      uint2 packed;
      packed.x = (uint32_t)f32_to_bf16(x0).bits | ((uint32_t)f32_to_bf16(x1).bits << 16);
      packed.y = (uint32_t)f32_to_bf16(x2).bits | ((uint32_t)f32_to_bf16(x3).bits << 16);
      *(uint2*)o = packed;
    }
  }
}

// A product a head: out[r, h ohs + n] = sum_k x[r, h K + k] w[h, n, k], bfloat16 operands on
// v_mfma_f32_16x16x16_bf16 (exact products, 32-bit sums).  A workgroup of four wavefronts takes 64 rows by 64
// columns of one head; a wavefront 16 rows by the 64 columns, its operands straight from memory (a head's weight
// is small and stays in the caches; the four wavefronts read the same columns).  K in steps of 16, ascending: a
// row's sums do not depend on what else is in the launch.
typedef short bf16x4_t __attribute__((ext_vector_type(4)));
typedef float f32x4_t __attribute__((ext_vector_type(4)));

template <typename TO>
__global__ __launch_bounds__(256) void linear_heads_kernel(const bf16_t* __restrict__ x, int ldx,
                                                           const bf16_t* __restrict__ w, TO* __restrict__ out, int ldo,
                                                           int rows, int N, int K, int ohs) {
  const int wave = threadIdx.x >> 6, lane = threadIdx.x & 63, c = lane & 15, g = lane >> 4;
  const int h = blockIdx.z, r0 = blockIdx.x * 64 + 16 * wave, n0 = blockIdx.y * 64;
  if (r0 >= rows) return;
  const bf16_t* xa = x + (long long)min(r0 + c, rows - 1) * ldx + (long long)h * K + 4 * g;
  const bf16_t* wb[4];
#pragma unroll
  for (int j = 0; j < 4; ++j) wb[j] = w + ((long long)h * N + min(n0 + 16 * j + c, N - 1)) * K + 4 * g;
  f32x4_t acc[4];
#pragma unroll
  for (int j = 0; j < 4; ++j) acc[j] = (f32x4_t){0.f, 0.f, 0.f, 0.f};
  for (int ks = 0; ks < K; ks += 16) {
    const bf16x4_t a = __builtin_bit_cast(bf16x4_t, *(const uint2*)(xa + ks));
#pragma unroll
    for (int j = 0; j < 4; ++j) {
      const bf16x4_t bv = __builtin_bit_cast(bf16x4_t, *(const uint2*)(wb[j] + ks));
      acc[j] = __builtin_amdgcn_mfma_f32_16x16x16bf16_1k(a, bv, acc[j], 0, 0, 0);
    }
  }
#pragma unroll
  for (int j = 0; j < 4; ++j) {
    const int n = n0 + 16 * j + c;
    if (n >= N) continue;
#pragma unroll
    for (int e = 0; e < 4; ++e) {
      const int r = r0 + 4 * g + e;
      if (r < rows) out[(long long)r * ldo + (long long)h * ohs + n] = from_f32<TO>(acc[j][e]);
    }
  }
}

}  // namespace

extern "C" int lq_rmsnorm_cols(const float* src, int lds_, const float* w, float eps, void* out, int out_dtype, int ldo,
                               int rows, int n, hipStream_t stream) {
  LQ_REQUIRE(rows > 0 && n > 0 && lds_ >= n && ldo >= n, "rmsnorm_cols: rows %d, columns %d, strides %d and %d", rows, n, lds_, ldo);
  LQ_REQUIRE(src && w && out, "rmsnorm_cols: null pointer");
  if (out_dtype == LQ_F32) rmsnorm_cols_kernel<float><<<rows, 256, 0, stream>>>(src, lds_, w, eps, (float*)out, ldo, n);
  else if (out_dtype == LQ_BF16) rmsnorm_cols_kernel<bf16_t><<<rows, 256, 0, stream>>>(src, lds_, w, eps, (bf16_t*)out, ldo, n);
  else LQ_REQUIRE(false, "rmsnorm_cols: unknown dtype %d", out_dtype);
  LQ_CHECK_LAUNCH("rmsnorm_cols");
  return 0;
}

extern "C" int lq_rotary(const float* src, int lds_, void* out, int out_dtype, int ldo, int rows, int heads, int size,
                         int out_head_stride, int dims, int interleaved, const double* freqs, float magnitude,
                         const int* row_pos, hipStream_t stream) {
  LQ_REQUIRE(rows > 0 && heads > 0 && size > 0, "rotary: rows %d, heads %d, size %d", rows, heads, size);
  LQ_REQUIRE(dims >= 2 && dims % 2 == 0 && dims <= size && dims <= 8192, "rotary: %d rotated entries of %d", dims, size);
  LQ_REQUIRE(out_head_stride >= size && lds_ >= heads * size && ldo >= (heads - 1) * out_head_stride + size,
             "rotary: a stride is smaller than what it steps over");
  LQ_REQUIRE(src && out && freqs && row_pos, "rotary: null pointer");
  const size_t lds_bytes = (size_t)dims * sizeof(float);
  if (out_dtype == LQ_F32)
    rotary_kernel<float><<<rows, 128, lds_bytes, stream>>>(src, lds_, (float*)out, ldo, heads, size, out_head_stride, dims,
                                                           interleaved, freqs, magnitude, row_pos);
  else if (out_dtype == LQ_BF16)
    rotary_kernel<bf16_t><<<rows, 128, lds_bytes, stream>>>(src, lds_, (bf16_t*)out, ldo, heads, size, out_head_stride, dims,
                                                            interleaved, freqs, magnitude, row_pos);
  else LQ_REQUIRE(false, "rotary: unknown dtype %d", out_dtype);
  LQ_CHECK_LAUNCH("rotary");
  return 0;
}

// src [rows, (heads + kv_heads) * key_dim + kv_heads * value_dim] float32 (stride lds_): queries, keys, values.
// dims = 0: no rotation (freqs may be null); norm_eps < 0: no norm.
extern "C" int lq_rotary_qkv(const float* src, int lds_, void* q_out, int ldq, void* k_out, int ldk, void* v_out, int ldv,
                             int out_dtype, int rows, int heads, int kv_heads, int key_dim, int value_dim, int dims,
                             int interleaved, const double* freqs, float magnitude, float norm_eps, const int* row_pos,
                             int value_width, hipStream_t stream) {
  // `value_width` > 0: so many value entries a row pass, in the place of kv_heads * value_dim (key heads that share
  // a value head)
  const int VW = value_width > 0 ? value_width : kv_heads * value_dim;
  LQ_REQUIRE(rows > 0 && heads > 0 && kv_heads > 0 && key_dim > 0 && value_dim > 0, "rotary_qkv: rows %d, heads %d and %d, sizes %d and %d",
             rows, heads, kv_heads, key_dim, value_dim);
  LQ_REQUIRE(dims >= 0 && dims % 2 == 0 && dims <= key_dim && dims <= 8192, "rotary_qkv: %d rotated entries of %d", dims, key_dim);
  LQ_REQUIRE(lds_ >= (heads + kv_heads) * key_dim + VW && ldq >= heads * key_dim && ldk >= kv_heads * key_dim &&
                 ldv >= VW, "rotary_qkv: a row stride is smaller than its row");
  LQ_REQUIRE(src && q_out && k_out && v_out && row_pos && (dims == 0 || freqs), "rotary_qkv: null pointer");
  const size_t lds_bytes = (size_t)dims * sizeof(float);
  // few rows (single tokens): a wavefront a head, so that no wavefront walks through its heads one after the other
  const int share = rows >= 512 ? 1 : (lq_ceil_div(heads + kv_heads, 4) < 64 ? lq_ceil_div(heads + kv_heads, 4) : 64);
  const dim3 grid(rows, share);
  if (out_dtype == LQ_F32)
    rotary_qkv_kernel<float><<<grid, 256, lds_bytes, stream>>>(src, lds_, (float*)q_out, ldq, (float*)k_out, ldk, (float*)v_out,
                                                               ldv, heads, kv_heads, key_dim, VW, dims, interleaved,
                                                               freqs, magnitude, norm_eps, row_pos);
  else if (out_dtype == LQ_BF16)
    rotary_qkv_kernel<bf16_t><<<grid, 256, lds_bytes, stream>>>(src, lds_, (bf16_t*)q_out, ldq, (bf16_t*)k_out, ldk,
                                                                (bf16_t*)v_out, ldv, heads, kv_heads, key_dim, VW, dims,
                                                                interleaved, freqs, magnitude, norm_eps, row_pos);
  else LQ_REQUIRE(false, "rotary_qkv: unknown dtype %d", out_dtype);
  LQ_CHECK_LAUNCH("rotary_qkv");
  return 0;
}

// bias: null or a number for every column of src; wq, wk: weights of unit_q and unit_k entries, or null (with
// `norm_qk` off: no norm of q and k); kcache and vcache null: q alone.
extern "C" int lq_qkv_norm_store(const float* src, int lds_, const float* bias, const float* wq, const float* wk, int unit_q,
                                 int unit_k, int norm_qk, int norm_v, int v_from_k, float eps, void* q_out, int ldq, int dtype,
                                 int rows, int heads, int kv_heads, int key_dim, int value_dim, const int* row_pos,
                                 const int* row_seq, const int* seq_slot, const int* block_table, int bt_stride, void* kcache,
                                 void* vcache, int block_size, const float* cos_sin, int dims, int interleaved,
                                 float magnitude, hipStream_t stream) {
  LQ_REQUIRE(cos_sin == nullptr || (dims >= 2 && dims % 2 == 0 && dims <= key_dim && unit_q == key_dim && unit_k == key_dim),
             "qkv_norm_store: %d rotated entries in units of %d and %d for heads of %d", dims, unit_q, unit_k, key_dim);
  LQ_REQUIRE(rows > 0 && rows <= 0x7fffffff && heads > 0 && kv_heads > 0 && key_dim > 0 && value_dim > 0,
             "qkv_norm_store: rows %d, heads %d and %d, sizes %d and %d", rows, heads, kv_heads, key_dim, value_dim);
  LQ_REQUIRE(!v_from_k || key_dim == value_dim, "qkv_norm_store: values that are the keys have their size (%d, %d)", key_dim, value_dim);
  const int QW = heads * key_dim, KW = kv_heads * key_dim, VW = kv_heads * value_dim;
  LQ_REQUIRE(unit_q > 0 && unit_k > 0 && QW % unit_q == 0 && KW % unit_k == 0, "qkv_norm_store: units of %d and %d entries", unit_q, unit_k);
  LQ_REQUIRE(lds_ >= QW + KW + (v_from_k ? 0 : VW) && ldq >= QW, "qkv_norm_store: a row stride is smaller than its row");
  LQ_REQUIRE(src && q_out && (kcache == nullptr) == (vcache == nullptr), "qkv_norm_store: null pointer");
  LQ_REQUIRE(kcache == nullptr || (row_pos && row_seq && seq_slot && block_table && block_size > 0 && bt_stride > 0),
             "qkv_norm_store: the cache needs the rows' places");
  LQ_REQUIRE(norm_qk || (wq == nullptr && wk == nullptr), "qkv_norm_store: weights without a norm");
  // (values go head by head where queries and keys do; they are only copied there)
  const int unit_v = norm_v || (unit_q == key_dim && unit_k == key_dim) ? value_dim : VW;
  QkvUnits a = {lds_, ldq, heads, kv_heads, key_dim, value_dim, unit_q, unit_k, norm_qk, norm_v, v_from_k,
                eps, bias, wq, wk, row_pos, row_seq, seq_slot, block_table, bt_stride, block_size,
                unit_v, cos_sin, cos_sin != nullptr ? dims : 0, interleaved, magnitude};
  const int units = QW / unit_q + (kcache ? KW / unit_k + VW / unit_v : 0);
  const bool wide = unit_q > 512 || unit_k > 512 || (kcache && unit_v > 512);
  const int gy = wide ? units : lq_ceil_div(units, 4);
  LQ_REQUIRE(gy <= 65535, "qkv_norm_store: too many heads");
  const dim3 grid(rows, gy);
  // what fits the kernel that keeps a unit in registers: everything in fours on whole vectors (the choice follows from
  // the model's sizes and the buffers' alignment, which are the same in every step)
  const int el = dtype == LQ_F32 ? 4 : 2;
  int most = unit_q > unit_k ? unit_q : unit_k;
  if (kcache != nullptr && unit_v > most) most = unit_v;
  const bool fours = key_dim % 4 == 0 && value_dim % 4 == 0 && lds_ % 4 == 0 && ldq % 4 == 0 && (uintptr_t)src % 16 == 0 &&
                     (uintptr_t)bias % 16 == 0 && (uintptr_t)wq % 16 == 0 && (uintptr_t)wk % 16 == 0 &&
                     (uintptr_t)q_out % (4 * el) == 0 && (uintptr_t)kcache % (4 * el) == 0 && most <= 16384;
#define LQ_QKV4(T, WIDE, PER)                                                                                        \
  qkv_norm_store4_kernel<T, WIDE, PER><<<grid, 256, 0, stream>>>(src, (T*)q_out, (T*)kcache, (T*)vcache, a)
#define LQ_QKV(T)                                                                                                    \
  do {                                                                                                               \
    if (fours && !wide && most <= 256) LQ_QKV4(T, false, 1);                                                         \
    else if (fours && !wide) LQ_QKV4(T, false, 2);                                                                   \
    else if (fours && most <= 4096) LQ_QKV4(T, true, 4);                                                             \
    else if (fours) LQ_QKV4(T, true, 16);                                                                            \
    else                                                                                                             \
    if (wide) qkv_norm_store_kernel<T, true><<<grid, 256, 0, stream>>>(src, (T*)q_out, (T*)kcache, (T*)vcache, a);   \
    else qkv_norm_store_kernel<T, false><<<grid, 256, 0, stream>>>(src, (T*)q_out, (T*)kcache, (T*)vcache, a);       \
  } while (0)
  if (dtype == LQ_F32) LQ_QKV(float);
  else if (dtype == LQ_BF16) LQ_QKV(bf16_t);
  else LQ_REQUIRE(false, "qkv_norm_store: unknown dtype %d", dtype);
#undef LQ_QKV
#undef LQ_QKV4
  LQ_CHECK_LAUNCH("qkv_norm_store");
  return 0;
}

// Whether lq_linear_heads takes these operands (else the caller runs a product a head).
extern "C" int lq_linear_heads_accepts(const void* x, const void* w, int in_dtype, int K, int ldx) {
  return in_dtype == LQ_BF16 && K % 16 == 0 && ldx % 4 == 0 && ((uintptr_t)x % 8) == 0 && ((uintptr_t)w % 8) == 0;
}

// x [rows, heads * K] (stride ldx), w [heads, N, K] dense, out: head h's N columns from column h * out_head_stride
extern "C" int lq_linear_heads(const void* x, int ldx, const void* w, void* out, int in_dtype, int out_dtype, int ldo,
                               int rows, int heads, int N, int K, int out_head_stride, hipStream_t stream) {
  LQ_REQUIRE(rows > 0 && heads > 0 && heads <= 65535 && N > 0 && K > 0, "linear_heads: rows %d, heads %d, N %d, K %d", rows,
             heads, N, K);
  LQ_REQUIRE(ldx >= heads * K && out_head_stride >= N && ldo >= (heads - 1) * out_head_stride + N,
             "linear_heads: a stride is smaller than what it steps over");
  LQ_REQUIRE(x && w && out, "linear_heads: null pointer");
  LQ_REQUIRE(lq_linear_heads_accepts(x, w, in_dtype, K, ldx), "linear_heads: bfloat16 operands, K in 16s, rows on 8 bytes");
  LQ_REQUIRE(lq_ceil_div(N, 64) <= 65535, "linear_heads: too many columns");
  dim3 grid(lq_ceil_div(rows, 64), lq_ceil_div(N, 64), heads);
  if (out_dtype == LQ_F32)
    linear_heads_kernel<float><<<grid, 256, 0, stream>>>((const bf16_t*)x, ldx, (const bf16_t*)w, (float*)out, ldo, rows, N, K,
                                                         out_head_stride);
  else if (out_dtype == LQ_BF16)
    linear_heads_kernel<bf16_t><<<grid, 256, 0, stream>>>((const bf16_t*)x, ldx, (const bf16_t*)w, (bf16_t*)out, ldo, rows, N,
                                                          K, out_head_stride);
  else LQ_REQUIRE(false, "linear_heads: unknown dtype %d", out_dtype);
  LQ_CHECK_LAUNCH("linear_heads");
  return 0;
}
