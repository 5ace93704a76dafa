// Linear attention with a fixed decay a head: S <- decay S + k v^T, o = S^T q, per head, the state 32-bit.
//
// q, k and v are 32-bit results of a product; on their way in they may pass silu (`act`), q and k may be rotated by the
// row's angles (`cs`: cos and sin, [rows][dims / 2][2]) and k is multiplied by `k_scale`.  The state of a head is
// [P values][N key entries].  `powers` [heads][CHUNK + 1] holds the decays' powers.
//
// Two ways, chosen by the step:
// * few tokens a sequence: `decay_walk_kernel` walks them one by one, the state in registers (a step of single tokens
//   streams the state through once);
// * longer portions: chunks of CHUNK tokens.  A first launch leaves what every chunk adds to the state,
//   sum_j decay^(n-1-j) k_j v_j^T; a second chains them (in every chunk's place the state that it starts from, the last
//   one's end in the cache); a third makes a chunk's results from its start, decay^(i+1) S^T q_i, and from its own
//   tokens, sum_(j<=i) decay^(i-j) (q_i . k_j) v_j.  The products are 32-bit on the matrix cores
//   (v_mfma_f32_16x16x4_f32).  Chunks count from a sequence's first row of the step.
// A row's result is made of its own sequence alone, in an order that follows from the row's place in its portion.
#include "device_math.h"

namespace {

constexpr int CHUNK = 64;
constexpr int PAD = 4;  // floats behind a row in LDS: rows four apart then lie 16 banks apart

struct DecayArgs {
  const float *q, *k, *v;
  int ldq, ldk, ldv;
  const float* powers;
  float *state, *out, *scratch;
  int ldo, heads, N, P, batch, rows, act;
  float k_scale;
  const float* cs;
  int dims, interleaved;
  float mag;
  const int *seq_slot, *cu_rows;
};

// Entry n of a head's row on its way in.  `cs`: the row's angles, null for values and where nothing is rotated.
__device__ inline float taken_in(const DecayArgs& a, const float* row, const float* cs, int n) {
  float v = activate(row[n], a.act);
  if (cs == nullptr || n >= a.dims) return v;
  const int half = a.dims >> 1;
  const int j = a.interleaved ? n >> 1 : n < half ? n : n - half;
  const bool first = a.interleaved ? !(n & 1) : n < half;
  const int mate = a.interleaved ? n ^ 1 : first ? n + half : n - half;
  const float c = cs[2 * j] * a.mag, s = cs[2 * j + 1] * a.mag, m = activate(row[mate], a.act);
  return first ? v * c - m * s : v * c + m * s;
}

// Entries n .. n + 3 (zeros from `size` on).  FOURS: size and the row's place allow whole vectors.
template <bool FOURS>
__device__ inline float4 taken_in4(const DecayArgs& a, const float* row, const float* cs, int n, int size) {
  if (FOURS && (cs == nullptr || n >= a.dims)) {
    if (n >= size) return make_float4(0.f, 0.f, 0.f, 0.f);
    const float4 v = *(const float4*)(row + n);
    return make_float4(activate(v.x, a.act), activate(v.y, a.act), activate(v.z, a.act), activate(v.w, a.act));
  }
  float4 v;
  v.x = n < size ? taken_in(a, row, cs, n) : 0.f;
  v.y = n + 1 < size ? taken_in(a, row, cs, n + 1) : 0.f;
  v.z = n + 2 < size ? taken_in(a, row, cs, n + 2) : 0.f;
  v.w = n + 3 < size ? taken_in(a, row, cs, n + 3) : 0.f;
  return v;
}

// ---------------------------------------------------------------- token by token
// `L` lanes (a power of two) share a column of the state, each with E runs of VEC entries; a workgroup of 256 threads
// has WALK columns for each of its 256 / L groups of lanes.
constexpr int WALK = 4;

template <int VEC, int E>
__global__ __launch_bounds__(256) void decay_walk_kernel(DecayArgs a, int L) {
  extern __shared__ __attribute__((aligned(16))) float lds[];  // q [N], k [N], padded to whole runs
  const int b = blockIdx.x / a.heads, h = blockIdx.x % a.heads, tid = threadIdx.x, l = tid & (L - 1), group = tid / L;
  const int groups = 256 / L, N = a.N, P = a.P, NP = E * VEC * L;
  float *qs = lds, *ks = lds + NP;
  const int r0 = a.cu_rows[b], r1 = a.cu_rows[b + 1];
  const float decay = a.powers[h * (CHUNK + 1) + 1];
  float* head = a.state + ((long long)a.seq_slot[b] * a.heads + h) * (long long)P * N;
  float S[WALK][E][VEC];
  int col[WALK];
#pragma unroll
  for (int w = 0; w < WALK; ++w) {
    col[w] = (blockIdx.y * WALK + w) * groups + group;
#pragma unroll
    for (int e = 0; e < E; ++e) {
      const int n = (e * L + l) * VEC;
      if constexpr (VEC == 4) {
        float4 s = make_float4(0.f, 0.f, 0.f, 0.f);
        if (col[w] < P && n < N) s = *(const float4*)(head + (long long)col[w] * N + n);
        S[w][e][0] = s.x, S[w][e][1] = s.y, S[w][e][2] = s.z, S[w][e][3] = s.w;
      } else {
        S[w][e][0] = col[w] < P && n < N ? head[(long long)col[w] * N + n] : 0.f;
      }
    }
  }
  for (int r = r0; r < r1; ++r) {
    const float* cs = a.cs != nullptr ? a.cs + (long long)r * a.dims : nullptr;
    const float *qr = a.q + (long long)r * a.ldq + h * N, *kr = a.k + (long long)r * a.ldk + h * N;
    __syncthreads();
    for (int n = tid; n < NP; n += 256) {
      qs[n] = n < N ? taken_in(a, qr, cs, n) : 0.f;
      ks[n] = n < N ? taken_in(a, kr, cs, n) * a.k_scale : 0.f;
    }
    __syncthreads();
#pragma unroll
    for (int w = 0; w < WALK; ++w) {
      const float v = col[w] < P ? activate(a.v[(long long)r * a.ldv + h * P + col[w]], a.act) : 0.f;
      float o = 0.f;
#pragma unroll
      for (int e = 0; e < E; ++e)
#pragma unroll
        for (int i = 0; i < VEC; ++i) {
          const int n = (e * L + l) * VEC + i;
          S[w][e][i] = fmaf(decay, S[w][e][i], ks[n] * v);
          o = fmaf(S[w][e][i], qs[n], o);
        }
      for (int off = 1; off < L; off <<= 1) o += __shfl_xor(o, off, LQ_WAVE);
      if (l == 0 && col[w] < P) a.out[(long long)r * a.ldo + h * P + col[w]] = o;
    }
  }
#pragma unroll
  for (int w = 0; w < WALK; ++w)
#pragma unroll
    for (int e = 0; e < E; ++e) {
      const int n = (e * L + l) * VEC;
      if (col[w] >= P || n >= N) continue;
      float* s = head + (long long)col[w] * N + n;
      if constexpr (VEC == 4) *(float4*)s = make_float4(S[w][e][0], S[w][e][1], S[w][e][2], S[w][e][3]);
      else *s = S[w][e][0];
    }
}

// ---------------------------------------------------------------- chunk by chunk
typedef float f32x4 __attribute__((ext_vector_type(4)));

// Sequence b's chunks have the numbers first_chunk(b), first_chunk(b) + 1, ...; rows / CHUNK + batch numbers hold the
// chunks of all sequences (some numbers between two sequences may stay unused).
__device__ inline int first_chunk(const DecayArgs& a, int b) { return a.cu_rows[b] / CHUNK + b; }

// The sequence that chunk number c belongs to, its first row r0 and its rows n (0 or less: an unused number).
__device__ inline int chunk_rows(const DecayArgs& a, int c, int& r0, int& n) {
  int lo = 0, hi = a.batch - 1;
  while (lo < hi) {
    const int mid = (lo + hi + 1) >> 1;
    if (first_chunk(a, mid) <= c) lo = mid;
    else hi = mid - 1;
  }
  r0 = a.cu_rows[lo] + (c - first_chunk(a, lo)) * CHUNK;
  n = min(CHUNK, a.cu_rows[lo + 1] - r0);
  return lo;
}

constexpr int SLICE = 128;  // value columns a workgroup at most

// The chunk's keys (scaled, times their decay to the chunk's end with `weigh`) and values, rows of 16 NS and of
// 16 pt + PAD floats in LDS; entries and rows that are not there are zeros.
template <int NS, bool FOURS>
__device__ inline void stage_chunk(const DecayArgs& a, int h, int r0, int n, int p0, int pt, const float* pw, bool weigh,
                                   float* kt, float* vt) {
  constexpr int NP = 16 * NS;
  for (int i = threadIdx.x; i < CHUNK * (NP / 4); i += 256) {
    const int t = i / (NP / 4), e = (i - t * (NP / 4)) * 4;
    float4 v = make_float4(0.f, 0.f, 0.f, 0.f);
    if (t < n) {
      const float* cs = a.cs != nullptr ? a.cs + (long long)(r0 + t) * a.dims : nullptr;
      v = taken_in4<FOURS>(a, a.k + (long long)(r0 + t) * a.ldk + h * a.N, cs, e, a.N);
      const float f = weigh ? a.k_scale * pw[n - 1 - t] : a.k_scale;
      v.x *= f, v.y *= f, v.z *= f, v.w *= f;
    }
    *(float4*)(kt + t * (NP + PAD) + e) = v;
  }
  const int PW = 16 * pt;
  for (int i = threadIdx.x; i < CHUNK * (PW / 4); i += 256) {
    const int t = i / (PW / 4), e = (i - t * (PW / 4)) * 4;
    float4 v = make_float4(0.f, 0.f, 0.f, 0.f);
    if (t < n) v = taken_in4<FOURS>(a, a.v + (long long)(r0 + t) * a.ldv + h * a.P, nullptr, p0 + e, a.P);
    *(float4*)(vt + t * (PW + PAD) + e) = v;
  }
}

// What a chunk adds to the state: [P][N] = sum_j v_j (decay^(n - 1 - j) k_j)^T, in the chunk's place of the scratch.
template <int NS, bool FOURS>
__global__ __launch_bounds__(256) void decay_chunk_state_kernel(DecayArgs a) {
  extern __shared__ __attribute__((aligned(16))) float lds[];
  constexpr int NP = 16 * NS;
  int r0, n;
  chunk_rows(a, blockIdx.x, r0, n);
  if (n <= 0) return;
  const int h = blockIdx.y, p0 = blockIdx.z * SLICE, pt = (min(SLICE, a.P - p0) + 15) / 16, PW = 16 * pt;
  float *kt = lds, *vt = lds + CHUNK * (NP + PAD);
  stage_chunk<NS, FOURS>(a, h, r0, n, p0, pt, a.powers + h * (CHUNK + 1), true, kt, vt);
  __syncthreads();
  const int wave = threadIdx.x >> 6, lane = threadIdx.x & 63, c = lane & 15, g = lane >> 4;
  float* to = a.scratch + ((long long)blockIdx.x * a.heads + h) * a.P * a.N;
  for (int t = wave; t < pt; t += 4) {
    f32x4 acc[NS];
#pragma unroll
    for (int s = 0; s < NS; ++s) acc[s] = (f32x4){0.f, 0.f, 0.f, 0.f};
    for (int j = 0; j < CHUNK / 16; ++j)
#pragma unroll
      for (int e = 0; e < 4; ++e) {
        const int tok = 16 * j + 4 * g + e;
        const float v = vt[tok * (PW + PAD) + 16 * t + c];
#pragma unroll
        for (int s = 0; s < NS; ++s)
          acc[s] = __builtin_amdgcn_mfma_f32_16x16x4f32(v, kt[tok * (NP + PAD) + 16 * s + c], acc[s], 0, 0, 0);
      }
#pragma unroll
    for (int s = 0; s < NS; ++s)
#pragma unroll
      for (int e = 0; e < 4; ++e) {
        const int p = p0 + 16 * t + 4 * g + e, m = 16 * s + c;
        if (p < a.P && m < a.N) to[(long long)p * a.N + m] = acc[s][e];
      }
  }
}

// In every chunk's place the state that the chunk starts from; the sequence's new state into the cache.
template <int VEC>
__global__ __launch_bounds__(256) void decay_chain_kernel(DecayArgs a) {
  const int b = blockIdx.x / a.heads, h = blockIdx.x % a.heads;
  const long long PN = (long long)a.P * a.N, idx = ((long long)blockIdx.y * 256 + threadIdx.x) * VEC;
  if (idx >= PN) return;
  const int rows = a.cu_rows[b + 1] - a.cu_rows[b], chunks = (rows + CHUNK - 1) / CHUNK;
  const float* pw = a.powers + h * (CHUNK + 1);
  const float whole = pw[CHUNK], last = pw[rows > 0 ? rows - (chunks - 1) * CHUNK : 0];
  float* cached = a.state + ((long long)a.seq_slot[b] * a.heads + h) * PN + idx;
  const long long stride = (long long)a.heads * PN;
  float* at = a.scratch + ((long long)first_chunk(a, b) * a.heads + h) * PN + idx;
  auto load = [](const float* p, float* v) {
    if constexpr (VEC == 4) {
      const float4 x = *(const float4*)p;
      v[0] = x.x, v[1] = x.y, v[2] = x.z, v[3] = x.w;
    } else {
      v[0] = *p;
    }
  };
  auto store = [](float* p, const float* v) {
    if constexpr (VEC == 4) *(float4*)p = make_float4(v[0], v[1], v[2], v[3]);
    else *p = v[0];
  };
  float S[VEC];
  load(cached, S);
  for (int c0 = 0; c0 < chunks; c0 += 4) {
    float add[4][VEC];  // four chunks' loads in flight together
#pragma unroll
    for (int i = 0; i < 4; ++i)
      if (c0 + i < chunks) load(at + (c0 + i) * stride, add[i]);
#pragma unroll
    for (int i = 0; i < 4; ++i)
      if (c0 + i < chunks) {
        store(at + (c0 + i) * stride, S);
        const float d = c0 + i + 1 < chunks ? whole : last;
#pragma unroll
        for (int j = 0; j < VEC; ++j) S[j] = fmaf(d, S[j], add[i][j]);
      }
  }
  if (chunks > 0) store(cached, S);
}

// A chunk's results.  Wavefront w has the rows 16 w .. + 15 of the chunk: the products of its queries with the keys up to
// its own rows, 16 keys by 16 queries at a time, each times the decay between them, straight into the product with the
// values; ahead of that the start state's share.
template <int NS, int PT, bool FOURS>
__global__ __launch_bounds__(256) void decay_chunk_out_kernel(DecayArgs a) {
  extern __shared__ __attribute__((aligned(16))) float lds[];
  constexpr int NP = 16 * NS, PW = 16 * PT;
  __shared__ float pw[CHUNK + 1];
  int r0, n;
  chunk_rows(a, blockIdx.x, r0, n);
  if (n <= 0) return;
  const int h = blockIdx.y, p0 = blockIdx.z * PW;
  float *kt = lds, *vt = lds + CHUNK * (NP + PAD);
  for (int i = threadIdx.x; i <= CHUNK; i += 256) pw[i] = a.powers[h * (CHUNK + 1) + i];
  stage_chunk<NS, FOURS>(a, h, r0, n, p0, PT, nullptr, false, kt, vt);
  __syncthreads();
  const int wave = threadIdx.x >> 6, lane = threadIdx.x & 63, c = lane & 15, g = lane >> 4;
  if (16 * wave >= n) return;
  const int i = 16 * wave + c;  // this lane's query row as an operand
  float4 q[NS];
  {
    const int r = r0 + min(i, n - 1);
    const float* cs = a.cs != nullptr ? a.cs + (long long)r * a.dims : nullptr;
    const float* row = a.q + (long long)r * a.ldq + h * a.N;
#pragma unroll
    for (int s = 0; s < NS; ++s) q[s] = taken_in4<FOURS>(a, row, cs, 16 * s + 4 * g, a.N);
  }
  f32x4 o[PT];  // o[d][e]: row 16 wave + 4 g + e, value column p0 + 16 d + c
  const float* start = a.scratch + ((long long)blockIdx.x * a.heads + h) * a.P * a.N;
#pragma unroll
  for (int d = 0; d < PT; ++d) {
    o[d] = (f32x4){0.f, 0.f, 0.f, 0.f};
    const int p = p0 + 16 * d + c;
    const float* col = start + (long long)min(p, a.P - 1) * a.N + 4 * g;
#pragma unroll
    for (int s = 0; s < NS; ++s) {
      const int m = 16 * s + 4 * g;
      float4 x;
      if (FOURS) {
        x = m < a.N ? *(const float4*)(col + 16 * s) : make_float4(0.f, 0.f, 0.f, 0.f);
      } else {
        x.x = m < a.N ? col[16 * s] : 0.f, x.y = m + 1 < a.N ? col[16 * s + 1] : 0.f;
        x.z = m + 2 < a.N ? col[16 * s + 2] : 0.f, x.w = m + 3 < a.N ? col[16 * s + 3] : 0.f;
      }
      o[d] = __builtin_amdgcn_mfma_f32_16x16x4f32(q[s].x, x.x, o[d], 0, 0, 0);
      o[d] = __builtin_amdgcn_mfma_f32_16x16x4f32(q[s].y, x.y, o[d], 0, 0, 0);
      o[d] = __builtin_amdgcn_mfma_f32_16x16x4f32(q[s].z, x.z, o[d], 0, 0, 0);
      o[d] = __builtin_amdgcn_mfma_f32_16x16x4f32(q[s].w, x.w, o[d], 0, 0, 0);
    }
  }
#pragma unroll
  for (int e = 0; e < 4; ++e) {
    const float f = pw[16 * wave + 4 * g + e + 1];
#pragma unroll
    for (int d = 0; d < PT; ++d) o[d][e] *= f;
  }
  for (int t = 0; t <= wave; ++t) {
    f32x4 st = (f32x4){0.f, 0.f, 0.f, 0.f};  // st[e]: key 16 t + 4 g + e with query i
    const float* kr = kt + (16 * t + c) * (NP + PAD) + 4 * g;
#pragma unroll
    for (int s = 0; s < NS; ++s) {
      const float4 x = *(const float4*)(kr + 16 * s);
      st = __builtin_amdgcn_mfma_f32_16x16x4f32(x.x, q[s].x, st, 0, 0, 0);
      st = __builtin_amdgcn_mfma_f32_16x16x4f32(x.y, q[s].y, st, 0, 0, 0);
      st = __builtin_amdgcn_mfma_f32_16x16x4f32(x.z, q[s].z, st, 0, 0, 0);
      st = __builtin_amdgcn_mfma_f32_16x16x4f32(x.w, q[s].w, st, 0, 0, 0);
    }
#pragma unroll
    for (int e = 0; e < 4; ++e) {
      const int j = 16 * t + 4 * g + e;
      st[e] = j <= i ? st[e] * pw[max(i - j, 0)] : 0.f;
    }
#pragma unroll
    for (int e = 0; e < 4; ++e) {
      const float* vr = vt + (16 * t + 4 * g + e) * (PW + PAD) + c;
#pragma unroll
      for (int d = 0; d < PT; ++d) o[d] = __builtin_amdgcn_mfma_f32_16x16x4f32(st[e], vr[16 * d], o[d], 0, 0, 0);
    }
  }
#pragma unroll
  for (int e = 0; e < 4; ++e) {
    const int row = 16 * wave + 4 * g + e;
    if (row >= n) continue;
    float* to = a.out + (long long)(r0 + row) * a.ldo + h * a.P;
#pragma unroll
    for (int d = 0; d < PT; ++d) {
      const int p = p0 + 16 * d + c;
      if (p < a.P) to[p] = o[d][e];
    }
  }
}

// The longest portion of a sequence from which a step is cut into chunks, and the largest keys that it takes: one
// decision for the query about scratch and for the launch.
constexpr int CHUNKS_FROM = 24;
constexpr int MAX_CHUNK_KEYS = 256;

long long chunk_floats(int rows, int batch, int heads, int N, int P, int max_rows) {
  if (max_rows < CHUNKS_FROM || N > MAX_CHUNK_KEYS) return 0;
  return ((long long)rows / CHUNK + batch) * heads * ((long long)P * N);
}

template <int NS>
bool large_lds(const void* kernel, int bytes) {
  return hipFuncSetAttribute(kernel, hipFuncAttributeMaxDynamicSharedMemorySize, bytes) == hipSuccess;
}

template <int NS, bool FOURS>
int launch_chunks(const DecayArgs& a, hipStream_t stream) {
  constexpr int NP = 16 * NS;
  const int chunks = a.rows / CHUNK + a.batch;
  const int pw = a.P < SLICE ? (a.P + 15) / 16 * 16 : SLICE;
  const int lds_k = CHUNK * (NP + PAD) * 4;
  constexpr int most = CHUNK * (NP + PAD + SLICE + PAD) * 4;
  static bool ready = false;
  if (!ready) {
    LQ_REQUIRE(large_lds<NS>((const void*)decay_chunk_state_kernel<NS, FOURS>, most) &&
                   large_lds<NS>((const void*)decay_chunk_out_kernel<NS, 2, FOURS>, most) &&
                   large_lds<NS>((const void*)decay_chunk_out_kernel<NS, 4, FOURS>, most) &&
                   large_lds<NS>((const void*)decay_chunk_out_kernel<NS, 8, FOURS>, most),
               "decay_scan: %d bytes of LDS are not to be had", most);
    ready = true;
  }
  decay_chunk_state_kernel<NS, FOURS><<<dim3(chunks, a.heads, lq_ceil_div(a.P, SLICE)), 256,
                                        lds_k + CHUNK * (pw + PAD) * 4, stream>>>(a);
  LQ_CHECK_LAUNCH("decay_scan(chunk states)");
  const long long PN = (long long)a.P * a.N;
  if (PN % 4 == 0 && (uintptr_t)a.state % 16 == 0 && (uintptr_t)a.scratch % 16 == 0)
    decay_chain_kernel<4><<<dim3(a.batch * a.heads, (unsigned)lq_ceil_div64(PN, 1024)), 256, 0, stream>>>(a);
  else
    decay_chain_kernel<1><<<dim3(a.batch * a.heads, (unsigned)lq_ceil_div64(PN, 256)), 256, 0, stream>>>(a);
  LQ_CHECK_LAUNCH("decay_scan(chain)");
#define LQ_DECAY_OUT(PT)                                                                                   \
  decay_chunk_out_kernel<NS, PT, FOURS><<<dim3(chunks, a.heads, lq_ceil_div(a.P, 16 * PT)), 256,             \
                                          lds_k + CHUNK * (16 * PT + PAD) * 4, stream>>>(a)
  if (a.P <= 32) LQ_DECAY_OUT(2);
  else if (a.P <= 64) LQ_DECAY_OUT(4);
  else LQ_DECAY_OUT(8);
#undef LQ_DECAY_OUT
  LQ_CHECK_LAUNCH("decay_scan(chunk results)");
  return 0;
}

template <bool FOURS>
int launch_chunks_by_keys(const DecayArgs& a, hipStream_t stream) {
  if (a.N <= 32) return launch_chunks<2, FOURS>(a, stream);
  if (a.N <= 64) return launch_chunks<4, FOURS>(a, stream);
  if (a.N <= 128) return launch_chunks<8, FOURS>(a, stream);
  return launch_chunks<16, FOURS>(a, stream);
}

}  // namespace

// Float32 entries of scratch with which a step of `rows` rows, the longest sequence bringing `max_rows`, is cut into
// chunks (0: it is walked token by token).
extern "C" long long lq_decay_scan_workspace(int rows, int batch, int heads, int N, int P, int max_rows) {
  if (rows <= 0 || batch <= 0 || heads <= 0 || N <= 0 || P <= 0) return 0;
  return chunk_floats(rows, batch, heads, N, P, max_rows);
}

// q and k [rows, heads * N], v [rows, heads * P] (strides ldq, ldk, ldv), powers [heads, 65], state [slots, heads, P, N],
// out [rows, heads * P]; rows lie sequence by sequence (cu_rows).  act: an activation's number (device_math.h, 0: none).
// cos_sin [rows, dims / 2, 2] or null.  `scratch`: lq_decay_scan_workspace(...) floats, or null (then token by token).
extern "C" int lq_decay_scan(const float* q, int ldq, const float* k, int ldk, const float* v, int ldv, const float* powers,
                             float* state, float* out, int ldo, int rows, int heads, int N, int P, float k_scale, int act,
                             const float* cos_sin, int dims, int interleaved, float magnitude, const int* seq_slot,
                             const int* cu_rows, int batch, int max_rows, float* scratch, long long scratch_floats,
                             hipStream_t stream) {
  LQ_REQUIRE(rows > 0 && heads > 0 && heads <= 65535 && N > 0 && N <= 1024 && P > 0 && batch > 0 && rows >= batch,
             "decay_scan: rows %d of %d sequences, %d heads of %d x %d (keys of at most 1024)", rows, batch, heads, N, P);
  LQ_REQUIRE(ldq >= heads * N && ldk >= heads * N && ldv >= heads * P && ldo >= heads * P,
             "decay_scan: a row stride is smaller than its row");
  LQ_REQUIRE(q && k && v && powers && state && out && seq_slot && cu_rows, "decay_scan: null pointer");
  LQ_REQUIRE(act == ACT_NONE || act == ACT_SILU, "decay_scan: unknown activation %d", act);
  LQ_REQUIRE(cos_sin == nullptr || (dims >= 2 && dims % 2 == 0 && dims <= N), "decay_scan: %d rotated entries of %d", dims, N);
  LQ_REQUIRE((long long)batch * heads <= 0x7fffffff && lq_ceil_div(P, 16) <= 65535, "decay_scan: too many heads or columns");
  DecayArgs a = {q, k, v, ldq, ldk, ldv, powers, state, out, scratch, ldo, heads, N, P, batch, rows, act, k_scale,
                 cos_sin, cos_sin != nullptr ? dims : 0, interleaved, magnitude, seq_slot, cu_rows};
  const long long need = scratch != nullptr ? chunk_floats(rows, batch, heads, N, P, max_rows) : 0;
  LQ_REQUIRE(need <= scratch_floats, "decay_scan: %lld floats of scratch for a step in chunks, %lld given", need, scratch_floats);
  if (need > 0) {
    const bool fours = N % 4 == 0 && P % 4 == 0 && ldq % 4 == 0 && ldk % 4 == 0 && ldv % 4 == 0 && (uintptr_t)q % 16 == 0 &&
                       (uintptr_t)k % 16 == 0 && (uintptr_t)v % 16 == 0 && (uintptr_t)scratch % 16 == 0;
    return fours ? launch_chunks_by_keys<true>(a, stream) : launch_chunks_by_keys<false>(a, stream);
  }
  const bool vec = N % 4 == 0 && (uintptr_t)state % 16 == 0;
  const int units = vec ? N / 4 : N;
  int L = 1;
  while (L < 64 && L < units) L <<= 1;
  const int E = lq_ceil_div(units, L);  // at most 4 runs of four, or 16 of one
  const dim3 grid((unsigned)(batch * heads), lq_ceil_div(P, WALK * (256 / L)));
#define LQ_WALK(VEC, E) decay_walk_kernel<VEC, E><<<grid, 256, 2 * (E) * (VEC) * L * sizeof(float), stream>>>(a, L)
  if (vec && E == 1) LQ_WALK(4, 1);
  else if (vec && E == 2) LQ_WALK(4, 2);
  else if (vec) LQ_WALK(4, 4);
  else if (E == 1) LQ_WALK(1, 1);
  else if (E <= 4) LQ_WALK(1, 4);
  else LQ_WALK(1, 16);
#undef LQ_WALK
  LQ_CHECK_LAUNCH("decay_scan(token by token)");
  return 0;
}
