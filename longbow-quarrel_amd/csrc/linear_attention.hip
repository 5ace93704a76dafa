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

// How the chunks' kernels take q, k and v in.  The fast ways ask for whole vectors of four everywhere, have no branch
// between their loads, so that a thread's loads are in flight together, and are made for what they name.
enum { TAKE_ANY = 0, TAKE_SILU = 1, TAKE_HALF = 2 };  // any; silu and no rotation; half-split pairs and no activation

// A quad of a head's row and what its rotation needs, as loaded.
template <int TAKE>
struct Quad {
  float4 v, mate, c0, c1;
};

// Entries n .. n + 3 of a head's row of `size` entries (TAKE_ANY: of the row itself, without loads ahead).
template <int TAKE>
__device__ inline void load_quad(const DecayArgs& a, Quad<TAKE>& q, const float* row, const float* cs, int n, int size) {
  if constexpr (TAKE == TAKE_ANY) return;
  const int at = min(n, size - 4);
  q.v = *(const float4*)(row + at);
  if constexpr (TAKE == TAKE_HALF) {
    const int half = a.dims >> 1, j = min(at < half ? at : at - half, half - 4);
    q.mate = *(const float4*)(row + (at < half ? at + half : min(at, a.dims - 4) - half));
    q.c0 = *(const float4*)(cs + 2 * j), q.c1 = *(const float4*)(cs + 2 * j + 4);
  }
}

// What becomes of it (zeros from `size` on, and where `there` is false).
template <int TAKE>
__device__ inline float4 use_quad(const DecayArgs& a, const Quad<TAKE>& q, const float* row, const float* cs, int n, int size,
                                  bool there) {
  float4 o = make_float4(0.f, 0.f, 0.f, 0.f);
  if constexpr (TAKE == TAKE_ANY) {
    if (!there) return o;
    o.x = n < size ? taken_in(a, row, cs, n) : 0.f;
    o.y = n + 1 < size ? taken_in(a, row, cs, n + 1) : 0.f;
    o.z = n + 2 < size ? taken_in(a, row, cs, n + 2) : 0.f;
    o.w = n + 3 < size ? taken_in(a, row, cs, n + 3) : 0.f;
    return o;
  } else {
    if constexpr (TAKE == TAKE_SILU) {
      o = make_float4(silu_f(q.v.x), silu_f(q.v.y), silu_f(q.v.z), silu_f(q.v.w));
    } else {
      const float sign = n < (a.dims >> 1) ? -a.mag : a.mag, m = a.mag;
      o.x = q.v.x * (q.c0.x * m) + q.mate.x * (q.c0.y * sign);
      o.y = q.v.y * (q.c0.z * m) + q.mate.y * (q.c0.w * sign);
      o.z = q.v.z * (q.c1.x * m) + q.mate.z * (q.c1.y * sign);
      o.w = q.v.w * (q.c1.z * m) + q.mate.w * (q.c1.w * sign);
      if (n >= a.dims) o = q.v;
    }
    return there && n < size ? o : make_float4(0.f, 0.f, 0.f, 0.f);
  }
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
    const float* vr = a.v + (long long)r * a.ldv + h * P;
    float v[WALK];
#pragma unroll
    for (int w = 0; w < WALK; ++w) v[w] = vr[min(col[w], P - 1)];
    __syncthreads();
    for (int n = tid; n < NP; n += 256) {
      qs[n] = n < N ? taken_in(a, qr, cs, n) : 0.f;
      ks[n] = n < N ? taken_in(a, kr, cs, n) * a.k_scale : 0.f;
    }
    __syncthreads();
#pragma unroll
    for (int w = 0; w < WALK; ++w) {
      const float val = activate(v[w], a.act);
      float o = 0.f;
#pragma unroll
      for (int e = 0; e < E; ++e)
#pragma unroll
        for (int i = 0; i < VEC; ++i) {
          const int n = (e * L + l) * VEC + i;
          S[w][e][i] = fmaf(decay, S[w][e][i], ks[n] * val);
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

constexpr int SLICE = 128;  // value columns a workgroup at most: two tiles of 16 a wavefront

// A chunk's q or k rows on their way in, as rows of 16 NS + PAD floats in LDS (entries and rows that are not there are
// zeros), times `scale` and, with `pw`, the decay to the chunk's end.
template <int NS, int TAKE>
__device__ inline void stage_rows(const DecayArgs& a, const float* src, int ld, int h, int r0, int n, float scale,
                                  const float* pw, float* to) {
  constexpr int NP = 16 * NS, BATCH = NS < 4 ? NS : 4;  // quads whose loads are in flight together
#pragma unroll 1
  for (int i0 = 0; i0 < NS; i0 += BATCH) {
    Quad<TAKE> quad[BATCH];
    float f[BATCH];
#pragma unroll
    for (int k = 0; k < BATCH; ++k) {
      const int i = (i0 + k) * 256 + threadIdx.x, t = i / (NP / 4), e = (i - t * (NP / 4)) * 4;
      const long long r = r0 + min(t, n - 1);
      load_quad<TAKE>(a, quad[k], src + r * ld + h * a.N, a.cs + r * a.dims, e, a.N);
      f[k] = pw != nullptr ? scale * pw[max(n - 1 - t, 0)] : scale;
    }
#pragma unroll
    for (int k = 0; k < BATCH; ++k) {
      const int i = (i0 + k) * 256 + threadIdx.x, t = i / (NP / 4), e = (i - t * (NP / 4)) * 4;
      const long long r = r0 + min(t, n - 1);
      float4 v = use_quad<TAKE>(a, quad[k], src + r * ld + h * a.N, a.cs != nullptr ? a.cs + r * a.dims : nullptr, e, a.N, t < n);
      v.x *= f[k], v.y *= f[k], v.z *= f[k], v.w *= f[k];
      *(float4*)(to + t * (NP + PAD) + e) = v;
    }
  }
}

// The chunk's values in column p of tokens 16 j + 4 g + e, straight from memory (a wavefront is alone in reading its
// columns).
template <int TAKE>
__device__ inline void load_values(const DecayArgs& a, float (&v)[CHUNK / 16][4], int h, int r0, int n, int g, int p) {
  const float* col = a.v + h * a.P + min(p, a.P - 1);
#pragma unroll
  for (int j = 0; j < CHUNK / 16; ++j)
#pragma unroll
    for (int e = 0; e < 4; ++e) v[j][e] = col[(long long)(r0 + min(16 * j + 4 * g + e, n - 1)) * a.ldv];
}
template <int TAKE>
__device__ inline void use_values(const DecayArgs& a, float (&v)[CHUNK / 16][4], int n, int g, int p) {
#pragma unroll
  for (int j = 0; j < CHUNK / 16; ++j)
#pragma unroll
    for (int e = 0; e < 4; ++e) {
      const float x = TAKE == TAKE_SILU ? silu_f(v[j][e]) : TAKE == TAKE_HALF ? v[j][e] : activate(v[j][e], a.act);
      v[j][e] = 16 * j + 4 * g + e < n && p < a.P ? x : 0.f;
    }
}

// What a chunk adds to the state: [P][N] = sum_j v_j (decay^(n - 1 - j) k_j)^T, in the chunk's place of the scratch.  A
// wavefront has two tiles of 16 columns of values, for all keys.
template <int NS, int TAKE>
__global__ __launch_bounds__(256) void decay_chunk_state_kernel(DecayArgs a) {
  extern __shared__ __attribute__((aligned(16))) float kt[];
  constexpr int NP = 16 * NS;
  int r0, n;
  chunk_rows(a, blockIdx.x, r0, n);
  if (n <= 0) return;
  const int h = blockIdx.y, wave = threadIdx.x >> 6, lane = threadIdx.x & 63, c = lane & 15, g = lane >> 4;
  const int p0 = blockIdx.z * SLICE + 16 * wave;  // the first tile's columns; the second's lie 64 on
  float v[2][CHUNK / 16][4];
#pragma unroll
  for (int t = 0; t < 2; ++t) load_values<TAKE>(a, v[t], h, r0, n, g, p0 + 64 * t + c);
  stage_rows<NS, TAKE>(a, a.k, a.ldk, h, r0, n, a.k_scale, a.powers + h * (CHUNK + 1), kt);
#pragma unroll
  for (int t = 0; t < 2; ++t) use_values<TAKE>(a, v[t], n, g, p0 + 64 * t + c);
  __syncthreads();
  if (p0 >= a.P) return;
  const bool two = p0 + 64 < a.P;
  float* to = a.scratch + ((long long)blockIdx.x * a.heads + h) * a.P * a.N;
  f32x4 acc[2][NS];
#pragma unroll
  for (int s = 0; s < NS; ++s) acc[0][s] = acc[1][s] = (f32x4){0.f, 0.f, 0.f, 0.f};
#pragma unroll
  for (int j = 0; j < CHUNK / 16; ++j) {
    if (16 * j >= n) break;
#pragma unroll
    for (int e = 0; e < 4; ++e) {
      const float* kr = kt + (16 * j + 4 * g + e) * (NP + PAD) + c;
#pragma unroll
      for (int s = 0; s < NS; ++s) {
        const float k = kr[16 * s];
        acc[0][s] = __builtin_amdgcn_mfma_f32_16x16x4f32(v[0][j][e], k, acc[0][s], 0, 0, 0);
        if (two) acc[1][s] = __builtin_amdgcn_mfma_f32_16x16x4f32(v[1][j][e], k, acc[1][s], 0, 0, 0);
      }
    }
  }
#pragma unroll
  for (int t = 0; t < 2; ++t)
#pragma unroll
    for (int s = 0; s < NS; ++s)
#pragma unroll
      for (int e = 0; e < 4; ++e) {
        const int p = p0 + 64 * t + 4 * g + e, m = 16 * s + c;
        if (p < a.P && m < a.N) to[(long long)p * a.N + m] = acc[t][s][e];
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

// A chunk's results, in two steps.  The scores first: wavefront w has the keys 16 w .. + 15 and makes their products with
// the queries from its own rows on, 16 keys by 16 queries at a time, each times the decay between them, into LDS.  Then a
// wavefront has two tiles of 16 columns of values, for all rows: the start state's share (an entry of the state is read
// by one wavefront alone and meets all rows' queries), and the scores' product with the values.
template <int NS, int TAKE>
__global__ __launch_bounds__(256) void decay_chunk_out_kernel(DecayArgs a) {
  extern __shared__ __attribute__((aligned(16))) float lds[];
  constexpr int NP = 16 * NS, T = CHUNK / 16, SROW = CHUNK + PAD;
  __shared__ float pw[CHUNK + 1];
  float *qt = lds, *sc = lds + CHUNK * (NP + PAD);  // queries [64][NP + PAD], scores [64][SROW]
  int r0, n;
  chunk_rows(a, blockIdx.x, r0, n);
  if (n <= 0) return;
  const int h = blockIdx.y, wave = threadIdx.x >> 6, lane = threadIdx.x & 63, c = lane & 15, g = lane >> 4;
  for (int i = threadIdx.x; i <= CHUNK; i += 256) pw[i] = a.powers[h * (CHUNK + 1) + i];
  float4 k[NS];  // this wavefront's keys as an operand: key 16 wave + c, entries 16 s + 4 g .. + 3
  {
    const int t = 16 * wave + c;
    const long long r = r0 + min(t, n - 1);
    const float *row = a.k + r * a.ldk + h * a.N, *cs = a.cs != nullptr ? a.cs + r * a.dims : nullptr;
    constexpr int BATCH = NS < 4 ? NS : 4;
#pragma unroll
    for (int s0 = 0; s0 < NS; s0 += BATCH) {
      Quad<TAKE> quad[BATCH];
#pragma unroll
      for (int j = 0; j < BATCH; ++j) load_quad<TAKE>(a, quad[j], row, cs, 16 * (s0 + j) + 4 * g, a.N);
#pragma unroll
      for (int j = 0; j < BATCH; ++j) {
        float4 x = use_quad<TAKE>(a, quad[j], row, cs, 16 * (s0 + j) + 4 * g, a.N, t < n);
        x.x *= a.k_scale, x.y *= a.k_scale, x.z *= a.k_scale, x.w *= a.k_scale;
        k[s0 + j] = x;
      }
    }
  }
  stage_rows<NS, TAKE>(a, a.q, a.ldq, h, r0, n, 1.f, nullptr, qt);
  __syncthreads();
  for (int i = wave; i < T; ++i) {
    if (16 * i >= n) break;
    f32x4 st = (f32x4){0.f, 0.f, 0.f, 0.f};  // st[e]: key 16 wave + 4 g + e with query 16 i + c
    const float* qr = qt + (16 * i + c) * (NP + PAD) + 4 * g;
#pragma unroll
    for (int s = 0; s < NS; ++s) {
      const float4 q = *(const float4*)(qr + 16 * s);
      st = __builtin_amdgcn_mfma_f32_16x16x4f32(k[s].x, q.x, st, 0, 0, 0);
      st = __builtin_amdgcn_mfma_f32_16x16x4f32(k[s].y, q.y, st, 0, 0, 0);
      st = __builtin_amdgcn_mfma_f32_16x16x4f32(k[s].z, q.z, st, 0, 0, 0);
      st = __builtin_amdgcn_mfma_f32_16x16x4f32(k[s].w, q.w, st, 0, 0, 0);
    }
    const int back = 16 * (i - wave) + c - 4 * g;  // query minus key, at e = 0
    float4 w;
    w.x = back >= 0 ? st[0] * pw[back] : 0.f;
    w.y = back >= 1 ? st[1] * pw[back - 1] : 0.f;
    w.z = back >= 2 ? st[2] * pw[back - 2] : 0.f;
    w.w = back >= 3 ? st[3] * pw[back - 3] : 0.f;
    *(float4*)(sc + (16 * i + c) * SROW + 16 * wave + 4 * g) = w;
  }
  __syncthreads();
  const float* start = a.scratch + ((long long)blockIdx.x * a.heads + h) * a.P * a.N;
#pragma unroll 1
  for (int d = 0; d < 2; ++d) {
    const int p = blockIdx.z * SLICE + 16 * (wave + 4 * d) + c;
    if (p - c >= a.P) break;
    f32x4 o[T];  // o[i][e]: row 16 i + 4 g + e, value column p
#pragma unroll
    for (int i = 0; i < T; ++i) o[i] = (f32x4){0.f, 0.f, 0.f, 0.f};
    const float* col = start + (long long)min(p, a.P - 1) * a.N;
    float4 x[NS];
#pragma unroll
    for (int s = 0; s < NS; ++s) {
      const int m = 16 * s + 4 * g;
      if constexpr (TAKE != TAKE_ANY) {  // (the queries are zeros from N on; what meets them must be a number)
        x[s] = *(const float4*)(col + min(m, a.N - 4));
      } else {
        x[s].x = m < a.N ? col[m] : 0.f, x[s].y = m + 1 < a.N ? col[m + 1] : 0.f;
        x[s].z = m + 2 < a.N ? col[m + 2] : 0.f, x[s].w = m + 3 < a.N ? col[m + 3] : 0.f;
      }
    }
    float v[T][4];
    load_values<TAKE>(a, v, h, r0, n, g, p);
    use_values<TAKE>(a, v, n, g, p);
#pragma unroll
    for (int s = 0; s < NS; ++s)
#pragma unroll
      for (int i = 0; i < T; ++i) {
        const float4 q = *(const float4*)(qt + (16 * i + c) * (NP + PAD) + 16 * s + 4 * g);
        o[i] = __builtin_amdgcn_mfma_f32_16x16x4f32(q.x, x[s].x, o[i], 0, 0, 0);
        o[i] = __builtin_amdgcn_mfma_f32_16x16x4f32(q.y, x[s].y, o[i], 0, 0, 0);
        o[i] = __builtin_amdgcn_mfma_f32_16x16x4f32(q.z, x[s].z, o[i], 0, 0, 0);
        o[i] = __builtin_amdgcn_mfma_f32_16x16x4f32(q.w, x[s].w, o[i], 0, 0, 0);
      }
#pragma unroll
    for (int i = 0; i < T; ++i) {
      if (16 * i >= n) break;
#pragma unroll
      for (int e = 0; e < 4; ++e) o[i][e] *= pw[16 * i + 4 * g + e + 1];
#pragma unroll
      for (int t = 0; t <= i; ++t) {
        const float4 w = *(const float4*)(sc + (16 * i + c) * SROW + 16 * t + 4 * g);
        o[i] = __builtin_amdgcn_mfma_f32_16x16x4f32(w.x, v[t][0], o[i], 0, 0, 0);
        o[i] = __builtin_amdgcn_mfma_f32_16x16x4f32(w.y, v[t][1], o[i], 0, 0, 0);
        o[i] = __builtin_amdgcn_mfma_f32_16x16x4f32(w.z, v[t][2], o[i], 0, 0, 0);
        o[i] = __builtin_amdgcn_mfma_f32_16x16x4f32(w.w, v[t][3], o[i], 0, 0, 0);
      }
#pragma unroll
      for (int e = 0; e < 4; ++e) {
        const int row = 16 * i + 4 * g + e;
        if (row < n && p < a.P) a.out[(long long)(r0 + row) * a.ldo + h * a.P + p] = o[i][e];
      }
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

bool large_lds(const void* kernel, int bytes) {
  return hipFuncSetAttribute(kernel, hipFuncAttributeMaxDynamicSharedMemorySize, bytes) == hipSuccess;
}

template <int NS, int TAKE>
int launch_chunks(const DecayArgs& a, hipStream_t stream) {
  constexpr int rows_bytes = CHUNK * (16 * NS + PAD) * 4, out_bytes = rows_bytes + CHUNK * (CHUNK + PAD) * 4;
  static bool ready = false;
  if (!ready) {
    LQ_REQUIRE(large_lds((const void*)decay_chunk_state_kernel<NS, TAKE>, rows_bytes) &&
                   large_lds((const void*)decay_chunk_out_kernel<NS, TAKE>, out_bytes),
               "decay_scan: %d bytes of LDS are not to be had", out_bytes);
    ready = true;
  }
  const dim3 grid(a.rows / CHUNK + a.batch, a.heads, lq_ceil_div(a.P, SLICE));
  decay_chunk_state_kernel<NS, TAKE><<<grid, 256, rows_bytes, stream>>>(a);
  LQ_CHECK_LAUNCH("decay_scan(chunk states)");
  const long long PN = (long long)a.P * a.N;
  if (PN % 4 == 0 && (uintptr_t)a.state % 16 == 0 && (uintptr_t)a.scratch % 16 == 0)
    decay_chain_kernel<4><<<dim3(a.batch * a.heads, (unsigned)lq_ceil_div64(PN, 1024)), 256, 0, stream>>>(a);
  else
    decay_chain_kernel<1><<<dim3(a.batch * a.heads, (unsigned)lq_ceil_div64(PN, 256)), 256, 0, stream>>>(a);
  LQ_CHECK_LAUNCH("decay_scan(chain)");
  decay_chunk_out_kernel<NS, TAKE><<<grid, 256, out_bytes, stream>>>(a);
  LQ_CHECK_LAUNCH("decay_scan(chunk results)");
  return 0;
}

template <int TAKE>
int launch_chunks_by_keys(const DecayArgs& a, hipStream_t stream) {
  if (a.N <= 32) return launch_chunks<2, TAKE>(a, stream);
  if (a.N <= 64) return launch_chunks<4, TAKE>(a, stream);
  if (a.N <= 128) return launch_chunks<8, TAKE>(a, stream);
  return launch_chunks<16, TAKE>(a, stream);
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
    const bool fours = N % 4 == 0 && ldq % 4 == 0 && ldk % 4 == 0 && (uintptr_t)q % 16 == 0 && (uintptr_t)k % 16 == 0 &&
                       (uintptr_t)scratch % 16 == 0;
    if (fours && act == ACT_SILU && cos_sin == nullptr) return launch_chunks_by_keys<TAKE_SILU>(a, stream);
    if (fours && act == ACT_NONE && cos_sin != nullptr && !interleaved && dims % 8 == 0 && (uintptr_t)cos_sin % 16 == 0)
      return launch_chunks_by_keys<TAKE_HALF>(a, stream);
    return launch_chunks_by_keys<TAKE_ANY>(a, stream);
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
