// Recurrences whose decay is a matrix of its own or whose gates are exponentials: the selective scan (a decay for every
// channel and state entry, one step size a channel) and the gates and output of a matrix memory with a running maximum.
// Everything is 32-bit arithmetic; inputs that are projections or convolutions come in the run's dtype, and an output
// that feeds a matrix product is rounded to it.
#include "device_math.h"

namespace {

// ---------------------------------------------------------------- the selective scan
// Per channel c and state entry n, with dt = softplus(raw + bias) one number a token and channel:
//   S[c, n] <- exp(dt A[c, n]) S[c, n] + dt x B[n],   y = sum_n S[c, n] C[n] + D[c] x,   out = y silu(z).
// A thread owns SLAB neighbouring state entries of one channel, LN threads share a channel (LN from the state size
// alone), a workgroup 256 / LN channels; sums over n are a thread's own entries in ascending order, then the exchange
// over the LN lanes.  B and C (shared by all channels), the channels' steps and inputs of TT tokens are staged in LDS,
// two buffers taking turns: the next chunk's loads are in flight while this chunk is computed token by token.
//
// A launch of few long sequences runs in segments side by side (as the state-space scan does): pass 1 from zero, each
// segment leaving its end state and the sum of its steps (its decay is exp(A sum dt)); a short kernel chains them; pass
// 2 runs the segments again from their true starts.
constexpr int SEL_SLAB = 8, SEL_TH = 256;
constexpr int SEL_SEGMENTS = 16, SEL_MIN_ROWS = 512;
constexpr float LOG2E = 1.4426950408889634f;

constexpr int sel_tokens(int ln) { return ln >= 64 ? 4 : ln >= 16 ? 8 : ln >= 4 ? 16 : 8; }
constexpr int sel_buffer(int ln) {  // B and C, then steps, inputs and results of the channels
  return sel_tokens(ln) * (2 * ln * SEL_SLAB + 3 * (SEL_TH / ln));
}

struct SelArgs {
  int ldx, lddt, ldb, ldc, ldz, ldo, channels, N;
  const float *dt_bias, *a_log, *d_skip;
  float* state;  // [slots][channels][N]
  const int *seq_slot, *cu_rows;
  int nseg, pass;  // nseg 1: no segments (pass 1 alone)
  float *seg_state, *seg_steps;  // [sequences][nseg][channels][N], [sequences][nseg][channels]
};

template <int LN, typename T>
__global__ __launch_bounds__(SEL_TH) void selective_scan_kernel(const T* __restrict__ x, const float* __restrict__ dt,
                                                                const T* __restrict__ Bm, const T* __restrict__ Cm,
                                                                const T* __restrict__ z, T* __restrict__ out, SelArgs a) {
  constexpr int COLS = SEL_TH / LN, NP = LN * SEL_SLAB, TT = sel_tokens(LN), BUF = sel_buffer(LN);
  constexpr int BPER = (TT * 2 * NP + SEL_TH - 1) / SEL_TH, XPER = (TT * COLS + SEL_TH - 1) / SEL_TH;
  __shared__ __attribute__((aligned(16))) float lds[2 * BUF];
  const int tid = threadIdx.x, l = tid % LN, col = tid / LN;
  const int b = blockIdx.y, p0 = blockIdx.x * COLS, ch = p0 + col, N = a.N;
  const bool live = ch < a.channels;
  long long r0 = a.cu_rows[b], r1 = a.cu_rows[b + 1];
  const int seg = blockIdx.z;
  const int nseg = (a.nseg > 1 && r1 - r0 >= SEL_MIN_ROWS) ? a.nseg : 1;
  if (seg >= nseg || (a.pass == 2 && seg == 0)) return;
  if (nseg > 1) {
    const long long len = ((r1 - r0 + nseg - 1) / nseg + TT - 1) / TT * TT;
    r0 = min(r1, r0 + seg * len);
    r1 = min(r1, r0 + len);
  }
  const bool write_y = a.pass == 2 || seg == 0;
  const int mine = live ? ch : 0;
  float* sp = a.state + ((long long)a.seq_slot[b] * a.channels + mine) * N;
  float* seg_sp = nseg > 1 ? a.seg_state + (((long long)b * a.nseg + seg) * a.channels + mine) * N : nullptr;
  const float* from = nseg > 1 && a.pass == 2 ? seg_sp : sp;
  const bool from_zero = nseg > 1 && a.pass == 1 && seg > 0;
  float* to = nseg == 1 ? sp : a.pass == 1 ? seg_sp : nullptr;
  float S[SEL_SLAB], A2[SEL_SLAB];
#pragma unroll
  for (int i = 0; i < SEL_SLAB; ++i) {
    const int n = l * SEL_SLAB + i;
    const bool has = live && n < N;
    S[i] = has && !from_zero ? from[n] : 0.f;
    A2[i] = has ? -expf(a.a_log[(long long)mine * N + n]) * LOG2E : 0.f;
  }
  const float D = a.d_skip[mine];
  float steps = 0.f;  // the sum of the segment's steps
  T bpre[BPER], xpre[XPER], zpre[XPER];
  float dpre[XPER];
  auto fetch = [&](long long c0, int nt) {  // the chunk's loads, into registers
#pragma unroll
    for (int j = 0; j < BPER; ++j) {
      const int e = tid + j * SEL_TH, t = e / (2 * NP), rem = e - t * 2 * NP, n = rem < NP ? rem : rem - NP;
      bpre[j] = from_f32<T>(0.f);
      if (t < nt && n < N) bpre[j] = rem < NP ? Bm[(c0 + t) * a.ldb + n] : Cm[(c0 + t) * a.ldc + n];
    }
#pragma unroll
    for (int j = 0; j < XPER; ++j) {
      const int e = tid + j * SEL_TH, t = e / COLS, c = p0 + e - t * COLS;
      xpre[j] = from_f32<T>(0.f), dpre[j] = 0.f;
      if (t < nt && c < a.channels) xpre[j] = x[(c0 + t) * a.ldx + c], dpre[j] = dt[(c0 + t) * a.lddt + c];
    }
  };
  auto stash = [&](float* buf) {  // registers to LDS; the step is made of its logit here
#pragma unroll
    for (int j = 0; j < BPER; ++j) {
      const int e = tid + j * SEL_TH;
      if (e < TT * 2 * NP) buf[e] = to_f32(bpre[j]);
    }
#pragma unroll
    for (int j = 0; j < XPER; ++j) {
      const int e = tid + j * SEL_TH, c = p0 + e % COLS;
      if (e >= TT * COLS) continue;
      buf[TT * 2 * NP + e] = softplus_f(dpre[j] + (c < a.channels ? a.dt_bias[c] : 0.f));
      buf[TT * (2 * NP + COLS) + e] = to_f32(xpre[j]);
    }
  };
  int cur = 0;
  if (r1 > r0) {
    fetch(r0, (int)min((long long)TT, r1 - r0));
    stash(lds);
  }
  __syncthreads();
  for (long long c0 = r0; c0 < r1; c0 += TT, cur ^= 1) {
    const int nt = (int)min((long long)TT, r1 - c0);
    const int next = (int)min((long long)TT, r1 - c0 - TT);
    if (next > 0) fetch(c0 + TT, next);
    if (write_y) {
#pragma unroll
      for (int j = 0; j < XPER; ++j) {  // this chunk's gates, for its results after the barrier
        const int e = tid + j * SEL_TH, t = e / COLS, c = p0 + e - t * COLS;
        zpre[j] = from_f32<T>(0.f);
        if (t < nt && c < a.channels) zpre[j] = z[(c0 + t) * a.ldz + c];
      }
    }
    float* buf = lds + cur * BUF;
    const float *bc = buf, *sdt = buf + TT * 2 * NP, *sx = sdt + TT * COLS;
    float* sy = buf + TT * (2 * NP + 2 * COLS);
#pragma unroll
    for (int t = 0; t < TT; ++t) {
      if (t >= nt) break;
      const float step = sdt[t * COLS + col], xv = sx[t * COLS + col], dx = step * xv;
      float bv[SEL_SLAB];
#pragma unroll
      for (int i = 0; i < SEL_SLAB; ++i) bv[i] = bc[t * 2 * NP + l * SEL_SLAB + i];
#pragma unroll
      for (int i = 0; i < SEL_SLAB; ++i)
        S[i] = fmaf(S[i], __builtin_amdgcn_exp2f(step * A2[i]), dx * bv[i]);
      steps += step;
      if (write_y) {
        float acc = 0.f, acc1 = 0.f;  // (two chains, even and odd entries)
#pragma unroll
        for (int i = 0; i < SEL_SLAB; i += 2) {
          acc = fmaf(S[i], bc[t * 2 * NP + NP + l * SEL_SLAB + i], acc);
          acc1 = fmaf(S[i + 1], bc[t * 2 * NP + NP + l * SEL_SLAB + i + 1], acc1);
        }
        acc = group_sum<LN>(acc + acc1);
        if (l == 0) sy[t * COLS + col] = fmaf(D, xv, acc);
      }
    }
    if (next > 0) stash(lds + (cur ^ 1) * BUF);
    __syncthreads();
    if (write_y) {
#pragma unroll
      for (int j = 0; j < XPER; ++j) {
        const int e = tid + j * SEL_TH, t = e / COLS, c = p0 + e - t * COLS;
        if (t < nt && c < a.channels) out[(c0 + t) * a.ldo + c] = from_f32<T>(sy[e] * silu_f(to_f32(zpre[j])));
      }
    }
  }
  if (live && to != nullptr) {
#pragma unroll
    for (int i = 0; i < SEL_SLAB; ++i) {
      const int n = l * SEL_SLAB + i;
      if (n < N) to[n] = S[i];
    }
  }
  if (live && nseg > 1 && a.pass == 1 && l == 0) a.seg_steps[((long long)b * a.nseg + seg) * a.channels + mine] = steps;
}

// A step of single tokens: the same operations on one token a sequence, straight from memory (nothing is shared by
// enough threads to be worth a stop in LDS).
template <int LN, bool WHOLE, typename T>
__global__ __launch_bounds__(SEL_TH) void selective_step_kernel(const T* __restrict__ x, const float* __restrict__ dt,
                                                                const T* __restrict__ Bm, const T* __restrict__ Cm,
                                                                const T* __restrict__ z, T* __restrict__ out, SelArgs a) {
  constexpr int COLS = SEL_TH / LN;
  const int l = threadIdx.x % LN, b = blockIdx.y, ch = blockIdx.x * COLS + (int)threadIdx.x / LN, N = a.N;
  const bool live = ch < a.channels;
  const int c = live ? ch : 0;
  const long long r = a.cu_rows[b];
  float* sp = a.state + ((long long)a.seq_slot[b] * a.channels + c) * N;
  float S[SEL_SLAB], A2[SEL_SLAB], bv[SEL_SLAB], cv[SEL_SLAB];
  if (WHOLE) {  // (every lane has its eight entries: they go as 16-byte loads)
    const float* ap = a.a_log + (long long)c * N + l * SEL_SLAB;
    const float4 a0 = *(const float4*)ap, a1 = *(const float4*)(ap + 4);
    const float4 s0 = *(const float4*)(sp + l * SEL_SLAB), s1 = *(const float4*)(sp + l * SEL_SLAB + 4);
#pragma unroll
    for (int i = 0; i < SEL_SLAB; ++i) {
      bv[i] = to_f32(Bm[r * a.ldb + l * SEL_SLAB + i]);
      cv[i] = to_f32(Cm[r * a.ldc + l * SEL_SLAB + i]);
    }
    A2[0] = a0.x, A2[1] = a0.y, A2[2] = a0.z, A2[3] = a0.w, A2[4] = a1.x, A2[5] = a1.y, A2[6] = a1.z, A2[7] = a1.w;
    S[0] = s0.x, S[1] = s0.y, S[2] = s0.z, S[3] = s0.w, S[4] = s1.x, S[5] = s1.y, S[6] = s1.z, S[7] = s1.w;
  } else {
#pragma unroll
    for (int i = 0; i < SEL_SLAB; ++i) {
      const int n = l * SEL_SLAB + i;
      const bool has = n < N;
      A2[i] = has ? a.a_log[(long long)c * N + n] : 0.f;
      bv[i] = has ? to_f32(Bm[r * a.ldb + n]) : 0.f;
      cv[i] = has ? to_f32(Cm[r * a.ldc + n]) : 0.f;
      S[i] = has ? sp[n] : 0.f;
    }
  }
  const float raw = dt[r * a.lddt + c], bias = a.dt_bias[c], xv = to_f32(x[r * a.ldx + c]), zv = to_f32(z[r * a.ldz + c]);
  const float D = a.d_skip[c];
  const float step = softplus_f(raw + bias), dx = step * xv;
  float acc = 0.f, acc1 = 0.f;
#pragma unroll
  for (int i = 0; i < SEL_SLAB; ++i) {
    A2[i] = WHOLE || l * SEL_SLAB + i < N ? -expf(A2[i]) * LOG2E : 0.f;
    S[i] = fmaf(S[i], __builtin_amdgcn_exp2f(step * A2[i]), dx * bv[i]);
  }
#pragma unroll
  for (int i = 0; i < SEL_SLAB; i += 2) {
    acc = fmaf(S[i], cv[i], acc);
    acc1 = fmaf(S[i + 1], cv[i + 1], acc1);
  }
  acc = group_sum<LN>(acc + acc1);
  if (!live) return;
  if (WHOLE) {
    *(float4*)(sp + l * SEL_SLAB) = make_float4(S[0], S[1], S[2], S[3]);
    *(float4*)(sp + l * SEL_SLAB + 4) = make_float4(S[4], S[5], S[6], S[7]);
  } else {
#pragma unroll
    for (int i = 0; i < SEL_SLAB; ++i) {
      const int n = l * SEL_SLAB + i;
      if (n < N) sp[n] = S[i];
    }
  }
  if (l == 0) out[r * a.ldo + c] = from_f32<T>(fmaf(D, xv, acc) * silu_f(zv));
}

// Between the two passes: segment 0 left the state at its true end, every other segment the state it reaches from zero
// and the sum of its steps.  In order, every segment's true start takes the place of what it left, and the last
// segment's true end goes into the cache.
__global__ __launch_bounds__(256) void selective_chain_kernel(SelArgs a) {
  const int b = blockIdx.y;
  if (a.cu_rows[b + 1] - a.cu_rows[b] < SEL_MIN_ROWS) return;
  const long long CN = (long long)a.channels * a.N, e = (long long)blockIdx.x * 256 + threadIdx.x;
  if (e >= CN) return;
  const long long c = e / a.N;
  const float A2 = -expf(a.a_log[e]) * LOG2E;
  float* seg = a.seg_state + (long long)b * a.nseg * CN + e;
  const float* steps = a.seg_steps + (long long)b * a.nseg * a.channels + c;
  float S = seg[0];
  for (int s = 1; s < a.nseg; ++s) {
    const float reached = seg[s * CN];
    seg[s * CN] = S;
    S = fmaf(__builtin_amdgcn_exp2f(steps[(long long)s * a.channels] * A2), S, reached);
  }
  a.state[(long long)a.seq_slot[b] * CN + e] = S;
}

int sel_lanes(int N) {
  int ln = 1;
  while (ln * SEL_SLAB < N) ln <<= 1;
  return ln;
}

long long selective_floats(int batch, int channels, int N, int max_rows) {
  if (max_rows < SEL_MIN_ROWS || N > 64 * SEL_SLAB) return 0;
  if ((long long)batch * lq_ceil_div(channels, SEL_TH / sel_lanes(N)) >= 4ll * lq_compute_units()) return 0;  // the chip is full as it is
  return (long long)batch * SEL_SEGMENTS * ((long long)channels * N + channels);
}

template <int LN, typename T>
void launch_selective(const void* x, const float* dt, const void* Bm, const void* Cm, const void* z, void* out, const SelArgs& a,
                      int batch, bool single, hipStream_t stream) {
  dim3 grid(lq_ceil_div(a.channels, SEL_TH / LN), batch, a.nseg);
  const bool whole = a.N == LN * SEL_SLAB && (uintptr_t)a.state % 16 == 0 && (uintptr_t)a.a_log % 16 == 0;
  if (single && whole)
    selective_step_kernel<LN, true, T><<<grid, SEL_TH, 0, stream>>>((const T*)x, dt, (const T*)Bm, (const T*)Cm, (const T*)z, (T*)out, a);
  else if (single)
    selective_step_kernel<LN, false, T><<<grid, SEL_TH, 0, stream>>>((const T*)x, dt, (const T*)Bm, (const T*)Cm, (const T*)z, (T*)out, a);
  else
    selective_scan_kernel<LN, T><<<grid, SEL_TH, 0, stream>>>((const T*)x, dt, (const T*)Bm, (const T*)Cm, (const T*)z, (T*)out, a);
}

template <typename T>
void dispatch_selective(const void* x, const float* dt, const void* Bm, const void* Cm, const void* z, void* out,
                        const SelArgs& a, int batch, bool single, hipStream_t stream) {
  switch (sel_lanes(a.N)) {
    case 1: return launch_selective<1, T>(x, dt, Bm, Cm, z, out, a, batch, single, stream);
    case 2: return launch_selective<2, T>(x, dt, Bm, Cm, z, out, a, batch, single, stream);
    case 4: return launch_selective<4, T>(x, dt, Bm, Cm, z, out, a, batch, single, stream);
    case 8: return launch_selective<8, T>(x, dt, Bm, Cm, z, out, a, batch, single, stream);
    case 16: return launch_selective<16, T>(x, dt, Bm, Cm, z, out, a, batch, single, stream);
    case 32: return launch_selective<32, T>(x, dt, Bm, Cm, z, out, a, batch, single, stream);
    default: return launch_selective<64, T>(x, dt, Bm, Cm, z, out, a, batch, single, stream);
  }
}

// ---------------------------------------------------------------- the gates of a matrix memory
// Per head, with i = cap tanh((raw_i + b_i) / cap) and f = log sigmoid(cap tanh((raw_f + b_f) / cap)) the logarithms of
// the gates and a running maximum m (zero before the first token):
//   m_t = max(f_t + m_(t-1), i_t);   decay = exp(f_t + m_(t-1) - m_t);   take = exp(i_t - m_t);   floor = exp(-m_t).
// A workgroup of WAVES wavefronts a (sequence, head), 64 tokens a wavefront at a time: a token is the map m -> max(F + m, I)
// with (F, I) = (f, i), maps compose to maps of the same form, so the running maxima of 64 tokens are a scan over the
// lanes, and a wavefront's start is the wavefronts' maps before it applied to the chunk's.
__device__ inline float soft_cap_f(float v, float cap) { return cap * tanhf(v / cap); }

template <int WAVES>
__global__ __launch_bounds__(64 * WAVES) void memory_gates_kernel(const float* __restrict__ zi, int ldi,
                                                                  const float* __restrict__ zf, int ldf,
                                                                  const float* __restrict__ bi, const float* __restrict__ bf,
                                                                  float cap, float* __restrict__ m_state,
                                                                  float* __restrict__ decay, float* __restrict__ take,
                                                                  float* __restrict__ floor_out, int heads,
                                                                  const int* __restrict__ seq_slot,
                                                                  const int* __restrict__ cu_rows) {
  __shared__ float whole_f[WAVES], whole_i[WAVES];
  const int b = blockIdx.x / heads, h = blockIdx.x % heads, wave = threadIdx.x >> 6, lane = threadIdx.x & 63;
  float* mp = m_state + (long long)seq_slot[b] * heads + h;
  float m = *mp;  // the maximum before the chunk (every thread holds it)
  const long long r0 = cu_rows[b], r1 = cu_rows[b + 1];
  for (long long c0 = r0; c0 < r1; c0 += 64 * WAVES) {
    const long long r = c0 + threadIdx.x;
    const bool live = r < r1;
    float i = -INFINITY, f = 0.f;  // (a lane past the end maps m to itself)
    if (live) {
      i = soft_cap_f(zi[r * ldi + h] + bi[h], cap);
      f = -softplus_f(-soft_cap_f(zf[r * ldf + h] + bf[h], cap));
    }
    float F = f, I = i;  // the composition of this lane's token with all before it in the wavefront
#pragma unroll
    for (int off = 1; off < 64; off <<= 1) {
      const float Fb = __shfl_up(F, off, 64), Ib = __shfl_up(I, off, 64);
      if (lane >= off) {
        I = fmaxf(Ib + F, I);
        F += Fb;
      }
    }
    float start = m;
    if constexpr (WAVES > 1) {
      if (lane == 63) whole_f[wave] = F, whole_i[wave] = I;
      __syncthreads();
      for (int w = 0; w < WAVES; ++w) {
        if (w == wave) start = m;
        m = fmaxf(whole_f[w] + m, whole_i[w]);
      }
      __syncthreads();  // (the next chunk writes the maps anew)
    }
    const float top = fmaxf(F + start, I);
    float before = __shfl_up(top, 1, 64);
    if (lane == 0) before = start;
    if (live) {
      decay[r * heads + h] = expf(f + before - top);
      take[r * heads + h] = expf(i - top);
      floor_out[r * heads + h] = expf(-top);
    }
    if constexpr (WAVES == 1) m = __shfl(top, 63, 64);
  }
  if (threadIdx.x == 0) *mp = m;
}

// The memory's answer from the scan's results.  y [rows, heads * (P + 1)]: a head's S^T q and, in its last column, n . q,
// both before q's scale: o = scale y / (max(|scale n . q|, floor) + eps0); then o divided by its root mean square over P,
// times a weight for every column, times the sigmoid of the gate.  One wavefront a (row, head), a head's entries in
// registers (PER a lane) where they fit.
template <typename T, int PER>
__global__ __launch_bounds__(256) void memory_out_kernel(const float* __restrict__ y, int ldy, const float* __restrict__ floor_in,
                                                         const float* __restrict__ z, int ldz, const float* __restrict__ w,
                                                         float scale, float eps0, float eps, T* __restrict__ out, int ldo,
                                                         int heads, int P) {
  const int r = blockIdx.x, h = blockIdx.y * 4 + (threadIdx.x >> 6), lane = threadIdx.x & 63;
  if (h >= heads) return;
  const float* yr = y + (long long)r * ldy + (long long)h * (P + 1);
  const float den = fmaxf(fabsf(scale * yr[P]), floor_in[(long long)r * heads + h]) + eps0;
  const float mul = scale / den;
  const float* zr = z + (long long)r * ldz + (long long)h * P;
  const float* wr = w + (long long)h * P;
  T* orow = out + (long long)r * ldo + (long long)h * P;
  float v[PER], g[PER];
  float ss = 0.f;
#pragma unroll
  for (int j = 0; j < PER; ++j) {
    const int d = lane + 64 * j;
    v[j] = d < P ? yr[d] * mul : 0.f;
    g[j] = d < P ? zr[d] : 0.f;
    ss = fmaf(v[j], v[j], ss);
  }
  for (int d = lane + 64 * PER; d < P; d += 64) ss = fmaf(yr[d] * mul, yr[d] * mul, ss);
  const float inv = 1.f / sqrtf(wave_sum(ss) / (float)P + eps);
#pragma unroll
  for (int j = 0; j < PER; ++j) {
    const int d = lane + 64 * j;
    if (d < P) orow[d] = from_f32<T>(v[j] * inv * wr[d] * sigmoid_f(g[j]));
  }
  for (int d = lane + 64 * PER; d < P; d += 64) orow[d] = from_f32<T>(yr[d] * mul * inv * wr[d] * sigmoid_f(zr[d]));
}

}  // namespace

extern "C" long long lq_selective_scan_workspace(int batch, int channels, int N, int max_rows) {
  if (batch <= 0 || channels <= 0 || N <= 0) return 0;
  return selective_floats(batch, channels, N, max_rows);
}

// x, z and out [rows, channels], B and C [rows, N] in one dtype, dt [rows, channels] 32-bit (before its softplus),
// dt_bias and d_skip [channels], a_log [channels, N], state [slots, channels, N]; rows lie sequence by sequence
// (cu_rows), every one of the `batch` sequences with at least one of the `rows`.  `max_rows`: the most rows a sequence
// brings (0: unknown); `scratch`: lq_selective_scan_workspace(...)
// floats, or null (then no segments).
extern "C" int lq_selective_scan(const void* x, int ldx, const float* dt, int lddt, const void* Bm, int ldb, const void* Cm,
                                 int ldc, const void* z, int ldz, const float* dt_bias, const float* a_log,
                                 const float* d_skip, float* state, void* out, int ldo, int dtype, int channels, int N,
                                 const int* seq_slot, const int* cu_rows, int batch, int rows, int max_rows, float* scratch,
                                 long long scratch_floats, hipStream_t stream) {
  LQ_REQUIRE(rows >= batch, "selective_scan: %d rows of %d sequences", rows, batch);
  const bool single = rows == batch;  // every sequence brings one token
  LQ_REQUIRE(channels > 0 && N > 0 && batch > 0 && batch <= 65535, "selective_scan: %d channels, state %d, %d sequences", channels, N, batch);
  LQ_REQUIRE(N <= 64 * SEL_SLAB, "selective_scan: state size %d is larger than %d", N, 64 * SEL_SLAB);
  LQ_REQUIRE(ldx >= channels && lddt >= channels && ldz >= channels && ldo >= channels && ldb >= N && ldc >= N,
             "selective_scan: a row stride is smaller than its row");
  LQ_REQUIRE(x && dt && Bm && Cm && z && dt_bias && a_log && d_skip && state && out && seq_slot && cu_rows,
             "selective_scan: null pointer");
  LQ_REQUIRE(dtype == LQ_F32 || dtype == LQ_BF16, "selective_scan: unknown dtype %d", dtype);
  const long long need = scratch != nullptr ? selective_floats(batch, channels, N, max_rows) : 0;
  LQ_REQUIRE(need <= scratch_floats, "selective_scan: %lld floats of scratch for a launch in segments, %lld given", need, scratch_floats);
  SelArgs a = {ldx, lddt, ldb, ldc, ldz, ldo, channels, N, dt_bias, a_log, d_skip, state, seq_slot, cu_rows, 1, 1, nullptr, nullptr};
  if (need > 0) {
    a.nseg = SEL_SEGMENTS;
    a.seg_state = scratch;
    a.seg_steps = scratch + (long long)batch * SEL_SEGMENTS * channels * N;
  }
  auto run = [&]() {
    if (dtype == LQ_F32) dispatch_selective<float>(x, dt, Bm, Cm, z, out, a, batch, single, stream);
    else dispatch_selective<bf16_t>(x, dt, Bm, Cm, z, out, a, batch, single, stream);
  };
  run();
  LQ_CHECK_LAUNCH("selective_scan");
  if (a.nseg > 1) {
    selective_chain_kernel<<<dim3((unsigned)lq_ceil_div64((long long)channels * N, 256), batch), 256, 0, stream>>>(a);
    LQ_CHECK_LAUNCH("selective_scan(chain)");
    a.pass = 2;
    run();
    LQ_CHECK_LAUNCH("selective_scan(second pass)");
  }
  return 0;
}

// zi and zf [rows, heads] (raw logits), bi and bf [heads], m_state [slots, heads]; decay, take and floor [rows, heads] dense;
// `rows` all sequences' rows together (for the launch's shape alone)
extern "C" int lq_memory_gates(const float* zi, int ldi, const float* zf, int ldf, const float* bi, const float* bf, float cap,
                               float* m_state, float* decay, float* take, float* floor_out, int heads, const int* seq_slot,
                               const int* cu_rows, int batch, int rows, hipStream_t stream) {
  LQ_REQUIRE(rows >= 0 && heads > 0 && batch > 0 && cap > 0.f && ldi >= heads && ldf >= heads, "memory_gates: %d heads, cap %g", heads, (double)cap);
  LQ_REQUIRE(zi && zf && bi && bf && m_state && decay && take && floor_out && seq_slot && cu_rows, "memory_gates: null pointer");
#define LQ_GATES(WAVES)                                                                                                     \
  memory_gates_kernel<WAVES><<<(unsigned)(batch * heads), 64 * WAVES, 0, stream>>>(zi, ldi, zf, ldf, bi, bf, cap, m_state, decay, \
                                                                                   take, floor_out, heads, seq_slot, cu_rows)
  if (rows > 64ll * batch) LQ_GATES(16);  // (some sequence brings more than a wavefront's tokens)
  else LQ_GATES(1);
#undef LQ_GATES
  LQ_CHECK_LAUNCH("memory_gates");
  return 0;
}

extern "C" int lq_memory_out(const float* y, int ldy, const float* floor_in, const float* z, int ldz, const float* w, float scale,
                             float eps0, float eps, void* out, int out_dtype, int ldo, int rows, int heads, int P,
                             hipStream_t stream) {
  LQ_REQUIRE(rows > 0 && heads > 0 && P > 0 && ldy >= heads * (P + 1) && ldz >= heads * P && ldo >= heads * P,
             "memory_out: rows %d, %d heads of %d, or a row stride is smaller than its row", rows, heads, P);
  LQ_REQUIRE(y && floor_in && z && w && out && lq_ceil_div(heads, 4) <= 65535, "memory_out: null pointer or too many heads");
  const dim3 grid(rows, lq_ceil_div(heads, 4));
  if (out_dtype == LQ_F32)
    memory_out_kernel<float, 8><<<grid, 256, 0, stream>>>(y, ldy, floor_in, z, ldz, w, scale, eps0, eps, (float*)out, ldo, heads, P);
  else if (out_dtype == LQ_BF16)
    memory_out_kernel<bf16_t, 8><<<grid, 256, 0, stream>>>(y, ldy, floor_in, z, ldz, w, scale, eps0, eps, (bf16_t*)out, ldo, heads, P);
  else LQ_REQUIRE(false, "memory_out: unknown dtype %d", out_dtype);
  LQ_CHECK_LAUNCH("memory_out");
  return 0;
}
