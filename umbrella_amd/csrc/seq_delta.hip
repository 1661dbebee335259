// Gated delta rule: a [D][E] fp32 matrix state per (sequence, value head), decayed by one number per token and corrected by what it
// already returns for the token's key,
//     S <- g_t S        u_t = beta_t (v_t - S^T k_t)        S <- S + k_t u_t^T        o_t = S^T q_t
// q and k are unit vectors (q times a constant) shared by H / Hk consecutive value heads; q, k and v come out of one input
// projection through a short causal convolution per channel and silu; beta = sigmoid(b), log g = -exp(A_log) softplus(a + dt_bias),
// one of each per value head.  Columns of proj from col0: [q (Hk D) | k (Hk D) | v (H E) | gate (H E) | b (H) | a (H)].
//
// The raw projections of the last positions are the sequence's state beside S: a ring of `taps` rows per slot, position p in row
// p % taps -- one row more than the convolution looks back, so that the row a token stores is none of those its own convolution
// reads and a single-token step can read and refresh the ring from several workgroups at once.
//
//   delta_step    steps of ONE token per sequence: convolution, unit norms, gates, recurrence and ring in one launch
//   delta_prep    longer steps: q, k, v, beta and log g of every token as the chunk kernels read them
//   delta_chunk_* longer steps: the recurrence in chunks of 64 tokens (below)
// Everything is fp32.  The convolution sums its taps oldest first whatever their source.
#include "seq_common.h"
#include <type_traits>

constexpr float DELTA_UNIT_EPS = 1e-6f;

__device__ __forceinline__ float delta_softplus(float z) { return fmaxf(z, 0.f) + log1pf(expf(-fabsf(z))); }

struct DeltaIn {
  const float* proj;                       // row t, columns from col0
  int ld, col0, Hk, H, D, E, taps;
  float* ring;                             // [slots][taps][C]
  const float *dt_bias, *a_log;            // [H]
  __device__ __forceinline__ int qk() const { return Hk * D; }
  __device__ __forceinline__ int C() const { return 2 * Hk * D + H * E; }
};

// convolved, activated channel c of token t (position p): taps of this step's rows or of the ring, loaded before any is used
template <typename P>
__device__ __forceinline__ float delta_channel(const DeltaIn& in, const typename El<P>::type* __restrict__ w,
                                               const int* __restrict__ slot_, int t, int p, int slot, int c) {
  const int taps = in.taps, C = in.C();
  float acc = 0.f;
  for (int j0 = 0; j0 < taps; j0 += 4) {
    float x[4], wv[4];
#pragma unroll
    for (int u = 0; u < 4; ++u) {
      const int j = j0 + u < taps ? j0 + u : taps - 1, d = taps - 1 - j;          // tap j looks d positions back
      const bool same = d == 0 || (t - d >= 0 && slot_[t - d] == slot);
      const float* src = (same || d > p) ? in.proj + (long)(same ? t - d : t) * in.ld + in.col0 + c
                                         : in.ring + ((long)slot * taps + (p - d) % taps) * C + c;
      x[u] = *src;
      wv[u] = (j0 + u < taps && d <= p) ? ldf<P>(w + (long)c * taps + j) : 0.f;
      if (d > p) x[u] = 0.f;
    }
#pragma unroll
    for (int u = 0; u < 4; ++u) acc += wv[u] * x[u];
  }
  return siluf_(acc);
}

// ---- one token per sequence.  Workgroup = (32 value columns, value head, row): thread (c = tid % 32, rg = tid / 32) keeps rows
// rg, rg + 8, .. of column c.  The state's rows are in flight while the convolution and the norms are formed in LDS; the two sums
// over the rows (S^T k and S^T q) meet once in a wave and once through LDS.
template <typename P, int RPT>
__global__ __launch_bounds__(256) void delta_step_kernel(float* __restrict__ o, float* __restrict__ state, DeltaIn in,
                                                         const typename El<P>::type* __restrict__ conv_w, const int* __restrict__ pos,
                                                         const int* __restrict__ slot_, float qscale) {
  extern __shared__ float sm[];
  const int t = blockIdx.z, h = blockIdx.y, e0 = blockIdx.x * 32, D = in.D, E = in.E, C = in.C(), rep = in.H / in.Hk, hk = h / rep;
  const int tid = threadIdx.x, wave = tid >> 6, lane = tid & 63, c = tid & 31, rg = tid >> 5;
  const int p = pos[t], slot = slot_[t];
  const bool c_ok = e0 + c < E;
  float* sp = state + (((long)slot * in.H + h) * D) * E + (c_ok ? e0 + c : 0);
  float S[RPT];
#pragma unroll
  for (int i = 0; i < RPT; ++i) {
    const int d = rg + 8 * i;
    S[i] = sp[(long)(d < D ? d : 0) * E];
  }
  float* qs = sm;                          // [D] q, [D] k, [32] v, [8] sums of squares and gates, [2][4][32] partial sums
  float* ks = qs + D;
  float* vs = ks + D;
  float* sc = vs + 32;
  float* red = sc + 8;
  const float* pr = in.proj + (long)t * in.ld + in.col0;
  float* rw = in.ring + ((long)slot * in.taps + p % in.taps) * C;
  const bool owner = blockIdx.x == 0 && h % rep == 0;                // of the q / k channels' ring entries
  for (int x = tid; x < 2 * D + 32; x += 256) {
    const int cc = x < D ? hk * D + x : (x < 2 * D ? in.qk() + hk * D + (x - D) : 2 * in.qk() + h * E + e0 + (x - 2 * D));
    if (x >= 2 * D && e0 + (x - 2 * D) >= E) { sm[x] = 0.f; continue; }
    sm[x] = delta_channel<P>(in, conv_w, slot_, t, p, slot, cc);
    if (x >= 2 * D || owner) rw[cc] = pr[cc];
  }
  if (tid == 0) {
    const int bc = in.C() + in.H * E + h;
    sc[2] = 1.f / (1.f + expf(-pr[bc]));
    sc[3] = expf(-expf(in.a_log[h]) * delta_softplus(pr[bc + in.H] + in.dt_bias[h]));
  }
  __syncthreads();
  if (wave < 2) {
    float ss = 0.f;
    for (int i = lane; i < D; i += 64) { const float v = sm[wave * D + i]; ss += v * v; }
    ss = wave_sum(ss);
    if (lane == 0) sc[wave] = 1.f / sqrtf(ss + DELTA_UNIT_EPS);
  }
  __syncthreads();
  const float fq = sc[0] * qscale, fk = sc[1], beta = sc[2], g = sc[3];
  const bool fresh = p == 0;
  float a = 0.f;
#pragma unroll
  for (int i = 0; i < RPT; ++i) {
    const int d = rg + 8 * i;
    S[i] = (fresh || d >= D) ? 0.f : g * S[i];
    a += S[i] * (d < D ? ks[d] * fk : 0.f);
  }
  a += __shfl_xor(a, 32, 64);
  if (lane < 32) red[wave * 32 + c] = a;
  __syncthreads();
  const float u = beta * (vs[c] - ((red[c] + red[32 + c]) + (red[64 + c] + red[96 + c])));
  float b = 0.f;
#pragma unroll
  for (int i = 0; i < RPT; ++i) {
    const int d = rg + 8 * i;
    if (d < D) {
      S[i] += ks[d] * fk * u;
      b += S[i] * (qs[d] * fq);
      if (c_ok) sp[(long)d * E] = S[i];
    }
  }
  b += __shfl_xor(b, 32, 64);
  if (lane < 32) red[128 + wave * 32 + c] = b;
  __syncthreads();
  if (tid < 32 && c_ok)
    o[((long)t * in.H + h) * E + e0 + c] = (red[128 + c] + red[160 + c]) + (red[192 + c] + red[224 + c]);
}

// ---- longer steps: one wave per (token, head slot): Hk q slots, Hk k slots, H v slots, one slot for the gates
template <typename P>
__global__ __launch_bounds__(256) void delta_prep_kernel(float* __restrict__ q, float* __restrict__ k, int ldqk, int Dp,
                                                         float* __restrict__ v, float* __restrict__ beta, float* __restrict__ lg,
                                                         DeltaIn in, const typename El<P>::type* __restrict__ conv_w,
                                                         const int* __restrict__ pos, const int* __restrict__ slot_, int T,
                                                         float qscale) {
  const int wave = threadIdx.x >> 6, lane = threadIdx.x & 63;
  const int per = 2 * in.Hk + in.H + 1;
  const long item = (long)blockIdx.x * 4 + wave;
  if (item >= (long)T * per) return;
  const int t = (int)(item / per), hs = (int)(item % per), D = in.D, E = in.E;
  const int p = pos[t], slot = slot_[t];
  if (hs < 2 * in.Hk) {
    const bool is_q = hs < in.Hk;
    const int hk = is_q ? hs : hs - in.Hk;
    float keep[4], ss = 0.f;                             // D <= 256
#pragma unroll
    for (int u = 0; u < 4; ++u) {
      const int i = lane + 64 * u;
      keep[u] = i < D ? delta_channel<P>(in, conv_w, slot_, t, p, slot, hs * D + i) : 0.f;
      ss += keep[u] * keep[u];
    }
    ss = wave_sum(ss);
    const float f = (is_q ? qscale : 1.f) / sqrtf(ss + DELTA_UNIT_EPS);
    float* row = (is_q ? q : k) + (long)t * ldqk + (long)hk * Dp;
#pragma unroll
    for (int u = 0; u < 4; ++u)
      if (lane + 64 * u < Dp) row[lane + 64 * u] = keep[u] * f;       // zeros from D to Dp
  } else if (hs < per - 1) {
    const int h = hs - 2 * in.Hk;
    for (int i = lane; i < E; i += 64)
      v[((long)t * in.H + h) * E + i] = delta_channel<P>(in, conv_w, slot_, t, p, slot, 2 * in.qk() + h * E + i);
  } else {
    const float* pr = in.proj + (long)t * in.ld + in.col0 + in.C() + in.H * E;
    for (int h = lane; h < in.H; h += 64) {
      beta[(long)t * in.H + h] = 1.f / (1.f + expf(-pr[h]));
      lg[(long)t * in.H + h] = -expf(in.a_log[h]) * delta_softplus(pr[in.H + h] + in.dt_bias[h]);
    }
  }
}

// ---- the recurrence in chunks of 64 tokens.  With c_t = log g_1 + .. + log g_t inside a chunk and S_0 the state before it,
//     u_t = beta_t (v_t - e^(c_t) S_0^T k_t - sum_{s < t} e^(c_t - c_s) (k_s . k_t) u_s)
// is a unit lower triangular system (I + A) U = diag(beta) V - diag(beta e^c) K S_0, A_ts = beta_t e^(c_t - c_s) (k_t . k_s).  So
//   (1) all chunks side by side: Uv = (I + A)^-1 diag(beta) V, Wk = (I + A)^-1 diag(beta e^c) K, M_ts = e^(c_t - c_s) (q_t . k_s), s <= t
//   (2) chunk after chunk, the state in registers: U = Uv - Wk S, o = diag(e^c) Q S + M U, S <- e^(c_end) S + K^T diag(e^(c_end - c)) U
// All products run on the true-fp32 matrix instruction 16x16x4.  Its operands pair up by lane group, so the order of k inside 16 is
// free: step i multiplies k = 4 (lane / 16) + i.  An accumulator tile (rows 4 (lane / 16) + r, column lane % 16) therefore IS the
// right-hand operand of the next product over those rows -- the triangular solve goes down its four 16-row blocks, and the state
// meets Wk, Q and K^T, without a value changing lanes.  Exponents are of non-positive numbers; prefix sums are kept in double, as
// a decay between two tokens is the exponential of a difference of two of them.
constexpr int DC_Q = 64;

struct DeltaChunk {
  const float *q, *k, *v, *beta, *lg;      // q, k [T][ldqk] groups of Dp (zero padded from D); v [T][H E]; beta, lg [T][H]
  float *wk, *uv, *m, *ec, *ew;            // [T][H Dp], [T][H Ep], [T][H 64], [H][T] e^(c_t), [H][T] e^(c_end - c_t)
  int T, ldqk, Hk, H, D, Dp, E, Ep;
  const int *seq_slot, *seq_row0, *seq_pos0, *seq_len;
};

__device__ __forceinline__ f32x4 mma4(f32x4 a, f32x4 b, f32x4 c) {
#pragma unroll
  for (int i = 0; i < 4; ++i) c = __builtin_amdgcn_mfma_f32_16x16x4f32(a[i], b[i], c, 0, 0, 0);
  return c;
}

// (1) grid (chunks, value heads, sequences)
__global__ __launch_bounds__(256) void delta_chunk_solve_kernel(DeltaChunk a) {
  extern __shared__ __attribute__((aligned(16))) float sm[];
  const int b = blockIdx.z, h = blockIdx.y, t0 = blockIdx.x * DC_Q, len = a.seq_len[b];
  if (t0 >= len) return;
  const int cnt = len - t0 < DC_Q ? len - t0 : DC_Q, H = a.H, Dp = a.Dp, LK = Dp + 4, hk = h / (H / a.Hk);
  const long row0 = (long)a.seq_row0[b] + t0;
  const int tid = threadIdx.x, wave = tid >> 6, lane = tid & 63, j = lane & 15, g = lane >> 4;
  double* cum = reinterpret_cast<double*>(sm);   // [64]
  float* be = sm + 128;                          // [64] beta (0 past the stretch)
  float* ecs = be + 64;                          // [64] e^(c_t)
  float* As = ecs + 64;                          // [64][68]: -A
  float* Td = As + 64 * 68;                      // [4][16][20]: inverses of the diagonal blocks of I + A
  float* Ks = Td + 4 * 16 * 20;                  // [64][LK]
  float* Qs = Ks + 64 * LK;                      // [64][LK]
  if (wave == 0) {
    double v = lane < cnt ? (double)a.lg[(row0 + lane) * H + h] : 0.0;
#pragma unroll
    for (int o = 1; o < 64; o <<= 1) {
      const double u = __shfl_up(v, o, 64);
      if (lane >= o) v += u;
    }
    cum[lane] = v;
    be[lane] = lane < cnt ? a.beta[(row0 + lane) * H + h] : 0.f;
    const float e = expf((float)v), w = expf((float)(__shfl(v, 63, 64) - v));
    ecs[lane] = e;
    if (lane < cnt) {
      a.ec[(long)h * a.T + row0 + lane] = e;
      a.ew[(long)h * a.T + row0 + lane] = w;
    }
  }
  const int dq = Dp >> 2;
  for (int x = tid; x < 64 * dq; x += 256) {
    const int s = x / dq, d = (x - s * dq) * 4;
    f32x4 kv = f32x4{0.f, 0.f, 0.f, 0.f}, qv = kv;
    if (s < cnt) {
      kv = *reinterpret_cast<const f32x4*>(a.k + (row0 + s) * a.ldqk + (long)hk * Dp + d);
      qv = *reinterpret_cast<const f32x4*>(a.q + (row0 + s) * a.ldqk + (long)hk * Dp + d);
    }
    *reinterpret_cast<f32x4*>(Ks + s * LK + d) = kv;
    *reinterpret_cast<f32x4*>(Qs + s * LK + d) = qv;
  }
  __syncthreads();
  // k . k and q . k, the ten 16 x 16 tiles on and below the diagonal of each
  for (int id = wave; id < 20; id += 4) {
    const int pair = id < 10 ? id : id - 10;
    const int rb = pair < 1 ? 0 : (pair < 3 ? 1 : (pair < 6 ? 2 : 3)), cb = pair - rb * (rb + 1) / 2;
    const float* X = (id < 10 ? Ks : Qs) + (16 * rb + j) * LK + 4 * g;
    const float* Y = Ks + (16 * cb + j) * LK + 4 * g;
    f32x4 acc = f32x4{0.f, 0.f, 0.f, 0.f};
    for (int k0 = 0; k0 < Dp; k0 += 16) acc = mma4(*reinterpret_cast<const f32x4*>(X + k0), *reinterpret_cast<const f32x4*>(Y + k0), acc);
    const int s = 16 * cb + j;
    const double cs = cum[s];
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int t = 16 * rb + 4 * g + r;
      const float e = s <= t ? expf((float)(cum[t] - cs)) : 0.f;
      if (id < 10) As[t * 68 + s] = s < t ? -be[t] * e * acc[r] : 0.f;
      else if (t < cnt) a.m[((row0 + t) * H + h) * 64 + s] = e * acc[r];
    }
  }
  __syncthreads();
  {                                              // wave w inverts diagonal block w: lane = column, rows one after another
    float x[16];
    const float* Ab = As + (16 * wave) * 68 + 16 * wave;
#pragma unroll
    for (int t = 0; t < 16; ++t) {
      x[t] = t == j ? 1.f : 0.f;
#pragma unroll
      for (int s = 0; s < t; ++s) x[t] += Ab[t * 68 + s] * x[s];
    }
    if (g == 0) {
#pragma unroll
      for (int t = 0; t < 16; ++t) Td[(wave * 16 + t) * 20 + j] = x[t];
    }
  }
  __syncthreads();
  const int nk = Dp >> 4, nt = nk + (a.Ep >> 4);
  for (int tile = wave; tile < nt; tile += 4) {
    const bool isW = tile < nk;
    const int col = 16 * (isW ? tile : tile - nk) + j;
    f32x4 U[4];
#pragma unroll
    for (int rb = 0; rb < 4; ++rb) {
      f32x4 acc;
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int t = 16 * rb + 4 * g + r;
        float x;
        if (isW) x = ecs[t] * Ks[t * LK + col];
        else x = (t < cnt && col < a.E) ? a.v[((row0 + t) * H + h) * a.E + col] : 0.f;
        acc[r] = be[t] * x;
      }
#pragma unroll
      for (int cb = 0; cb < rb; ++cb) acc = mma4(*reinterpret_cast<const f32x4*>(As + (16 * rb + j) * 68 + 16 * cb + 4 * g), U[cb], acc);
      U[rb] = mma4(*reinterpret_cast<const f32x4*>(Td + (rb * 16 + j) * 20 + 4 * g), acc, f32x4{0.f, 0.f, 0.f, 0.f});
    }
    float* dst = isW ? a.wk + (row0 * H + h) * Dp + col : a.uv + (row0 * H + h) * a.Ep + col;
    const long lds = (long)H * (isW ? Dp : a.Ep);
#pragma unroll
    for (int rb = 0; rb < 4; ++rb)
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int t = 16 * rb + 4 * g + r;
        if (t < cnt) dst[t * lds] = U[rb][r];
      }
  }
}

// (2) grid (16-column slices, value heads, sequences).  Wave w keeps TPW 16-row tiles of the state slice (from tile w TPW) as
// accumulators; the waves' shares of Wk S and Q S meet in LDS; wave w owns read-out rows 16 w .. of the chunk.
template <int TPW> struct DeltaFrag {
  f32x4 wk[4][TPW], q[4][TPW], kt[4][TPW], m[4], uv[4], ew[4], ec;
  float eq;
};

template <int TPW, bool PRE>
__global__ __launch_bounds__(256) void delta_chunk_scan_kernel(float* __restrict__ o, float* __restrict__ state, DeltaChunk a) {
  extern __shared__ __attribute__((aligned(16))) float red[];        // [2][4 waves][8 tiles][256]
  const int b = blockIdx.z, h = blockIdx.y, H = a.H, Dp = a.Dp, D = a.D, E = a.E;
  const int n = a.seq_len[b];
  if (n <= 0) return;
  const int tid = threadIdx.x, lane = tid & 63, j = lane & 15, g = lane >> 4, hk = h / (H / a.Hk);
  const int wave = __builtin_amdgcn_readfirstlane(tid >> 6);         // uniform: what depends on it stays in scalar registers
  const int col = blockIdx.x * 16 + j;
  const bool c_ok = col < E;
  const long row0 = a.seq_row0[b];
  float* sp = state + (((long)a.seq_slot[b] * H + h) * D) * E + (c_ok ? col : 0);
  const bool fresh = a.seq_pos0[b] == 0;
  f32x4 S[TPW];
#pragma unroll
  for (int x = 0; x < TPW; ++x)
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int d = 16 * (wave * TPW + x) + 4 * g + r;
      S[x][r] = (!fresh && c_ok && d < D) ? sp[(long)d * E] : 0.f;
    }
  const f32x4 zero = f32x4{0.f, 0.f, 0.f, 0.f};
  const int nch = (n + DC_Q - 1) / DC_Q;
  const int ldw = H * Dp, ldu = H * a.Ep, ldm = H * 64, ldk = a.ldqk;
  // The operands of a chunk.  Every load is unconditional: a row past the stretch reads the last row instead, and what it brings
  // has no effect -- its weight ew is 0, M is 0 above the diagonal, its read-out is not stored.  In a full chunk the row of lane
  // (j, g) is its lane part plus a uniform part, so an address is a scalar base and one of a few lane offsets.
  auto load = [&](int ch, DeltaFrag<TPW>& f) {
    const int cnt = n - ch * DC_Q < DC_Q ? n - ch * DC_Q : DC_Q;
    const long base = row0 + (long)ch * DC_Q;
    const float* wk = a.wk + base * ldw + (long)h * Dp + 16 * wave * TPW;
    const float* q = a.q + base * ldk + (long)hk * Dp + 16 * wave * TPW;
    const float* k = a.k + base * ldk + (long)hk * Dp + 16 * wave * TPW;
    const float* uv = a.uv + base * ldu + (long)h * a.Ep + blockIdx.x * 16;
    const float* m = a.m + base * ldm + (long)h * 64;
    const float* ec = a.ec + (long)h * a.T + base;
    const float* ew = a.ew + (long)h * a.T + base;
    auto fill = [&](auto full) {
      // row of an operand whose lanes run over rows (u + j) / over groups of four rows (u + 4 g + r): uniform and lane part
      auto at_j = [&](const float* p, int ld, int u) {
        return full ? p + u * ld + (unsigned)(j * ld) : p + (unsigned)((u + j < cnt ? u + j : cnt - 1) * ld);
      };
      auto at_g = [&](const float* p, int ld, int u) {
        return full ? p + u * ld + (unsigned)(4 * g * ld) : p + (unsigned)((u + 4 * g < cnt ? u + 4 * g : cnt - 1) * ld);
      };
#pragma unroll
      for (int i = 0; i < 4; ++i) {
#pragma unroll
        for (int x = 0; x < TPW; ++x) {
          if (16 * (wave * TPW + x) < Dp) {                          // uniform
            f.wk[i][x] = *reinterpret_cast<const f32x4*>(at_j(wk + 16 * x, ldw, 16 * i) + 4 * g);
            f.q[i][x] = *reinterpret_cast<const f32x4*>(at_j(q + 16 * x, ldk, 16 * i) + 4 * g);
#pragma unroll
            for (int r = 0; r < 4; ++r) f.kt[i][x][r] = at_g(k + 16 * x, ldk, 16 * i + r)[j];
          } else {
            f.wk[i][x] = f.q[i][x] = f.kt[i][x] = zero;
          }
        }
#pragma unroll
        for (int r = 0; r < 4; ++r) {
          f.uv[i][r] = at_g(uv, ldu, 16 * i + r)[j];
          f.ew[i][r] = at_g(ew, 1, 16 * i + r)[0];
          if (!full && 16 * i + 4 * g + r >= cnt) f.ew[i][r] = 0.f;
        }
        if (i <= wave) f.m[i] = *reinterpret_cast<const f32x4*>(at_j(m + 16 * i, ldm, 16 * wave) + 4 * g);
        else f.m[i] = zero;
      }
#pragma unroll
      for (int r = 0; r < 4; ++r) f.ec[r] = at_g(ec, 1, 16 * wave + r)[0];
    };
    if (cnt == DC_Q) fill(std::true_type{});
    else fill(std::false_type{});
    f.eq = ec[cnt - 1];
  };
  auto compute = [&](int ch, const DeltaFrag<TPW>& f) {
    const int cnt = n - ch * DC_Q < DC_Q ? n - ch * DC_Q : DC_Q;
    float* rb = red + (ch & 1) * (4 * 8 * 256);
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      f32x4 w = zero, q = zero;
#pragma unroll
      for (int x = 0; x < TPW; ++x) { w = mma4(f.wk[i][x], S[x], w); q = mma4(f.q[i][x], S[x], q); }
      *reinterpret_cast<f32x4*>(rb + (wave * 8 + i) * 256 + lane * 4) = w;
      *reinterpret_cast<f32x4*>(rb + (wave * 8 + 4 + i) * 256 + lane * 4) = q;
    }
    __syncthreads();
    f32x4 U[4], out = zero;
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      f32x4 s = *reinterpret_cast<const f32x4*>(rb + i * 256 + lane * 4);
#pragma unroll
      for (int w = 1; w < 4; ++w) s += *reinterpret_cast<const f32x4*>(rb + (w * 8 + i) * 256 + lane * 4);
      U[i] = f.uv[i] - s;
    }
#pragma unroll
    for (int w = 0; w < 4; ++w) out += *reinterpret_cast<const f32x4*>(rb + (w * 8 + 4 + wave) * 256 + lane * 4);
    out *= f.ec;
#pragma unroll
    for (int i = 0; i < 4; ++i)
      if (i <= wave) out = mma4(f.m[i], U[i], out);
#pragma unroll
    for (int x = 0; x < TPW; ++x) S[x] *= f.eq;
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const f32x4 ue = U[i] * f.ew[i];
#pragma unroll
      for (int x = 0; x < TPW; ++x) S[x] = mma4(f.kt[i][x], ue, S[x]);
    }
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int t = 16 * wave + 4 * g + r;
      if (t < cnt && c_ok) o[((row0 + (long)ch * DC_Q + t) * H + h) * E + col] = out[r];
    }
  };
  if constexpr (PRE) {                           // the next chunk's operands are in flight while a chunk is worked on
    DeltaFrag<TPW> f0, f1;
    load(0, f0);
    for (int ch = 0; ch < nch; ch += 2) {
      if (ch + 1 < nch) load(ch + 1, f1);
      compute(ch, f0);
      if (ch + 1 < nch) {
        if (ch + 2 < nch) load(ch + 2, f0);
        compute(ch + 1, f1);
      }
    }
  } else {
    for (int ch = 0; ch < nch; ++ch) {
      DeltaFrag<TPW> f;
      load(ch, f);
      compute(ch, f);
    }
  }
#pragma unroll
  for (int x = 0; x < TPW; ++x)
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int d = 16 * (wave * TPW + x) + 4 * g + r;
      if (c_ok && d < D) sp[(long)d * E] = S[x][r];
    }
}

static inline int up16(int n) { return (n + 15) & ~15; }
static inline size_t delta_solve_lds(int Dp) {
  return ((size_t)128 + 64 + 64 + 64 * 68 + 4 * 16 * 20 + 2 * 64 * (size_t)(Dp + 4)) * sizeof(float);
}
static inline bool delta_in_ok(const float* proj, int ld, int col0, const void* conv_w, const float* ring, const float* dt_bias,
                               const float* a_log, int T, int Hk, int H, int D, int E, int taps) {
  return T >= 1 && Hk >= 1 && H >= 1 && H % Hk == 0 && H <= 65535 && D >= 1 && D <= 256 && E >= 1 && taps >= 1 && proj && conv_w && ring &&
         dt_bias && a_log && col0 >= 0 && ld >= col0 + 2 * Hk * D + 2 * H * E + 2 * H;
}

extern "C" int umb_delta_step(float* o, float* state, const float* proj, int ld, int col0, const void* conv_w, float* ring,
                              const float* dt_bias, const float* a_log, const int* pos, const int* slot, int T, int Hk, int H, int D,
                              int E, int taps, int dtype, hipStream_t st) {
  if (!delta_in_ok(proj, ld, col0, conv_w, ring, dt_bias, a_log, T, Hk, H, D, E, taps) || T > 65535 || !o || !state || !pos || !slot)
    return UMB_EINVAL;
  const DeltaIn in{proj, ld, col0, Hk, H, D, E, taps, ring, dt_bias, a_log};
  const size_t lds = (size_t)(2 * D + 32 + 8 + 256) * sizeof(float);
  const float qscale = 1.f / sqrtf((float)D);
  const dim3 grid((E + 31) / 32, H, T);
#define DELTA_STEP(RPT) \
  hipLaunchKernelGGL((delta_step_kernel<P, RPT>), grid, dim3(256), lds, st, o, state, in, (const El_*)conv_w, pos, slot, qscale)
  DISPATCH_SEQ_DTYPE(dtype, {
    typedef typename El<P>::type El_;
    if (D <= 32) DELTA_STEP(4);
    else if (D <= 64) DELTA_STEP(8);
    else if (D <= 128) DELTA_STEP(16);
    else DELTA_STEP(32);
  })
#undef DELTA_STEP
  UMB_LAUNCH_CHECK();
  return UMB_OK;
}

extern "C" int umb_delta_prep(float* q, float* k, int ldqk, float* v, float* beta, float* log_g, const float* proj, int ld, int col0,
                              const void* conv_w, float* ring, const float* dt_bias, const float* a_log, const int* pos,
                              const int* slot, int T, int Hk, int H, int D, int E, int taps, int dtype, hipStream_t st) {
  if (!delta_in_ok(proj, ld, col0, conv_w, ring, dt_bias, a_log, T, Hk, H, D, E, taps) || !q || !k || ldqk < Hk * up16(D) || !v || !beta ||
      !log_g || !pos || !slot)
    return UMB_EINVAL;
  const DeltaIn in{proj, ld, col0, Hk, H, D, E, taps, ring, dt_bias, a_log};
  const long items = (long)T * (2 * Hk + H + 1);
  DISPATCH_SEQ_DTYPE(dtype, {
    typedef typename El<P>::type El_;
    hipLaunchKernelGGL(delta_prep_kernel<P>, dim3((unsigned)((items + 3) / 4)), dim3(256), 0, st, q, k, ldqk, up16(D), v, beta, log_g, in,
                       (const El_*)conv_w, pos, slot, T, 1.f / sqrtf((float)D));
  })
  UMB_LAUNCH_CHECK();
  return UMB_OK;
}

extern "C" long umb_delta_scan_floats(int T, int H, int D, int E) {
  if (T < 1 || H < 1 || D < 1 || D > 256 || E < 1 || delta_solve_lds(up16(D)) > 160 * 1024) return 0;
  return (long)T * H * (up16(D) + up16(E) + 64 + 2) + 16;
}

extern "C" int umb_delta_scan(float* o, float* state, const float* q, const float* k, int ldqk, const float* v, const float* beta,
                              const float* log_g, const int* seq_slot, const int* seq_row0, const int* seq_pos0, const int* seq_len,
                              int T, int B, int max_len, int Hk, int H, int D, int E, float* scratch, long scratch_floats,
                              hipStream_t st) {
  const long need = umb_delta_scan_floats(T, H, D, E);
  if (need == 0 || need > scratch_floats || !scratch || B < 1 || B > 65535 || H > 65535 || max_len < 1 || max_len > T || Hk < 1 || H % Hk ||
      ldqk < Hk * up16(D) || ldqk % 4 || !o || !state || !q || !k || !v || !beta || !log_g || !seq_slot || !seq_row0 || !seq_pos0 ||
      !seq_len || ((uintptr_t)q | (uintptr_t)k | (uintptr_t)scratch) % 16)
    return UMB_EINVAL;
  const int Dp = up16(D), Ep = up16(E);
  const long n = (long)T * H;
  float* wk = scratch;
  float* m = wk + n * Dp;
  float* uv = m + n * 64;
  float* ec = uv + n * Ep;
  DeltaChunk a{q, k, v, beta, log_g, wk, uv, m, ec, ec + n, T, ldqk, Hk, H, D, Dp, E, Ep, seq_slot, seq_row0, seq_pos0, seq_len};
  const size_t lds1 = delta_solve_lds(Dp), lds2 = (size_t)2 * 4 * 8 * 256 * sizeof(float);
  if (ensure_dynamic_lds<delta_chunk_solve_kernel>(lds1) != UMB_OK) return UMB_EHIP;
  hipLaunchKernelGGL(delta_chunk_solve_kernel, dim3((max_len + DC_Q - 1) / DC_Q, H, B), dim3(256), lds1, st, a);
#define DELTA_SCAN(TPW, PRE)                                                                                              \
  do {                                                                                                                    \
    if (ensure_dynamic_lds<delta_chunk_scan_kernel<TPW, PRE>>(lds2) != UMB_OK) return UMB_EHIP;                           \
    hipLaunchKernelGGL((delta_chunk_scan_kernel<TPW, PRE>), dim3(Ep / 16, H, B), dim3(256), lds2, st, o, state, a);       \
  } while (0)
  if (Dp <= 64) DELTA_SCAN(1, true);
  else if (Dp <= 128) DELTA_SCAN(2, true);
  else DELTA_SCAN(4, false);
#undef DELTA_SCAN
  UMB_LAUNCH_CHECK();
  return UMB_OK;
}
