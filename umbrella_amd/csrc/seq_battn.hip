// Causal softmax attention with a learned bias by distance, grouped query heads, over the paged key/value store.
//     q_i = unit_rms(W_q h_i) * w_q * temp(i)       k_j = unit_rms(W_k h_j) * w_k       v_j = unit_rms(W_v h_j)
//     score(i, j, h) = q_i . k_j * scale + bias[h][min(i - j, n_dist - 1)]      (j <= i, i - j < window)
//     out_i = c * sigmoid(gate_i[h]) * softmax_j(score) . v
// With softcap > 0 the scaled product is capped before the bias joins it: softcap tanh(q . k scale / softcap).
// temp(i) = 1 + coef ln(floor((i + 1) / every) + 1) sharpens the queries of long contexts; the bias table is indexed by the
// clamped distance itself (whatever bucketing a design uses is expanded into it at load).  Keys and values are cached as
// normed (storage dtype); queries, scores, weights, maxima and sums are fp32 (expf, not the fast intrinsic).
//
// The general form (umb_attn_*, UmbAttnForm) adds, each by parameter:
//   chunk   position i sees only keys of its own run of `chunk` positions, counted from position 0 of the sequence
//   sink    a per-head score that joins the softmax denominator with no key and no value
//   maps    2: differential attention -- every head has two query / key maps over the SAME values (a cached key row is [map 1 |
//           map 2]); with a1, a2 their softmax outputs o = a1 - lambda a2, and the head's o over its root mean square goes out.
//           The two maps of a head are two rows of one workgroup: the value rows are read once for both.
//   keep_first   the first keep_first positions stay visible (at their true distance) whatever the window and the chunk hide:
//           the walk over the keys takes those of them that lie before its first position in front, as one range
//   gate_elem    the output gate is a row of H E columns, one sigmoid per output element, instead of one per head
// and its prep adds rotary positions (either pair layout, a constant on cos and sin), norms by choice, queries alone (a
// layer that reads another layer's keys and values), and values mixed with those of another layer (UmbValueMix): what is cached is
// (1 - lambda) v + lambda first, with `first` the same tokens' values as an earlier layer's prep left them.
//
// prep: one wave per (token, head slot): query heads -> fp32 q, key heads -> cache K, value heads -> cache V.
// attend (vector pipe, any dtype and head size): workgroup = (token, RH query heads of ONE key/value head, so one pass over
// the keys serves them all); waves take 64-key rounds by round number; score phase lane = key, value phase lane = value
// column with eight keys' rows in flight; per-wave running maximum / denominator, merged through LDS in wave order.  Which
// keys land in which wave and round depends on the query's position alone -- never on the batch or on how a prompt was cut.
#include "seq_common.h"

static inline bool bsa_kv_ok(const UmbPagedKV* kv) { return kv && kv->k && kv->v && kv->pages && kv->page >= 1 && kv->max_pages >= 1; }

// HQ = H maps query slots, GK = G maps key slots (key slot x: key/value head x / maps, map x % maps), G value slots (GV = 0: none)
struct AttnPrep {
  int HQ, GK, G, GV, D, E, maps;
  int norm_qk, norm_v;                     // unit RMS (times the weight, where there is one) of q and k; of v
  int rot_dims, layout;
  float rot_mult;
  float temp_coef;
  int temp_every;
  float eps;
  UmbValueMix mix;                         // first: values to mix in; keep: where this layer's own go (fp32 rows of G E); null: neither
};

template <typename P>
__global__ __launch_bounds__(256) void attn_prep_kernel(float* __restrict__ q, UmbPagedKV kv, const float* __restrict__ proj, int ld,
                                                        const typename El<P>::type* __restrict__ w_q,
                                                        const typename El<P>::type* __restrict__ w_k, const int* __restrict__ pos,
                                                        const int* __restrict__ slot, const float* __restrict__ freq, int T,
                                                        AttnPrep a) {
  typedef typename El<P>::type El_;
  const int wave = threadIdx.x >> 6, lane = threadIdx.x & 63;
  const int per = a.HQ + a.GK + a.GV;
  const long item = (long)blockIdx.x * 4 + wave;
  if (item >= (long)T * per) return;
  const int t = (int)(item / per), hs = (int)(item % per);
  const bool is_v = hs >= a.HQ + a.GK, is_q = hs < a.HQ;
  const int n = is_v ? a.E : a.D, D = a.D;
  const int col = is_v ? (a.HQ + a.GK) * D + (hs - a.HQ - a.GK) * a.E : hs * D;
  const float* src = proj + (long)t * ld + col;
  float f = 1.f;
  if (is_v ? a.norm_v : a.norm_qk) {
    float ss = 0.f;
    for (int i = lane; i < n; i += 64) { const float v = src[i]; ss += v * v; }
    ss = wave_sum(ss);
    f = 1.f / sqrtf(ss / (float)n + a.eps);
  }
  const int p = pos[t];
  if (is_v) {
    const int g = hs - a.HQ - a.GK;
    El_* row = reinterpret_cast<El_*>(kv.v) + pkv_tok(kv, slot[t], p, g, a.G, a.E);
    const long o = ((long)t * a.G + g) * a.E;
    for (int i = lane; i < n; i += 64) {
      float v = src[i] * f;
      if (a.mix.keep) a.mix.keep[o + i] = v;
      if (a.mix.first) v = (1.f - a.mix.lambda) * v + a.mix.lambda * a.mix.first[o + i];
      stf<P>(row + i, v);
    }
    return;
  }
  const El_* w = is_q ? w_q : w_k;
  const float temp = is_q && a.temp_every > 0 ? 1.f + a.temp_coef * logf((float)((p + 1) / a.temp_every + 1)) : 1.f;
  const int ks = hs - a.HQ;
  El_* krow = is_q ? nullptr : reinterpret_cast<El_*>(kv.k) + pkv_tok(kv, slot[t], p, ks / a.maps, a.G, a.maps * D) + (ks % a.maps) * D;
  float* qrow = q + ((long)t * a.HQ + (is_q ? hs : 0)) * D;
  const int half = a.rot_dims >> 1;
  for (int i = lane; i < n; i += 64) {
    float v = src[i] * f * (w ? ldf<P>(w + i) : 1.f);
    if (i < a.rot_dims) {
      int fi, other;
      bool first;
      if (a.layout == 0) { first = i < half; fi = first ? i : i - half; other = first ? i + half : i - half; }
      else { first = (i & 1) == 0; fi = i >> 1; other = i ^ 1; }
      const float u = src[other] * f * (w ? ldf<P>(w + other) : 1.f);
      float sn, cs;
      sincosf((float)p * freq[fi], &sn, &cs);
      sn *= a.rot_mult;
      cs *= a.rot_mult;
      v = first ? v * cs - u * sn : v * cs + u * sn;
    }
    if (is_q) qrow[i] = v * temp;
    else stf<P>(krow + i, v);
  }
}

constexpr int BSA_MAXC = 8;      // value columns per lane: E <= 512

// RH rows of the workgroup = RH / MAPS query heads with MAPS maps each (row r: head r / MAPS, map r % MAPS)
template <typename P, int RH, int NC, int NW, int MAPS>
__global__ __launch_bounds__(NW * 64) void bsa_attend_kernel(typename El<P>::type* __restrict__ out, int ldo,
                                                             const float* __restrict__ q, UmbPagedKV kv,
                                                             const float* __restrict__ proj, int ld, int gate_col,
                                                             const float* __restrict__ bias, int n_dist,
                                                             const int* __restrict__ pos, const int* __restrict__ slot_, int H,
                                                             int G, int D, int E, int window, float scale, float out_scale,
                                                             float softcap, UmbAttnForm form, float* __restrict__ part,
                                                             int nsplit) {
  static_assert(RH % MAPS == 0, "rows are whole heads");
  typedef typename El<P>::type El_;
  extern __shared__ float lds[];
  constexpr int KB = 8;
  const int split = blockIdx.z;                         // nsplit > 1: the workgroup takes every nsplit-th group of NW rounds
  const int wave = threadIdx.x >> 6, lane = threadIdx.x & 63;
  const int Dp = (D + 3) & ~3, Ep = (E + 3) & ~3, Mp = Dp > Ep ? Dp : Ep;
  // [RH][Dp] queries (later [NW][RH][Ep] partial sums), [NW][2 RH] maxima and denominators, per wave [RH][64] weights + offsets
  float* q_s = lds;
  float* ml_s = lds + NW * RH * Mp;
  float* w_s = ml_s + NW * 2 * RH + wave * (RH * 64 + 128);
  long* off_s = reinterpret_cast<long*>(w_s + RH * 64);
  const int t = blockIdx.x, hpg = H / G;
  constexpr int RR = RH / MAPS;
  const int h0 = blockIdx.y * RR, g = h0 / hpg;           // RR divides H / G: the block's heads share key/value head g
  const int i = pos[t], slot = slot_[t];
  for (int x = threadIdx.x; x < RH * D; x += NW * 64) {
    const int r = x / D, d = x % D;
    q_s[r * Dp + d] = q[(((long)t * H + h0) * MAPS + r) * D + d];
  }
  __syncthreads();
  int j_lo = i - window + 1 > 0 ? i - window + 1 : 0;
  if (form.chunk > 0) j_lo = max(j_lo, i / form.chunk * form.chunk);
  const int kept = min(form.keep_first, j_lo);          // first positions in front of the walk: keys 0 .. kept - 1, then j_lo .. i
  const int n_keys = kept + i - j_lo + 1;
  const bool vec = (D & 7) == 0 && sizeof(El_) == 2;
  float acc[RH][NC], m_run[RH], l_run[RH];
#pragma unroll
  for (int r = 0; r < RH; ++r) {
    m_run[r] = -INFINITY;
    l_run[r] = 0.f;
#pragma unroll
    for (int c = 0; c < NC; ++c) acc[r][c] = 0.f;
  }
  int dcl[NC];
#pragma unroll
  for (int c = 0; c < NC; ++c) dcl[c] = lane + 64 * c < E ? lane + 64 * c : E - 1;
  for (int base = (split * NW + wave) * 64; base < n_keys; base += nsplit * NW * 64) {
    const int kx = base + lane;
    float s[RH];
#pragma unroll
    for (int r = 0; r < RH; ++r) s[r] = 0.f;
    long off = 0;
    int dist = 0;
    if (kx < n_keys) {
      const int j = kx < kept ? kx : j_lo + kx - kept;
      dist = i - j;
      const El_* kr = reinterpret_cast<const El_*>(kv.k) + pkv_tok(kv, slot, j, g, G, MAPS * D);
      off = pkv_tok(kv, slot, j, g, G, E);
      bool done = false;
      if constexpr (sizeof(El_) == 2) {
        if (vec) {
#pragma unroll
          for (int mp = 0; mp < MAPS; ++mp)
          for (int d = 0; d < D; d += 64) {              // eight 16-byte loads in flight, then their 64 x RH products
            u32x4 kk[8];
#pragma unroll
            for (int u = 0; u < 8; ++u) kk[u] = *reinterpret_cast<const u32x4*>(kr + mp * D + (d + 8 * u < D ? d + 8 * u : 0));
#pragma unroll
            for (int u = 0; u < 8; ++u) {
              if (d + 8 * u >= D) break;
#pragma unroll
              for (int e = 0; e < 4; ++e) {
                const float k0 = lo_f<P>(kk[u][e]), k1 = hi_f<P>(kk[u][e]);
                const int dd = d + 8 * u + 2 * e;
#pragma unroll
                for (int r = mp; r < RH; r += MAPS) s[r] += q_s[r * Dp + dd] * k0 + q_s[r * Dp + dd + 1] * k1;
              }
            }
          }
          done = true;
        }
      }
      if (!done) {
#pragma unroll
        for (int mp = 0; mp < MAPS; ++mp)
          for (int d = 0; d < D; ++d) {
            const float kd = ldf<P>(kr + mp * D + d);
#pragma unroll
            for (int r = mp; r < RH; r += MAPS) s[r] += q_s[r * Dp + d] * kd;
          }
      }
    }
    const int bi = dist < n_dist ? dist : n_dist - 1;
#pragma unroll
    for (int r = 0; r < RH; ++r) {
      float sc = s[r] * scale;
      if (softcap > 0.f) sc = softcap * tanhf(sc / softcap);          // capped score; the bias (if any) is added to the capped value
      const float sv = kx < n_keys ? sc + (bias ? bias[(long)(h0 + r / MAPS) * n_dist + bi] : 0.f) : -INFINITY;
      const float m_new = fmaxf(m_run[r], wave_max(sv));          // finite: every round has at least one key
      const float fac = expf(m_run[r] - m_new);                   // 0 on the first round (m_run = -inf)
      const float pw = kx < n_keys ? expf(sv - m_new) : 0.f;
      l_run[r] = l_run[r] * fac + wave_sum(pw);
      m_run[r] = m_new;
#pragma unroll
      for (int c = 0; c < NC; ++c) acc[r][c] *= fac;
      w_s[r * 64 + lane] = pw;
    }
    off_s[lane] = off;
    __builtin_amdgcn_fence(__ATOMIC_SEQ_CST, "wavefront");
    __builtin_amdgcn_wave_barrier();
    const int cnt = n_keys - base < 64 ? n_keys - base : 64;
    for (int j0 = 0; j0 < cnt; j0 += KB) {
      float vv[KB][NC];
#pragma unroll
      for (int u = 0; u < KB; ++u) {
        const long oj = off_s[j0 + u < cnt ? j0 + u : cnt - 1];
#pragma unroll
        for (int c = 0; c < NC; ++c) vv[u][c] = ldf<P>(reinterpret_cast<const El_*>(kv.v) + oj + dcl[c]);
      }
#pragma unroll
      for (int u = 0; u < KB; ++u) {
#pragma unroll
        for (int r = 0; r < RH; ++r) {
          const float wj = j0 + u < cnt ? w_s[r * 64 + j0 + u] : 0.f;
#pragma unroll
          for (int c = 0; c < NC; ++c) acc[r][c] += wj * vv[u][c];
        }
      }
    }
    __builtin_amdgcn_fence(__ATOMIC_SEQ_CST, "wavefront");
    __builtin_amdgcn_wave_barrier();
  }
  __syncthreads();                                  // every wave is done with the queries: their LDS becomes the partials
#pragma unroll
  for (int r = 0; r < RH; ++r) {
#pragma unroll
    for (int c = 0; c < NC; ++c) {
      const int d = lane + 64 * c;
      if (d < E) lds[(wave * RH + r) * Ep + d] = acc[r][c];
    }
    if (lane == 0) { ml_s[(wave * RH + r) * 2] = m_run[r]; ml_s[(wave * RH + r) * 2 + 1] = l_run[r]; }
  }
  __syncthreads();
  // row r of the waves' partials merged in wave order: unnormalised output of column d, maximum and denominator
  auto merged = [&](int r, int d, float& M, float& L) -> float {
    M = -INFINITY;
#pragma unroll
    for (int w = 0; w < NW; ++w) M = fmaxf(M, ml_s[(w * RH + r) * 2]);
    float o = 0.f;
    L = 0.f;
#pragma unroll
    for (int w = 0; w < NW; ++w) {
      const float mw = ml_s[(w * RH + r) * 2];
      const float f = mw == -INFINITY ? 0.f : expf(mw - M);
      o += lds[(w * RH + r) * Ep + d] * f;
      L += ml_s[(w * RH + r) * 2 + 1] * f;
    }
    return o;
  };
  auto gate_of = [&](int h, int d) {
    return gate_col >= 0 ? 1.f / (1.f + expf(-proj[(long)t * ld + gate_col + (form.gate_elem ? h * E + d : h)])) : 1.f;
  };
  if (MAPS == 1 || nsplit > 1) {
    for (int x = threadIdx.x; x < RH * E; x += NW * 64) {
      const int r = x / E, d = x % E;
      float M, L;
      const float o = merged(r, d, M, L);
      if (nsplit > 1) {                                // partial result of this split: [t][row][split][E + 2] = o.., M, L
        float* pr = part + ((((long)t * H + h0) * MAPS + r) * nsplit + split) * (E + 2);
        pr[d] = o;
        if (d == 0) { pr[E] = M; pr[E + 1] = L; }
        continue;
      }
      if (form.sink) L += expf(form.sink[h0 + r] - M);
      stf<P>(out + (long)t * ldo + (long)(h0 + r) * E + d, out_scale * gate_of(h0 + r, d) * (o / L));
    }
  } else {
    // a wave per head: o = a1 - lambda a2 over its root mean square
    for (int rr = wave; rr < RR; rr += NW) {
      float v[NC], ss = 0.f;
#pragma unroll
      for (int c = 0; c < NC; ++c) {
        const int d = dcl[c];
        float M, L1, L2;
        float o = merged(MAPS * rr, d, M, L1);
        if (form.sink) L1 += expf(form.sink[h0 + rr] - M);
        const float a2 = merged(MAPS * rr + MAPS - 1, d, M, L2);
        if (form.sink) L2 += expf(form.sink[h0 + rr] - M);
        o = o / L1 - form.lambda * (a2 / L2);
        v[c] = o;
        if (lane + 64 * c < E) ss += o * o;
      }
      ss = wave_sum(ss);
      const float f = out_scale / sqrtf(ss / (float)E + form.eps);
#pragma unroll
      for (int c = 0; c < NC; ++c)
        if (lane + 64 * c < E) stf<P>(out + (long)t * ldo + (long)(h0 + rr) * E + dcl[c], v[c] * f * gate_of(h0 + rr, dcl[c]));
    }
  }
}

// the splits of one (token, head) merged: lane s holds split s's maximum and denominator (a split that had no key carries
// M = -inf, L = 0), the factors go round by shuffles, every sum runs over the splits in order
template <typename P, int MAPS>
__global__ __launch_bounds__(64) void bsa_merge_kernel(typename El<P>::type* __restrict__ out, int ldo, const float* __restrict__ part,
                                                       const float* __restrict__ proj, int ld, int gate_col, int H, int E,
                                                       int nsplit, float out_scale, UmbAttnForm form) {
  const int t = blockIdx.x, h = blockIdx.y, lane = threadIdx.x;
  auto gate_of = [&](int d) {
    return gate_col >= 0 ? 1.f / (1.f + expf(-proj[(long)t * ld + gate_col + (form.gate_elem ? h * E + d : h)])) : 1.f;
  };
  const float* pr[MAPS];
  float f[MAPS][16], inv[MAPS];
#pragma unroll
  for (int mp = 0; mp < MAPS; ++mp) {
    pr[mp] = part + (((long)t * H + h) * MAPS + mp) * nsplit * (E + 2);
    const float ms = lane < nsplit ? pr[mp][lane * (E + 2) + E] : -INFINITY;
    const float ls = lane < nsplit ? pr[mp][lane * (E + 2) + E + 1] : 0.f;
    const float M = wave_max(ms);
    const float fs = ms == -INFINITY ? 0.f : expf(ms - M);
    float L = 0.f;
#pragma unroll
    for (int s = 0; s < 16; ++s) {
      f[mp][s] = __shfl(fs, s, 64);
      L += __shfl(ls * fs, s, 64);
    }
    if (form.sink) L += expf(form.sink[h] - M);
    inv[mp] = 1.f / L;
  }
  auto column = [&](int mp, int d) -> float {
    float v[16];
#pragma unroll
    for (int s = 0; s < 16; ++s) v[s] = pr[mp][(s < nsplit ? s : nsplit - 1) * (E + 2) + d];
    float o = 0.f;
#pragma unroll
    for (int s = 0; s < 16; ++s) o += s < nsplit ? v[s] * f[mp][s] : 0.f;
    return o * inv[mp];
  };
  typename El<P>::type* orow = out + (long)t * ldo + (long)h * E;
  if constexpr (MAPS == 1) {
    for (int d = lane; d < E; d += 64) stf<P>(orow + d, column(0, d) * (out_scale * gate_of(d)));
  } else {
    float v[BSA_MAXC], ss = 0.f;
#pragma unroll
    for (int c = 0; c < BSA_MAXC; ++c) {
      const int d = lane + 64 * c;
      if (64 * c < E) {                                  // uniform
        const float o = d < E ? column(0, d) - form.lambda * column(1, d) : 0.f;
        v[c] = o;
        ss += o * o;
      }
    }
    ss = wave_sum(ss);
    const float c0 = out_scale / sqrtf(ss / (float)E + form.eps);
#pragma unroll
    for (int c = 0; c < BSA_MAXC; ++c)
      if (lane + 64 * c < E) stf<P>(orow + lane + 64 * c, v[c] * (c0 * gate_of(lane + 64 * c)));
  }
}

static inline bool form_ok(const UmbAttnForm* f) { return !f || ((f->maps == 1 || f->maps == 2) && f->chunk >= 0 && f->keep_first >= 0); }
static inline int form_gate_cols(const UmbAttnForm& f, int H, int E) { return f.gate_elem ? H * E : H; }

extern "C" int umb_attn_prep_mix(float* q, const UmbPagedKV* kv, const float* proj, int ld, int append, const void* w_q, const void* w_k,
                                 int norm_qk, int norm_v, const int* pos, const int* slot, const float* freq, int rot_dims, int layout,
                                 float rot_mult, int T, int H, int G, int D, int E, int maps, float temp_coef, int temp_every, float eps,
                                 const UmbValueMix* mix, int dtype, hipStream_t st) {
  if (T < 1 || H < 1 || G < 1 || H % G || D < 1 || E < 1 || maps < 1 || maps > 2 || rot_dims < 0 || rot_dims > D || (rot_dims & 1) ||
      (rot_dims && !freq) || layout < 0 || layout > 1 || !q || (append && !bsa_kv_ok(kv)) || !proj || !pos || !slot ||
      ld < maps * H * D + (append ? maps * G * D + G * E : 0))
    return UMB_EINVAL;
  AttnPrep a{maps * H, append ? maps * G : 0, G, append ? G : 0, D, E, maps, norm_qk, norm_v, rot_dims, layout, rot_mult,
             temp_coef, temp_every, eps, mix ? *mix : UmbValueMix{nullptr, nullptr, 0.f, 0.f}};
  const UmbPagedKV none{};
  const long items = (long)T * (a.HQ + a.GK + a.GV);
  DISPATCH_SEQ_DTYPE(dtype, {
    typedef typename El<P>::type El_;
    hipLaunchKernelGGL(attn_prep_kernel<P>, dim3((unsigned)((items + 3) / 4)), dim3(256), 0, st, q, append ? *kv : none, proj, ld,
                       (const El_*)w_q, (const El_*)w_k, pos, slot, freq, T, a);
  })
  UMB_LAUNCH_CHECK();
  return UMB_OK;
}

extern "C" int umb_attn_prep(float* q, const UmbPagedKV* kv, const float* proj, int ld, int append, const void* w_q, const void* w_k,
                             int norm_qk, int norm_v, const int* pos, const int* slot, const float* freq, int rot_dims, int layout,
                             float rot_mult, int T, int H, int G, int D, int E, int maps, float temp_coef, int temp_every, float eps,
                             int dtype, hipStream_t st) {
  return umb_attn_prep_mix(q, kv, proj, ld, append, w_q, w_k, norm_qk, norm_v, pos, slot, freq, rot_dims, layout, rot_mult, T, H, G, D, E,
                           maps, temp_coef, temp_every, eps, nullptr, dtype, st);
}

extern "C" int umb_bsa_prep(float* q, const UmbPagedKV* kv, const float* proj, int ld, const void* w_q, const void* w_k,
                            const int* pos, const int* slot, int T, int H, int G, int D, int E, float temp_coef, int temp_every,
                            float eps, int dtype, hipStream_t st) {
  return umb_attn_prep(q, kv, proj, ld, 1, w_q, w_k, 1, 1, pos, slot, nullptr, 0, 0, 1.f, T, H, G, D, E, 1, temp_coef, temp_every, eps,
                       dtype, st);
}

template <typename P, int RH, int NC, int NW, int MAPS>
static int bsa_launch(dim3 grid, size_t lds, hipStream_t st, void* out, int ldo, const float* q, const UmbPagedKV& kv,
                      const float* proj, int ld, int gate_col, const float* bias, int n_dist, const int* pos, const int* slot, int H,
                      int G, int D, int E, int window, float scale, float out_scale, float softcap, const UmbAttnForm& form,
                      float* scratch, int nsplit) {
  typedef typename El<P>::type El_;
  if (ensure_dynamic_lds<bsa_attend_kernel<P, RH, NC, NW, MAPS>>(lds) != UMB_OK) return UMB_EHIP;
  hipLaunchKernelGGL((bsa_attend_kernel<P, RH, NC, NW, MAPS>), grid, dim3(NW * 64), lds, st, (El_*)out, ldo, q, kv, proj, ld, gate_col,
                     bias, n_dist, pos, slot, H, G, D, E, window, scale, out_scale, softcap, form, scratch, nsplit);
  return UMB_OK;
}

extern "C" int umb_attn_attend(void* out, int ldo, const float* q, const UmbPagedKV* kv, const float* proj, int ld, int gate_col,
                               const float* bias, int n_dist, const int* pos, const int* slot, int T, int H, int G, int D, int E,
                               int window, float scale, float out_scale, float softcap, const UmbAttnForm* form_, float* scratch,
                               long scratch_floats, int dtype, hipStream_t st) {
  if (T < 1 || H < 1 || G < 1 || H % G || D < 1 || E < 1 || E > 64 * BSA_MAXC || window < 1 || !out || !q || !bsa_kv_ok(kv) ||
      !pos || !slot || ldo < H * E || (bias && n_dist < 1) || !form_ok(form_))
    return UMB_EINVAL;
  const UmbAttnForm form = form_ ? *form_ : UmbAttnForm{1, 0, nullptr, 0.f, 0.f, 0, 0};
  if (gate_col >= 0 && (!proj || ld < gate_col + form_gate_cols(form, H, E))) return UMB_EINVAL;
  const int maps = form.maps;
  const int hpg = H / G, nc = (E + 63) / 64;
  const int Dp = (D + 3) & ~3, Ep = (E + 3) & ~3, Mp = Dp > Ep ? Dp : Ep;
  // rows (head, map) of one workgroup: query heads of one key/value head, as many as divide the group and fit the register budget
  int rh = nc <= 2 ? 8 : (nc <= 4 ? 4 : 2);
  while (rh > maps && hpg % (rh / maps)) rh >>= 1;
  // A handful of (token, head block) items leaves most of the chip idle while each walks all its keys: with scratch for the
  // partial results the keys of an item are dealt to several workgroups (whole groups of four 64-key rounds by number, so the
  // order of every sum is a function of the position and of the step's row count only) and merged by a second launch.
  const int hblocks = H * maps / rh;
  const long items = (long)T * hblocks;
  int nsplit = 1;
  if (scratch && items <= 64) {                          // fewer than ~2048 waves in all with sixteen waves per item
    nsplit = (int)(512 / items) < 16 ? (int)(512 / items) : 16;
    // keys of one chunk or window only: no more workgroups than there can be groups of four rounds
    const long most = (long)(form.chunk > 0 && form.chunk < window ? form.chunk : window) + form.keep_first;
    if (nsplit > (most + 255) / 256) nsplit = (int)((most + 255) / 256);
    while (nsplit > 1 && (long)T * H * maps * nsplit * (E + 2) > scratch_floats) nsplit >>= 1;
  }
  const dim3 grid(T, hblocks, nsplit);
  int nw = (nsplit > 1 || items >= 1024) ? 4 : 16;
  auto lds_of = [&](int w) { return ((size_t)w * rh * Mp + (size_t)w * 2 * rh + (size_t)w * (rh * 64 + 128)) * sizeof(float); };
  if (nw == 16 && lds_of(16) > 128 * 1024) nw = 4;
  if (lds_of(nw) > 160 * 1024) return UMB_EINVAL;
  const size_t lds = lds_of(nw);
#define BSA_GO(RH, NC, NW, MAPS)                                                                                             \
  SEQ_TRY_((bsa_launch<P, RH, NC, NW, MAPS>(grid, lds, st, out, ldo, q, *kv, proj, ld, gate_col, bias, n_dist, pos, slot, H, G, D,   \
                                           E, window, scale, out_scale, softcap, form, scratch, nsplit)))
#define SEQ_TRY_(call) do { const int rc__ = (call); if (rc__ != UMB_OK) return rc__; } while (0)
#define BSA_NW(RH, NC, MAPS)                                                                                                 \
  do { if (nw == 16) BSA_GO(RH, NC, 16, MAPS); else BSA_GO(RH, NC, 4, MAPS); } while (0)
#define BSA_RH(NC)                                                                                                           \
  do {                                                                                                                       \
    if (maps == 2) { if (rh == 8) BSA_NW(8, NC, 2); else if (rh == 4) BSA_NW(4, NC, 2); else BSA_NW(2, NC, 2); }              \
    else if (rh == 8) BSA_NW(8, NC, 1); else if (rh == 4) BSA_NW(4, NC, 1); else if (rh == 2) BSA_NW(2, NC, 1);               \
    else BSA_NW(1, NC, 1);                                                                                                   \
  } while (0)
  DISPATCH_SEQ_DTYPE(dtype, {
    typedef typename El<P>::type El_;
    if (nc <= 1) BSA_RH(1);
    else if (nc <= 2) BSA_RH(2);
    else if (nc <= 4) {
      if (maps == 2) { if (rh == 4) BSA_NW(4, 4, 2); else BSA_NW(2, 4, 2); }
      else if (rh == 4) BSA_NW(4, 4, 1); else if (rh == 2) BSA_NW(2, 4, 1); else BSA_NW(1, 4, 1);
    } else {
      if (maps == 2) BSA_NW(2, 8, 2); else if (rh == 2) BSA_NW(2, 8, 1); else BSA_NW(1, 8, 1);
    }
    if (nsplit > 1) {
      if (maps == 2)
        hipLaunchKernelGGL((bsa_merge_kernel<P, 2>), dim3(T, H), dim3(64), 0, st, (El_*)out, ldo, scratch, proj, ld, gate_col, H, E,
                           nsplit, out_scale, form);
      else
        hipLaunchKernelGGL((bsa_merge_kernel<P, 1>), dim3(T, H), dim3(64), 0, st, (El_*)out, ldo, scratch, proj, ld, gate_col, H, E,
                           nsplit, out_scale, form);
    }
  })
#undef BSA_RH
#undef BSA_NW
#undef BSA_GO
#undef SEQ_TRY_
  UMB_LAUNCH_CHECK();
  return UMB_OK;
}

extern "C" int umb_bsa_attend(void* out, int ldo, const float* q, const UmbPagedKV* kv, const float* proj, int ld, int gate_col,
                              const float* bias, int n_dist, const int* pos, const int* slot, int T, int H, int G, int D, int E,
                              int window, float scale, float out_scale, float softcap, float* scratch, long scratch_floats,
                              int dtype, hipStream_t st) {
  return umb_attn_attend(out, ldo, q, kv, proj, ld, gate_col, bias, n_dist, pos, slot, T, H, G, D, E, window, scale, out_scale,
                         softcap, nullptr, scratch, scratch_floats, dtype, st);
}

// ---- prompt attention on the matrix pipe (16-bit storage; D a multiple of 8, E a multiple of 16).
// Workgroup = (16 consecutive positions of one sequence, one key/value head, a block of 4 HPW of its query heads); wave w owns
// HPW heads.  The tile's keys -- from the first position's window start to the last position -- are walked in steps of 32 by
// the whole workgroup: the step's 32 cached key rows and value rows are staged ONCE into LDS (keys as cached: the A operand of
// S^T = K Q^T; values transposed: the A operand of O^T += V^T P^T) and serve every head of the workgroup; the next step's rows
// are in flight in registers while the current one is used.  Per step and head: two 16-key score tiles; the bias of the
// lane's eight (query, key) pairs, fetched by distance before the products are issued; online softmax in fp32 with base-2
// exponents, accumulators rescaled only when a maximum moved; the lane's eight weights ARE its share of the B operand of the
// value product.  Scores and weights keep fp32 accuracy on the 16-bit pipe: the fp32 queries and the fp32 weights enter as
// high + low 16-bit halves (two products each, 2^-17 relative).
constexpr float BSA_LOG2E = 1.4426950408889634f;

template <typename P> __device__ __forceinline__ void split2(float a, float b, unsigned& hi, unsigned& lo) {
  const u16 ah = P::from_f(a), bh = P::from_f(b);
  hi = (unsigned)ah | ((unsigned)bh << 16);
  lo = pack2<P>(a - P::to_f(ah), b - P::to_f(bh));
}

// HPW rows per wave = HPW / MAPS heads with MAPS maps each; every map has its part of the staged key rows, the value fragments of
// a step serve all rows
template <typename P, int NSM, int NVM, int HPW, int MAPS>
__global__ __launch_bounds__(256) void bsa_attend_mfma_kernel(u16* __restrict__ out, int ldo, const float* __restrict__ q,
                                                              UmbPagedKV kv, const float* __restrict__ proj, int ld, int gate_col,
                                                              const float* __restrict__ bias, int n_dist,
                                                              const int* __restrict__ seq_slot, const int* __restrict__ seq_row0,
                                                              const int* __restrict__ seq_pos0, const int* __restrict__ seq_len,
                                                              int H, int G, int D, int E, int window, float scale, float out_scale,
                                                              float softcap, UmbAttnForm form) {
  extern __shared__ __attribute__((aligned(16))) u16 bsa_lds[];
  static_assert(HPW % MAPS == 0, "a wave owns whole heads");
  constexpr int HW = HPW / MAPS;                      // heads per wave
  constexpr int NLK = (NSM * 4 * MAPS + 7) / 8, NLV = (NVM * 2 + 7) / 8;     // 16-byte chunks of a key / value row per staging thread
  const int wave = threadIdx.x >> 6, lane = threadIdx.x & 63, j = lane & 15, g4 = lane >> 4;
  const int DK = MAPS * D, LD = DK + 8;               // LDS row stride of the key tile: 16 bytes of padding spread the banks
  const int ns = (D + 31) >> 5, nv = E >> 4, nck = DK >> 3, ncv = E >> 3;
  constexpr int LT = 36;                              // row stride of the transposed value tile: 32 keys + 8 bytes of padding
  u16* k_s = bsa_lds;                                 // [32][LD]
  u16* v_t = bsa_lds + 32 * LD;                       // [E][LT]
  const int b = blockIdx.y;
  // How many keys a tile sees depends on its place in the chunk (or, without a window, in the sequence).  Workgroups that share a CU
  // are about 256 apart in launch order, which is the same tile of another head block: every other run of 256 takes the tiles from the
  // far end, so a CU's workgroups add up to about the same work.
  const int row = b + (int)gridDim.y * (int)blockIdx.z, run = gridDim.x < 256 ? 256 / gridDim.x : 1;
  const int tile = (row / run) & 1 ? (int)(gridDim.x - 1 - blockIdx.x) : (int)blockIdx.x;
  const int n = seq_len[b], q0 = tile * 16;
  if (q0 >= n) return;                                // the whole workgroup
  const int hpg = H / G, hblocks = (hpg + 4 * HW - 1) / (4 * HW);
  const int g = blockIdx.z / hblocks;
  const int hl0 = ((blockIdx.z % hblocks) * 4 + wave) * HW;         // first of the wave's heads inside the group
  const bool active = hl0 < hpg;                      // a wave without heads still stages rows and meets the barriers
  const int slot = seq_slot[b], row0 = seq_row0[b], pos0 = seq_pos0[b];
  const int nq = n - q0 < 16 ? n - q0 : 16;
  const int i_first = pos0 + q0, i_last = i_first + nq - 1;
  const bool q_ok = j < nq;
  const int i_j = i_first + (q_ok ? j : nq - 1);
  const long qrow = row0 + q0 + (q_ok ? j : nq - 1);
  int j_lo = i_first - window + 1 > 0 ? i_first - window + 1 : 0;
  int c_lo = 0;                                       // first position of the query's own chunk
  if (form.chunk > 0) {
    j_lo = max(j_lo, i_first / form.chunk * form.chunk);
    c_lo = i_j / form.chunk * form.chunk;
  }
  const int kept = min(form.keep_first, j_lo);        // first positions in front of the walk: step rows 0 .. kept - 1, then j_lo .. i_last
  const int j_off = j_lo - kept;
  const int total = kept + i_last - j_lo + 1;
  const float scale2 = scale * BSA_LOG2E;
  const u16* kbase = reinterpret_cast<const u16*>(kv.k);
  const u16* vbase = reinterpret_cast<const u16*>(kv.v);
  u32x4 qh[HPW][NSM], ql[HPW][NSM];
  f32x4 o[HPW][NVM];
  float m_run[HPW], l_run[HPW];
  bool h_ok[HPW];
  int hd[HPW];
#pragma unroll
  for (int hh = 0; hh < HPW; ++hh) {
    h_ok[hh] = hl0 + hh / MAPS < hpg;
    hd[hh] = g * hpg + (h_ok[hh] ? hl0 + hh / MAPS : hpg - 1);
    const float* qr = q + ((qrow * H + hd[hh]) * MAPS + hh % MAPS) * D;
#pragma unroll
    for (int s = 0; s < NSM; ++s) {
      const int d = 32 * s + 8 * g4;
      qh[hh][s] = u32x4{0u, 0u, 0u, 0u};
      ql[hh][s] = u32x4{0u, 0u, 0u, 0u};
      if (s < ns && d < D) {
        const f32x4 a = *reinterpret_cast<const f32x4*>(qr + d), c = *reinterpret_cast<const f32x4*>(qr + d + 4);
        unsigned hi[4], lo[4];
        split2<P>(a[0], a[1], hi[0], lo[0]);
        split2<P>(a[2], a[3], hi[1], lo[1]);
        split2<P>(c[0], c[1], hi[2], lo[2]);
        split2<P>(c[2], c[3], hi[3], lo[3]);
        qh[hh][s] = u32x4{hi[0], hi[1], hi[2], hi[3]};
        ql[hh][s] = u32x4{lo[0], lo[1], lo[2], lo[3]};
      }
    }
#pragma unroll
    for (int dt = 0; dt < NVM; ++dt) o[hh][dt] = f32x4{0.f, 0.f, 0.f, 0.f};
    m_run[hh] = -INFINITY;
    l_run[hh] = 0.f;
  }
  // staging role of a thread: key row sm of the step, 16-byte chunks sc, sc + 8, ... of that row (keys and values)
  const int sm = threadIdx.x & 31, sc = threadIdx.x >> 5;
  u32x4 stk[NLK], stv[NLV];
  auto fetch = [&](int base) {
    const int kx = base + sm;
    const bool ok = kx < total;
    const int jk = kx < kept ? kx : j_off + kx;
    const long offk = ok ? pkv_tok(kv, slot, jk, g, G, DK) : 0;
    const long offv = ok ? pkv_tok(kv, slot, jk, g, G, E) : 0;
#pragma unroll
    for (int u = 0; u < NLK; ++u) {
      const int ch = sc + 8 * u;
      stk[u] = (ok && ch < nck) ? *reinterpret_cast<const u32x4*>(kbase + offk + 8 * ch) : u32x4{0u, 0u, 0u, 0u};
    }
#pragma unroll
    for (int u = 0; u < NLV; ++u) {
      const int ch = sc + 8 * u;
      stv[u] = (ok && ch < ncv) ? *reinterpret_cast<const u32x4*>(vbase + offv + 8 * ch) : u32x4{0u, 0u, 0u, 0u};
    }
  };
  fetch(0);
  for (int base = 0; base < total; base += 32) {
    __syncthreads();                                  // every wave is done with the previous tile
#pragma unroll
    for (int u = 0; u < NLK; ++u) {
      const int ch = sc + 8 * u;
      if (ch < nck) *reinterpret_cast<u32x4*>(k_s + sm * LD + 8 * ch) = stk[u];
    }
#pragma unroll
    for (int u = 0; u < NLV; ++u) {
      const int ch = sc + 8 * u;
      if (ch < ncv) {
#pragma unroll
        for (int e = 0; e < 4; ++e) {
          v_t[(8 * ch + 2 * e) * LT + sm] = (u16)(stv[u][e] & 0xffffu);
          v_t[(8 * ch + 2 * e + 1) * LT + sm] = (u16)(stv[u][e] >> 16);
        }
      }
    }
    __syncthreads();
    if (base + 32 < total) fetch(base + 32);          // in flight while this step is used
    if (!active) continue;
    // which of the lane's eight keys this query sees, and at what distance: the same for every head
    bool vis[8];
    int di[8];
#pragma unroll
    for (int e = 0; e < 8; ++e) {
      const int kx = base + 16 * (e >> 2) + 4 * g4 + (e & 3);
      const int jt = kx < kept ? kx : j_off + kx;
      vis[e] = q_ok && jt <= i_j && ((jt > i_j - window && jt >= c_lo) || jt < form.keep_first);
      const int dd = i_j - jt;
      di[e] = dd < 0 ? 0 : (dd < n_dist ? dd : n_dist - 1);
    }
    float bv[HPW][8];
#pragma unroll
    for (int hh = 0; hh < HPW; ++hh)
#pragma unroll
      for (int e = 0; e < 8; ++e) bv[hh][e] = bias ? bias[(long)hd[hh] * n_dist + di[e]] : 0.f;
    f32x4 sc2[HPW][2];
#pragma unroll
    for (int u = 0; u < 2; ++u) {
#pragma unroll
      for (int hh = 0; hh < HPW; ++hh) sc2[hh][u] = f32x4{0.f, 0.f, 0.f, 0.f};
      const u16* kr = k_s + (16 * u + j) * LD;
#pragma unroll
      for (int s = 0; s < NSM; ++s) {
        const int d = 32 * s + 8 * g4;
        if (s < ns) {
#pragma unroll
          for (int mp = 0; mp < MAPS; ++mp) {
            const u32x4 kf = d < D ? *reinterpret_cast<const u32x4*>(kr + mp * D + d) : u32x4{0u, 0u, 0u, 0u};
#pragma unroll
            for (int hh = mp; hh < HPW; hh += MAPS) {
              sc2[hh][u] = P::mfma(kf, ql[hh][s], sc2[hh][u]);
              sc2[hh][u] = P::mfma(kf, qh[hh][s], sc2[hh][u]);
            }
          }
        }
      }
    }
    u32x4 ph[HPW], pl[HPW];
#pragma unroll
    for (int hh = 0; hh < HPW; ++hh) {
      // maxima and exponents in base 2 (scale2 = scale log2 e): one v_exp_f32 per weight
      float sv[8], mx = -INFINITY;
#pragma unroll
      for (int e = 0; e < 8; ++e) {
        float raw = sc2[hh][e >> 2][e & 3] * scale2;
        if (softcap > 0.f) raw = softcap * tanhf(sc2[hh][e >> 2][e & 3] * scale / softcap) * BSA_LOG2E;      // capped, then to base 2
        sv[e] = vis[e] ? raw + bv[hh][e] * BSA_LOG2E : -INFINITY;
        mx = fmaxf(mx, sv[e]);
      }
      mx = fmaxf(mx, __shfl_xor(mx, 16, 64));
      mx = fmaxf(mx, __shfl_xor(mx, 32, 64));
      const float m_new = fmaxf(m_run[hh], mx);
      const float m_ref = m_new == -INFINITY ? 0.f : m_new;          // a row that has seen no key yet: all weights 0
      const float fac = __builtin_amdgcn_exp2f(m_run[hh] - m_ref);
      float w[8], sum = 0.f;
#pragma unroll
      for (int e = 0; e < 8; ++e) {
        w[e] = __builtin_amdgcn_exp2f(sv[e] - m_ref);
        sum += w[e];
      }
      sum += __shfl_xor(sum, 16, 64);
      sum += __shfl_xor(sum, 32, 64);
      l_run[hh] = l_run[hh] * fac + sum;
      m_run[hh] = m_new;
      if (__ballot(fac != 1.f)) {                                    // the maximum moved for some row of the tile
#pragma unroll
        for (int dt = 0; dt < NVM; ++dt) {
          if (dt < nv) { o[hh][dt][0] *= fac; o[hh][dt][1] *= fac; o[hh][dt][2] *= fac; o[hh][dt][3] *= fac; }
        }
      }
      unsigned hi[4], lo[4];
#pragma unroll
      for (int e = 0; e < 4; ++e) split2<P>(w[2 * e], w[2 * e + 1], hi[e], lo[e]);
      ph[hh] = u32x4{hi[0], hi[1], hi[2], hi[3]};
      pl[hh] = u32x4{lo[0], lo[1], lo[2], lo[3]};
    }
    // O^T[d][query] += V^T[d][keys] P^T[keys][query]: lane (d row j of tile dt, quad g4) reads its 8 keys' values
#pragma unroll
    for (int dt = 0; dt < NVM; ++dt) {
      if (dt < nv) {
        const u16* vr = v_t + (16 * dt + j) * LT + 4 * g4;
        const u32x2 t0 = *reinterpret_cast<const u32x2*>(vr), t1 = *reinterpret_cast<const u32x2*>(vr + 16);
        const u32x4 va = u32x4{t0[0], t0[1], t1[0], t1[1]};
#pragma unroll
        for (int hh = 0; hh < HPW; ++hh) {
          o[hh][dt] = P::mfma(va, pl[hh], o[hh][dt]);
          o[hh][dt] = P::mfma(va, ph[hh], o[hh][dt]);
        }
      }
    }
  }
  // lane holds O^T[d = 16 dt + 4 g4 + rr][query j]
  if (q_ok && active) {
#pragma unroll
    for (int hh = 0; hh < HPW; hh += MAPS) {
      if (!h_ok[hh]) continue;
      const bool gate_head = gate_col >= 0 && !form.gate_elem;
      const float gt = gate_head ? 1.f / (1.f + expf(-proj[qrow * ld + gate_col + hd[hh]])) : 1.f;
      const float* ge = gate_col >= 0 && form.gate_elem ? proj + qrow * ld + gate_col + (long)hd[hh] * E : nullptr;
      float l[MAPS];
#pragma unroll
      for (int mp = 0; mp < MAPS; ++mp)
        l[mp] = l_run[hh + mp] + (form.sink ? __builtin_amdgcn_exp2f(form.sink[hd[hh]] * BSA_LOG2E - m_run[hh + mp]) : 0.f);
      float inv = out_scale * gt / l[0];
      if constexpr (MAPS == 2) {                      // o = a1 - lambda a2 over the root mean square of the head's E columns
        const float i1 = 1.f / l[0], i2 = form.lambda / l[1];
        float ss = 0.f;
#pragma unroll
        for (int dt = 0; dt < NVM; ++dt) {
          if (dt < nv) {
#pragma unroll
            for (int rr = 0; rr < 4; ++rr) {
              const float v = o[hh][dt][rr] * i1 - o[hh + 1][dt][rr] * i2;
              o[hh][dt][rr] = v;
              ss += v * v;
            }
          }
        }
        ss += __shfl_xor(ss, 16, 64);                 // the query's column quads: lanes j, j + 16, j + 32, j + 48 (all active)
        ss += __shfl_xor(ss, 32, 64);
        inv = out_scale * gt / sqrtf(ss / (float)E + form.eps);
      }
      u16* orow = out + qrow * ldo + (long)hd[hh] * E;
#pragma unroll
      for (int dt = 0; dt < NVM; ++dt) {
        if (dt < nv) {
#pragma unroll
          for (int rr = 0; rr < 4; ++rr) {
            const int d = 16 * dt + 4 * g4 + rr;
            float v = o[hh][dt][rr] * inv;
            if (ge) v /= 1.f + expf(-ge[d]);
            orow[d] = P::from_f(v);
          }
        }
      }
    }
  }
}

extern "C" int umb_bsa_attend_tiled_ok(int H, int G, int D, int E, int dtype) {
  return H >= 1 && G >= 1 && H % G == 0 && (dtype == UMB_SEQ_BF16 || dtype == UMB_SEQ_F16) && D >= 8 && D % 8 == 0 && D <= 256 &&
         E >= 16 && E % 16 == 0 && E <= 256;
}

extern "C" int umb_attn_attend_tiled(void* out, int ldo, const float* q, const UmbPagedKV* kv, const float* proj, int ld,
                                     int gate_col, const float* bias, int n_dist, const int* seq_slot, const int* seq_row0,
                                     const int* seq_pos0, const int* seq_len, int B, int max_len, int H, int G, int D, int E,
                                     int window, float scale, float out_scale, float softcap, const UmbAttnForm* form_, int dtype,
                                     hipStream_t st) {
  if (B < 1 || B > 65535 || max_len < 1 || window < 1 || !out || !q || !bsa_kv_ok(kv) || !seq_slot || !seq_row0 || !seq_pos0 ||
      !seq_len || ldo < H * E || (bias && n_dist < 1) || !umb_bsa_attend_tiled_ok(H, G, D, E, dtype) || !form_ok(form_))
    return UMB_EINVAL;
  if (!bias) n_dist = 1;
  const UmbAttnForm form = form_ ? *form_ : UmbAttnForm{1, 0, nullptr, 0.f, 0.f, 0, 0};
  if (gate_col >= 0 && (!proj || ld < gate_col + form_gate_cols(form, H, E))) return UMB_EINVAL;
  const int hpg = H / G, maps = form.maps;
  const size_t lds = ((size_t)32 * (maps * D + 8) + (size_t)E * 36) * sizeof(u16);
#define BSA_MFMA(NSM, NVM, HPW, MAPS)                                                                                      \
  do {                                                                                                                     \
    const int hblocks = (hpg + 4 * (HPW / MAPS) - 1) / (4 * (HPW / MAPS));                                                 \
    if ((long)G * hblocks > 65535) return UMB_EINVAL;                                                                      \
    const dim3 grid((max_len + 15) / 16, B, G * hblocks);                                                                  \
    if (ensure_dynamic_lds<bsa_attend_mfma_kernel<P, NSM, NVM, HPW, MAPS>>(lds) != UMB_OK) return UMB_EHIP;                \
    hipLaunchKernelGGL((bsa_attend_mfma_kernel<P, NSM, NVM, HPW, MAPS>), grid, dim3(256), lds, st, (u16*)out, ldo, q, *kv, \
                       proj, ld, gate_col, bias, n_dist, seq_slot, seq_row0, seq_pos0, seq_len, H, G, D, E, window, scale, \
                       out_scale, softcap, form);                                                                          \
  } while (0)
#define BSA_MFMA_SHAPE()                                                                                                   \
  if (maps == 2) { if (D <= 128 && E <= 128) BSA_MFMA(4, 8, 2, 2); else BSA_MFMA(8, 16, 2, 2); }                           \
  else if (D <= 64 && E <= 64) { if (hpg > 4) BSA_MFMA(2, 4, 2, 1); else BSA_MFMA(2, 4, 1, 1); }                           \
  else if (D <= 128 && E <= 128) { if (hpg > 4) BSA_MFMA(4, 8, 2, 1); else BSA_MFMA(4, 8, 1, 1); }                         \
  else BSA_MFMA(8, 16, 1, 1)
  if (dtype == UMB_SEQ_BF16) { using P = BF16; BSA_MFMA_SHAPE(); }
  else { using P = F16; BSA_MFMA_SHAPE(); }
#undef BSA_MFMA_SHAPE
#undef BSA_MFMA
  UMB_LAUNCH_CHECK();
  return UMB_OK;
}

extern "C" int umb_bsa_attend_tiled(void* out, int ldo, const float* q, const UmbPagedKV* kv, const float* proj, int ld,
                                    int gate_col, const float* bias, int n_dist, const int* seq_slot, const int* seq_row0,
                                    const int* seq_pos0, const int* seq_len, int B, int max_len, int H, int G, int D, int E,
                                    int window, float scale, float out_scale, float softcap, int dtype, hipStream_t st) {
  return umb_attn_attend_tiled(out, ldo, q, kv, proj, ld, gate_col, bias, n_dist, seq_slot, seq_row0, seq_pos0, seq_len, B, max_len, H,
                               G, D, E, window, scale, out_scale, softcap, nullptr, dtype, st);
}
