// Linear recurrences with a matrix state per head: the gated delta rule
//     S <- g * S;  u = beta (v - S^T k);  S <- S + k u^T;  o = S^T q
// (g a decay per key channel, or per head: HEAD_DELTA), retention (g one constant
// per head, u = v) and the matrix memory of log gates i, f (MEMORY)
//     m' = max(f + m, i);  S <- e^{f+m-m'} S + e^{i-m'} k v^T;  n alike with k alone;
//     o = S^T q / (max(|n.q|, e^{-m'}) + 1e-6).
//
// Everything between the projections and the output product is 32-bit, in
// bf16 models too, so the matrix work runs on v_mfma_f32_16x16x4_f32.
//
// Prompts: chunks of 16 tokens. With b_t the running sum of log g inside a
// chunk, S0 the state before it and all powers taken as differences <= 0,
//     U = T (V - K~ S0)          K~_t = e^{b_t} k_t
//     O = Q~ S0 + A U            Q~_t = e^{b_t} q_t
//     S = e^{b_C} S0 + K^^T U    K^_t = e^{b_C - b_t} k_t
//     A_ts = sum_c q_tc k_sc e^{b_tc - b_sc}                     (s <= t)
//     T = (I + strict_lower(beta_t sum_c k_tc k_sc e^{b_tc - b_sc}))^-1 diag(beta)
// chunk_prepare computes all that does not depend on S0, one workgroup per
// (chunk, head), convolutions or rotation included; chunk_scan walks the
// chunks, one workgroup per (sequence, head, 16 value columns), its four waves
// owning slices of the key channels. An accumulator tile of the state is
// directly the B operand of the next product if the contraction takes channels
// in the order 4g + r (g = lane / 16), which every A operand is stored for: no
// lane ever shuffles.
// A memory's running maxima are a scan of their own ahead of all that
// (memory_gates): with them the chunk's weights are known, every exponent is at
// most 0 up to rounding, and what is left is retention with weights that depend on
// the token. Its normaliser n is one more value column, of ones.
//
// Single tokens: one workgroup per (sequence, head) does everything from the
// projection to the gated, normed head in one pass over the state.
//
// Convolution inputs of the last ``taps`` tokens live in a ring indexed by
// position: a decode step writes place pos % taps and reads only the others,
// so workgroups that share a key head do not race.
#include "elem.h"
#include <torch/extension.h>
#include <c10/hip/HIPStream.h>

#define CUR_STREAM c10::hip::getCurrentHIPStream().stream()
#define CHUNK 16
#define MAX_TAPS 8

enum { DELTA = 0, RETAIN = 1, HEAD_DELTA = 2, MEMORY = 3 };
constexpr bool is_delta(int mode) { return mode == DELTA || mode == HEAD_DELTA; }

// what the rules' kernels read
struct RecArgs {
  const void* proj;    // [T, stride]
  long stride;
  int q0, k0, v0, b0;  // columns of q, k, v and beta (delta rules)
  int H, G, d, e, taps, rot;
  const float* conv_w;
  const float* a_log;
  const float* dt_bias;
  const float* norm;   // [e], MEMORY: [H * e]; RETAIN has none
  const void* z;       // [T, zstride]: decay pre-activations per channel or head
  long zstride;
  const void* gate;    // [T, gstride]: output gate pre-activations of all heads
  long gstride;
  const float* decay;
  const float* cos_sin;
  float eps;
  int i0, f0;          // columns of the log gates (MEMORY)
  const float *i_bias, *f_bias;
  float cap;
  float *nstate, *mstate;  // [slots, H, d], [slots, H]
  float* state;        // [slots, H, d, e]
  void* ring;          // [slots, taps, 2*G*d + H*e]
  const int* starts;
  const int* slots;
  void* out;           // [T, ostride]
  long ostride;
  float oscale;
};

// ring channel of a projection's channel i: q, then k, then v
DEVINL int ring_width(const RecArgs& a) { return 2 * a.G * a.d + a.H * a.e; }

// conv input ``back`` tokens before local row t of a portion that begins at
// position start and packed row row0
template <typename T>
DEVINL float conv_in(const RecArgs& a, int col, int ch, int row0, int t, int back,
                     int start, int slot) {
  const int at = t - back;
  if (at >= 0) return ldf((const T*)a.proj + (long)(row0 + at) * a.stride + col);
  const int pos = start + at;
  if (pos < 0) return 0.f;
  return ldf((const T*)a.ring + ((long)slot * a.taps + pos % a.taps) * ring_width(a) + ch);
}

// x[j]: the convolution inputs of local rows off - (MAX_TAPS - 1) + j, enough for
// CHUNK outputs; rows past the portion's end repeat its last row (not used)
template <typename T>
DEVINL void conv_inputs(const RecArgs& a, int col, int ch, int row0, int off, int n,
                        int start, int slot, float (&x)[CHUNK + MAX_TAPS - 1]) {
  const T* p = (const T*)a.proj + (long)(row0 + off) * a.stride + col;
#pragma unroll
  for (int t = 0; t < CHUNK; ++t)
    x[MAX_TAPS - 1 + t] = ldf(p + (long)min(t, n - 1) * a.stride);
  if (off >= MAX_TAPS - 1) {
#pragma unroll
    for (int j = 1; j < MAX_TAPS; ++j) x[MAX_TAPS - 1 - j] = ldf(p - (long)j * a.stride);
  } else {
#pragma unroll
    for (int j = 1; j < MAX_TAPS; ++j)
      x[MAX_TAPS - 1 - j] = j < a.taps
          ? conv_in<T>(a, col, ch, row0, off, j, start, slot) : 0.f;
  }
}

DEVINL void conv_weights(const RecArgs& a, int ch, float (&w)[MAX_TAPS]) {
#pragma unroll
  for (int j = 0; j < MAX_TAPS; ++j)
    w[j] = j < a.taps ? a.conv_w[(long)ch * a.taps + a.taps - 1 - j] : 0.f;
}

DEVINL float conv_at(const float (&w)[MAX_TAPS], const float (&x)[CHUNK + MAX_TAPS - 1],
                     int t) {
  float y = 0.f;
#pragma unroll
  for (int j = 0; j < MAX_TAPS; ++j) y += w[j] * x[MAX_TAPS - 1 + t - j];
  return silu_f(y);
}

DEVINL float log_decay(const RecArgs& a, float neg_exp_a, float z, int i) {
  return neg_exp_a * softplus_f(z + a.dt_bias[i]);
}

// ------------------------------------------------------------------ prompts

// v after convolution and silu (delta rules) or as projected: [T, H*e] fp32
template <typename T, int MODE>
__global__ __launch_bounds__(256) void value_prepare_kernel(
    RecArgs a, const int* __restrict__ cu, const int* __restrict__ cseq,
    const int* __restrict__ coff, float* __restrict__ vf) {
  const int s = cseq[blockIdx.x], off = coff[blockIdx.x];
  const int row0 = cu[s], n = min(CHUNK, cu[s + 1] - row0 - off);
  const int slot = a.slots[s], start = a.starts[s];
  const int c = blockIdx.y * 256 + threadIdx.x;
  const int HE = a.H * a.e;
  if (c >= HE || slot < 0) return;
  if constexpr (!is_delta(MODE)) {
    for (int t = 0; t < n; ++t) {
      const long row = row0 + off + t;
      vf[row * HE + c] = ldf((const T*)a.proj + row * a.stride + a.v0 + c);
    }
    return;
  }
  const int ch = 2 * a.G * a.d + c;
  float w[MAX_TAPS], x[CHUNK + MAX_TAPS - 1];
  conv_weights(a, ch, w);
  conv_inputs<T>(a, a.v0 + c, ch, row0, off, n, start, slot, x);
#pragma unroll
  for (int t = 0; t < CHUNK; ++t)
    if (t < n) vf[(long)(row0 + off + t) * HE + c] = conv_at(w, x, t);
}

// Log gates of a memory's tokens, [T, H] each, and the running maxima m; m0 [S, H]:
// the maxima before the portions
struct GateSpace {
  float *f, *i, *m, *m0;
};

DEVINL void memory_gate(const RecArgs& a, float zi, float zf, int h, float& i, float& f) {
  i = a.cap * tanhf((zi + a.i_bias[h]) / a.cap);
  f = -softplus_f(-a.cap * tanhf((zf + a.f_bias[h]) / a.cap));
}

// One workgroup per (head, sequence). Tokens are maps m -> max(F + m, A); their
// composition (F, A) after (F', A') is (F + F', max(F + A', A)), a prefix scan.
template <typename T>
__global__ __launch_bounds__(1024) void memory_gates_kernel(RecArgs a,
                                                            const int* __restrict__ cu,
                                                            GateSpace w) {
  __shared__ float wf[16], wa[16], carry;
  const int h = blockIdx.x, s = blockIdx.y, slot = a.slots[s];
  if (slot < 0) return;
  const int row0 = cu[s], len = cu[s + 1] - row0;
  const int tid = threadIdx.x, lane = tid % WAVE, wave = tid / WAVE;
  float m = a.starts[s] > 0 ? a.mstate[(long)slot * a.H + h] : 0.f;
  if (tid == 0) w.m0[(long)s * a.H + h] = m;
  for (int t0 = 0; t0 < len; t0 += 1024) {
    const int t = t0 + tid;
    const long at = (long)(row0 + t) * a.H + h;
    float F = 0.f, A = -INFINITY;
    if (t < len) {
      const T* p = (const T*)a.proj + (long)(row0 + t) * a.stride;
      memory_gate(a, ldf(p + a.i0 + h), ldf(p + a.f0 + h), h, A, F);
      w.i[at] = A;
      w.f[at] = F;
    }
#pragma unroll
    for (int off = 1; off < WAVE; off <<= 1) {
      const float pf = __shfl_up(F, off, WAVE), pa = __shfl_up(A, off, WAVE);
      if (lane >= off) {
        A = fmaxf(F + pa, A);
        F += pf;
      }
    }
    if (lane == WAVE - 1) {
      wf[wave] = F;
      wa[wave] = A;
    }
    __syncthreads();
    float before = m;
    for (int v = 0; v < wave; ++v) before = fmaxf(wf[v] + before, wa[v]);
    const float now = fmaxf(F + before, A);
    if (t < len) w.m[at] = now;
    if (tid == 1023) carry = now;
    __syncthreads();
    m = carry;  // past the end tokens change nothing
  }
  if (tid == 0) a.mstate[(long)slot * a.H + h] = m;
}

// Workspace of one (chunk, head), fp32: Q~, K~ (delta rules) and K^ in the order the
// scan's lanes load them, 256 values per 16 channels: [tile][lane][4], where
// lane 16 g + i holds channels 4g .. 4g+3 of token i (Q~, K~) or tokens
// 4g .. 4g+3 of channel i (K^); e^{b_C} [dp], one of them but for DELTA; A, T (delta rules) [16][16]
struct ChunkSpace {
  float *q, *k, *kt, *g, *a, *t;
  int dp;
};

template <typename T, int MODE>
__global__ __launch_bounds__(256) void chunk_prepare_kernel(
    RecArgs a, const int* __restrict__ cu, const int* __restrict__ cseq,
    const int* __restrict__ coff, ChunkSpace w, GateSpace mg) {
  extern __shared__ __attribute__((aligned(16))) float lds[];
  __shared__ float beta[CHUNK];
  __shared__ float red[4];
  __shared__ float pair[4][2][CHUNK * CHUNK];
  // with one decay per token: the factors of Q~ and K~, and of K^, and the exponents
  // whose differences weigh the pairs
  __shared__ float lg[CHUNK], fq[CHUNK], fk[CHUNK], px[CHUNK], py[CHUNK], fg;
  const int dp = w.dp, ld = dp + 4;
  float* sq = lds;              // [16][ld]
  float* sk = sq + CHUNK * ld;
  float* sb = sk + CHUNK * ld;  // running log decay per channel (DELTA)
  const int h = blockIdx.y, s = cseq[blockIdx.x], off = coff[blockIdx.x];
  const int row0 = cu[s], n = min(CHUNK, cu[s + 1] - row0 - off);
  const int slot = a.slots[s], start = a.starts[s];
  if (slot < 0) return;
  const int tid = threadIdx.x, lane = tid % WAVE, wave = tid / WAVE;
  const int hk = h / (a.H / a.G);
  const T* proj = (const T*)a.proj;
  const float lam = MODE == RETAIN ? logf(fmaxf(a.decay[h], 1e-30f)) : 0.f;
  const float nea = is_delta(MODE) ? -expf(a.a_log[h]) : 0.f;

  // ---- q, k (convolution + silu, or rotation) and the running log decay
  for (int i = tid; i < 2 * dp; i += 256) {
    const bool is_k = i >= dp;
    const int c = is_k ? i - dp : i;
    float* dst = (is_k ? sk : sq) + c;
    const int col = (is_k ? a.k0 : a.q0) + hk * a.d + c;
    if constexpr (is_delta(MODE)) {
      const int ch = (is_k ? a.G * a.d : 0) + hk * a.d + c;
      float cw[MAX_TAPS], x[CHUNK + MAX_TAPS - 1];
      if (c < a.d) {
        conv_weights(a, ch, cw);
        conv_inputs<T>(a, col, ch, row0, off, n, start, slot, x);
      }
#pragma unroll
      for (int t = 0; t < CHUNK; ++t)
        dst[t * ld] = t < n && c < a.d ? conv_at(cw, x, t) : 0.f;
    } else {
      const int half = a.rot / 2;
      const float sc = is_k == (MODE == RETAIN) ? rsqrtf((float)a.d) : 1.f;
      for (int t = 0; t < CHUNK; ++t) {
        float y = 0.f;
        if (t < n && c < a.d) {
          const T* p = proj + (long)(row0 + off + t) * a.stride + col;
          y = ldf(p);
          if (c < a.rot) {
            const float* cs = a.cos_sin + (long)(start + off + t) * a.rot;
            const int f = c < half ? c : c - half;
            y = c < half ? y * cs[f] - ldf(p + half) * cs[half + f]
                         : y * cs[f] + ldf(p - half) * cs[half + f];
          }
        }
        dst[t * ld] = y * sc;
      }
    }
  }
  if constexpr (MODE == DELTA) {
    const T* z = (const T*)a.z + (long)(row0 + off) * a.zstride + h * a.d;
#pragma unroll 4
    for (int x = tid; x < CHUNK * dp; x += 256) {
      const int t = x / dp, c = x % dp;
      sb[t * ld + c] = t < n && c < a.d
          ? log_decay(a, nea, ldf(z + t * a.zstride + c), h * a.d + c) : 0.f;
    }
  }
  if (tid < CHUNK) {
    const long row = row0 + off + min(tid, n - 1);
    const bool in = tid < n;
    if constexpr (is_delta(MODE))
      beta[tid] = in ? sigmoid_f(ldf(proj + row * a.stride + a.b0 + h)) : 0.f;
    if constexpr (MODE != DELTA) {
      float x = lam;
      if constexpr (MODE == HEAD_DELTA)
        x = log_decay(a, nea, ldf((const T*)a.z + row * a.zstride + h), h);
      if constexpr (MODE == MEMORY) x = mg.f[row * a.H + h];
      lg[tid] = in ? x : 0.f;
    }
  }
  __syncthreads();
  if (MODE != DELTA && tid < CHUNK) {
    float b = 0.f, bc = 0.f;
#pragma unroll
    for (int u = 0; u < CHUNK; ++u) {
      bc += lg[u];
      if (u <= tid) b += lg[u];
    }
    const bool in = tid < n;
    float before = 0.f, m = 0.f, mc = 0.f, put = 0.f;
    if constexpr (MODE == MEMORY) {
      const long row = row0 + off;
      before = off ? mg.m[(row - 1) * a.H + h] : mg.m0[(long)s * a.H + h];
      m = mg.m[(row + min(tid, n - 1)) * a.H + h];
      mc = mg.m[(row + n - 1) * a.H + h];
      put = mg.i[(row + min(tid, n - 1)) * a.H + h];
    }
    fq[tid] = in ? expf(b + before - m) : 0.f;
    fk[tid] = in ? expf(bc - b + put - mc) : 0.f;
    px[tid] = in ? b - m : 0.f;
    py[tid] = in ? b - put : 0.f;
    if (tid == 0) fg = expf(bc + before - mc);
  }
  bool safe = true;  // every e^{-b} of the chunk is moderate
  if constexpr (MODE == DELTA) {
    float lowest = 0.f;
    for (int c = tid; c < dp; c += 256) {
      float b = 0.f;
#pragma unroll
      for (int t = 0; t < CHUNK; ++t) {
        b += sb[t * ld + c];
        sb[t * ld + c] = b;
      }
      lowest = fminf(lowest, b);
    }
    lowest = -wave_max(-lowest);
    if (lane == 0) red[wave] = lowest;
  }
  if constexpr (is_delta(MODE)) {
    // unit vectors; q also takes d^-1/2
    for (int t = wave * 4; t < wave * 4 + 4; ++t) {
      float q2 = 0.f, k2 = 0.f;
      for (int c = lane; c < dp; c += WAVE) {
        q2 += sq[t * ld + c] * sq[t * ld + c];
        k2 += sk[t * ld + c] * sk[t * ld + c];
      }
      const float qi = rsqrtf(wave_sum(q2) + 1e-6f) * rsqrtf((float)a.d);
      const float ki = rsqrtf(wave_sum(k2) + 1e-6f);
      for (int c = lane; c < dp; c += WAVE) {
        sq[t * ld + c] *= qi;
        sk[t * ld + c] *= ki;
      }
    }
  }
  __syncthreads();
  if constexpr (MODE == DELTA)
    safe = fminf(fminf(red[0], red[1]), fminf(red[2], red[3])) > -30.f;

  // ---- Q~, K~, K^ out; A and K K^T on the matrix cores, waves splitting tiles
  const long ws = (long)blockIdx.x * a.H + h;
  const int i = lane & 15, g = lane >> 4;
  floatx4 aqk = {0.f, 0.f, 0.f, 0.f}, akk = {0.f, 0.f, 0.f, 0.f};
  for (int tile = wave; tile * 16 < dp; tile += 4) {
    const int c0 = tile * 16 + 4 * g;
    const floatx4 q = *reinterpret_cast<const floatx4*>(sq + i * ld + c0);
    const floatx4 k = *reinterpret_cast<const floatx4*>(sk + i * ld + c0);
    floatx4 qe, ke, kt, kn, ge;
    const long wt = (ws * (dp / 16) + tile) * 256 + lane * 4;
#pragma unroll
    for (int r = 0; r < 4; ++r) {  // K^ with the lanes along the channels
      const int t = 4 * g + r, c = tile * 16 + i;
      const float kv = sk[t * ld + c];
      kt[r] = kv * (MODE == DELTA ? expf(sb[(CHUNK - 1) * ld + c] - sb[t * ld + c])
                                  : fk[t]);
    }
    *reinterpret_cast<floatx4*>(w.kt + wt) = kt;
    if constexpr (MODE == DELTA) {
      const floatx4 b = *reinterpret_cast<const floatx4*>(sb + i * ld + c0);
      const floatx4 bc =
          *reinterpret_cast<const floatx4*>(sb + (CHUNK - 1) * ld + c0);
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const float eb = expf(b[r]);
        qe[r] = q[r] * eb;
        ke[r] = k[r] * eb;
        kn[r] = safe ? k[r] * expf(-b[r]) : 0.f;
        ge[r] = expf(bc[r]);
      }
      *reinterpret_cast<floatx4*>(w.k + wt) = ke;
    } else {
      qe = q * fq[i];
      ge = floatx4{fg, fg, fg, fg};
      if constexpr (MODE == HEAD_DELTA)
        *reinterpret_cast<floatx4*>(w.k + wt) = k * fq[i];
    }
    *reinterpret_cast<floatx4*>(w.q + wt) = qe;
    if (i == 0 && (MODE == DELTA || c0 == 0))
      *reinterpret_cast<floatx4*>(w.g + ws * dp + c0) = ge;
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      if constexpr (MODE == DELTA) {
        aqk = __builtin_amdgcn_mfma_f32_16x16x4f32(qe[r], kn[r], aqk, 0, 0, 0);
        akk = __builtin_amdgcn_mfma_f32_16x16x4f32(ke[r], kn[r], akk, 0, 0, 0);
      } else {
        aqk = __builtin_amdgcn_mfma_f32_16x16x4f32(q[r], k[r], aqk, 0, 0, 0);
        if constexpr (MODE == HEAD_DELTA)
          akk = __builtin_amdgcn_mfma_f32_16x16x4f32(k[r], k[r], akk, 0, 0, 0);
      }
    }
  }
#pragma unroll
  for (int r = 0; r < 4; ++r) {
    pair[wave][0][(4 * g + r) * CHUNK + i] = aqk[r];
    if constexpr (is_delta(MODE)) pair[wave][1][(4 * g + r) * CHUNK + i] = akk[r];
  }
  __syncthreads();
  const int t = tid / CHUNK, u = tid % CHUNK;
  float sqk = 0.f, skk = 0.f;
  if (MODE != DELTA || safe) {
#pragma unroll
    for (int v = 0; v < 4; ++v) {
      sqk += pair[v][0][tid];
      if constexpr (is_delta(MODE)) skk += pair[v][1][tid];
    }
  } else if (u <= t) {
    // strong decay: take every power as one exponential of the difference
    for (int c = 0; c < a.d; ++c) {
      const float x = expf(sb[t * ld + c] - sb[u * ld + c]) * sk[u * ld + c];
      sqk += sq[t * ld + c] * x;
      skk += sk[t * ld + c] * x;
    }
  }
  if constexpr (MODE != DELTA) {
    const float f = u <= t && t < n ? expf(px[t] - py[u]) : 0.f;
    sqk *= f;
    skk *= f;
  }
  if constexpr (!is_delta(MODE)) {
    w.a[ws * 256 + tid] = sqk;
    return;
  }
  w.a[ws * 256 + tid] = u <= t ? sqk : 0.f;
  __syncthreads();
  pair[0][0][tid] = u < t ? beta[t] * skk : 0.f;
  __syncthreads();
  // column ``tid`` of the unit lower triangular inverse, then times beta
  if (tid < CHUNK) {
    float x[CHUNK];
#pragma unroll
    for (int r = 0; r < CHUNK; ++r) {
      float y = r == tid ? 1.f : 0.f;
#pragma unroll
      for (int v = 0; v < r; ++v) y -= pair[0][0][r * CHUNK + v] * x[v];
      x[r] = y;
    }
#pragma unroll
    for (int r = 0; r < CHUNK; ++r) w.t[ws * 256 + r * CHUNK + tid] = x[r] * beta[tid];
  }
}

// NTW: 16-channel tiles of the state per wave (key channels <= 64 * NTW). A memory's
// extra column tile makes one workgroup more than fit at two per CU in the usual
// sizes: it takes three, with one operand set less in flight.
template <int MODE, int NTW>
__global__ __launch_bounds__(256, NTW > 2 ? 1 : MODE == MEMORY ? 3 : 2) void chunk_scan_kernel(
    RecArgs a, const int* __restrict__ cu, const int* __restrict__ cfirst,
    ChunkSpace w, const float* __restrict__ vf, float* __restrict__ of,
    float* __restrict__ den, int S) {
  __shared__ floatx4 part[2][4][2][WAVE];
  // all column tiles of one (sequence, head) on one XCD: they share its L2
  const int NE = (a.e + (MODE == MEMORY) + 15) / 16, groups = S * a.H;
  const int band = blockIdx.x / (8 * NE), in = blockIdx.x % (8 * NE);
  const int group = band * 8 + in % 8, et = in / 8;
  if (group >= groups) return;
  const int s = group / a.H, h = group % a.H;
  const int slot = a.slots[s];
  const int len = cu[s + 1] - cu[s];
  if (slot < 0 || len == 0) return;
  const int lane = threadIdx.x % WAVE, wave = threadIdx.x / WAVE;
  const int i = lane & 15, g = lane >> 4;
  const int col = et * 16 + i;
  const bool cv = col < a.e;
  const bool cn = MODE == MEMORY && col == a.e;  // the normaliser's column
  const int dp = w.dp, RT = dp / 16, HE = a.H * a.e;
  float* state = a.state + ((long)slot * a.H + h) * a.d * a.e;
  float* nstate = MODE == MEMORY ? a.nstate + ((long)slot * a.H + h) * a.d : nullptr;

  floatx4 st[NTW];
  const bool fresh = a.starts[s] == 0;
#pragma unroll
  for (int x = 0; x < NTW; ++x)
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int row = (wave * NTW + x) * 16 + 4 * g + r;
      st[x][r] = fresh || row >= a.d || !(cv || cn) ? 0.f
                 : cn ? nstate[row] : state[(long)row * a.e + col];
    }

  // one chunk's operands; in three sets, a chunk's loads have two chunks' time to
  // arrive
  constexpr int SETS = MODE == MEMORY ? 2 : 3;
  constexpr int NG = MODE == DELTA ? NTW : 1;  // decays per channel, or one
  struct Frags {
    floatx4 q[NTW], k[NTW], t[NTW], gd[NG], v, am, tm;
  };
  const int nch = (len + CHUNK - 1) / CHUNK;
  const long base = cu[s];
  auto fetch = [&](int c, Frags& f) {
    const long ws = (long)(cfirst[s] + c) * a.H + h;
    const int n = min(CHUNK, len - c * CHUNK);
#pragma unroll
    for (int x = 0; x < NTW; ++x) {
      // a wave without this tile loads the last one and zeroes it on use
      const int tile = min(wave * NTW + x, RT - 1);
      const long o = (ws * RT + tile) * 256 + lane * 4;
      f.q[x] = ld4(w.q + o);
      if (is_delta(MODE)) f.k[x] = ld4(w.k + o);
      f.t[x] = ld4(w.kt + o);
      if constexpr (MODE == DELTA) f.gd[x] = ld4(w.g + ws * dp + tile * 16 + 4 * g);
    }
    if constexpr (MODE != DELTA) f.gd[0][0] = w.g[ws * dp];
#pragma unroll
    for (int r = 0; r < 4; ++r)
      f.v[r] = vf[(base + c * CHUNK + min(4 * g + r, n - 1)) * HE + h * a.e +
                  min(col, a.e - 1)];
    f.am = ld4(w.a + ws * 256 + i * CHUNK + 4 * g);
    if (is_delta(MODE)) f.tm = ld4(w.t + ws * 256 + i * CHUNK + 4 * g);
  };
  auto step = [&](int c, Frags& f) {
    const int n = min(CHUNK, len - c * CHUNK);
    const long row0 = base + c * CHUNK;
    floatx4 qa[NTW], ka[NTW], ta[NTW], gd[NG];
#pragma unroll
    for (int x = 0; x < NTW; ++x) {
      const float in = wave * NTW + x < RT ? 1.f : 0.f;
      qa[x] = f.q[x];  // meets a zero state where the tile is not there
      if (is_delta(MODE)) ka[x] = f.k[x];
      ta[x] = f.t[x] * in;
      if constexpr (MODE == DELTA) gd[x] = f.gd[x];
    }
    const float g0 = MODE == DELTA ? 0.f : f.gd[0][0];
    floatx4 u;
#pragma unroll
    for (int r = 0; r < 4; ++r)
      u[r] = 4 * g + r >= n ? 0.f : cv ? f.v[r] : cn ? 1.f : 0.f;
    const floatx4 am = f.am;
    floatx4 tm = {0.f, 0.f, 0.f, 0.f};
    if (is_delta(MODE)) tm = f.tm;

    // this wave's channels of Q~ S0 and K~ S0
    floatx4 o = {0.f, 0.f, 0.f, 0.f}, ks = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int x = 0; x < NTW; ++x)
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        o = __builtin_amdgcn_mfma_f32_16x16x4f32(qa[x][r], st[x][r], o, 0, 0, 0);
        if (is_delta(MODE))
          ks = __builtin_amdgcn_mfma_f32_16x16x4f32(ka[x][r], st[x][r], ks, 0, 0, 0);
      }
    const int buf = c & 1;
    part[buf][wave][0][lane] = o;
    if (is_delta(MODE)) part[buf][wave][1][lane] = ks;
    __syncthreads();
    if (is_delta(MODE)) {
#pragma unroll
      for (int v = 0; v < 4; ++v) u -= part[buf][v][1][lane];
      floatx4 y = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int r = 0; r < 4; ++r)
        y = __builtin_amdgcn_mfma_f32_16x16x4f32(tm[r], u[r], y, 0, 0, 0);
      u = y;
    }
    if (wave == (c & 3)) {
      floatx4 y = part[buf][0][0][lane];
#pragma unroll
      for (int v = 1; v < 4; ++v) y += part[buf][v][0][lane];
#pragma unroll
      for (int r = 0; r < 4; ++r)
        y = __builtin_amdgcn_mfma_f32_16x16x4f32(am[r], u[r], y, 0, 0, 0);
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int t = 4 * g + r;
        if (t < n && cv) of[(row0 + t) * HE + h * a.e + col] = y[r];
        if (t < n && cn) den[(row0 + t) * a.H + h] = y[r];
      }
    }
#pragma unroll
    for (int x = 0; x < NTW; ++x) {
      if constexpr (MODE == DELTA) st[x] *= gd[x];
      else st[x] *= g0;
#pragma unroll
      for (int r = 0; r < 4; ++r)
        st[x] = __builtin_amdgcn_mfma_f32_16x16x4f32(ta[x][r], u[r], st[x], 0, 0, 0);
    }
    if (c + SETS < nch) fetch(c + SETS, f);
  };
  Frags f0, f1, f2;
  fetch(0, f0);
  if (nch > 1) fetch(1, f1);
  if (SETS > 2 && nch > 2) fetch(2, f2);
  for (int c = 0; c < nch; c += SETS) {
    step(c, f0);
    if (c + 1 < nch) step(c + 1, f1);
    if constexpr (SETS > 2)
      if (c + 2 < nch) step(c + 2, f2);
  }
#pragma unroll
  for (int x = 0; x < NTW; ++x)
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int row = (wave * NTW + x) * 16 + 4 * g + r;
      if (row < a.d && cv) state[(long)row * a.e + col] = st[x][r];
      if (row < a.d && cn) nstate[row] = st[x][r];
    }
}

// raw convolution inputs of the portion's last tokens into the ring
template <typename T>
__global__ void ring_update_kernel(RecArgs a, const int* __restrict__ cu) {
  const int s = blockIdx.y, slot = a.slots[s];
  if (slot < 0) return;
  const int n = cu[s + 1] - cu[s], C = ring_width(a), qk = a.G * a.d;
  const int c = blockIdx.x * blockDim.x + threadIdx.x;
  if (c >= C) return;
  const int col = c < qk ? a.q0 + c : c < 2 * qk ? a.k0 + c - qk : a.v0 + c - 2 * qk;
  for (int t = max(0, n - a.taps); t < n; ++t)
    ((T*)a.ring)[((long)slot * a.taps + (a.starts[s] + t) % a.taps) * C + c] =
        ((const T*)a.proj)[(long)(cu[s] + t) * a.stride + col];
}

// what a memory's head is divided by
DEVINL float memory_norm(float den, float m) { return fmaxf(fabsf(den), expf(-m)) + 1e-6f; }

template <int MODE>
DEVINL float gate_act(float x) {
  return MODE == DELTA || MODE == MEMORY ? sigmoid_f(x) : silu_f(x);
}

// o / rms(o) per head, times weight and gate: 4 values per lane, GL lanes per
// (token, head); e = 4 GL at most
template <typename T, int MODE, int GL>
__global__ __launch_bounds__(256) void head_norm_gate4_kernel(
    RecArgs a, const float* __restrict__ of, const float* __restrict__ den,
    const float* __restrict__ m, long TH) {
  const long id = ((long)blockIdx.x * 256 + threadIdx.x) / GL;
  const int c = threadIdx.x % GL * 4;
  const long th = min(id, TH - 1);
  const long t = th / a.H;
  const int h = th % a.H;
  const bool in = c < a.e;
  floatx4 o = {0.f, 0.f, 0.f, 0.f}, g = o;
  if (in) {
    o = ld4(of + th * a.e + c);
    g = ld4((const T*)a.gate + t * a.gstride + h * a.e + c);
  }
  if constexpr (MODE == MEMORY) o *= 1.f / memory_norm(den[th], m[th]);
  const float inv = rsqrtf(
      group_sum<GL>(o[0] * o[0] + o[1] * o[1] + o[2] * o[2] + o[3] * o[3]) / a.e + a.eps);
  if (!in || id >= TH) return;
  const float sc = inv * a.oscale;
  floatx4 y;
#pragma unroll
  for (int r = 0; r < 4; ++r) y[r] = o[r] * sc * gate_act<MODE>(g[r]);
  if constexpr (MODE != RETAIN) y *= ld4(a.norm + (MODE == MEMORY ? h * a.e : 0) + c);
  st4((T*)a.out + t * a.ostride + h * a.e + c, y);
}

// The same for any head width: one wave per (token, head)
template <typename T, int MODE>
__global__ __launch_bounds__(256) void head_norm_gate_kernel(
    RecArgs a, const float* __restrict__ of, const float* __restrict__ den,
    const float* __restrict__ m, long TH) {
  const long wid = (long)blockIdx.x * 4 + threadIdx.x / WAVE;
  const int lane = threadIdx.x % WAVE;
  if (wid >= TH) return;
  const long t = wid / a.H;
  const int h = wid % a.H;
  const float* o = of + wid * a.e;
  const float f = MODE == MEMORY ? 1.f / memory_norm(den[wid], m[wid]) : 1.f;
  float ss = 0.f;
  for (int c = lane; c < a.e; c += WAVE) ss += o[c] * f * (o[c] * f);
  const float inv = rsqrtf(wave_sum(ss) / a.e + a.eps);
  for (int c = lane; c < a.e; c += WAVE) {
    float y = o[c] * f * inv *
              gate_act<MODE>(ldf((const T*)a.gate + t * a.gstride + h * a.e + c));
    if constexpr (MODE != RETAIN) y *= a.norm[(MODE == MEMORY ? h * a.e : 0) + c];
    stf((T*)a.out + t * a.ostride + h * a.e + c, y * a.oscale);
  }
}

// ------------------------------------------------------------ single tokens

DEVINL float block_sum_n(float x, float* red) {
  x = wave_sum(x);
  __syncthreads();
  if ((threadIdx.x & 63) == 0) red[threadIdx.x >> 6] = x;
  __syncthreads();
  float y = 0.f;
  for (int i = 0; i < (int)blockDim.x / WAVE; ++i) y += red[i];
  return y;
}

// VW value columns and up to R key channels per thread
template <typename T, int MODE, int VW, int R>
__global__ __launch_bounds__(1024) void recurrence_decode_kernel(RecArgs a, int CG) {
  extern __shared__ __attribute__((aligned(16))) float lds[];
  __shared__ float red[16];
  const int h = blockIdx.x, b = blockIdx.y;
  const int d = a.d, e = a.e, tid = threadIdx.x, NT = blockDim.x;
  T* out = (T*)a.out + b * a.ostride + (long)h * e;
  const int slot = a.slots[b];
  if (slot < 0) {  // idle row of a captured batch
    for (int c = tid; c < e; c += NT) stf(out + c, 0.f);
    return;
  }
  float* sq = lds;
  float* sk = sq + d;
  float* sg = sk + d;
  float* sv = sg + d;          // v, then u
  float* so = sv + CG * VW;    // [RG][CG * VW] partial sums
  const int pos = a.starts[b];
  const int cg = tid % CG, rg = tid / CG, RG = NT / CG;
  const bool cv = cg * VW < e;
  float* state = a.state + ((long)slot * a.H + h) * d * e + cg * VW;
  const T* proj = (const T*)a.proj + b * a.stride;
  const T* z = (const T*)a.z + b * a.zstride;
  const T* gate = (const T*)a.gate + b * a.gstride + (long)h * e;

  // the state is on its way while q, k, v are prepared
  float st[R][VW];
#pragma unroll
  for (int j = 0; j < R; ++j) {
    const int row = rg + RG * j;
    if (row < d && cv && pos > 0) {
      if constexpr (VW == 4) {
        const floatx4 v = ld4(state + (long)row * e);
#pragma unroll
        for (int x = 0; x < 4; ++x) st[j][x] = v[x];
      } else {
        st[j][0] = state[(long)row * e];
      }
    } else {
#pragma unroll
      for (int x = 0; x < VW; ++x) st[j][x] = 0.f;
    }
  }

  const int rep = a.H / a.G, hk = h / rep;
  float den = 1.f;  // MEMORY: what the head is divided by
  if constexpr (is_delta(MODE)) {
    const int C = ring_width(a);
    T* ring = (T*)a.ring + (long)slot * a.taps * C;
    for (int c = tid; c < 2 * d + e; c += NT) {
      const bool qk = c < 2 * d, is_k = qk && c >= d;
      const int i = qk ? hk * d + (is_k ? c - d : c) : h * e + c - 2 * d;
      const int ch = (qk ? (is_k ? a.G * d : 0) : 2 * a.G * d) + i;
      const T raw = proj[(qk ? (is_k ? a.k0 : a.q0) : a.v0) + i];
      const float* cw = a.conv_w + (long)ch * a.taps;
      float y = cw[a.taps - 1] * ldf(&raw);
      for (int j = 1; j < a.taps && j <= pos; ++j)
        y += cw[a.taps - 1 - j] * ldf(ring + (long)((pos - j) % a.taps) * C + ch);
      y = silu_f(y);
      if (qk) (is_k ? sk : sq)[is_k ? c - d : c] = y;
      else sv[c - 2 * d] = y;
      // the heads that share a key head would write the same value
      if (!qk || h % rep == 0) ring[(long)(pos % a.taps) * C + ch] = raw;
    }
    const float nea = -expf(a.a_log[h]);
    const float gh = MODE == DELTA ? 0.f : expf(log_decay(a, nea, ldf(z + h), h));
    for (int c = tid; c < d; c += NT)
      sg[c] = MODE == DELTA ? expf(log_decay(a, nea, ldf(z + h * d + c), h * d + c)) : gh;
    __syncthreads();
    float q2 = 0.f, k2 = 0.f;
    for (int c = tid; c < d; c += NT) {
      q2 += sq[c] * sq[c];
      k2 += sk[c] * sk[c];
    }
    const float qi = rsqrtf(block_sum_n(q2, red) + 1e-6f) * rsqrtf((float)d);
    const float ki = rsqrtf(block_sum_n(k2, red) + 1e-6f);
    for (int c = tid; c < d; c += NT) {
      sq[c] *= qi;
      sk[c] *= ki;
    }
  } else {
    float keep = 0.f, put = 1.f, m = 0.f;
    const float before = MODE == MEMORY && pos > 0 ? a.mstate[(long)slot * a.H + h] : 0.f;
    if constexpr (MODE == RETAIN) {
      keep = a.decay[h];
    } else {
      float i, f;
      memory_gate(a, ldf(proj + a.i0 + h), ldf(proj + a.f0 + h), h, i, f);
      m = fmaxf(f + before, i);
      keep = expf(f + before - m);
      put = expf(i - m);
    }
    const int half = a.rot / 2;
    const float* cs = a.cos_sin + (long)pos * a.rot;
    for (int c = tid; c < 2 * d; c += NT) {
      const bool is_k = c >= d;
      const int i = is_k ? c - d : c;
      const T* p = proj + (is_k ? a.k0 : a.q0) + h * d + i;
      float y = ldf(p);
      if (i < a.rot) {
        const int f = i < half ? i : i - half;
        y = i < half ? y * cs[f] - ldf(p + half) * cs[half + f]
                     : y * cs[f] + ldf(p - half) * cs[half + f];
      }
      if (is_k == (MODE == RETAIN)) y *= rsqrtf((float)d);
      (is_k ? sk : sq)[i] = is_k ? y * put : y;
    }
    for (int c = tid; c < e; c += NT) sv[c] = ldf(proj + a.v0 + h * e + c);
    for (int c = tid; c < d; c += NT) sg[c] = keep;
    if constexpr (MODE == MEMORY) {
      __syncthreads();
      float* ns = a.nstate + ((long)slot * a.H + h) * d;
      float nq = 0.f;
      for (int c = tid; c < d; c += NT) {
        const float x = (pos > 0 ? keep * ns[c] : 0.f) + sk[c];
        ns[c] = x;
        nq += x * sq[c];
      }
      den = memory_norm(block_sum_n(nq, red), m);  // everyone has read mstate
      if (tid == 0) a.mstate[(long)slot * a.H + h] = m;
    }
  }
  __syncthreads();

  float sum[VW];
  if constexpr (is_delta(MODE)) {
#pragma unroll
    for (int x = 0; x < VW; ++x) sum[x] = 0.f;
#pragma unroll
    for (int j = 0; j < R; ++j) {
      const int row = rg + RG * j;
      if (row < d) {
        const float g = sg[row], k = sk[row];
#pragma unroll
        for (int x = 0; x < VW; ++x) {
          st[j][x] *= g;
          sum[x] += st[j][x] * k;
        }
      }
    }
#pragma unroll
    for (int x = 0; x < VW; ++x) so[rg * CG * VW + cg * VW + x] = sum[x];
    __syncthreads();
    const float beta = sigmoid_f(ldf(proj + a.b0 + h));
    for (int c = tid; c < e; c += NT) {
      float y = 0.f;
      for (int r = 0; r < RG; ++r) y += so[r * CG * VW + c];
      sv[c] = beta * (sv[c] - y);
    }
    __syncthreads();
  }
#pragma unroll
  for (int x = 0; x < VW; ++x) sum[x] = 0.f;
  float u[VW];
#pragma unroll
  for (int x = 0; x < VW; ++x) u[x] = cv ? sv[cg * VW + x] : 0.f;
#pragma unroll
  for (int j = 0; j < R; ++j) {
    const int row = rg + RG * j;
    if (row < d) {
      const float k = sk[row], q = sq[row], g = is_delta(MODE) ? 1.f : sg[row];
#pragma unroll
      for (int x = 0; x < VW; ++x) {
        st[j][x] = g * st[j][x] + k * u[x];
        sum[x] += st[j][x] * q;
      }
      if (cv) {
        if constexpr (VW == 4) {
          floatx4 v;
#pragma unroll
          for (int x = 0; x < 4; ++x) v[x] = st[j][x];
          st4(state + (long)row * e, v);
        } else {
          state[(long)row * e] = st[j][0];
        }
      }
    }
  }
#pragma unroll
  for (int x = 0; x < VW; ++x) so[rg * CG * VW + cg * VW + x] = sum[x];
  __syncthreads();
  float ss = 0.f;
  for (int c = tid; c < e; c += NT) {
    float y = 0.f;
    for (int r = 0; r < RG; ++r) y += so[r * CG * VW + c];
    if constexpr (MODE == MEMORY) y /= den;
    sv[c] = y;  // u is no longer needed
    ss += y * y;
  }
  const float inv = rsqrtf(block_sum_n(ss, red) / e + a.eps);
  for (int c = tid; c < e; c += NT) {
    float y = sv[c] * inv * gate_act<MODE>(ldf(gate + c));
    if constexpr (MODE != RETAIN) y *= a.norm[(MODE == MEMORY ? h * e : 0) + c];
    stf(out + c, y * a.oscale);
  }
}

// --------------------------------------------------------------------- host

static void check_common(const RecArgs& a, const torch::Tensor& proj,
                         const torch::Tensor& state, const torch::Tensor& starts,
                         const torch::Tensor& slots, const torch::Tensor& out) {
  TORCH_CHECK(proj.is_cuda() && proj.dim() == 2 && proj.stride(1) == 1 &&
              (proj.dtype() == torch::kBFloat16 || proj.dtype() == torch::kFloat32));
  TORCH_CHECK(state.is_contiguous() && state.dtype() == torch::kFloat32 &&
              state.dim() == 4 && state.size(1) == a.H && state.size(2) == a.d &&
              state.size(3) == a.e, "state must be fp32 [slots, H, d, e]");
  TORCH_CHECK(a.G > 0 && a.H % a.G == 0 && a.d >= 1 && a.e >= 1);
  TORCH_CHECK(a.d <= 512 && a.e <= 1024, "head sizes up to 512 x 1024");
  TORCH_CHECK(starts.dtype() == torch::kInt32 && slots.dtype() == torch::kInt32 &&
              starts.numel() == slots.numel() && starts.is_contiguous());
  TORCH_CHECK(out.dtype() == proj.dtype() && out.size(0) == proj.size(0) &&
              out.stride(1) == 1);
}

template <int MODE>
static void run_prefill(RecArgs a, const torch::Tensor& proj, const torch::Tensor& cu,
                        const torch::Tensor& cseq, const torch::Tensor& coff,
                        const torch::Tensor& cfirst) {
  const int NC = cseq.numel(), S = cu.numel() - 1;
  const long T_ = proj.size(0);
  TORCH_CHECK(cu.dtype() == torch::kInt32 && cseq.dtype() == torch::kInt32 &&
              coff.dtype() == torch::kInt32 && cfirst.dtype() == torch::kInt32 &&
              coff.numel() == NC && cfirst.numel() == S + 1);
  if (T_ == 0 || NC == 0) return;
  const int dp = (a.d + 15) / 16 * 16;
  const long WH = (long)NC * a.H, HE = (long)a.H * a.e;
  auto f32 = proj.options().dtype(torch::kFloat32);
  auto vf = torch::empty({T_, HE}, f32), of = torch::empty({T_, HE}, f32);
  // one workspace: q~ [k~] k^ g A [T] [log gates, maxima, denominators]
  constexpr bool RULE = is_delta(MODE);
  const long nq = WH * CHUNK * dp, ng = WH * dp, na = WH * 256, TH = T_ * a.H;
  const long total = nq * (RULE ? 3 : 2) + ng + na * (RULE ? 2 : 1) +
                     (MODE == MEMORY ? 4 * TH + (long)S * a.H : 0);
  auto space = torch::empty({total}, f32);
  ChunkSpace w;
  float* p = space.data_ptr<float>();
  auto take = [&](long n) { float* r = p; p += n; return r; };
  w.dp = dp;
  w.q = take(nq);
  w.k = RULE ? take(nq) : nullptr;
  w.kt = take(nq);
  w.g = take(ng);
  w.a = take(na);
  w.t = RULE ? take(na) : nullptr;
  GateSpace mg = {};
  float* den = nullptr;
  if (MODE == MEMORY) {
    mg.f = take(TH);
    mg.i = take(TH);
    mg.m = take(TH);
    den = take(TH);
    mg.m0 = take((long)S * a.H);
  }
  auto stream = CUR_STREAM;
  const int* cup = cu.data_ptr<int>();
  const int* sp = cseq.data_ptr<int>();
  const int* op = coff.data_ptr<int>();
  const size_t lds = (size_t)(MODE == DELTA ? 3 : 2) * CHUNK * (dp + 4) * 4;
  DISPATCH_ELEM(proj.dtype() == torch::kBFloat16, {
    if constexpr (MODE == MEMORY)
      hipLaunchKernelGGL((memory_gates_kernel<T>), dim3(a.H, S), dim3(1024), 0, stream, a,
                         cup, mg);
    hipLaunchKernelGGL((value_prepare_kernel<T, MODE>), dim3(NC, (HE + 255) / 256),
                       dim3(256), 0, stream, a, cup, sp, op, vf.data_ptr<float>());
    if (lds > 48 * 1024)
      (void)hipFuncSetAttribute((const void*)chunk_prepare_kernel<T, MODE>,
                                hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds);
    hipLaunchKernelGGL((chunk_prepare_kernel<T, MODE>), dim3(NC, a.H), dim3(256), lds,
                       stream, a, cup, sp, op, w, mg);
  });
  const int NE = (a.e + (MODE == MEMORY) + 15) / 16;
  const dim3 grid((S * a.H + 7) / 8 * 8 * NE);
#define SCAN(N)                                                                  \
  hipLaunchKernelGGL((chunk_scan_kernel<MODE, N>), grid, dim3(256), 0, stream, a, \
                     cup, cfirst.data_ptr<int>(), w, vf.data_ptr<float>(),       \
                     of.data_ptr<float>(), den, S)
  if (dp <= 64) SCAN(1);
  else if (dp <= 128) SCAN(2);
  else if (dp <= 256) SCAN(4);
  else SCAN(8);
#undef SCAN
  DISPATCH_ELEM(proj.dtype() == torch::kBFloat16, {
    if (RULE)
      hipLaunchKernelGGL((ring_update_kernel<T>),
                         dim3((2 * a.G * a.d + a.H * a.e + 255) / 256, S), dim3(256), 0,
                         stream, a, cup);
    const bool four = ((a.e | a.gstride | a.ostride) & 3) == 0 && a.e <= 256 &&
                      (((size_t)a.out | (size_t)a.gate) & 15) % (4 * sizeof(T)) == 0;
    auto finish = [&](auto kern, int per) {
      hipLaunchKernelGGL(kern, dim3((TH + per - 1) / per), dim3(256), 0, stream, a,
                         of.data_ptr<float>(), den, mg.m, TH);
    };
    if (four && a.e <= 128) finish(head_norm_gate4_kernel<T, MODE, 32>, 8);
    else if (four) finish(head_norm_gate4_kernel<T, MODE, 64>, 4);
    else finish(head_norm_gate_kernel<T, MODE>, 4);
  });
  HIP_CHECK_KERNEL();
}

template <int MODE>
static void run_decode(RecArgs a, const torch::Tensor& proj) {
  const int B = proj.size(0);
  if (B == 0) return;
  const int VW = a.e % 4 == 0 ? 4 : 1;
  int CG = 1;
  while (CG * VW < a.e) CG *= 2;
  int NT = 256;
  while (NT < 1024 && (NT < CG || (a.d + NT / CG - 1) / (NT / CG) > 16)) NT *= 2;
  TORCH_CHECK(CG <= NT, "value width ", a.e, " not supported");
  const int rows = (a.d + NT / CG - 1) / (NT / CG);
  const size_t lds = (size_t)(3 * a.d + CG * VW + NT * VW) * 4;
  auto stream = CUR_STREAM;
  DISPATCH_ELEM(proj.dtype() == torch::kBFloat16, {
    auto launch = [&](auto kern) {
      hipLaunchKernelGGL(kern, dim3(a.H, B), dim3(NT), lds, stream, a, CG);
    };
    if (VW == 4) {
      if (rows <= 4) launch(recurrence_decode_kernel<T, MODE, 4, 4>);
      else if (rows <= 16) launch(recurrence_decode_kernel<T, MODE, 4, 16>);
      else if (rows <= 32) launch(recurrence_decode_kernel<T, MODE, 4, 32>);
      else TORCH_CHECK(false, "state ", a.d, " x ", a.e, " too large per head");
    } else {
      if (rows <= 16) launch(recurrence_decode_kernel<T, MODE, 1, 16>);
      else if (rows <= 128) launch(recurrence_decode_kernel<T, MODE, 1, 128>);
      else TORCH_CHECK(false, "state ", a.d, " x ", a.e, " too large per head");
    }
  });
  HIP_CHECK_KERNEL();
}

static const void* column(const torch::Tensor& t, long c) {
  return (const char*)t.data_ptr() + c * t.element_size();
}

// all but the decay's and the gate's pre-activations
static RecArgs rule_args(const torch::Tensor& proj,
                         const torch::Tensor& conv_w, const torch::Tensor& a_log,
                         const torch::Tensor& dt_bias, const torch::Tensor& norm,
                         long H, long G, long d, long e, long taps, long q0, long k0,
                         long v0, long b0, double eps, const torch::Tensor& state,
                         const torch::Tensor& ring, const torch::Tensor& starts,
                         const torch::Tensor& slots, const torch::Tensor& out, long col,
                         double oscale) {
  RecArgs a = {};
  a.proj = proj.data_ptr();
  a.stride = proj.stride(0);
  a.q0 = q0; a.k0 = k0; a.v0 = v0; a.b0 = b0;
  a.H = H; a.G = G; a.d = d; a.e = e; a.taps = taps;
  check_common(a, proj, state, starts, slots, out);
  for (auto* t : {&conv_w, &a_log, &dt_bias, &norm})
    TORCH_CHECK(t->dtype() == torch::kFloat32 && t->is_contiguous());
  const long C = 2 * G * d + H * e;
  TORCH_CHECK(taps >= 1 && taps <= MAX_TAPS, "convolution taps 1..", MAX_TAPS);
  TORCH_CHECK(conv_w.numel() == C * taps && a_log.numel() == H && norm.numel() == e);
  TORCH_CHECK(ring.is_contiguous() && ring.dtype() == proj.dtype() &&
              ring.size(0) == state.size(0) && ring.size(1) == taps && ring.size(2) == C);
  TORCH_CHECK(std::max({q0 + G * d, k0 + G * d, v0 + H * e, b0 + H}) <= proj.size(1) &&
              col + H * e <= out.size(1));
  a.conv_w = conv_w.data_ptr<float>();
  a.a_log = a_log.data_ptr<float>();
  a.dt_bias = dt_bias.data_ptr<float>();
  a.norm = norm.data_ptr<float>();
  a.eps = eps;
  a.state = state.data_ptr<float>();
  a.ring = ring.data_ptr();
  a.starts = starts.data_ptr<int>();
  a.slots = slots.data_ptr<int>();
  a.out = (char*)out.data_ptr() + col * out.element_size();
  a.ostride = out.stride(0);
  a.oscale = oscale;
  return a;
}

static RecArgs delta_args(const torch::Tensor& proj, const torch::Tensor& z,
                          const torch::Tensor& conv_w, const torch::Tensor& a_log,
                          const torch::Tensor& dt_bias, const torch::Tensor& norm,
                          long H, long G, long d, long e, long taps, long q0, long k0,
                          long v0, long b0, double eps, const torch::Tensor& state,
                          const torch::Tensor& ring, const torch::Tensor& starts,
                          const torch::Tensor& slots, const torch::Tensor& out, long col,
                          double oscale) {
  auto a = rule_args(proj, conv_w, a_log, dt_bias, norm, H, G, d, e, taps, q0, k0, v0, b0,
                     eps, state, ring, starts, slots, out, col, oscale);
  TORCH_CHECK(dt_bias.numel() == H * d);
  TORCH_CHECK(z.dtype() == proj.dtype() && z.stride(1) == 1 &&
              z.size(0) == proj.size(0) && z.size(1) == H * (d + e));
  a.z = z.data_ptr();
  a.gate = column(z, H * d);
  a.zstride = a.gstride = z.stride(0);
  return a;
}

static RecArgs head_delta_args(const torch::Tensor& proj, const torch::Tensor& conv_w,
                               const torch::Tensor& a_log, const torch::Tensor& dt_bias,
                               const torch::Tensor& norm, long H, long G, long d, long e,
                               long taps, long q0, long k0, long v0, long b0, long a0,
                               long g0, double eps, const torch::Tensor& state,
                               const torch::Tensor& ring, const torch::Tensor& starts,
                               const torch::Tensor& slots, const torch::Tensor& out,
                               long col, double oscale) {
  auto a = rule_args(proj, conv_w, a_log, dt_bias, norm, H, G, d, e, taps, q0, k0, v0, b0,
                     eps, state, ring, starts, slots, out, col, oscale);
  TORCH_CHECK(dt_bias.numel() == H && a0 + H <= proj.size(1) && g0 + H * e <= proj.size(1));
  a.z = column(proj, a0);
  a.gate = column(proj, g0);
  a.zstride = a.gstride = proj.stride(0);
  return a;
}

void delta_prefill(torch::Tensor proj, torch::Tensor z, torch::Tensor conv_w,
                   torch::Tensor a_log, torch::Tensor dt_bias, torch::Tensor norm,
                   long H, long G, long d, long e, long taps, long q0, long k0, long v0,
                   long b0, double eps, torch::Tensor state, torch::Tensor ring,
                   torch::Tensor cu, torch::Tensor cseq, torch::Tensor coff,
                   torch::Tensor cfirst, torch::Tensor starts, torch::Tensor slots,
                   torch::Tensor out, long col, double oscale) {
  auto a = delta_args(proj, z, conv_w, a_log, dt_bias, norm, H, G, d, e, taps, q0, k0,
                      v0, b0, eps, state, ring, starts, slots, out, col, oscale);
  TORCH_CHECK(starts.numel() == cu.numel() - 1);
  run_prefill<DELTA>(a, proj, cu, cseq, coff, cfirst);
}

void delta_decode(torch::Tensor proj, torch::Tensor z, torch::Tensor conv_w,
                  torch::Tensor a_log, torch::Tensor dt_bias, torch::Tensor norm,
                  long H, long G, long d, long e, long taps, long q0, long k0, long v0,
                  long b0, double eps, torch::Tensor state, torch::Tensor ring,
                  torch::Tensor starts, torch::Tensor slots, torch::Tensor out, long col,
                  double oscale) {
  auto a = delta_args(proj, z, conv_w, a_log, dt_bias, norm, H, G, d, e, taps, q0, k0,
                      v0, b0, eps, state, ring, starts, slots, out, col, oscale);
  TORCH_CHECK(starts.numel() == proj.size(0));
  run_decode<DELTA>(a, proj);
}

void head_delta_prefill(torch::Tensor proj, torch::Tensor conv_w, torch::Tensor a_log,
                        torch::Tensor dt_bias, torch::Tensor norm, long H, long G, long d,
                        long e, long taps, long q0, long k0, long v0, long b0, long a0,
                        long g0, double eps, torch::Tensor state, torch::Tensor ring,
                        torch::Tensor cu, torch::Tensor cseq, torch::Tensor coff,
                        torch::Tensor cfirst, torch::Tensor starts, torch::Tensor slots,
                        torch::Tensor out, long col, double oscale) {
  auto a = head_delta_args(proj, conv_w, a_log, dt_bias, norm, H, G, d, e, taps, q0, k0, v0,
                           b0, a0, g0, eps, state, ring, starts, slots, out, col, oscale);
  TORCH_CHECK(starts.numel() == cu.numel() - 1);
  run_prefill<HEAD_DELTA>(a, proj, cu, cseq, coff, cfirst);
}

void head_delta_decode(torch::Tensor proj, torch::Tensor conv_w, torch::Tensor a_log,
                       torch::Tensor dt_bias, torch::Tensor norm, long H, long G, long d,
                       long e, long taps, long q0, long k0, long v0, long b0, long a0,
                       long g0, double eps, torch::Tensor state, torch::Tensor ring,
                       torch::Tensor starts, torch::Tensor slots, torch::Tensor out,
                       long col, double oscale) {
  auto a = head_delta_args(proj, conv_w, a_log, dt_bias, norm, H, G, d, e, taps, q0, k0, v0,
                           b0, a0, g0, eps, state, ring, starts, slots, out, col, oscale);
  TORCH_CHECK(starts.numel() == proj.size(0));
  run_decode<HEAD_DELTA>(a, proj);
}

static RecArgs memory_args(const torch::Tensor& proj, const torch::Tensor& i_bias,
                           const torch::Tensor& f_bias, const torch::Tensor& norm, long H,
                           long d, long e, long q0, long k0, long v0, long i0, long f0,
                           long g0, double cap, double eps, const torch::Tensor& state,
                           const torch::Tensor& nstate, const torch::Tensor& mstate,
                           const torch::Tensor& starts, const torch::Tensor& slots,
                           const torch::Tensor& out, long col, double oscale) {
  RecArgs a = {};
  a.proj = proj.data_ptr();
  a.stride = proj.stride(0);
  a.q0 = q0; a.k0 = k0; a.v0 = v0; a.i0 = i0; a.f0 = f0;
  a.H = H; a.G = H; a.d = d; a.e = e;
  check_common(a, proj, state, starts, slots, out);
  for (auto* t : {&i_bias, &f_bias, &norm, &nstate, &mstate})
    TORCH_CHECK(t->dtype() == torch::kFloat32 && t->is_contiguous());
  TORCH_CHECK(i_bias.numel() == H && f_bias.numel() == H && norm.numel() == H * e);
  TORCH_CHECK(nstate.dim() == 3 && nstate.size(0) == state.size(0) && nstate.size(1) == H &&
              nstate.size(2) == d && mstate.dim() == 2 && mstate.size(0) == state.size(0) &&
              mstate.size(1) == H, "normalisers [slots, H, d], maxima [slots, H]");
  TORCH_CHECK(std::max({q0 + H * d, k0 + H * d, v0 + H * e, g0 + H * e, i0 + H, f0 + H}) <=
                  proj.size(1) && col + H * e <= out.size(1));
  TORCH_CHECK(cap > 0, "gate cap");
  a.i_bias = i_bias.data_ptr<float>();
  a.f_bias = f_bias.data_ptr<float>();
  a.norm = norm.data_ptr<float>();
  a.gate = column(proj, g0);
  a.gstride = proj.stride(0);
  a.cap = cap;
  a.eps = eps;
  a.state = state.data_ptr<float>();
  a.nstate = nstate.data_ptr<float>();
  a.mstate = mstate.data_ptr<float>();
  a.starts = starts.data_ptr<int>();
  a.slots = slots.data_ptr<int>();
  a.out = (char*)out.data_ptr() + col * out.element_size();
  a.ostride = out.stride(0);
  a.oscale = oscale;
  return a;
}

void memory_prefill(torch::Tensor proj, torch::Tensor i_bias, torch::Tensor f_bias,
                    torch::Tensor norm, long H, long d, long e, long q0, long k0, long v0,
                    long i0, long f0, long g0, double cap, double eps, torch::Tensor state,
                    torch::Tensor nstate, torch::Tensor mstate, torch::Tensor cu,
                    torch::Tensor cseq, torch::Tensor coff, torch::Tensor cfirst,
                    torch::Tensor starts, torch::Tensor slots, torch::Tensor out, long col,
                    double oscale) {
  auto a = memory_args(proj, i_bias, f_bias, norm, H, d, e, q0, k0, v0, i0, f0, g0, cap, eps,
                       state, nstate, mstate, starts, slots, out, col, oscale);
  TORCH_CHECK(starts.numel() == cu.numel() - 1);
  run_prefill<MEMORY>(a, proj, cu, cseq, coff, cfirst);
}

void memory_decode(torch::Tensor proj, torch::Tensor i_bias, torch::Tensor f_bias,
                   torch::Tensor norm, long H, long d, long e, long q0, long k0, long v0,
                   long i0, long f0, long g0, double cap, double eps, torch::Tensor state,
                   torch::Tensor nstate, torch::Tensor mstate, torch::Tensor starts,
                   torch::Tensor slots, torch::Tensor out, long col, double oscale) {
  auto a = memory_args(proj, i_bias, f_bias, norm, H, d, e, q0, k0, v0, i0, f0, g0, cap, eps,
                       state, nstate, mstate, starts, slots, out, col, oscale);
  TORCH_CHECK(starts.numel() == proj.size(0));
  run_decode<MEMORY>(a, proj);
}

static RecArgs retention_args(const torch::Tensor& proj, const torch::Tensor& decay,
                              const torch::Tensor& cos_sin, long H, long d, long e,
                              long rot, long q0, long k0, long v0, long g0, double eps,
                              const torch::Tensor& state, const torch::Tensor& starts,
                              const torch::Tensor& slots, const torch::Tensor& out) {
  RecArgs a = {};
  a.proj = proj.data_ptr();
  a.stride = proj.stride(0);
  a.q0 = q0; a.k0 = k0; a.v0 = v0;
  a.gate = column(proj, g0);
  a.gstride = proj.stride(0);
  a.H = H; a.G = H; a.d = d; a.e = e; a.rot = rot;
  check_common(a, proj, state, starts, slots, out);
  TORCH_CHECK(decay.dtype() == torch::kFloat32 && decay.numel() == H);
  TORCH_CHECK(rot % 2 == 0 && rot <= d && cos_sin.dtype() == torch::kFloat32 &&
              cos_sin.is_contiguous() && cos_sin.size(1) == rot);
  TORCH_CHECK(std::max({q0 + H * d, k0 + H * d, v0 + H * e, g0 + H * e}) <= proj.size(1) &&
              H * e <= out.size(1));
  a.decay = decay.data_ptr<float>();
  a.cos_sin = cos_sin.data_ptr<float>();
  a.eps = eps;
  a.state = state.data_ptr<float>();
  a.starts = starts.data_ptr<int>();
  a.slots = slots.data_ptr<int>();
  a.out = out.data_ptr();
  a.ostride = out.stride(0);
  a.oscale = 1.f;
  return a;
}

void retention_prefill(torch::Tensor proj, torch::Tensor decay, torch::Tensor cos_sin,
                       long H, long d, long e, long rot, long q0, long k0, long v0,
                       long g0, double eps, torch::Tensor state, torch::Tensor cu,
                       torch::Tensor cseq, torch::Tensor coff, torch::Tensor cfirst,
                       torch::Tensor starts, torch::Tensor slots, torch::Tensor out) {
  auto a = retention_args(proj, decay, cos_sin, H, d, e, rot, q0, k0, v0, g0, eps, state,
                          starts, slots, out);
  TORCH_CHECK(starts.numel() == cu.numel() - 1);
  run_prefill<RETAIN>(a, proj, cu, cseq, coff, cfirst);
}

void retention_decode(torch::Tensor proj, torch::Tensor decay, torch::Tensor cos_sin,
                      long H, long d, long e, long rot, long q0, long k0, long v0,
                      long g0, double eps, torch::Tensor state, torch::Tensor starts,
                      torch::Tensor slots, torch::Tensor out) {
  auto a = retention_args(proj, decay, cos_sin, H, d, e, rot, q0, k0, v0, g0, eps, state,
                          starts, slots, out);
  TORCH_CHECK(starts.numel() == proj.size(0));
  run_decode<RETAIN>(a, proj);
}
