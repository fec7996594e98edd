// Flash-style causal prefill attention over the paged KV cache (gfx950).
//
// MFMA structure (CDNA4, v_mfma_f32_32x32x16_bf16):
//  * swapped QK^T — compute S^T = mfma(A=K-tile, B=Q^T-tile) so each lane
//    owns ONE q column (q = lane&31) and the softmax row-reduce is
//    per-lane over registers + one shfl_xor(32) with its half-wave partner
//    (no cross-lane softmax, no P staging through LDS);
//  * P -> PV A-fragments in-register via bf16 packing + v_permlane32_swap
//    (the cvt_pk/permlane redistribution idiom);
//  * K tile staged in LDS row-major with the ((row&15)<<4) XOR byte-swizzle
//    (ds_read_b128 would otherwise be up-to-16-way bank-conflicted at
//    D=128); V staged TRANSPOSED [D][KVBLK+8] so the PV B-fragment read is
//    a contiguous 16-B ds_read per lane;
//  * O accumulates in registers (col d = lane&31 per d-tile); the epilogue
//    transposes through LDS so global stores are coalesced 16-B rows.
//
// Geometry: 8 waves/WG (512 threads); the WG covers HG = min(G, 4) query
// heads of ONE kv head x (8/HG)*32 query rows, so every staged K/V tile
// feeds 8 waves of MFMA (GQA heads share the stage — staging bandwidth was
// the 156-TF bound of the 4-wave/1-head structure).  KV tiles of 64 keys,
// two 32-key MFMA steps each.
// BIAS adds a per-head distance penalty, linear, logarithmic or none, and a sliding
// window or chunks of positions (tiles and MFMA steps wholly outside of what a wave
// sees are skipped), lets keys and values differ in width, and writes scaled columns
// of a wider output. A sink starts every row's softmax from a term without key or
// value. EXTRA: GATED takes a sink and multiplies the head by a sigmoid gate; TAILED
// takes a key's last dimensions from a row that all heads share; TURNED turns the
// result back and gates its channels, in fp32 (head_turn.h).
// Covers fresh prefill and append-prefill (chunked agent turns) since K/V
// are read from the paged cache with an absolute-position causal bound.
#include "head_turn.h"
#include <torch/extension.h>
#include <c10/hip/HIPStream.h>

#define CUR_STREAM c10::hip::getCurrentHIPStream().stream()

typedef __attribute__((ext_vector_type(4))) float f32x4;

DEVINL unsigned int pack2_bf16(float lo, float hi) {
  return ((unsigned int)f32_to_bf16(hi) << 16) | f32_to_bf16(lo);
}

#define LN2 0.69314718f  // the hardware's logarithm has base 2
enum { NO_BIAS = 0, LINEAR_BIAS = 1, LOG_BIAS = 2, FLAT_BIAS = 3 };
enum { PLAIN = 0, GATED = 1, TAILED = 2, TURNED = 3 };
#define TURN_STRIDE 40  // row stride of a wave's 32 x 32 results in LDS

// shared last dimensions of the keys: key t's are row t, its own come first in kc
struct KeyTail {
  const __hip_bfloat16* rows;
  long stride;
  int width;  // columns there are; the rest of D is zeros
  int own;    // dimensions in kc, a multiple of 8
};

union frag_u {
  unsigned int u[4];
  bf16x8 v;
};

template <int D, int DV, int HG, bool FP8, int BIAS, int EXTRA>  // HG = query heads per workgroup
__global__ __launch_bounds__(512, 1) void prefill_kernel(
    const __hip_bfloat16* __restrict__ q,   // [T, qstride], heads D apart
    const void* __restrict__ kc,  // [NP, Hkv, P, D] bf16 | fp8 e4m3
    const void* __restrict__ vc,
    __hip_bfloat16* __restrict__ out,       // [T, ostride], heads dv apart
    const int* __restrict__ block_seq,      // [NB] seq index of this q-block
    const int* __restrict__ block_qoff,     // [NB] q-row offset within the seq
    const int* __restrict__ cu_q,           // [S+1]
    const int* __restrict__ block_tables,   // [S, MP]
    const int* __restrict__ ctx_lens,       // [S]
    int Hq, int Hkv, int P, int MP, float scale,
    long qstride, long ostride, int dv, float oscale,
    const float* __restrict__ slopes, const float* __restrict__ rates, int window,
    int chunk, const float* __restrict__ sink,  // [Hq], or null unless GATED
    const __hip_bfloat16* __restrict__ gate, long gstride,  // [T, gstride]
    KeyTail tail, HeadTurn turn) {
  constexpr int KVB = 64;           // keys staged per tile
  constexpr int NC = D / 16;        // Q^T fragments (MFMA K-chunks of QK^T)
  constexpr int NDT = DV / 32;      // 32-wide d-tiles of O
  constexpr int VROW = KVB + 8;     // padded V^T row length (elements)
  // K-tile XOR swizzle mask: a row has D/8 16-B slots, so the swizzle may
  // only permute within that many slots (at D=64, (row&15)<<4 would escape
  // the 128-B row)
  // (at D=192 a row is 1.5 times all banks: pairs of rows share a permutation)
  constexpr int SWZ = D == 192 ? 7 : (D / 8) - 1;
  constexpr int SWZ_SHIFT = D == 192 ? 1 : 0;
  constexpr int QS = 8 / HG;          // 32-row q sub-blocks per WG
  const int nb = gridDim.x - 1 - blockIdx.x;  // late rows see most keys: first
  const int seq = block_seq[nb];
  const int qoff = block_qoff[nb];
  const int q_start = cu_q[seq];
  const int qlen = cu_q[seq + 1] - q_start;
  const int ctx = ctx_lens[seq];
  const int* bt = block_tables + (long)seq * MP;

  const int tid = threadIdx.x;
  const int wave = tid / WAVE;
  const int lane = tid % WAVE;
  const int col = lane & 31;   // q column owned by this lane (within wave's 32)
  const int half = lane >> 5;  // half-wave
  // wave -> (query head, q sub-block): heads vary fastest so the HG heads
  // of one sub-block sit on consecutive waves
  const int h = blockIdx.y * HG + (wave % HG);
  const int kvh = h / (Hq / Hkv);
  const int qsub = wave / HG;

  extern __shared__ __attribute__((aligned(16))) char smem[];
  short* kbuf = (short*)smem;                       // [KVB][D] XOR-swizzled
  short* vtbuf = (short*)(smem + KVB * D * 2);      // [D][VROW] transposed
  // [8][32] after K, V^T and the epilogue's four 32 x DV tiles
  float* scratch = (float*)(smem + max(KVB * D * 2 + DV * VROW * 2, 256 * DV));
  float* wsc = scratch + wave * 32;

  // ---- Q fragments (B-operand of swapped QK^T): held for the whole block
  const int qrow = qoff + qsub * 32 + col;  // local q row in this seq
  const bool qvalid = qrow < qlen;
  const long qbase = (q_start + (qvalid ? qrow : 0)) * qstride + (long)h * D;
  frag_u qf[NC];
#pragma unroll
  for (int c = 0; c < NC; ++c) {
    if (qvalid) {
      const shortx8 v =
          *reinterpret_cast<const shortx8*>(q + qbase + c * 16 + half * 8);
      qf[c].u[0] = ((const unsigned int*)&v)[0];
      qf[c].u[1] = ((const unsigned int*)&v)[1];
      qf[c].u[2] = ((const unsigned int*)&v)[2];
      qf[c].u[3] = ((const unsigned int*)&v)[3];
    } else {
      qf[c].u[0] = qf[c].u[1] = qf[c].u[2] = qf[c].u[3] = 0u;
    }
  }

  const int q_abs = ctx - qlen + qrow;  // absolute position of this lane's q
  const bool has_sink = EXTRA == GATED || (BIAS && sink);
  float m = has_sink ? sink[h] : -1e30f, l = has_sink ? 1.f : 0.f;
  floatx16 o[NDT];
#pragma unroll
  for (int dt = 0; dt < NDT; ++dt)
#pragma unroll
    for (int r = 0; r < 16; ++r) o[dt][r] = 0.f;

  // keys needed by this q block: up to the last row's absolute position
  const int blk_rows = min(qlen - qoff, QS * 32);
  const int kend = min(ctx, ctx - qlen + qoff + blk_rows);
  const int ntiles = (kend + KVB - 1) / KVB;
  // absolute position of the wave's first (smallest) q row
  const int q_abs_min = ctx - qlen + qoff + qsub * 32;

  // this head's penalty per token of distance, or of ln(1 + rate * distance);
  // first key any row here sees
  const float slope = BIAS && BIAS != FLAT_BIAS
                          ? slopes[h] * (BIAS == LOG_BIAS ? LN2 : 1.f) : 0.f;
  const float rate = BIAS == LOG_BIAS ? rates[h] : 0.f;
  const int win = BIAS && window > 0 ? window : 0x3fffffff;
  // first key a query at position x sees (negative: all)
  auto first_seen = [&](int x) {
    const int lo = x - win + 1;
    return BIAS && chunk > 0 ? max(lo, x - x % chunk) : lo;
  };
  const int tile0 = BIAS ? max(0, first_seen(ctx - qlen + qoff)) / KVB : 0;
  const int lo = BIAS ? first_seen(q_abs) : 0;
  const int lo_min = BIAS ? first_seen(q_abs_min) : 0;
  const int lo_max = BIAS ? first_seen(q_abs_min + 31) : 0;

  for (int tile = tile0; tile < ntiles; ++tile) {
    const int kbase = tile * KVB;
    // ---- stage K (swizzled) and V^T cooperatively: 512 threads
    __syncthreads();
    auto load8 = [&](const void* cache, long base) -> shortx8 {
      if constexpr (FP8)
        return fp8x8_to_bf16x8(
            *reinterpret_cast<const u64b*>((const unsigned char*)cache + base));
      else
        return *reinterpret_cast<const shortx8*>((const __hip_bfloat16*)cache + base);
    };
#pragma unroll
    for (int i = 0; i < KVB * (D > DV ? D : DV) / (512 * 8); ++i) {
      const int c = tid + i * 512;
      constexpr int W8 = (D > DV ? D : DV) / 8;
      const int row = c / W8;
      const int d0 = (c % W8) * 8;
      const int t = kbase + row;
      shortx8 kv8 = {0, 0, 0, 0, 0, 0, 0, 0};
      shortx8 vv8 = {0, 0, 0, 0, 0, 0, 0, 0};
      if (t < ctx) {
        const long slot = ((long)bt[t / P] * Hkv + kvh) * P + (t % P);
        if constexpr (EXTRA == TAILED) {
          const long key = (long)bt[t / P] * P + t % P;
          if (d0 < tail.own)
            kv8 = load8(kc, slot * tail.own + d0);
          else if (d0 < D && d0 - tail.own < tail.width)
            kv8 = load8(tail.rows, key * tail.stride + d0 - tail.own);
        } else {
          if (D >= DV || d0 < D) kv8 = load8(kc, slot * D + d0);
        }
        if (DV >= D || d0 < DV) vv8 = load8(vc, slot * DV + d0);
      }
      if (D >= DV || d0 < D) {
        const int kb = (row * D * 2 + ((d0 * 2) ^ (((row >> SWZ_SHIFT) & SWZ) << 4))) / 2;
        *reinterpret_cast<shortx8*>(kbuf + kb) = kv8;
      }
      if (DV >= D || d0 < DV) {
#pragma unroll
        for (int j = 0; j < 8; ++j) vtbuf[(d0 + j) * VROW + row] = vv8[j];
      }
    }
    __syncthreads();

    // ---- two 32-key MFMA steps (waves skip steps beyond their causal bound)
    const int wave_kend = min(kend, q_abs_min + 32);
#pragma unroll
    for (int s = 0; s < 2; ++s) {
      const int ks = kbase + s * 32;  // absolute key base of this step
      if (ks >= wave_kend) break;
      if (BIAS && ks + 31 < lo_min) continue;  // before all that the wave sees
      // S^T = K * Q^T : rows k, cols q
      floatx16 st;
#pragma unroll
      for (int r = 0; r < 16; ++r) st[r] = 0.f;
      const int krow = s * 32 + col;  // this lane's A-row in the K tile
#pragma unroll
      for (int c = 0; c < NC; ++c) {
        const int kb =
            (krow * D * 2 +
             (((c * 16 + half * 8) * 2) ^ (((krow >> SWZ_SHIFT) & SWZ) << 4))) / 2;
        frag_u kf;
        const shortx8 kv = *reinterpret_cast<const shortx8*>(kbuf + kb);
        kf.u[0] = ((const unsigned int*)&kv)[0];
        kf.u[1] = ((const unsigned int*)&kv)[1];
        kf.u[2] = ((const unsigned int*)&kv)[2];
        kf.u[3] = ((const unsigned int*)&kv)[3];
        st = __builtin_amdgcn_mfma_f32_32x32x16_bf16(kf.v, qf[c].v, st, 0, 0, 0);
      }
      // ---- mask + scale (S^T reg r holds key row R = (r&3)+8*(r>>2)+4*half)
      float p[16];
      // distance of key row 4 * half, and the logarithm's argument there
      const float dist0 = (float)(q_abs - ks - 4 * half);
      const float arg0 = 1.f + rate * dist0;
      const bool need_mask = (ks + 31 > q_abs_min) || (ks + 31 >= ctx) ||
                             (BIAS && ks < lo_max);
#pragma unroll
      for (int r = 0; r < 16; ++r) {
        const int k_abs = ks + (r & 3) + 8 * (r >> 2) + 4 * half;
        float sv = st[r] * scale;
        if constexpr (BIAS != NO_BIAS) {
          // a row that has seen only masked keys yet holds weights of
          // exp(0); its first visible key rescales them to zero
          const float step = (float)((r & 3) + 8 * (r >> 2));
          if constexpr (BIAS != FLAT_BIAS)
            sv -= slope * (BIAS == LOG_BIAS ? __builtin_amdgcn_logf(arg0 - rate * step)
                                            : dist0 - step);
          if (need_mask && (k_abs > q_abs || k_abs >= ctx || k_abs < lo))
            sv = -1e30f;
        } else {
          if (need_mask && (k_abs > q_abs || k_abs >= ctx)) sv = -3.0e4f;
        }
        p[r] = sv;
      }
      // ---- online softmax (per-lane column view)
      float tmax = p[0];
#pragma unroll
      for (int r = 1; r < 16; ++r) tmax = fmaxf(tmax, p[r]);
      tmax = fmaxf(tmax, __shfl_xor(tmax, 32, WAVE));
      const float mn = fmaxf(m, tmax);
      const float alpha = __expf(m - mn);
      m = mn;
      float psum = 0.f;
#pragma unroll
      for (int r = 0; r < 16; ++r) {
        p[r] = __expf(p[r] - mn);
        psum += p[r];
      }
      psum += __shfl_xor(psum, 32, WAVE);
      l = l * alpha + psum;
      // ---- rescale O by alpha of each O-row's q (broadcast via LDS)
      if (half == 0) wsc[col] = alpha;
      asm volatile("s_waitcnt lgkmcnt(0)" ::: "memory");
      __builtin_amdgcn_sched_barrier(0);
#pragma unroll
      for (int g = 0; g < 4; ++g) {
        const f32x4 av = *reinterpret_cast<const f32x4*>(wsc + 4 * half + 8 * g);
#pragma unroll
        for (int dt = 0; dt < NDT; ++dt) {
#pragma unroll
          for (int j = 0; j < 4; ++j) o[dt][4 * g + j] *= av[j];
        }
      }
      // ---- P -> bf16 A-fragments (pack + permlane32_swap)
      frag_u pf[2];
#pragma unroll
      for (int c = 0; c < 2; ++c) {
        unsigned int a0 = pack2_bf16(p[c * 8 + 0], p[c * 8 + 1]);
        unsigned int a1 = pack2_bf16(p[c * 8 + 2], p[c * 8 + 3]);
        unsigned int b0 = pack2_bf16(p[c * 8 + 4], p[c * 8 + 5]);
        unsigned int b1 = pack2_bf16(p[c * 8 + 6], p[c * 8 + 7]);
        {
          auto r0 = __builtin_amdgcn_permlane32_swap(a0, b0, false, false);
          a0 = r0[0];
          b0 = r0[1];
          auto r1 = __builtin_amdgcn_permlane32_swap(a1, b1, false, false);
          a1 = r1[0];
          b1 = r1[1];
        }
        pf[c].u[0] = a0;
        pf[c].u[1] = a1;
        pf[c].u[2] = b0;
        pf[c].u[3] = b1;
      }
      // ---- PV: O[dt] += P * V  (B-frag = 16-B row read of transposed V)
#pragma unroll
      for (int c = 0; c < 2; ++c) {
#pragma unroll
        for (int dt = 0; dt < NDT; ++dt) {
          const int d = dt * 32 + col;
          const int kloc = s * 32 + c * 16 + half * 8;
          frag_u vf;
          const shortx8 vv =
              *reinterpret_cast<const shortx8*>(vtbuf + d * VROW + kloc);
          vf.u[0] = ((const unsigned int*)&vv)[0];
          vf.u[1] = ((const unsigned int*)&vv)[1];
          vf.u[2] = ((const unsigned int*)&vv)[2];
          vf.u[3] = ((const unsigned int*)&vv)[3];
          o[dt] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(pf[c].v, vf.v, o[dt], 0, 0, 0);
        }
      }
    }
  }

  // ---- epilogue: divide by l (per q row), transpose via LDS, store rows
  if constexpr (EXTRA == GATED) {  // divided by l, times the gate
    const long grow = (q_start + (qvalid ? qrow : 0)) * gstride + h;
    l *= 1.f + __expf(-bf16_to_f32(((const unsigned short*)gate)[grow]));
  }
  if (half == 0) wsc[col] = l;
  asm volatile("s_waitcnt lgkmcnt(0)" ::: "memory");
  __builtin_amdgcn_sched_barrier(0);
  float linv[4][4];
#pragma unroll
  for (int g = 0; g < 4; ++g) {
    const f32x4 lv = *reinterpret_cast<const f32x4*>(wsc + 4 * half + 8 * g);
#pragma unroll
    for (int j = 0; j < 4; ++j) linv[g][j] = oscale / lv[j];
  }
  if constexpr (EXTRA == TURNED) {
    // 32 x 32 results at a time through the wave's own LDS; a lane then holds 16
    // neighbouring channels of one row
    __syncthreads();
    float* ob = (float*)smem + wave * (32 * TURN_STRIDE);
    const int r = lane >> 1, c0 = (lane & 1) * 16, qr = qoff + qsub * 32 + r;
    const long row = q_start + qr;
    const float* cs = turn.cs ? turn.cs + (long)(ctx - qlen + qr) * dv : nullptr;
    const bf16_t* gp = turn.gate ? (const bf16_t*)turn.gate + row * turn.gstride + h * dv
                                 : nullptr;
    bf16_t* orow = (bf16_t*)out + row * ostride + (long)h * dv;
    const bool vec = ((dv | ostride | turn.gstride | ((long)out >> 1) |
                       ((long)turn.gate >> 1)) & 7) == 0;
#pragma unroll
    for (int dt = 0; dt < NDT; ++dt) {
#pragma unroll
      for (int g = 0; g < 4; ++g)
#pragma unroll
        for (int j = 0; j < 4; ++j)
          ob[(j + 8 * g + 4 * half) * TURN_STRIDE + col] = o[dt][4 * g + j] * linv[g][j];
      asm volatile("s_waitcnt lgkmcnt(0)" ::: "memory");
      __builtin_amdgcn_sched_barrier(0);
#pragma unroll
      for (int i = 0; i < 16; i += 8) {
        const int d = dt * 32 + c0 + i;
        if (qr >= qlen || d >= dv) continue;
        float y[8];
        const float* src = ob + r * TURN_STRIDE + c0 + i;
#pragma unroll
        for (int k = 0; k < 8; ++k) y[k] = src[k];
        if (vec) {
          if (cs) {
            const floatx4 c = ld4(cs + d / 2), sn = ld4(cs + (dv + d) / 2);
#pragma unroll
            for (int k = 0; k < 4; ++k) turn_pair(y[2 * k], y[2 * k + 1], c[k], -sn[k]);
          }
          if (gp) {
            const shortx8 gv = *reinterpret_cast<const shortx8*>(gp + d);
#pragma unroll
            for (int k = 0; k < 8; ++k) y[k] *= sigmoid_f(bf16_to_f32((unsigned short)gv[k]));
          }
          shortx8 v;
#pragma unroll
          for (int k = 0; k < 8; ++k) v[k] = (short)f32_to_bf16(y[k]);
          *reinterpret_cast<shortx8*>(orow + d) = v;
        } else {
#pragma unroll
          for (int k = 0; k < 8; k += 2) {
            if (cs && d + k < dv)
              turn_pair(y[k], y[k + 1], cs[(d + k) / 2], -cs[(dv + d + k) / 2]);
#pragma unroll
            for (int x = k; x < k + 2; ++x)
              if (d + x < dv) stf(orow + d + x, gp ? y[x] * sigmoid_f(ldf(gp + d + x)) : y[x]);
          }
        }
      }
    }
    return;
  }
  // everyone done with K/V buffers; reuse as O staging in two rounds of
  // 4 waves (8 waves' staging would not fit the K+V area)
#pragma unroll
  for (int round = 0; round < 2; ++round) {
    __syncthreads();
    if ((wave >> 2) != round) continue;
    short* obuf = (short*)smem + (wave & 3) * 32 * DV;
#pragma unroll
    for (int dt = 0; dt < NDT; ++dt) {
      const int d = dt * 32 + col;
#pragma unroll
      for (int g = 0; g < 4; ++g) {
#pragma unroll
        for (int j = 0; j < 4; ++j) {
          const int r = (j) + 8 * g + 4 * half;  // q row within the wave's 32
          obuf[r * DV + d] = (short)f32_to_bf16(o[dt][4 * g + j] * linv[g][j]);
        }
      }
    }
    asm volatile("s_waitcnt lgkmcnt(0)" ::: "memory");
    __builtin_amdgcn_sched_barrier(0);
    // each lane stores half a row (DV/2 elems = DV bytes) with 16-B stores
    const int r = lane >> 1;            // 0..31
    const int seg = (lane & 1) * (DV / 2);
    const int qr = qoff + qsub * 32 + r;
    if (qr < qlen) {
      __hip_bfloat16* orow = out + (long)(q_start + qr) * ostride + (long)h * dv;
      if (!BIAS || ((dv | ostride | ((long)out >> 1)) & 7) == 0) {
#pragma unroll
        for (int i = 0; i < DV / 16; ++i) {
          if (BIAS && seg + i * 8 >= dv) break;
          const shortx8 v =
              *reinterpret_cast<const shortx8*>(obuf + r * DV + seg + i * 8);
          *reinterpret_cast<shortx8*>(orow + seg + i * 8) = v;
        }
      } else {  // head width or column not a multiple of 8
        for (int i = seg; i < min(dv, seg + DV / 2); ++i)
          *(short*)(orow + i) = obuf[r * DV + i];
      }
    }
  }
}

// query heads per workgroup: the GQA group shares each staged K/V tile
static int heads_per_block(int G) { return G % 4 == 0 ? 4 : G % 2 == 0 ? 2 : 1; }

template <int D, int DV>
static size_t prefill_lds() {
  return std::max<size_t>(64 * D * 2 + DV * (64 + 8) * 2, 256 * DV) + 8 * 32 * 4;
}
template <int D, int DV>
static size_t turned_lds() {
  return std::max<size_t>(prefill_lds<D, DV>(), 8 * 32 * TURN_STRIDE * 4);
}

torch::Tensor attention_prefill_paged(torch::Tensor q, torch::Tensor kc,
                                      torch::Tensor vc, torch::Tensor bt,
                                      torch::Tensor cu_q, torch::Tensor ctx,
                                      double scale) {
  TORCH_CHECK(q.is_cuda() && q.dtype() == torch::kBFloat16, "bf16 GPU only");
  const int T = q.size(0), Hq = q.size(1), D = q.size(2);
  const int Hkv = kc.size(1), P = kc.size(2), MP = bt.size(1);
  TORCH_CHECK(D == 128 || D == 64, "head_dim must be 64 or 128, got ", D);
  auto out = torch::empty_like(q);
  if (T == 0) return out;
  TORCH_CHECK(Hq % Hkv == 0, "GQA requires Hq % Hkv == 0");
  const int HG = heads_per_block(Hq / Hkv);
  const int QROWS = 32 * (8 / HG);  // q rows covered per workgroup
  // host-side q-block map (cu_q is tiny; engine built it on CPU this step)
  auto cu_cpu = cu_q.to(torch::kCPU);
  const int* cu = cu_cpu.data_ptr<int>();
  const int S = cu_cpu.numel() - 1;
  std::vector<int> bseq, boff;
  for (int s = 0; s < S; ++s) {
    const int qlen = cu[s + 1] - cu[s];
    for (int off = 0; off < qlen; off += QROWS) {
      bseq.push_back(s);
      boff.push_back(off);
    }
  }
  const int NB = bseq.size();
  auto opts = torch::TensorOptions().dtype(torch::kInt32).device(q.device());
  auto bseq_t = torch::from_blob(bseq.data(), {NB}, torch::kInt32).to(opts.device());
  auto boff_t = torch::from_blob(boff.data(), {NB}, torch::kInt32).to(opts.device());

  const bool fp8 = kc.dtype() == torch::kFloat8_e4m3fn;
  dim3 grid(NB, Hq / HG), block(512);
  auto stream = CUR_STREAM;
#define PLAUNCH1(DD, HGV, F8)                                                 \
  hipLaunchKernelGGL((prefill_kernel<DD, DD, HGV, F8, NO_BIAS, PLAIN>), grid, block,   \
                     (prefill_lds<DD, DD>()), stream,                         \
                     (const __hip_bfloat16*)q.data_ptr(),                     \
                     kc.data_ptr(), vc.data_ptr(),                            \
                     (__hip_bfloat16*)out.data_ptr(),                         \
                     bseq_t.data_ptr<int>(), boff_t.data_ptr<int>(),          \
                     cu_q.data_ptr<int>(), bt.data_ptr<int>(),                \
                     ctx.data_ptr<int>(), Hq, Hkv, P, MP, (float)scale,       \
                     (long)Hq * D, (long)Hq * D, D, 1.f, nullptr, nullptr, 0, \
                     0, nullptr, nullptr, 0, KeyTail{}, HeadTurn{})
#define PLAUNCH(DD, HGV)                                                      \
  if (fp8) { PLAUNCH1(DD, HGV, true); } else { PLAUNCH1(DD, HGV, false); }
#define PLAUNCH_D(DD)                                                         \
  switch (HG) {                                                               \
    case 1: PLAUNCH(DD, 1); break;                                            \
    case 2: PLAUNCH(DD, 2); break;                                            \
    default: PLAUNCH(DD, 4); break;                                           \
  }
  if (D == 128) {
    PLAUNCH_D(128)
  } else {
    PLAUNCH_D(64)
  }
#undef PLAUNCH_D
#undef PLAUNCH
#undef PLAUNCH1
  HIP_CHECK_KERNEL();
  return out;
}

// query rows one workgroup of biased_attention_prefill covers
long biased_prefill_rows(long G) { return 32 * (8 / heads_per_block((int)G)); }

void biased_attention_prefill(torch::Tensor q, torch::Tensor kc, torch::Tensor vc,
                              torch::Tensor bt, torch::Tensor cu_q, torch::Tensor ctx,
                              torch::Tensor bseq, torch::Tensor boff, double scale,
                              long window, long chunk, c10::optional<torch::Tensor> slopes,
                              c10::optional<torch::Tensor> rates,
                              c10::optional<torch::Tensor> sink,
                              c10::optional<torch::Tensor> turn,
                              c10::optional<torch::Tensor> gate, torch::Tensor out,
                              long col, long dv, double oscale) {
  TORCH_CHECK(q.is_cuda() && q.dtype() == torch::kBFloat16 && q.is_contiguous());
  const int T = q.size(0), Hq = q.size(1), D = q.size(2);
  const int Hkv = kc.size(1), P = kc.size(2), MP = bt.size(1), DV = vc.size(3);
  TORCH_CHECK(Hq % Hkv == 0 && kc.size(3) == D && vc.size(1) == Hkv && vc.size(2) == P);
  TORCH_CHECK(kc.dtype() == torch::kBFloat16 && vc.dtype() == torch::kBFloat16 &&
              kc.is_contiguous() && vc.is_contiguous() && bt.is_contiguous());
  TORCH_CHECK(out.dtype() == torch::kBFloat16 && out.size(0) == T && out.stride(1) == 1 &&
              dv <= DV && col + Hq * dv <= out.size(1));
  for (auto* t : {&slopes, &rates, &sink})
    TORCH_CHECK(!*t || ((*t)->numel() == Hq && (*t)->dtype() == torch::kFloat32));
  const HeadTurn ht = head_turn(turn, gate, slopes || rates, q, Hq, dv);
  TORCH_CHECK(bseq.dtype() == torch::kInt32 && boff.dtype() == torch::kInt32 &&
              bseq.numel() == boff.numel() && cu_q.dtype() == torch::kInt32 &&
              cu_q.numel() == ctx.numel() + 1 && bt.size(0) == ctx.numel());
  const int NB = bseq.numel();
  if (T == 0 || NB == 0) return;
  const int HG = heads_per_block(Hq / Hkv);
  dim3 grid(NB, Hq / HG), block(512);
  const float* rp = rates ? rates->data_ptr<float>() : nullptr;
  const float* sp = slopes ? slopes->data_ptr<float>() : nullptr;
  const float* snk = sink ? sink->data_ptr<float>() : nullptr;
#define BLAUNCH1(DD, DVV, HGV, BB, XX, LDS)                                     \
  hipLaunchKernelGGL((prefill_kernel<DD, DVV, HGV, false, BB, XX>), grid, block, \
                     (LDS<DD, DVV>()), CUR_STREAM,                              \
                     (const __hip_bfloat16*)q.data_ptr(), kc.data_ptr(),        \
                     vc.data_ptr(), (__hip_bfloat16*)out.data_ptr() + col,      \
                     bseq.data_ptr<int>(), boff.data_ptr<int>(),                \
                     cu_q.data_ptr<int>(), bt.data_ptr<int>(),                  \
                     ctx.data_ptr<int>(), Hq, Hkv, P, MP, (float)scale,         \
                     (long)Hq * D, out.stride(0), (int)dv, (float)oscale,       \
                     sp, rp, (int)window, (int)chunk, snk, nullptr, 0, KeyTail{}, ht)
#define BLAUNCH(DD, DVV, HGV)                                                   \
  if (!sp) { BLAUNCH1(DD, DVV, HGV, FLAT_BIAS, TURNED, turned_lds); }           \
  else if (rp) { BLAUNCH1(DD, DVV, HGV, LOG_BIAS, PLAIN, prefill_lds); }        \
  else { BLAUNCH1(DD, DVV, HGV, LINEAR_BIAS, PLAIN, prefill_lds); }
#define BLAUNCH_HG(DD, DVV)                    \
  switch (HG) {                                \
    case 1: BLAUNCH(DD, DVV, 1); break;        \
    case 2: BLAUNCH(DD, DVV, 2); break;        \
    default: BLAUNCH(DD, DVV, 4); break;       \
  }
  if (D == 64 && DV == 64) { BLAUNCH_HG(64, 64) }
  else if (D == 64 && DV == 128) { BLAUNCH_HG(64, 128) }
  else if (D == 128 && DV == 64) { BLAUNCH_HG(128, 64) }
  else if (D == 128 && DV == 128) { BLAUNCH_HG(128, 128) }
  else TORCH_CHECK(false, "unsupported cache head widths ", D, ", ", DV);
#undef BLAUNCH_HG
#undef BLAUNCH
#undef BLAUNCH1
  HIP_CHECK_KERNEL();
}

// q [T, H, D] (rows may be strided), kc [NP, H, P, D], vc [NP, H, P, DV], gate
// [T, H] pre-activations (rows may be strided) -> out [T, H * DV]
void sink_attention_prefill(torch::Tensor q, torch::Tensor kc, torch::Tensor vc,
                            torch::Tensor bt, torch::Tensor cu_q, torch::Tensor ctx,
                            torch::Tensor bseq, torch::Tensor boff, double scale,
                            torch::Tensor sink, torch::Tensor gate, torch::Tensor out) {
  const int T = q.size(0), H = q.size(1), D = q.size(2);
  const int P = kc.size(2), MP = bt.size(1), DV = vc.size(3);
  TORCH_CHECK(q.is_cuda() && q.dtype() == torch::kBFloat16 && q.stride(2) == 1 &&
              q.stride(1) == D && q.stride(0) % 8 == 0 &&
              (reinterpret_cast<uintptr_t>(q.data_ptr()) & 15) == 0, "queries");
  TORCH_CHECK(kc.dtype() == torch::kBFloat16 && vc.dtype() == torch::kBFloat16 &&
              kc.is_contiguous() && vc.is_contiguous() && bt.is_contiguous() &&
              kc.size(1) == H && vc.size(1) == H && kc.size(3) == D && vc.size(2) == P &&
              vc.size(0) == kc.size(0), "keys and values");
  TORCH_CHECK(out.dtype() == torch::kBFloat16 && out.is_contiguous() && out.size(0) == T &&
              out.size(1) == (long)H * DV);
  TORCH_CHECK(gate.dtype() == torch::kBFloat16 && gate.size(0) == T && gate.size(1) == H &&
              gate.stride(1) == 1 && sink.numel() == H && sink.dtype() == torch::kFloat32);
  TORCH_CHECK(bseq.dtype() == torch::kInt32 && boff.dtype() == torch::kInt32 &&
              bseq.numel() == boff.numel() && cu_q.dtype() == torch::kInt32 &&
              bt.dtype() == torch::kInt32 && ctx.dtype() == torch::kInt32 &&
              cu_q.numel() == ctx.numel() + 1 && bt.size(0) == ctx.numel());
  const int NB = bseq.numel();
  if (T == 0 || NB == 0) return;
  dim3 grid(NB, H), block(512);
#define SLAUNCH(DD, DVV)                                                        \
  hipLaunchKernelGGL((prefill_kernel<DD, DVV, 1, false, NO_BIAS, GATED>), grid,    \
                     block, (prefill_lds<DD, DVV>()), CUR_STREAM,               \
                     (const __hip_bfloat16*)q.data_ptr(), kc.data_ptr(),        \
                     vc.data_ptr(), (__hip_bfloat16*)out.data_ptr(),            \
                     bseq.data_ptr<int>(), boff.data_ptr<int>(),                \
                     cu_q.data_ptr<int>(), bt.data_ptr<int>(),                  \
                     ctx.data_ptr<int>(), H, H, P, MP, (float)scale,            \
                     q.stride(0), out.stride(0), DV, 1.f, nullptr, nullptr, 0,  \
                     0, sink.data_ptr<float>(),                                 \
                     (const __hip_bfloat16*)gate.data_ptr(), gate.stride(0),    \
                     KeyTail{}, HeadTurn{})
  if (D == 64 && DV == 64) { SLAUNCH(64, 64); }
  else if (D == 64 && DV == 128) { SLAUNCH(64, 128); }
  else if (D == 128 && DV == 64) { SLAUNCH(128, 64); }
  else if (D == 128 && DV == 128) { SLAUNCH(128, 128); }
  else TORCH_CHECK(false, "unsupported head widths ", D, ", ", DV);
#undef SLAUNCH
  HIP_CHECK_KERNEL();
}

// q [T, H, D] (rows may be strided) against keys of which every head has ``own`` first
// dimensions in kc [NP, H, 1, own] and all heads share the others, tail [NP, n] (rows
// may be strided; zeros follow up to D); vc [NP, H, 1, DV] -> out [T, H * DV]
void tailed_attention_prefill(torch::Tensor q, torch::Tensor kc, torch::Tensor vc,
                              torch::Tensor tail, torch::Tensor bt, torch::Tensor cu_q,
                              torch::Tensor ctx, torch::Tensor bseq, torch::Tensor boff,
                              double scale, long window, torch::Tensor out) {
  const int T = q.size(0), H = q.size(1), D = q.size(2);
  const int MP = bt.size(1), DV = vc.size(3), own = kc.size(3);
  TORCH_CHECK(q.is_cuda() && q.dtype() == torch::kBFloat16 && q.stride(2) == 1 &&
              q.stride(1) == D && q.stride(0) % 8 == 0 &&
              (reinterpret_cast<uintptr_t>(q.data_ptr()) & 15) == 0, "queries");
  TORCH_CHECK(kc.dtype() == torch::kBFloat16 && vc.dtype() == torch::kBFloat16 &&
              kc.is_contiguous() && vc.is_contiguous() && bt.is_contiguous() &&
              kc.size(1) == H && vc.size(1) == H && kc.size(2) == 1 && vc.size(2) == 1 &&
              own < D && own % 8 == 0 && vc.size(0) == kc.size(0), "keys and values");
  TORCH_CHECK(tail.dtype() == torch::kBFloat16 && tail.dim() == 2 && tail.stride(1) == 1 &&
              tail.size(0) == kc.size(0) && tail.size(1) % 8 == 0 &&
              tail.stride(0) % 8 == 0 &&
              (reinterpret_cast<uintptr_t>(tail.data_ptr()) & 15) == 0, "shared key part");
  TORCH_CHECK(out.dtype() == torch::kBFloat16 && out.is_contiguous() && out.size(0) == T &&
              out.size(1) == (long)H * DV);
  TORCH_CHECK(bseq.dtype() == torch::kInt32 && boff.dtype() == torch::kInt32 &&
              bseq.numel() == boff.numel() && cu_q.dtype() == torch::kInt32 &&
              bt.dtype() == torch::kInt32 && ctx.dtype() == torch::kInt32 &&
              cu_q.numel() == ctx.numel() + 1 && bt.size(0) == ctx.numel());
  const int NB = bseq.numel();
  if (T == 0 || NB == 0) return;
  dim3 grid(NB, H), block(512);
  const KeyTail kt = {(const __hip_bfloat16*)tail.data_ptr(), tail.stride(0),
                      (int)tail.size(1), own};
#define TLAUNCH(DD, DVV)                                                        \
  hipLaunchKernelGGL((prefill_kernel<DD, DVV, 1, false, FLAT_BIAS, TAILED>), grid, \
                     block, (prefill_lds<DD, DVV>()), CUR_STREAM,               \
                     (const __hip_bfloat16*)q.data_ptr(), kc.data_ptr(),        \
                     vc.data_ptr(), (__hip_bfloat16*)out.data_ptr(),            \
                     bseq.data_ptr<int>(), boff.data_ptr<int>(),                \
                     cu_q.data_ptr<int>(), bt.data_ptr<int>(),                  \
                     ctx.data_ptr<int>(), H, H, 1, MP, (float)scale,            \
                     q.stride(0), out.stride(0), DV, 1.f, nullptr, nullptr,     \
                     (int)window, 0, nullptr, nullptr, 0, kt, HeadTurn{})
#define TLAUNCH_D(DD)                       \
  if (D == DD && DV == 64) { TLAUNCH(DD, 64); } \
  else if (D == DD && DV == 128) { TLAUNCH(DD, 128); } else
  TLAUNCH_D(64) TLAUNCH_D(128) TLAUNCH_D(192)
  TORCH_CHECK(false, "unsupported head widths ", D, ", ", DV);
#undef TLAUNCH_D
#undef TLAUNCH
  HIP_CHECK_KERNEL();
}
