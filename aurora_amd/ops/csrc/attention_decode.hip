// Paged-KV decode attention for gfx950 (one new token per sequence).
//
// Memory-bound by the KV read; the kernel streams each (seq, kv_head)'s
// pages once at 16 B/lane and amortises the read over all G grouped query
// heads (GQA).  Two levers keep it at streaming rate:
//  * token-group software pipelining: each D/8-lane group prefetches K/V
//    for 4 tokens before the (serial) online-softmax updates, so the
//    memory system always has 8 x 16 B loads in flight per lane-group
//    (the naive one-token loop is latency-bound through the o-rescale
//    dependency chain: measured 1.07 TB/s at B=16 -> this structure);
//  * flash-decode context splits: grid.z partitions the context into
//    contiguous chunks so small batches still put >=512 workgroups on the
//    256-CU chip; per-chunk (m, l, o) partials combine in a second kernel.
//
// Replaces the per-token provider round-trip of the reference agent loop
// (reference: server/chat/backend/agent/llm.py:192) with an in-process
// batched decode step.
#include "head_turn.h"
#include <torch/extension.h>
#include <c10/hip/HIPStream.h>

#define CUR_STREAM c10::hip::getCurrentHIPStream().stream()

#ifndef TUNR
#define TUNR 4  // tokens prefetched per group iteration (8 measured neutral)
#endif

enum { NO_BIAS = 0, LINEAR_BIAS = 1, LOG_BIAS = 2, FLAT_BIAS = 3 };

// BIAS: a distance penalty per head or none (see attention_prefill.hip), a window or
// chunks of positions; sink: one more term of the denominator per head, or null;
// FLAT_BIAS results may be turned back and gated
template <int D, int DV, int G, bool FP8, int BIAS>
__global__ __launch_bounds__(256) void paged_decode_kernel(
    const __hip_bfloat16* __restrict__ q,   // [B, Hq, D]
    const void* __restrict__ kc,  // [NP, Hkv, P, D] bf16 | fp8 e4m3
    const void* __restrict__ vc,
    __hip_bfloat16* __restrict__ out,       // [B, ostride], heads dv apart (CS==1)
    float* __restrict__ part,               // [CS, B, Hq, DV+2] (CS>1)
    const int* __restrict__ block_tables,   // [B, MP]
    const int* __restrict__ ctx_lens,       // [B]
    int Hkv, int NG,                        // NG: head groups per kv head
    int P, int MP, int CS, float scale,
    long ostride, int dv, float oscale,
    const float* __restrict__ slopes, const float* __restrict__ rates, int window,
    int chunk_of, const float* __restrict__ sink, HeadTurn turn) {
  constexpr int GL = (D > DV ? D : DV) / 8;  // lanes per token-group
  constexpr int TPW = WAVE / GL;   // token-groups per wave
  constexpr int NW = 4;            // waves per workgroup
  constexpr int NPART = NW * TPW;  // in-block partials to combine

  const int b = blockIdx.x;
  const int kvh = blockIdx.y / NG;
  const int h0 = blockIdx.y * G;  // first query head of this workgroup
  const int Hq = gridDim.y * G;
  const int cs = blockIdx.z;
  const int L = ctx_lens[b];
  // contiguous chunk of the visible context for this split
  int first = BIAS && window > 0 ? max(0, L - window) : 0;
  if (BIAS && chunk_of > 0) first = max(first, L - 1 - (L - 1) % chunk_of);
  const int chunk = (L - first + CS - 1) / CS;
  const int t_lo = first + cs * chunk;
  const int t_hi = min(L, t_lo + chunk);
  const int tid = threadIdx.x;
  const int wave = tid / WAVE;
  const int lane = tid % WAVE;
  const int grp = lane / GL;   // token-group within the wave
  const int sub = lane % GL;   // 16-B slot within the token row

  shortx8 qf[G];
#pragma unroll
  for (int g = 0; g < G; ++g) {
    if (DV > D && sub * 8 >= D)
      qf[g] = shortx8{0, 0, 0, 0, 0, 0, 0, 0};
    else
      qf[g] = *reinterpret_cast<const shortx8*>(
          q + ((long)b * Hq + h0 + g) * D + sub * 8);
  }
  float slope[G], rate[G];
#pragma unroll
  for (int g = 0; g < G; ++g) {
    slope[g] = BIAS && BIAS != FLAT_BIAS ? slopes[h0 + g] : 0.f;
    rate[g] = BIAS == LOG_BIAS ? rates[h0 + g] : 0.f;
  }
  // 16-B column of a key / value row this lane reads (lanes past the narrower
  // of the two re-read its last column and contribute nothing)
  const int ksub = min(sub * 8, D - 8), vsub = min(sub * 8, DV - 8);

  float m[G], l[G], o[G][8];
#pragma unroll
  for (int g = 0; g < G; ++g) {
    m[g] = -1e30f;
    l[g] = 0.f;
#pragma unroll
    for (int j = 0; j < 8; ++j) o[g][j] = 0.f;
  }

  const int* bt = block_tables + (long)b * MP;
  const int stride = NW * TPW;
  // groups stride the chunk; TUNR tokens prefetched per iteration
  for (int t0 = t_lo + (wave * TPW + grp) * TUNR; t0 < t_hi;
       t0 += stride * TUNR) {
    shortx8 kf[TUNR], vf[TUNR];
    int nt = 0;
    if constexpr (FP8) {
      // fp8 cache: half the KV stream bytes (the kernel is KV-bound at
      // ~6.15 TB/s in bf16); 8-byte loads, convert
      // to bf16 fragments in-register
      u64b k8[TUNR], v8[TUNR];
#pragma unroll
      for (int u = 0; u < TUNR; ++u) {
        const int t = t0 + u;
        const int tc = min(t, t_hi - 1);
        const long row = ((long)bt[tc / P] * Hkv + kvh) * P + (tc % P);
        k8[u] = *reinterpret_cast<const u64b*>((const unsigned char*)kc + row * D + ksub);
        v8[u] = *reinterpret_cast<const u64b*>((const unsigned char*)vc + row * DV + vsub);
      }
#pragma unroll
      for (int u = 0; u < TUNR; ++u) {
        kf[u] = fp8x8_to_bf16x8(k8[u]);
        vf[u] = fp8x8_to_bf16x8(v8[u]);
      }
    } else {
#pragma unroll
      for (int u = 0; u < TUNR; ++u) {
        const int t = t0 + u;
        const int tc = min(t, t_hi - 1);  // clamped prefetch (masked below)
        const long row = ((long)bt[tc / P] * Hkv + kvh) * P + (tc % P);
        kf[u] = *reinterpret_cast<const shortx8*>((const __hip_bfloat16*)kc + row * D + ksub);
        vf[u] = *reinterpret_cast<const shortx8*>((const __hip_bfloat16*)vc + row * DV + vsub);
      }
    }
#pragma unroll
    for (int u = 0; u < TUNR; ++u) {
      if (t0 + u >= t_hi) break;
      float s[G];
#pragma unroll
      for (int g = 0; g < G; ++g) {
        s[g] = group_sum<GL>(dot8_bf16_fast(kf[u], qf[g])) * scale;
        if constexpr (BIAS == LINEAR_BIAS || BIAS == LOG_BIAS) {
          const float dist = (float)(L - 1 - t0 - u);
          s[g] -= slope[g] * (BIAS == LOG_BIAS ? __logf(1.f + rate[g] * dist) : dist);
        }
        // defer-style rescale: the running max rarely grows, so the O/l
        // rescale (8*G VALU per token) is branch-skipped when it does not
        if (s[g] > m[g]) {
          const float alpha = __expf(m[g] - s[g]);
          m[g] = s[g];
          l[g] *= alpha;
#pragma unroll
          for (int j = 0; j < 8; ++j) o[g][j] *= alpha;
        }
        const float pv = __expf(s[g] - m[g]);
        l[g] += pv;
#pragma unroll
        for (int j = 0; j < 8; ++j)
          o[g][j] += pv * bf16_to_f32((unsigned short)vf[u][j]);
      }
    }
  }

  // ---- combine the NPART in-block partials per head through LDS ----
  __shared__ float s_m[G][NPART];
  __shared__ float s_l[G][NPART];
  __shared__ float s_o[G][NPART][DV];
  const int pidx = wave * TPW + grp;
#pragma unroll
  for (int g = 0; g < G; ++g) {
    if (sub == 0) {
      s_m[g][pidx] = m[g];
      s_l[g][pidx] = l[g];
    }
#pragma unroll
    for (int j = 0; j < 8; ++j)
      if (DV >= D || sub * 8 < DV) s_o[g][pidx][sub * 8 + j] = o[g][j];
  }
  __syncthreads();
  for (int gd = tid; gd < G * DV; gd += blockDim.x) {
    const int g = gd / DV, d = gd % DV;
    const bool ends = BIAS && CS == 1 && sink;  // the sink counts once
    const float first = ends ? sink[h0 + g] : -1e30f;
    float M = first;
#pragma unroll 4
    for (int i = 0; i < NPART; ++i) M = fmaxf(M, s_m[g][i]);
    float Lsum = ends ? __expf(first - M) : 0.f, O = 0.f;
#pragma unroll 4
    for (int i = 0; i < NPART; ++i) {
      const float w = __expf(s_m[g][i] - M);
      Lsum += w * s_l[g][i];
      O += w * s_o[g][i][d];
    }
    const long hq = (long)b * Hq + h0 + g;
    if (CS == 1) {
      float y = O / Lsum * oscale;
      if constexpr (BIAS == FLAT_BIAS) y = turned<bf16_t>(turn, y, b, L - 1, h0 + g, d, dv);
      if (!BIAS || d < dv)
        *(unsigned short*)(out + b * ostride + (long)(h0 + g) * dv + d) = f32_to_bf16(y);
    } else {
      // emit an un-normalised chunk partial: {o*w-sum, m, l}
      float* dst = part + ((long)cs * gridDim.x * Hq + hq) * (DV + 2);
      dst[d] = O;
      if (d == 0) {
        dst[DV] = M;
        dst[DV + 1] = Lsum;
      }
    }
  }
}

// combine CS chunk partials -> out; one wave per (b, h)
template <int D>
__global__ void decode_combine_kernel(const float* __restrict__ part,
                                      __hip_bfloat16* __restrict__ out,
                                      int CS, long BH, int Hq, long ostride,
                                      int dv, float oscale,
                                      const float* __restrict__ sink, HeadTurn turn,
                                      const int* __restrict__ ctx_lens) {
  const long bh = blockIdx.x * (blockDim.x / WAVE) + threadIdx.x / WAVE;
  if (bh >= BH) return;
  const int lane = threadIdx.x % WAVE;
  const float first = sink ? sink[bh % Hq] : -1e30f;
  float M = first;
  for (int s = 0; s < CS; ++s)
    M = fmaxf(M, part[((long)s * BH + bh) * (D + 2) + D]);
  float Lsum = sink ? __expf(first - M) : 0.f;
  for (int s = 0; s < CS; ++s) {
    const float* p = part + ((long)s * BH + bh) * (D + 2);
    Lsum += __expf(p[D] - M) * p[D + 1];
  }
  for (int d = lane; d < dv; d += WAVE) {
    float O = 0.f;
    for (int s = 0; s < CS; ++s) {
      const float* p = part + ((long)s * BH + bh) * (D + 2);
      O += __expf(p[D] - M) * p[d];
    }
    float y = O / Lsum * oscale;
    if (turn.cs || turn.gate)
      y = turned<bf16_t>(turn, y, bh / Hq, ctx_lens[bh / Hq] - 1, bh % Hq, d, dv);
    *(unsigned short*)(out + bh / Hq * ostride + bh % Hq * dv + d) = f32_to_bf16(y);
  }
}

// query heads sharing one K/V stream: the largest tile that divides the group
static int head_tile(int G) { return G % 8 == 0 ? 8 : G % 4 == 0 ? 4 : G % 2 == 0 ? 2 : 1; }

template <int D, int DV, bool FP8, int BIAS>
static void decode_launch(const torch::Tensor& q, const torch::Tensor& kc,
                          const torch::Tensor& vc, const torch::Tensor& bt,
                          const torch::Tensor& ctx, __hip_bfloat16* out, long ostride,
                          int dv, float scale, float oscale, const float* slopes,
                          const float* rates, int window, int chunk, const float* sink,
                          const HeadTurn& turn, int CS) {
  const int B = q.size(0), Hq = q.size(1);
  const int Hkv = kc.size(1), P = kc.size(2), MP = bt.size(1);
  const int G = Hq / Hkv, GT = head_tile(G);
  torch::Tensor part;
  if (CS > 1)
    part = torch::empty({CS, (long)B * Hq, DV + 2}, q.options().dtype(torch::kFloat32));
  float* pp = CS > 1 ? part.data_ptr<float>() : nullptr;
  dim3 grid(B, Hkv * (G / GT), CS), block(256);
  auto stream = CUR_STREAM;
#define LAUNCH(GG)                                                              \
  hipLaunchKernelGGL((paged_decode_kernel<D, DV, GG, FP8, BIAS>), grid, block,  \
                     0, stream, (const __hip_bfloat16*)q.data_ptr(),            \
                     kc.data_ptr(), vc.data_ptr(), out, pp, bt.data_ptr<int>(), \
                     ctx.data_ptr<int>(), Hkv, G / GT, P, MP, CS, scale,        \
                     ostride, dv, oscale, slopes, rates, window, chunk, sink, turn)
  switch (GT) {
    case 8: LAUNCH(8); break;
    case 4: LAUNCH(4); break;
    case 2: LAUNCH(2); break;
    default: LAUNCH(1); break;
  }
#undef LAUNCH
  if (CS > 1) {
    const long BH = (long)B * Hq;
    hipLaunchKernelGGL((decode_combine_kernel<DV>), dim3((BH + 3) / 4), dim3(256), 0,
                       stream, pp, out, CS, BH, Hq, ostride, dv, oscale, sink, turn,
                       ctx.data_ptr<int>());
  }
  HIP_CHECK_KERNEL();
}

torch::Tensor paged_attention_decode(torch::Tensor q, torch::Tensor kc,
                                     torch::Tensor vc, torch::Tensor bt,
                                     torch::Tensor ctx, double scale) {
  TORCH_CHECK(q.is_cuda() && q.dtype() == torch::kBFloat16, "bf16 GPU only");
  const int B = q.size(0), Hq = q.size(1), D = q.size(2), Hkv = kc.size(1);
  TORCH_CHECK(Hq % Hkv == 0, "GQA requires Hq % Hkv == 0");
  TORCH_CHECK(D == 128 || D == 64, "unsupported head_dim ", D);
  auto out = torch::empty_like(q);
  if (B == 0) return out;
  // context splits: fill target ~1024 WGs. At B=64 the LDS-bound residency
  // is only 2 WGs/CU, so deeper splits buy memory-level parallelism
  const int CS = std::max(1, std::min(8, 1024 / std::max(B * Hkv, 1)));
  auto* o = (__hip_bfloat16*)out.data_ptr();
  const long stride = (long)Hq * D;
  const bool fp8 = kc.dtype() == torch::kFloat8_e4m3fn;
#define RUN(DD, F8) \
  decode_launch<DD, DD, F8, NO_BIAS>(q, kc, vc, bt, ctx, o, stride, D, (float)scale, \
                                     1.f, nullptr, nullptr, 0, 0, nullptr, HeadTurn{}, CS)
  if (D == 128) { if (fp8) RUN(128, true); else RUN(128, false); }
  else { if (fp8) RUN(64, true); else RUN(64, false); }
#undef RUN
  return out;
}

void biased_attention_decode(torch::Tensor q, torch::Tensor kc, torch::Tensor vc,
                             torch::Tensor bt, torch::Tensor ctx, double scale,
                             long window, long chunk, c10::optional<torch::Tensor> slopes,
                             c10::optional<torch::Tensor> rates,
                             c10::optional<torch::Tensor> sink,
                             c10::optional<torch::Tensor> turn,
                             c10::optional<torch::Tensor> gate, torch::Tensor out,
                             long col, long dv, double oscale) {
  TORCH_CHECK(q.is_cuda() && q.dtype() == torch::kBFloat16 && q.is_contiguous());
  const int B = q.size(0), Hq = q.size(1), D = q.size(2);
  const int Hkv = kc.size(1), DV = vc.size(3);
  TORCH_CHECK(Hq % Hkv == 0 && kc.size(3) == D && vc.size(1) == Hkv &&
              vc.size(2) == kc.size(2));
  TORCH_CHECK(kc.dtype() == torch::kBFloat16 && vc.dtype() == torch::kBFloat16 &&
              kc.is_contiguous() && vc.is_contiguous() && bt.is_contiguous());
  TORCH_CHECK(out.dtype() == torch::kBFloat16 && out.size(0) == B && out.stride(1) == 1 &&
              dv <= DV && col + Hq * dv <= out.size(1));
  for (auto* t : {&slopes, &rates, &sink})
    TORCH_CHECK(!*t || ((*t)->numel() == Hq && (*t)->dtype() == torch::kFloat32));
  const HeadTurn ht = head_turn(turn, gate, slopes || rates, q, Hq, dv);
  TORCH_CHECK(ctx.numel() == B && bt.size(0) == B && bt.dtype() == torch::kInt32 &&
              ctx.dtype() == torch::kInt32);
  if (B == 0) return;
  // a split of fewer than 64 visible keys is not worth its combine
  int CS = std::max(1, std::min(8, 1024 / std::max(B * Hkv, 1)));
  for (long seen : {window, chunk})
    if (seen > 0) CS = std::max(1, std::min(CS, (int)((seen + 63) / 64)));
  auto* o = (__hip_bfloat16*)out.data_ptr() + col;
  const float* rp = rates ? rates->data_ptr<float>() : nullptr;
  const float* sp = slopes ? slopes->data_ptr<float>() : nullptr;
  const float* snk = sink ? sink->data_ptr<float>() : nullptr;
#define RUN1(DD, DVV, BB)                                                        \
  decode_launch<DD, DVV, false, BB>(q, kc, vc, bt, ctx, o, out.stride(0),        \
                                    (int)dv, (float)scale, (float)oscale,        \
                                    sp, rp, (int)window, (int)chunk, snk, ht, CS)
#define RUN(DD, DVV)                         \
  if (!sp) RUN1(DD, DVV, FLAT_BIAS);         \
  else if (rp) RUN1(DD, DVV, LOG_BIAS);      \
  else RUN1(DD, DVV, LINEAR_BIAS)
  if (D == 64 && DV == 64) { RUN(64, 64); }
  else if (D == 64 && DV == 128) { RUN(64, 128); }
  else if (D == 128 && DV == 64) { RUN(128, 64); }
  else if (D == 128 && DV == 128) { RUN(128, 128); }
  else TORCH_CHECK(false, "unsupported cache head widths ", D, ", ", DV);
#undef RUN
#undef RUN1
}
