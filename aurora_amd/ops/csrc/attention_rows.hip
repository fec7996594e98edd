// Attention for any head width and for float32: one wave per (query row, head),
// 64 keys at a time; with a distance bias, a window or chunks and a sink, the result
// turned back and gated (head_turn.h), or over shared latents (rows whose first
// columns are the values).
//
// The matrix-core kernels (attention_prefill / attention_decode) serve bf16
// heads up to 128 wide; this one serves everything else. Each lane scores its
// own key of the tile from an LDS copy of the query, the online softmax is a
// pair of wave reductions, and for the values the lanes own output columns.
#include "head_turn.h"
#include <torch/extension.h>
#include <c10/hip/HIPStream.h>

#define CUR_STREAM c10::hip::getCurrentHIPStream().stream()
#define ROWS_MAX_DV 512
#define ROWS_MAX_LATENT 1024

template <typename T, int MAX_DV>
__global__ __launch_bounds__(256) void attention_rows_kernel(
    const T* __restrict__ q,  // [T, Hq, DK]
    const T* __restrict__ kc, const T* __restrict__ vc,  // [NP, Hkv, P, DK|DV]
    const int* __restrict__ bt, const int* __restrict__ cu,
    const int* __restrict__ ctx, const int* __restrict__ row_seq,
    const int* __restrict__ row_off, const float* __restrict__ slopes,
    const float* __restrict__ rates,  // [Hq]: penalty of ln(1 + rate * distance)
    const float* __restrict__ sink,  // [Hq] each, or null
    T* __restrict__ out, long ostride, int T_, int Hq, int Hkv, int DK, int DV,
    int dv, int P, int MP, float scale, int window, int chunk, float oscale,
    HeadTurn turn) {
  extern __shared__ float qs[];
  const long wid = (long)blockIdx.x * 4 + threadIdx.x / WAVE;
  const int lane = threadIdx.x % WAVE;
  const bool live = wid < (long)T_ * Hq;
  const int t = live ? wid / Hq : 0;
  const int h = live ? wid % Hq : 0;
  float* qv = qs + (threadIdx.x / WAVE) * DK;
  if (live)
    for (int i = lane; i < DK; i += WAVE) qv[i] = ldf(q + ((long)t * Hq + h) * DK + i);
  __syncthreads();
  if (!live) return;
  const int seq = row_seq ? row_seq[t] : t;
  const int len = cu ? cu[seq + 1] - cu[seq] : 1;
  const int pos = ctx[seq] - len + (row_off ? row_off[t] : 0);
  const int kvh = h / (Hq / Hkv);
  const float slope = slopes ? slopes[h] : 0.f, rate = rates ? rates[h] : 0.f;
  const int* pages = bt + (long)seq * MP;
  int lo = window > 0 ? max(0, pos - window + 1) : 0;
  if (chunk > 0) lo = max(lo, pos - pos % chunk);
  // a sink is one more term of the denominator
  float m = sink ? sink[h] : -1e30f, l = sink ? 1.f : 0.f, acc[MAX_DV / WAVE];
#pragma unroll
  for (int j = 0; j < MAX_DV / WAVE; ++j) acc[j] = 0.f;
  for (int k0 = lo; k0 <= pos; k0 += WAVE) {
    const int key = k0 + lane;
    const bool seen = key <= pos;
    const int kk = min(key, pos);
    const long row = ((long)pages[kk / P] * Hkv + kvh) * P + kk % P;
    float s = 0.f;
    for (int i = 0; i < DK; ++i) s += qv[i] * ldf(kc + row * DK + i);
    const float dist = (float)(pos - kk);
    s = seen ? s * scale - slope * (rates ? logf(1.f + rate * dist) : dist) : -1e30f;
    const float mn = fmaxf(m, wave_max(s));
    const float alpha = expf(m - mn);
    const float p = seen ? expf(s - mn) : 0.f;
    m = mn;
    l = l * alpha + wave_sum(p);
#pragma unroll
    for (int j = 0; j < MAX_DV / WAVE; ++j) acc[j] *= alpha;
    const int n = min(WAVE, pos - k0 + 1);
    for (int i = 0; i < n; ++i) {
      const float pi = __shfl(p, i, WAVE);
      const long ri = __shfl(row, i, WAVE);
#pragma unroll
      for (int j = 0; j < MAX_DV / WAVE; ++j)
        if (lane + j * WAVE < dv) acc[j] += pi * ldf(vc + ri * DV + lane + j * WAVE);
    }
  }
#pragma unroll
  for (int j = 0; j < MAX_DV / WAVE; ++j) {
    const int d = lane + j * WAVE;
    if (j * WAVE >= dv) break;
    const float y = turned<T>(turn, acc[j] / l * oscale, t, pos, h, d, dv);
    if (d < dv) stf(out + t * ostride + h * dv + d, y);
  }
}

void biased_attention_rows(torch::Tensor q, torch::Tensor kc, torch::Tensor vc,
                           torch::Tensor bt, c10::optional<torch::Tensor> cu,
                           torch::Tensor ctx, c10::optional<torch::Tensor> row_seq,
                           c10::optional<torch::Tensor> row_off, double scale,
                           long window, long chunk, c10::optional<torch::Tensor> slopes,
                           c10::optional<torch::Tensor> rates,
                           c10::optional<torch::Tensor> sink,
                           c10::optional<torch::Tensor> turn,
                           c10::optional<torch::Tensor> gate, torch::Tensor out, long col,
                           long dv, double oscale) {
  const int T_ = q.size(0), Hq = q.size(1), DK = q.size(2);
  const int Hkv = kc.size(1), P = kc.size(2), MP = bt.size(1), DV = vc.size(3);
  TORCH_CHECK(q.is_cuda() && q.is_contiguous() && kc.is_contiguous() &&
              vc.is_contiguous() && bt.is_contiguous());
  TORCH_CHECK(kc.size(3) == DK && Hq % Hkv == 0 && dv <= DV && DV <= ROWS_MAX_DV,
              "head width ", DV, " not supported (at most ", ROWS_MAX_DV, ")");
  TORCH_CHECK(DK <= 2048, "keys of ", DK, " numbers");
  for (auto* t : {&slopes, &rates, &sink})
    TORCH_CHECK(!*t || ((*t)->numel() == Hq && (*t)->dtype() == torch::kFloat32));
  const HeadTurn ht = head_turn(turn, gate, slopes || rates, q, Hq, dv);
  TORCH_CHECK(kc.dtype() == q.dtype() && vc.dtype() == q.dtype() && out.dtype() == q.dtype());
  TORCH_CHECK(out.size(0) == T_ && out.stride(1) == 1 && col + Hq * dv <= out.size(1));
  TORCH_CHECK(bt.dtype() == torch::kInt32 && ctx.dtype() == torch::kInt32);
  if (cu) {
    TORCH_CHECK(row_seq && row_off && row_seq->numel() == T_ && row_off->numel() == T_ &&
                cu->numel() == ctx.numel() + 1);
  } else {
    TORCH_CHECK(ctx.numel() == T_);
  }
  TORCH_CHECK(bt.size(0) == ctx.numel());
  if (T_ == 0) return;
  const int* cup = cu ? cu->data_ptr<int>() : nullptr;
  const int* rsp = cu ? row_seq->data_ptr<int>() : nullptr;
  const int* rop = cu ? row_off->data_ptr<int>() : nullptr;
  const dim3 grid(((long)T_ * Hq + 3) / 4);
  DISPATCH_ELEM(q.dtype() == torch::kBFloat16, {
    hipLaunchKernelGGL(
        (attention_rows_kernel<T, ROWS_MAX_DV>), grid, dim3(256), 4 * DK * 4, CUR_STREAM, (const T*)q.data_ptr(),
        (const T*)kc.data_ptr(), (const T*)vc.data_ptr(), bt.data_ptr<int>(),
        cup, ctx.data_ptr<int>(), rsp, rop, slopes ? slopes->data_ptr<float>() : nullptr,
        rates ? rates->data_ptr<float>() : nullptr,
        sink ? sink->data_ptr<float>() : nullptr, (T*)out.data_ptr() + col, out.stride(0), T_, Hq, Hkv, DK,
        DV, (int)dv, P, MP, (float)scale, (int)window, (int)chunk, (float)oscale, ht);
  });
  HIP_CHECK_KERNEL();
}

// q [T, H, C] against the latent cache [NP, 1, P, C], whose first R columns are the
// values too -> out [T, H, R]
void latent_attention_rows(torch::Tensor q, torch::Tensor cache, torch::Tensor bt,
                           c10::optional<torch::Tensor> cu, torch::Tensor ctx,
                           c10::optional<torch::Tensor> row_seq,
                           c10::optional<torch::Tensor> row_off, double scale,
                           c10::optional<torch::Tensor> sink, long window,
                           torch::Tensor out) {
  const int T_ = q.size(0), H = q.size(1), C = q.size(2), R = out.size(2);
  const int P = cache.size(2), MP = bt.size(1);
  TORCH_CHECK(q.is_cuda() && q.is_contiguous() && cache.is_contiguous() &&
              bt.is_contiguous() && out.is_contiguous() && out.size(0) == T_ &&
              out.size(1) == H);
  TORCH_CHECK(cache.size(1) == 1 && cache.size(3) == C && R <= C && C <= 2048 &&
              R <= ROWS_MAX_LATENT, "latents of ", R, " numbers");
  TORCH_CHECK(!sink || (sink->numel() == H && sink->dtype() == torch::kFloat32));
  TORCH_CHECK(cache.dtype() == q.dtype() && out.dtype() == q.dtype());
  TORCH_CHECK(bt.dtype() == torch::kInt32 && ctx.dtype() == torch::kInt32 &&
              bt.size(0) == ctx.numel());
  if (cu) {
    TORCH_CHECK(row_seq && row_off && row_seq->numel() == T_ && row_off->numel() == T_ &&
                cu->numel() == ctx.numel() + 1);
  } else {
    TORCH_CHECK(ctx.numel() == T_);
  }
  if (T_ == 0) return;
  const dim3 grid(((long)T_ * H + 3) / 4);
  DISPATCH_ELEM(q.dtype() == torch::kBFloat16, {
    auto launch = [&](auto kern) {
      hipLaunchKernelGGL(
          kern, grid, dim3(256), 4 * C * 4, CUR_STREAM, (const T*)q.data_ptr(),
          (const T*)cache.data_ptr(), (const T*)cache.data_ptr(), bt.data_ptr<int>(),
          cu ? cu->data_ptr<int>() : nullptr, ctx.data_ptr<int>(),
          cu ? row_seq->data_ptr<int>() : nullptr, cu ? row_off->data_ptr<int>() : nullptr,
          (const float*)nullptr, (const float*)nullptr,
          sink ? sink->data_ptr<float>() : nullptr, (T*)out.data_ptr(), (long)H * R, T_,
          H, 1, C, C, R, P, MP, (float)scale, (int)window, 0, 1.f, HeadTurn{});
    };
    if (R <= ROWS_MAX_DV) launch(attention_rows_kernel<T, ROWS_MAX_DV>);
    else launch(attention_rows_kernel<T, ROWS_MAX_LATENT>);
  });
  HIP_CHECK_KERNEL();
}
