// What surrounds the mixers of the layer-listed decoders: the embedding of
// tokens and token pairs, the causal convolution added to a sublayer's input, and
// the activations of the dense feed-forwards.
//
// The two kernels with a past keep it in state slots. Rows that read a sequence's
// past and the store of its new past belong to one thread (convolution, per
// channel) or one workgroup (embedding, the portion's first row), so a portion
// never races with itself. Slot -1 marks an idle row of a captured batch.
#include "elem.h"
#include <torch/extension.h>
#include <c10/hip/HIPStream.h>

#define CUR_STREAM c10::hip::getCurrentHIPStream().stream()
#define CONV_ROWS 16      // rows per workgroup of the convolution
#define CONV_MAX_TAPS 16  // a block's past must not reach past the block before it

// ---------------------------------------------------------------- embedding

// One workgroup per token: table row * scale + pair row, normed, in fp32.
template <typename T, int V>
__global__ __launch_bounds__(256) void embed_pairs_kernel(
    const long* __restrict__ ids, const T* __restrict__ table, float scale,
    const T* __restrict__ pairs, long buckets, long mul_prev, long mul_cur,
    const float* __restrict__ weight, float eps, int* __restrict__ prev,
    const int* __restrict__ cu, const int* __restrict__ starts,
    const int* __restrict__ slots, float* __restrict__ out, int S, int W) {
  extern __shared__ __attribute__((aligned(16))) float row[];
  __shared__ float red[4];
  const int t = blockIdx.x;
  int seq = t, first = t, last = t;
  if (cu) {
    int lo = 0, hi = S;  // cu[lo] <= t < cu[hi]
    while (hi - lo > 1) {
      const int mid = (lo + hi) / 2;
      if (cu[mid] <= t) lo = mid; else hi = mid;
    }
    seq = lo;
    first = cu[seq];
    last = cu[seq + 1] - 1;
  }
  const int slot = slots[seq];
  const long id = ids[t];
  long pair = buckets;
  const bool past = t > first || (starts[seq] > 0 && slot >= 0);
  if (past) {
    const long before = t > first ? ids[t - 1] : (long)prev[slot];
    pair = (before * mul_prev + id * mul_cur) % buckets;
    if (pair < 0) pair += buckets;
  }
  const T* a = table + id * W;
  const T* b = pairs + pair * W;
  float ss = 0.f;
  for (int i = threadIdx.x * V; i < W; i += 256 * V) {
    if constexpr (V == 4) {
      const floatx4 v = ld4(a + i) * scale + ld4(b + i);
      *(floatx4*)(row + i) = v;
#pragma unroll
      for (int j = 0; j < 4; ++j) ss += v[j] * v[j];
    } else {
      const float v = ldf(a + i) * scale + ldf(b + i);
      row[i] = v;
      ss += v * v;
    }
  }
  const float inv = rsqrtf(block_sum4(ss, red) / W + eps);
  // every thread has read the past by now
  if (t == first && slot >= 0 && threadIdx.x == 0) prev[slot] = (int)ids[last];
  float* y = out + (long)t * W;
  for (int i = threadIdx.x * V; i < W; i += 256 * V) {
    if constexpr (V == 4) st4(y + i, *(const floatx4*)(row + i) * inv * ld4(weight + i));
    else y[i] = row[i] * inv * weight[i];
  }
}

void embed_pairs(torch::Tensor ids, torch::Tensor table, double scale,
                 torch::Tensor pairs, long mul_prev, long mul_cur, torch::Tensor weight,
                 double eps, torch::Tensor prev, c10::optional<torch::Tensor> cu,
                 torch::Tensor starts, torch::Tensor slots, torch::Tensor out) {
  const int T_ = ids.numel(), W = table.size(1), S = slots.numel();
  TORCH_CHECK(ids.is_cuda() && ids.dtype() == torch::kInt64 && ids.is_contiguous());
  TORCH_CHECK(table.is_contiguous() && pairs.is_contiguous() && pairs.size(1) == W &&
              pairs.dtype() == table.dtype() && pairs.size(0) > 1, "embedding tables");
  TORCH_CHECK(weight.numel() == W && weight.dtype() == torch::kFloat32 && W <= 16384);
  TORCH_CHECK(out.dtype() == torch::kFloat32 && out.is_contiguous() &&
              out.size(0) == T_ && out.size(1) == W);
  TORCH_CHECK(prev.dtype() == torch::kInt32 && prev.is_contiguous() &&
              prev.numel() == prev.size(0));
  TORCH_CHECK(starts.numel() == S && starts.dtype() == torch::kInt32 &&
              slots.dtype() == torch::kInt32 && starts.is_contiguous());
  if (cu) {
    TORCH_CHECK(cu->numel() == S + 1 && cu->dtype() == torch::kInt32);
  } else {
    TORCH_CHECK(S == T_);
  }
  if (T_ == 0) return;
  DISPATCH_ELEM(table.dtype() == torch::kBFloat16, {
    auto launch = [&](auto kern) {
      hipLaunchKernelGGL(kern, dim3(T_), dim3(256), (size_t)W * 4, CUR_STREAM,
                         (const long*)ids.data_ptr(), (const T*)table.data_ptr(),
                         (float)scale, (const T*)pairs.data_ptr(), pairs.size(0) - 1,
                         mul_prev, mul_cur, weight.data_ptr<float>(), (float)eps,
                         prev.data_ptr<int>(), cu ? cu->data_ptr<int>() : nullptr,
                         starts.data_ptr<int>(), slots.data_ptr<int>(),
                         out.data_ptr<float>(), S, W);
    };
    if (W % 4 == 0) launch(embed_pairs_kernel<T, 4>);
    else launch(embed_pairs_kernel<T, 1>);
  });
  HIP_CHECK_KERNEL();
}

// -------------------------------------------------------------- convolution

// V channels per thread, CONV_ROWS rows of one sequence; TAPS 0: any number,
// inputs read again for every tap (V = 1).
template <typename T, int V, int TAPS>
__global__ __launch_bounds__(256) void short_conv_kernel(
    const T* __restrict__ h, const float* __restrict__ w /* [taps, W] */,
    T* __restrict__ ring,
    const int* __restrict__ cu, const int* __restrict__ bseq, const int* __restrict__ boff,
    const int* __restrict__ starts, const int* __restrict__ slots, T* __restrict__ out,
    int W, int taps_) {
  const int c = (blockIdx.y * 256 + threadIdx.x) * V;
  if (c >= W) return;
  const int taps = TAPS ? TAPS : taps_;
  const int seq = cu ? bseq[blockIdx.x] : blockIdx.x;
  const int off = cu ? boff[blockIdx.x] : 0;
  const int row0 = cu ? cu[seq] : seq;
  const int len = cu ? cu[seq + 1] - row0 : 1;
  const int n = min(CONV_ROWS, len - off);
  const int slot = slots[seq], start = starts[seq];
  const int keep = taps - 1, ring_len = TAPS == 1 ? 1 : keep;
  T* rg = ring + (long)max(slot, 0) * keep * W + c;
  // channel v of local row t (may be negative: the sequence's past)
  auto input = [&](int t, float (&x)[V]) {
    const T* p = nullptr;
    if (t >= 0) p = h + (long)(row0 + t) * W + c;
    else if (slot >= 0 && start + t >= 0) p = rg + (long)((start + t) % ring_len) * W;
    if constexpr (V % 4 == 0) {
#pragma unroll
      for (int v = 0; v < V; v += 4) {
        floatx4 y = {0.f, 0.f, 0.f, 0.f};
        if (p) y = ld4(p + v);
#pragma unroll
        for (int i = 0; i < 4; ++i) x[v + i] = y[i];
      }
    } else {
#pragma unroll
      for (int v = 0; v < V; ++v) x[v] = p ? ldf(p + v) : 0.f;
    }
  };
  auto store = [&](int t, const float (&y)[V]) {
    T* p = out + (long)(row0 + t) * W + c;
    if constexpr (V % 4 == 0) {
#pragma unroll
      for (int v = 0; v < V; v += 4) st4(p + v, floatx4{y[v], y[v + 1], y[v + 2], y[v + 3]});
    } else {
#pragma unroll
      for (int v = 0; v < V; ++v) stf(p + v, y[v]);
    }
  };
  if constexpr (TAPS > 0) {
    float win[TAPS][V], wt[TAPS][V];  // win[j]: input TAPS - 1 - j rows back
#pragma unroll
    for (int j = 0; j < TAPS; ++j)
#pragma unroll
      for (int v = 0; v < V; ++v) wt[j][v] = w[(long)j * W + c + v];
#pragma unroll
    for (int j = 1; j < TAPS; ++j) input(off - TAPS + j, win[j]);
    for (int t = 0; t < n; ++t) {
#pragma unroll
      for (int j = 0; j + 1 < TAPS; ++j)
#pragma unroll
        for (int v = 0; v < V; ++v) win[j][v] = win[j + 1][v];
      input(off + t, win[TAPS - 1]);
      float y[V];
#pragma unroll
      for (int v = 0; v < V; ++v) y[v] = win[TAPS - 1][v];
#pragma unroll
      for (int j = 0; j < TAPS; ++j)
#pragma unroll
        for (int v = 0; v < V; ++v) y[v] += wt[j][v] * win[j][v];
      store(off + t, y);
    }
  } else {
    for (int t = 0; t < n; ++t) {
      float y[V], x[V];
      input(off + t, y);
      for (int j = 0; j < taps; ++j) {
        input(off + t - keep + j, x);
#pragma unroll
        for (int v = 0; v < V; ++v) y[v] += w[(long)j * W + c + v] * x[v];
      }
      store(off + t, y);
    }
  }
  // only the first block reads the past, and it has
  if (off == 0 && slot >= 0)
    for (int t = max(0, len - keep); t < len; ++t) {
      T* p = rg + (long)((start + t) % ring_len) * W;
#pragma unroll
      for (int v = 0; v < V; ++v) p[v] = h[(long)(row0 + t) * W + c + v];
    }
}

long short_conv_rows() { return CONV_ROWS; }

void short_conv_add(torch::Tensor h, torch::Tensor w, torch::Tensor ring,
                    c10::optional<torch::Tensor> cu, c10::optional<torch::Tensor> bseq,
                    c10::optional<torch::Tensor> boff, torch::Tensor starts,
                    torch::Tensor slots, torch::Tensor out) {
  const int T_ = h.size(0), W = h.size(1), taps = w.size(0), S = slots.numel();
  TORCH_CHECK(h.is_cuda() && h.is_contiguous() && out.is_contiguous() &&
              out.sizes() == h.sizes() && out.dtype() == h.dtype());
  TORCH_CHECK(w.is_contiguous() && w.size(1) == W && w.dtype() == torch::kFloat32);
  TORCH_CHECK(taps >= 1 && taps <= CONV_MAX_TAPS, "a convolution of ", taps, " taps");
  TORCH_CHECK(ring.is_contiguous() && ring.dtype() == h.dtype() && ring.dim() == 3 &&
              ring.size(1) == taps - 1 && ring.size(2) == W, "convolution state");
  TORCH_CHECK(starts.numel() == S && starts.dtype() == torch::kInt32 &&
              slots.dtype() == torch::kInt32);
  int blocks = T_;
  if (cu) {
    TORCH_CHECK(bseq && boff && bseq->numel() == boff->numel() &&
                cu->numel() == S + 1 && cu->dtype() == torch::kInt32 &&
                bseq->dtype() == torch::kInt32 && boff->dtype() == torch::kInt32);
    blocks = bseq->numel();
  } else {
    TORCH_CHECK(S == T_);
  }
  if (T_ == 0 || blocks == 0) return;
  DISPATCH_ELEM(h.dtype() == torch::kBFloat16, {
    constexpr int VW = 16 / sizeof(T);
    auto launch = [&](auto kern, int v) {
      const int per = 256 * v;
      hipLaunchKernelGGL(kern, dim3(blocks, (W + per - 1) / per), dim3(256), 0, CUR_STREAM,
                         (const T*)h.data_ptr(), w.data_ptr<float>(), (T*)ring.data_ptr(),
                         cu ? cu->data_ptr<int>() : nullptr,
                         cu ? bseq->data_ptr<int>() : nullptr,
                         cu ? boff->data_ptr<int>() : nullptr, starts.data_ptr<int>(),
                         slots.data_ptr<int>(), (T*)out.data_ptr(), W, taps);
    };
    if (W % VW) launch(short_conv_kernel<T, 1, 0>, 1);
    else if (taps == 1) launch(short_conv_kernel<T, VW, 1>, VW);
    else if (taps == 2) launch(short_conv_kernel<T, VW, 2>, VW);
    else if (taps == 3) launch(short_conv_kernel<T, VW, 3>, VW);
    else if (taps == 4) launch(short_conv_kernel<T, VW, 4>, VW);
    else if (taps == 5) launch(short_conv_kernel<T, VW, 5>, VW);
    else if (taps == 6) launch(short_conv_kernel<T, VW, 6>, VW);
    else launch(short_conv_kernel<T, 1, 0>, 1);
  });
  HIP_CHECK_KERNEL();
}

// -------------------------------------------------------------------- xIELU

// above zero: softplus(p) z^2 + z/2; below: (1/2 + softplus(q)) (e^z - 1 - z) + z/2
template <typename T, int V>
__global__ __launch_bounds__(256) void xielu_kernel(const T* __restrict__ z, long stride,
                                                    const float* __restrict__ act,
                                                    T* __restrict__ out, long total, int F) {
  const float up = softplus_f(act[0]), down = 0.5f + softplus_f(act[1]);
  const long i = ((long)blockIdx.x * 256 + threadIdx.x) * V;
  if (i >= total) return;
  const T* p = z + i / F * stride + i % F;
  auto f = [&](float x) {
    // 16-bit: e^z - 1 taken as it stands is off by 1e-7 at most, which shows only
    // next to inputs (and so results) of 1e-5
    const float y = fminf(x, 0.f);
    const float low = down * ((sizeof(T) == 2 ? __expf(y) - 1.f : expm1f(y)) - y);
    return (x > 0.f ? up * x * x : low) + 0.5f * x;
  };
  if constexpr (V % 4 == 0) {
#pragma unroll
    for (int v = 0; v < V; v += 4) {
      floatx4 x = ld4(p + v);
#pragma unroll
      for (int j = 0; j < 4; ++j) x[j] = f(x[j]);
      st4(out + i + v, x);
    }
  } else {
    stf(out + i, f(ldf(p)));
  }
}

torch::Tensor xielu(torch::Tensor z, torch::Tensor act) {
  TORCH_CHECK(z.is_cuda() && z.dim() == 2 && z.stride(1) == 1);
  TORCH_CHECK(act.numel() == 2 && act.dtype() == torch::kFloat32 && act.is_contiguous());
  const int T_ = z.size(0), F = z.size(1);
  auto out = torch::empty({T_, F}, z.options());
  const long total = (long)T_ * F;
  if (total == 0) return out;
  DISPATCH_ELEM(z.dtype() == torch::kBFloat16, {
    constexpr int VW = 16 / sizeof(T);
    auto launch = [&](auto kern, int v) {
      hipLaunchKernelGGL(kern, dim3((total + 256 * v - 1) / (256 * v)), dim3(256), 0,
                         CUR_STREAM, (const T*)z.data_ptr(), z.stride(0),
                         act.data_ptr<float>(), (T*)out.data_ptr(), total, F);
    };
    const bool vec = F % VW == 0 && z.stride(0) % VW == 0 &&
                     (reinterpret_cast<uintptr_t>(z.data_ptr()) & 15) == 0;
    if (vec) launch(xielu_kernel<T, VW>, VW);
    else launch(xielu_kernel<T, 1>, 1);
  });
  HIP_CHECK_KERNEL();
  return out;
}

// ---------------------------------------------------- gelu, relu^2, silu GLU

// f(a, b) of the columns i and i + F of z [T, stride] (GLU), or f(a, 0)
template <typename T, int V, bool GLU, typename Fn>
__global__ __launch_bounds__(256) void activation_kernel(const T* __restrict__ z, long stride,
                                                         T* __restrict__ out, long total,
                                                         int F, Fn f) {
  const long i = ((long)blockIdx.x * 256 + threadIdx.x) * V;
  if (i >= total) return;
  const T* p = z + i / F * stride + i % F;
  if constexpr (V % 4 == 0) {
#pragma unroll
    for (int v = 0; v < V; v += 4) {
      floatx4 a = ld4(p + v), b = {0.f, 0.f, 0.f, 0.f};
      if constexpr (GLU) b = ld4(p + F + v);
#pragma unroll
      for (int j = 0; j < 4; ++j) a[j] = f(a[j], b[j]);
      st4(out + i + v, a);
    }
  } else {
    stf(out + i, f(ldf(p), GLU ? ldf(p + F) : 0.f));
  }
}

struct ExactGelu {
  DEVINL float operator()(float x, float) const {
    return 0.5f * x * (1.f + erff(x * 0.70710678f));
  }
};
struct SquaredRelu {
  DEVINL float operator()(float x, float) const {
    const float y = fmaxf(x, 0.f);
    return y * y;
  }
};
struct SiluTimes {
  DEVINL float operator()(float g, float u) const { return silu_f(g) * u; }
};

template <bool GLU, typename Fn>
static torch::Tensor activate(const torch::Tensor& z, long F, Fn f) {
  TORCH_CHECK(z.is_cuda() && z.dim() == 2 && z.stride(1) == 1 && F >= 1 &&
              z.size(1) >= (GLU ? 2 : 1) * F);
  const long T_ = z.size(0), total = T_ * F;
  auto out = torch::empty({T_, F}, z.options());
  if (total == 0) return out;
  DISPATCH_ELEM(z.dtype() == torch::kBFloat16, {
    constexpr int VW = 16 / sizeof(T);
    auto launch = [&](auto kern, int v) {
      hipLaunchKernelGGL(kern, dim3((total + 256 * v - 1) / (256 * v)), dim3(256), 0,
                         CUR_STREAM, (const T*)z.data_ptr(), z.stride(0),
                         (T*)out.data_ptr(), total, (int)F, f);
    };
    const bool vec = F % VW == 0 && z.stride(0) % VW == 0 &&
                     (reinterpret_cast<uintptr_t>(z.data_ptr()) & 15) == 0;
    if (vec) launch(activation_kernel<T, VW, GLU, Fn>, VW);
    else launch(activation_kernel<T, 1, GLU, Fn>, 1);
  });
  HIP_CHECK_KERNEL();
  return out;
}

torch::Tensor gelu(torch::Tensor z) { return activate<false>(z, z.size(1), ExactGelu{}); }

torch::Tensor relu2(torch::Tensor z) { return activate<false>(z, z.size(1), SquaredRelu{}); }

// z [T, 2 F or more]: gate columns, then up columns
torch::Tensor silu_glu(torch::Tensor z, long F) { return activate<true>(z, F, SiluTimes{}); }
