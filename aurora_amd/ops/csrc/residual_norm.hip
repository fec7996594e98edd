// Residual-stream kernels of the layer-listed decoders.
//
// residual_rmsnorm: the residual is ONE fp32 tensor. The kernel that norms it
// also adds what came before: a sub-layer's output, scaled by its residual gate
// if it has one, or the chosen experts' rows with their routing weights (so no
// separate combine pass exists), and the vector that marks a pass of a repeated
// span. What the sub-layer and the experts give together may be normed before it is
// added. In steps of single tokens the kernel also adds the next sublayer's input
// convolution to the result. One workgroup per row, the row lives in LDS
// between the sum of squares and the scaling: x is read and written once,
// everything else once.
//
// bias_kv_write: splits the fused projection, adds the biases in fp32, and
// scatters K/V to the paged cache; heads are stored at the cache's width.
#include "elem.h"
#include <torch/extension.h>
#include <c10/hip/HIPStream.h>

#define CUR_STREAM c10::hip::getCurrentHIPStream().stream()

// the sub-layer's output is multiplied by sigmoid(pre + bias)
template <typename T>
struct ResidualGate {
  const T* pre;  // [T, stride], null: no gate
  long stride;
  const float* bias;
};

// causal convolution of the normed rows, one token per sequence: the ring holds
// position p's row at p mod (taps - 1); slot -1 has no past and stores nothing
template <typename T>
struct ConvTail {
  const float* w;  // [taps, W], the last row the present; null: no convolution
  int taps;
  T* ring;         // [slots, taps - 1, W]
  const int* pos;
  const int* slots;
  T* out;          // [T, W]
};

// NTHR threads per row: 1024 where few wide rows would leave the chip waiting. POST:
// the result is normed, times ``post``, before it is added
template <typename T, int V, int NTHR, bool POST>
__global__ __launch_bounds__(NTHR) void residual_rmsnorm_kernel(
    float* __restrict__ x, const float* __restrict__ weight,
    const T* __restrict__ delta, ResidualGate<T> rg, const T* __restrict__ y,
    const int* __restrict__ place, const float* __restrict__ gate, int top,
    const float* __restrict__ post, const float* __restrict__ step, T* __restrict__ out,
    ConvTail<T> cv, int W, float eps, float offset) {
  extern __shared__ __attribute__((aligned(16))) float row[];
  __shared__ float red[NTHR / WAVE];
  const long base = (long)blockIdx.x * W;
  const int* pl = place + (long)blockIdx.x * top;
  const float* gt = gate + (long)blockIdx.x * top;
  const T* pre = rg.pre ? rg.pre + blockIdx.x * rg.stride : nullptr;
  float ss = 0.f;
  if constexpr (POST) {
    typedef __attribute__((ext_vector_type(V))) float vec;
    auto loadf = [](const float* p) {
      if constexpr (V == 4) return ld4(p);
      else return vec(*p);
    };
    auto load = [](const T* p) {
      if constexpr (V == 4) return ld4(p);
      else return vec(ldf(p));
    };
    auto store = [](float* p, vec v) {
      if constexpr (V == 4) st4(p, v);
      else *p = v[0];
    };
    float rs = 0.f;
    for (int i = threadIdx.x * V; i < W; i += NTHR * V) {
      vec r = vec(0.f);
      if (delta) r = load(delta + base + i);
      if (y)
        for (int j = 0; j < top; ++j) r += gt[j] * load(y + (long)pl[j] * W + i);
      store(row + i, r);
#pragma unroll
      for (int j = 0; j < V; ++j) rs += r[j] * r[j];
    }
    const float rinv = rsqrtf(block_sum<NTHR / WAVE>(rs, red) / W + eps);
    for (int i = threadIdx.x * V; i < W; i += NTHR * V) {  // what the thread wrote
      vec v = loadf(x + base + i) + loadf(row + i) * rinv * loadf(post + i);
      if (step) v += loadf(step + i);
      store(row + i, v);
      store(x + base + i, v);
#pragma unroll
      for (int j = 0; j < V; ++j) ss += v[j] * v[j];
    }
  } else
  for (int i = threadIdx.x * V; i < W; i += NTHR * V) {
    float v[V];
    if constexpr (V == 4) {
      floatx4 a = ld4(x + base + i);
      if (delta) {
        floatx4 d = ld4(delta + base + i);
        if (pre) {
          const floatx4 g = ld4(pre + i) + ld4(rg.bias + i);
#pragma unroll
          for (int j = 0; j < 4; ++j) d[j] *= sigmoid_f(g[j]);
        }
        a += d;
      }
      if (y) {
        for (int j = 0; j < top; ++j) a += gt[j] * ld4(y + (long)pl[j] * W + i);
      }
      if (step) a += ld4(step + i);
#pragma unroll
      for (int j = 0; j < 4; ++j) v[j] = a[j];
      *reinterpret_cast<floatx4*>(row + i) = a;
      if (delta || y || step) st4(x + base + i, a);
    } else {
      float a = x[base + i];
      if (delta) {
        const float d = ldf(delta + base + i);
        a += pre ? d * sigmoid_f(ldf(pre + i) + rg.bias[i]) : d;
      }
      if (y)
        for (int j = 0; j < top; ++j) a += gt[j] * ldf(y + (long)pl[j] * W + i);
      if (step) a += step[i];
      v[0] = a;
      row[i] = a;
      x[base + i] = a;
    }
#pragma unroll
    for (int j = 0; j < V; ++j) ss += v[j] * v[j];
  }
  const float inv = rsqrtf(block_sum<NTHR / WAVE>(ss, red) / W + eps);
  const int keep = cv.taps - 1;
  const int slot = cv.w ? cv.slots[blockIdx.x] : -1;
  const int pos = cv.w ? cv.pos[blockIdx.x] : 0;
  T* ring = cv.ring + (long)max(slot, 0) * keep * W;
  const int known = slot >= 0 ? min(keep, pos) : 0;  // rows of the past
  for (int i = threadIdx.x * V; i < W; i += NTHR * V) {
    if constexpr (V == 4) {
      const floatx4 a = *reinterpret_cast<const floatx4*>(row + i);
      st4(out + base + i, a * inv * (offset + ld4(weight + i)));
    } else {
      stf(out + base + i, row[i] * inv * (offset + weight[i]));
    }
    if (!cv.w) continue;
    // from here on the row as stored; its place in the ring is the oldest row's,
    // read before
    const float* w = cv.w + (long)keep * W + i;
    T* mine = slot >= 0 && keep > 0 ? ring + (long)(pos % keep) * W + i : nullptr;
    if constexpr (V == 4) {
      const floatx4 y = ld4(out + base + i);
      floatx4 u = y + y * ld4(w);
#pragma unroll 4
      for (int b = 1; b <= known; ++b)
        u += ld4(w - (long)b * W) * ld4(ring + (long)((pos - b) % keep) * W + i);
      st4(cv.out + base + i, u);
      if (mine) st4(mine, y);
    } else {
      const float y = ldf(out + base + i);
      float u = y + y * *w;
      for (int b = 1; b <= known; ++b)
        u += w[-(long)b * W] * ldf(ring + (long)((pos - b) % keep) * W + i);
      stf(cv.out + base + i, u);
      if (mine) stf(mine, y);
    }
  }
}

std::vector<torch::Tensor> residual_rmsnorm(
    torch::Tensor x, torch::Tensor weight, c10::optional<torch::Tensor> delta,
    c10::optional<torch::Tensor> gate_pre, c10::optional<torch::Tensor> gate_bias,
    c10::optional<torch::Tensor> y, c10::optional<torch::Tensor> place,
    c10::optional<torch::Tensor> gate, c10::optional<torch::Tensor> post,
    c10::optional<torch::Tensor> step, c10::optional<torch::Tensor> conv_w, c10::optional<torch::Tensor> ring,
    c10::optional<torch::Tensor> pos, c10::optional<torch::Tensor> slots, double eps,
    double offset, bool to_bf16) {
  TORCH_CHECK(x.is_cuda() && x.dim() == 2 && x.is_contiguous() &&
              x.dtype() == torch::kFloat32, "residual must be fp32 [T, W]");
  const int T_ = x.size(0), W = x.size(1);
  TORCH_CHECK(weight.numel() == W && weight.dtype() == torch::kFloat32);
  TORCH_CHECK(W <= 32768, "row too wide for LDS");
  const auto dt = to_bf16 ? torch::kBFloat16 : torch::kFloat32;
  std::vector<torch::Tensor> out = {torch::empty({T_, W}, x.options().dtype(dt))};
  if (delta)
    TORCH_CHECK(delta->is_contiguous() && delta->sizes() == x.sizes() &&
                delta->dtype() == dt, "delta");
  if (gate_pre)
    TORCH_CHECK(delta && gate_bias && gate_pre->sizes() == x.sizes() &&
                gate_pre->stride(1) == 1 && gate_pre->dtype() == dt &&
                gate_bias->numel() == W && gate_bias->dtype() == torch::kFloat32,
                "residual gate");
  int top = 0;
  if (y) {
    TORCH_CHECK(place && gate && y->is_contiguous() && y->size(1) == W &&
                y->dtype() == dt && place->is_contiguous() && gate->is_contiguous() &&
                place->dtype() == torch::kInt32 && gate->dtype() == torch::kFloat32 &&
                place->size(0) == T_ && place->sizes() == gate->sizes(), "expert rows");
    top = place->size(1);
  }
  if (post)
    TORCH_CHECK(post->numel() == W && post->dtype() == torch::kFloat32 &&
                post->is_contiguous() && !gate_pre && (delta || y), "norm of the result");
  if (step) TORCH_CHECK(step->numel() == W && step->dtype() == torch::kFloat32);
  if (conv_w) {
    TORCH_CHECK(ring && pos && slots && conv_w->is_contiguous() && conv_w->size(1) == W &&
                conv_w->dtype() == torch::kFloat32 && ring->dim() == 3 &&
                ring->is_contiguous() && ring->dtype() == dt && ring->size(2) == W &&
                ring->size(1) == conv_w->size(0) - 1, "input convolution");
    TORCH_CHECK(pos->numel() == T_ && slots->numel() == T_ &&
                pos->dtype() == torch::kInt32 && slots->dtype() == torch::kInt32);
    out.push_back(torch::empty_like(out[0]));
  }
  if (T_ == 0) return out;
  const size_t lds = (size_t)W * 4;
  DISPATCH_ELEM(to_bf16, {
    ResidualGate<T> rg = {nullptr, 0, nullptr};
    if (gate_pre)
      rg = {(const T*)gate_pre->data_ptr(), gate_pre->stride(0), gate_bias->data_ptr<float>()};
    ConvTail<T> cv = {nullptr, 1, nullptr, nullptr, nullptr, nullptr};
    if (conv_w)
      cv = {conv_w->data_ptr<float>(), (int)conv_w->size(0), (T*)ring->data_ptr(),
            pos->data_ptr<int>(), slots->data_ptr<int>(), (T*)out[1].data_ptr()};
    auto launch = [&](auto kern, int threads) {
      hipLaunchKernelGGL(
          kern, dim3(T_), dim3(threads), lds, CUR_STREAM, x.data_ptr<float>(),
          weight.data_ptr<float>(), delta ? (const T*)delta->data_ptr() : nullptr, rg,
          y ? (const T*)y->data_ptr() : nullptr,
          y ? place->data_ptr<int>() : nullptr, y ? gate->data_ptr<float>() : nullptr,
          top, post ? post->data_ptr<float>() : nullptr, step ? step->data_ptr<float>() : nullptr, (T*)out[0].data_ptr(), cv, W,
          (float)eps, (float)offset);
    };
    const bool vec = W % 4 == 0 && (!gate_pre || (gate_pre->stride(0) % 4 == 0 &&
                     (reinterpret_cast<uintptr_t>(gate_pre->data_ptr()) & 15) == 0));
    const bool wide = vec && T_ <= 256 && W > 1024;
    if (post) {
      if (wide) launch(residual_rmsnorm_kernel<T, 4, 1024, true>, 1024);
      else if (vec) launch(residual_rmsnorm_kernel<T, 4, 256, true>, 256);
      else launch(residual_rmsnorm_kernel<T, 1, 256, true>, 256);
    } else {
      if (wide) launch(residual_rmsnorm_kernel<T, 4, 1024, false>, 1024);
      else if (vec) launch(residual_rmsnorm_kernel<T, 4, 256, false>, 256);
      else launch(residual_rmsnorm_kernel<T, 1, 256, false>, 256);
    }
  });
  HIP_CHECK_KERNEL();
  return out;
}

// V elements per thread (16 bytes): query heads first, then key, then value heads
template <typename T, int V>
__global__ __launch_bounds__(256) void bias_kv_write_vec_kernel(
    const T* __restrict__ proj, long stride, int q0, int k0, int v0,
    const float* __restrict__ bias, const int* __restrict__ slots,
    T* __restrict__ q_out, T* __restrict__ kc, T* __restrict__ vc, long total, int Hq,
    int Hkv, int d, int dv, int DK, int DV, int P) {
  const long id = (long)blockIdx.x * 256 + threadIdx.x;
  if (id >= total) return;
  const int per = (Hq * DK + Hkv * (DK + DV)) / V;  // threads per token
  const int t = id / per;
  int x = (id % per) * V;
  int col, b0, n;
  T* dst;
  if (x < Hq * DK) {
    const int h = x / DK;
    n = d;
    dst = q_out + (long)t * Hq * DK + x;
    x -= h * DK;
    col = q0 + h * d;
    b0 = h * d;
  } else {
    const int slot = slots[t];
    if (slot < 0) return;
    x -= Hq * DK;
    const bool key = x < Hkv * DK;
    if (!key) x -= Hkv * DK;
    const int width = key ? DK : DV;
    const int h = x / width;
    n = key ? d : dv;
    x -= h * width;
    dst = (key ? kc : vc) + (((long)(slot / P) * Hkv + h) * P + slot % P) * width + x;
    col = (key ? k0 : v0) + h * n;
    b0 = (Hq + (key ? 0 : Hkv)) * d + h * n;
  }
  const T* src = proj + (long)t * stride + col + x;
#pragma unroll
  for (int i = 0; i < V; i += 4) {
    floatx4 y = {0.f, 0.f, 0.f, 0.f};
    if (x + i < n) y = ld4(src + i) + ld4(bias + b0 + x + i);
    st4(dst + i, y);
  }
}

// any size: one wave per (token, head)
template <typename T>
__global__ __launch_bounds__(256) void bias_kv_write_kernel(
    const T* __restrict__ proj, long stride, int q0, int k0, int v0,
    const float* __restrict__ bias, const int* __restrict__ slots,
    T* __restrict__ q_out, T* __restrict__ kc, T* __restrict__ vc, int T_, int Hq,
    int Hkv, int d, int dv, int DK, int DV, int P) {
  const int HT = Hq + 2 * Hkv;
  const long wid = (long)blockIdx.x * 4 + threadIdx.x / WAVE;
  const int lane = threadIdx.x % WAVE;
  if (wid >= (long)T_ * HT) return;
  const int t = wid / HT;
  int h = wid % HT;
  int col, b0, n, width;
  T* dst;
  if (h < Hq) {
    col = q0 + h * d;
    b0 = h * d;
    n = d;
    width = DK;
    dst = q_out + ((long)t * Hq + h) * DK;
  } else {
    const int slot = slots[t];
    if (slot < 0) return;
    const bool key = h < Hq + Hkv;
    h -= key ? Hq : Hq + Hkv;
    n = key ? d : dv;
    width = key ? DK : DV;
    col = (key ? k0 : v0) + h * n;
    b0 = (Hq + (key ? 0 : Hkv)) * d + h * n;
    dst = (key ? kc : vc) + (((long)(slot / P) * Hkv + h) * P + slot % P) * width;
  }
  const T* src = proj + (long)t * stride + col;
  for (int i = lane; i < width; i += WAVE)
    stf(dst + i, i < n ? ldf(src + i) + bias[b0 + i] : 0.f);
}

torch::Tensor bias_kv_write(torch::Tensor proj, long q0, long k0, long v0,
                            torch::Tensor bias, torch::Tensor slots,
                            torch::Tensor kc, torch::Tensor vc, long Hq, long Hkv,
                            long d, long dv) {
  TORCH_CHECK(proj.is_cuda() && proj.dim() == 2 && proj.stride(1) == 1);
  TORCH_CHECK(kc.dtype() == proj.dtype() && vc.dtype() == proj.dtype());
  TORCH_CHECK(kc.is_contiguous() && vc.is_contiguous() && kc.size(1) == Hkv &&
              vc.size(1) == Hkv && kc.size(2) == vc.size(2));
  const int T_ = proj.size(0), DK = kc.size(3), DV = vc.size(3), P = kc.size(2);
  TORCH_CHECK(DK >= d && DV >= dv, "cache heads narrower than the model's");
  TORCH_CHECK(q0 + Hq * d <= proj.size(1) && k0 + Hkv * d <= proj.size(1) &&
              v0 + Hkv * dv <= proj.size(1));
  TORCH_CHECK(bias.numel() == Hq * d + Hkv * (d + dv) &&
              bias.dtype() == torch::kFloat32);
  TORCH_CHECK(slots.numel() == T_ && slots.dtype() == torch::kInt32);
  auto q = torch::empty({(long)T_, Hq, (long)DK}, proj.options());
  if (T_ == 0) return q;
  const long waves = (long)T_ * (Hq + 2 * Hkv);
  if ((((d | dv | DK | DV | q0 | k0 | v0) & 7) | (proj.stride(0) & 7)) == 0) {
    DISPATCH_ELEM(proj.dtype() == torch::kBFloat16, {
      constexpr int V = 16 / sizeof(T);
      const long total = (long)T_ * ((Hq * DK + Hkv * (DK + DV)) / V);
      hipLaunchKernelGGL((bias_kv_write_vec_kernel<T, V>), dim3((total + 255) / 256),
                         dim3(256), 0, CUR_STREAM, (const T*)proj.data_ptr(),
                         proj.stride(0), (int)q0, (int)k0, (int)v0,
                         bias.data_ptr<float>(), slots.data_ptr<int>(), (T*)q.data_ptr(),
                         (T*)kc.data_ptr(), (T*)vc.data_ptr(), total, (int)Hq, (int)Hkv,
                         (int)d, (int)dv, DK, DV, P);
    });
    HIP_CHECK_KERNEL();
    return q;
  }
  DISPATCH_ELEM(proj.dtype() == torch::kBFloat16, {
    hipLaunchKernelGGL((bias_kv_write_kernel<T>), dim3((waves + 3) / 4), dim3(256), 0,
                       CUR_STREAM, (const T*)proj.data_ptr(), proj.stride(0), (int)q0,
                       (int)k0, (int)v0, bias.data_ptr<float>(), slots.data_ptr<int>(),
                       (T*)q.data_ptr(), (T*)kc.data_ptr(), (T*)vc.data_ptr(), T_,
                       (int)Hq, (int)Hkv, (int)d, (int)dv, DK, DV, P);
  });
  HIP_CHECK_KERNEL();
  return q;
}
