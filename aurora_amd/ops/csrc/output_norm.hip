// Residual-stream kernels of decoders that norm their sublayers' OUTPUTS.
//
// output_norm: one kernel per sublayer. The result r is put together (a dense
// output, scaled by one sigmoid gate per row if it has one, plus the chosen
// experts' rows with their routing weights), its layer norm is added to the fp32
// residual, and what goes on is written twice: as the residual and as the next
// sublayer's input. After a layer the same kernel keeps the layer's result and
// replaces the residual by the weighted sum of all results kept so far, the
// embedding first; after the last layer it takes the final norm as well. One
// workgroup per row, the row lives in LDS between the passes.
//
// normed_qkv: splits the fused projection, norms queries and keys per head or over
// all heads of a token, rotates and scales them, and scatters keys and values to the
// paged cache, heads stored at the cache's width. Values may be the plain keys.
#include "elem.h"
#include <torch/extension.h>
#include <c10/hip/HIPStream.h>

#define CUR_STREAM c10::hip::getCurrentHIPStream().stream()

template <typename T>
struct OutputArgs {
  const float* src;      // [T, W]
  float* x;              // [T, W], may be src
  const float *w, *b;    // [W]
  const T* delta;        // [T, W] or null
  const T* gate;         // one number per row, gstride apart, or null
  long gstride;
  const T* y;            // expert rows, or null
  const int* place;      // [T, top]
  const float* share;    // [T, top]
  int top;
  float* kept;           // [room, T, W] or null: no depth average
  const float* coefs;    // [depth + 1]
  int depth;
  bool room;             // entry ``depth`` exists
  const float *fw, *fb;  // [W] or null: no final norm
  T* out;                // [T, W]
  int W;
  float eps;
};

template <typename T, int V, int NTHR>
__global__ __launch_bounds__(NTHR) void output_norm_kernel(OutputArgs<T> a, long TW) {
  extern __shared__ __attribute__((aligned(16))) float row[];
  __shared__ float red[NTHR / WAVE];
  typedef __attribute__((ext_vector_type(V))) float vec;
  const int W = a.W;
  const long base = (long)blockIdx.x * W;
  auto loadf = [](const float* p) {
    if constexpr (V == 4) return ld4(p);
    else return vec(*p);
  };
  auto load = [](const T* p) {
    if constexpr (V == 4) return ld4(p);
    else return vec(ldf(p));
  };
  auto storef = [](float* p, vec v) {
    if constexpr (V == 4) st4(p, v);
    else *p = v[0];
  };
  auto store = [](T* p, vec v) {
    if constexpr (V == 4) st4(p, v);
    else stf(p, v[0]);
  };
  auto each = [&](auto f) {
    for (int i = threadIdx.x * V; i < W; i += NTHR * V) f(i);
  };
  auto sum = [](vec v) {
    float s = 0.f;
#pragma unroll
    for (int j = 0; j < V; ++j) s += v[j];
    return s;
  };
  auto total = [&](float s) { return block_sum<NTHR / WAVE>(s, red); };
  // 1 / sqrt(mean of the squared deviations + eps); a thread reads what it wrote
  auto inverse = [&](float mean) {
    float ss = 0.f;
    each([&](int i) {
      const vec d = loadf(row + i) - mean;
      ss += sum(d * d);
    });
    return rsqrtf(total(ss) / W + a.eps);
  };

  const int* pl = a.place + (long)blockIdx.x * a.top;
  const float* sh = a.share + (long)blockIdx.x * a.top;
  const float g = a.gate ? sigmoid_f(ldf(a.gate + blockIdx.x * a.gstride)) : 1.f;
  float s = 0.f;
  each([&](int i) {
    vec r = vec(0.f);
    if (a.delta) r = g * load(a.delta + base + i);
    if (a.y)
      for (int j = 0; j < a.top; ++j) r += sh[j] * load(a.y + (long)pl[j] * W + i);
    storef(row + i, r);
    s += sum(r);
  });
  const float mean = total(s) / W, inv = inverse(mean);
  s = 0.f;
  each([&](int i) {
    vec v = loadf(a.src + base + i) + (loadf(row + i) - mean) * inv * loadf(a.w + i) +
            loadf(a.b + i);
    if (a.kept) {
      float* k = a.kept + base + i;
      if (a.room) storef(k + a.depth * TW, v);
      v *= a.coefs[a.depth];
#pragma unroll 4
      for (int j = 0; j < a.depth; ++j) v += a.coefs[j] * loadf(k + j * TW);
    }
    storef(a.x + base + i, v);
    if (!a.fw) {
      store(a.out + base + i, v);
    } else {
      storef(row + i, v);
      s += sum(v);
    }
  });
  if (!a.fw) return;
  const float fmean = total(s) / W, finv = inverse(fmean);
  each([&](int i) {
    store(a.out + base + i,
          (loadf(row + i) - fmean) * finv * loadf(a.fw + i) + loadf(a.fb + i));
  });
}

torch::Tensor output_norm(torch::Tensor src, torch::Tensor x, torch::Tensor weight,
                          torch::Tensor bias, c10::optional<torch::Tensor> delta,
                          c10::optional<torch::Tensor> gate, c10::optional<torch::Tensor> y,
                          c10::optional<torch::Tensor> place,
                          c10::optional<torch::Tensor> share,
                          c10::optional<torch::Tensor> kept,
                          c10::optional<torch::Tensor> coefs,
                          c10::optional<torch::Tensor> fw, c10::optional<torch::Tensor> fb,
                          double eps, bool to_bf16) {
  TORCH_CHECK(src.is_cuda() && src.dim() == 2 && src.is_contiguous() && x.is_contiguous() &&
              src.dtype() == torch::kFloat32 && x.dtype() == torch::kFloat32 &&
              x.sizes() == src.sizes(), "residual must be fp32 [T, W]");
  const int T_ = src.size(0), W = src.size(1);
  auto vector = [&](const torch::Tensor& t) {
    return t.numel() == W && t.dtype() == torch::kFloat32 && t.is_contiguous();
  };
  TORCH_CHECK(vector(weight) && vector(bias), "norm weight and bias");
  TORCH_CHECK(W <= 32768, "row too wide for LDS");
  const auto dt = to_bf16 ? torch::kBFloat16 : torch::kFloat32;
  if (delta)
    TORCH_CHECK(delta->is_contiguous() && delta->sizes() == src.sizes() &&
                delta->dtype() == dt, "delta");
  if (gate)
    TORCH_CHECK(delta && gate->dim() == 1 && gate->size(0) == T_ && gate->dtype() == dt,
                "row gate");
  int top = 0;
  if (y) {
    TORCH_CHECK(place && share && y->is_contiguous() && y->size(1) == W &&
                y->dtype() == dt && place->is_contiguous() && share->is_contiguous() &&
                place->dtype() == torch::kInt32 && share->dtype() == torch::kFloat32 &&
                place->size(0) == T_ && place->sizes() == share->sizes(), "expert rows");
    top = place->size(1);
  }
  if (kept)
    TORCH_CHECK(coefs && coefs->numel() >= 2 && coefs->dtype() == torch::kFloat32 &&
                coefs->is_contiguous() && kept->is_contiguous() && kept->dim() == 3 &&
                kept->dtype() == torch::kFloat32 && kept->size(1) == T_ &&
                kept->size(2) == W && kept->size(0) >= coefs->numel() - 1, "depth average");
  if (fw) TORCH_CHECK(fb && vector(*fw) && vector(*fb), "final norm");
  auto out = torch::empty({T_, W}, src.options().dtype(dt));
  if (T_ == 0) return out;
  DISPATCH_ELEM(to_bf16, {
    OutputArgs<T> a = {};
    a.src = src.data_ptr<float>();
    a.x = x.data_ptr<float>();
    a.w = weight.data_ptr<float>();
    a.b = bias.data_ptr<float>();
    if (delta) a.delta = (const T*)delta->data_ptr();
    if (gate) {
      a.gate = (const T*)gate->data_ptr();
      a.gstride = gate->stride(0);
    }
    if (y) {
      a.y = (const T*)y->data_ptr();
      a.place = place->data_ptr<int>();
      a.share = share->data_ptr<float>();
      a.top = top;
    }
    if (kept) {
      a.kept = kept->data_ptr<float>();
      a.coefs = coefs->data_ptr<float>();
      a.depth = (int)coefs->numel() - 1;
      a.room = a.depth < kept->size(0);
    }
    if (fw) {
      a.fw = fw->data_ptr<float>();
      a.fb = fb->data_ptr<float>();
    }
    a.out = (T*)out.data_ptr();
    a.W = W;
    a.eps = eps;
    auto launch = [&](auto kern, int threads) {
      const size_t lds = (size_t)W * 4;
      if (lds > 48 * 1024)
        (void)hipFuncSetAttribute((const void*)kern,
                                  hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds);
      hipLaunchKernelGGL(kern, dim3(T_), dim3(threads), lds, CUR_STREAM, a, (long)T_ * W);
    };
    if (W % 4 == 0 && T_ <= 256 && W > 1024) launch(output_norm_kernel<T, 4, 1024>, 1024);
    else if (W % 4 == 0) launch(output_norm_kernel<T, 4, 256>, 256);
    else launch(output_norm_kernel<T, 1, 256>, 256);
  });
  HIP_CHECK_KERNEL();
  return out;
}

// -------------------------------------------------------------- normed heads

struct HeadArgs {
  const void* proj;    // [T, stride]
  long stride;
  int q0, k0, v0;      // columns; v0 = k0: values are plain keys
  const float *qw, *kw;
  const float* cos_sin;  // [positions, rot] or null
  int rot;
  float coef;          // query temperature; 0: none
  int every;
  const int *pos, *slots;  // [T]
  void *q, *kc, *vc;   // [T, Hq, DK], [pages, Hkv, P, DK | DV]
  int Hq, Hkv, d, dv, DK, DV, P;
  int GL;              // lanes per head in the norms
  float eps;
};

// one workgroup per token; V elements (16 bytes) per access, then d, dv, DK, DV, rot
// and the columns are multiples of 8
template <typename T, int V, bool WHOLE>
__global__ __launch_bounds__(256) void normed_qkv_kernel(HeadArgs a) {
  extern __shared__ __attribute__((aligned(16))) float lds[];
  __shared__ float red[4];
  const int t = blockIdx.x, tid = threadIdx.x, d = a.d, HT = a.Hq + a.Hkv;
  const T* proj = (const T*)a.proj + (long)t * a.stride;
  float* row = lds;              // [HT][d] as projected
  float* inv = lds + HT * d;     // [HT]
  // elements as fp32, four at a time where V allows
  constexpr int C = V >= 4 ? 4 : 1;
  typedef __attribute__((ext_vector_type(C))) float vec;
  auto load = [](const T* p) {
    if constexpr (C == 4) return ld4(p);
    else return vec(ldf(p));
  };
  auto loadf = [](const float* p) {
    if constexpr (C == 4) return ld4(p);
    else return vec(*p);
  };

  const int per = 256 / a.GL, sub = tid % a.GL;
  float q2 = 0.f, k2 = 0.f;
  for (int h = tid / a.GL; h < HT; h += per) {
    const T* src = proj + (h < a.Hq ? a.q0 + h * d : a.k0 + (h - a.Hq) * d);
    float s = 0.f;
    for (int c = sub * V; c < d; c += a.GL * V) {
#pragma unroll
      for (int v = 0; v < V; v += C) {
        const vec x = load(src + c + v);
        *reinterpret_cast<vec*>(row + h * d + c + v) = x;
#pragma unroll
        for (int j = 0; j < C; ++j) s += x[j] * x[j];
      }
    }
    if constexpr (WHOLE) {
      (h < a.Hq ? q2 : k2) += s;
    } else {
      for (int off = a.GL / 2; off > 0; off >>= 1) s += __shfl_xor(s, off, WAVE);
      if (sub == 0) inv[h] = rsqrtf(s / d + a.eps);
    }
  }
  float qi = 0.f, ki = 0.f;
  if constexpr (WHOLE) {
    qi = rsqrtf(block_sum4(q2, red) / (a.Hq * d) + a.eps);
    ki = rsqrtf(block_sum4(k2, red) / (a.Hkv * d) + a.eps);
  } else {
    __syncthreads();
  }
  const int pos = a.pos[t], slot = a.slots[t];
  const float temp = a.coef == 0.f ? 1.f
      : 1.f + a.coef * logf((float)((pos + 1) / a.every + 1));
  const int half = a.rot / 2;
  const float* cs = a.cos_sin + (long)pos * a.rot;
  const int nq = a.Hq * a.DK, nk = a.Hkv * a.DK, all = nq + nk + a.Hkv * a.DV;
  const long page = slot < 0 ? 0 : slot / a.P, place = slot < 0 ? 0 : slot % a.P;
  for (int x = tid * V; x < all; x += 256 * V) {
    const bool is_q = x < nq, is_v = x >= nq + nk;
    if (!is_q && slot < 0) break;  // an idle row has no place in the cache
    const int y = is_q ? x : is_v ? x - nq - nk : x - nq;
    const int width = is_v ? a.DV : a.DK, h = y / width, c = y % width;
    T* dst;
    if (is_q) dst = (T*)a.q + (long)t * nq + y;
    else dst = (T*)(is_v ? a.vc : a.kc) + ((page * a.Hkv + h) * a.P + place) * width + c;
    const int n = is_v ? a.dv : d, hh = is_q ? h : a.Hq + h;
    const float* src = row + hh * d;
    const float* w = (is_q ? a.qw : a.kw) + (WHOLE ? h * d : 0);
    const float f = is_v ? 1.f : (WHOLE ? (is_q ? qi : ki) : inv[hh]) * (is_q ? temp : 1.f);
#pragma unroll
    for (int v = 0; v < V; v += C) {
      const int i = c + v;
      vec r = vec(0.f);
      if (i < n) {
        if (is_v) {
          r = a.v0 == a.k0 ? loadf(src + i) : load(proj + a.v0 + h * n + i);
        } else {
          r = loadf(src + i) * loadf(w + i);
          if (i < half)
            r = r * loadf(cs + i) -
                loadf(src + half + i) * loadf(w + half + i) * loadf(cs + half + i);
          else if (i < a.rot)
            r = r * loadf(cs + i - half) +
                loadf(src + i - half) * loadf(w + i - half) * loadf(cs + i);
          r *= f;
        }
      }
      if constexpr (C == 4) st4(dst + v, r);
      else stf(dst, r[0]);
    }
  }
}

torch::Tensor normed_qkv(torch::Tensor proj, long q0, long k0, long v0, torch::Tensor qw,
                         torch::Tensor kw, bool whole, double eps,
                         c10::optional<torch::Tensor> cos_sin, double coef, long every,
                         torch::Tensor pos, torch::Tensor slots, torch::Tensor kc,
                         torch::Tensor vc, long Hq, long Hkv, long d, long dv) {
  TORCH_CHECK(proj.is_cuda() && proj.dim() == 2 && proj.stride(1) == 1);
  TORCH_CHECK(kc.dtype() == proj.dtype() && vc.dtype() == proj.dtype() && kc.is_contiguous() &&
              vc.is_contiguous() && kc.size(1) == Hkv && vc.size(1) == Hkv &&
              kc.size(2) == vc.size(2) && kc.size(0) == vc.size(0), "caches");
  const int T_ = proj.size(0), DK = kc.size(3), DV = vc.size(3), P = kc.size(2);
  TORCH_CHECK(DK >= d && DV >= dv, "cache heads narrower than the model's");
  TORCH_CHECK(Hkv >= 1 && Hq % Hkv == 0 && (v0 != k0 || d == dv));
  TORCH_CHECK(q0 + Hq * d <= proj.size(1) && k0 + Hkv * d <= proj.size(1) &&
              v0 + Hkv * dv <= proj.size(1));
  TORCH_CHECK(qw.numel() == (whole ? Hq * d : d) && kw.numel() == (whole ? Hkv * d : d) &&
              qw.dtype() == torch::kFloat32 && kw.dtype() == torch::kFloat32 &&
              qw.is_contiguous() && kw.is_contiguous(), "norm weights");
  TORCH_CHECK(pos.numel() == T_ && pos.dtype() == torch::kInt32 && pos.is_contiguous() &&
              slots.numel() == T_ && slots.dtype() == torch::kInt32 && slots.is_contiguous());
  TORCH_CHECK(every >= 1);
  HeadArgs a = {};
  if (cos_sin) {
    TORCH_CHECK(cos_sin->dtype() == torch::kFloat32 && cos_sin->is_contiguous() &&
                cos_sin->dim() == 2 && cos_sin->size(1) % 2 == 0 && cos_sin->size(1) <= d);
    a.cos_sin = cos_sin->data_ptr<float>();
    a.rot = cos_sin->size(1);
  }
  auto q = torch::empty({(long)T_, Hq, (long)DK}, proj.options());
  if (T_ == 0) return q;
  a.proj = proj.data_ptr();
  a.stride = proj.stride(0);
  a.q0 = q0; a.k0 = k0; a.v0 = v0;
  a.qw = qw.data_ptr<float>();
  a.kw = kw.data_ptr<float>();
  a.coef = coef;
  a.every = every;
  a.pos = pos.data_ptr<int>();
  a.slots = slots.data_ptr<int>();
  a.q = q.data_ptr();
  a.kc = kc.data_ptr();
  a.vc = vc.data_ptr();
  a.Hq = Hq; a.Hkv = Hkv; a.d = d; a.dv = dv; a.DK = DK; a.DV = DV; a.P = P;
  a.eps = eps;
  const size_t lds = (size_t)(Hq + Hkv) * (d + 1) * 4;
  TORCH_CHECK(lds <= 150 * 1024, "queries and keys of a token too wide for LDS");
  DISPATCH_ELEM(proj.dtype() == torch::kBFloat16, {
    constexpr int VW = 16 / sizeof(T);
    const bool vec = ((d | dv | DK | DV | q0 | k0 | v0 | a.rot | proj.stride(0)) & 7) == 0 &&
                     (reinterpret_cast<uintptr_t>(a.proj) & 15) == 0;
    const int V = vec ? VW : 1;
    a.GL = 1;
    while (a.GL < WAVE && a.GL * V < d) a.GL *= 2;
    auto launch = [&](auto kern) {
      if (lds > 48 * 1024)
        (void)hipFuncSetAttribute((const void*)kern,
                                  hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds);
      hipLaunchKernelGGL(kern, dim3(T_), dim3(256), lds, CUR_STREAM, a);
    };
    if (vec && whole) launch(normed_qkv_kernel<T, VW, true>);
    else if (vec) launch(normed_qkv_kernel<T, VW, false>);
    else if (whole) launch(normed_qkv_kernel<T, 1, true>);
    else launch(normed_qkv_kernel<T, 1, false>);
  });
  HIP_CHECK_KERNEL();
  return q;
}
