// Routed experts with a clamped GLU,
//     act = g sigmoid(alpha g) (u + shift),  g = min(gate, limit), u = clamp(up)
// (without a limit, alpha 1 and shift 0: silu(gate) up), or a squared relu, act =
// max(up, 0)^2, chosen by one of three routers:
//     z = W_r h + b (fp32), the ``top`` largest, softmax over the chosen;
//     s = sigmoid(W_r h) (fp32), the ``top`` largest of s + c among the best groups of
//     neighbours (by the sum of their two largest), weights s / sum s * scale;
//     s = softmax(W_r h) (fp32) over all, the ``top`` largest among the best groups (by
//     their largest), weights s * scale
// as route -> sort -> gathered up product with the activation in its epilogue
// -> down product. Rows stay sorted by expert; the residual-norm kernel adds
// each token's weighted rows, so no scatter pass exists. Nothing is read back
// to the host and all shapes are static: prompts and captured decode steps run
// the same code, only the row tile differs. A grid block looks up its (expert,
// row tile) in a device table; blocks past its end leave at once, so experts
// nobody chose cost no weight traffic.
#include "elem.h"
#include <torch/extension.h>
#include <c10/hip/HIPStream.h>

#define CUR_STREAM c10::hip::getCurrentHIPStream().stream()
#define MAX_EXPERTS 1024

union mfrag {
  shortx8 s;
  bf16x8 v;
};

// ------------------------------------------------------------------- router

enum { CHOSEN_SOFTMAX = 0, GROUPED_SIGMOID = 1, GROUPED_SOFTMAX = 2 };

// one workgroup per 16 tokens; its waves split the contraction. GROUPED_SIGMOID: bias
// is the scores' correction; GROUPED_SOFTMAX: there is none
template <typename T, bool MATRIX16, int ROUTER>
__global__ __launch_bounds__(1024) void moe_route_kernel(
    const T* __restrict__ h, const T* __restrict__ router,
    const float* __restrict__ bias, int* __restrict__ sel, float* __restrict__ gate,
    int T_, int W, int E, int top, int groups, int keep, float scale) {
  constexpr bool GROUPED = ROUTER != CHOSEN_SOFTMAX;
  extern __shared__ float logits[];  // [16][E]
  __shared__ float part[16][16][64];
  const int lane = threadIdx.x % WAVE, wave = threadIdx.x / WAVE;
  const int i = lane & 15, g = lane >> 4;
  const int t0 = blockIdx.x * 16;
  const long arow = (long)min(t0 + i, T_ - 1) * W;
  for (int e0 = 0; e0 < E; e0 += 64) {
    floatx4 acc[4];
    long brow[4];
#pragma unroll
    for (int j = 0; j < 4; ++j) {
      acc[j] = floatx4{0.f, 0.f, 0.f, 0.f};
      brow[j] = (long)min(e0 + j * 16 + i, E - 1) * W;
    }
    if constexpr (MATRIX16) {  // bf16 operands, W a multiple of 8
      for (int k = wave * 32; k < W; k += 512) {
        const int kk = k + g * 8;
        mfrag a, b;
        a.s = shortx8{0, 0, 0, 0, 0, 0, 0, 0};
        b.s = a.s;
        if (kk < W) a.s = *reinterpret_cast<const shortx8*>(h + arow + kk);
#pragma unroll
        for (int j = 0; j < 4; ++j) {
          if (e0 + j * 16 >= E) break;
          if (kk < W) b.s = *reinterpret_cast<const shortx8*>(router + brow[j] + kk);
          acc[j] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(a.v, b.v, acc[j], 0, 0, 0);
        }
      }
    } else {
      for (int k = wave * 4; k < W; k += 64) {
        const int kk = k + g;
        const float a = kk < W ? ldf(h + arow + kk) : 0.f;
#pragma unroll
        for (int j = 0; j < 4; ++j) {
          if (e0 + j * 16 >= E) break;
          const float b = kk < W ? ldf(router + brow[j] + kk) : 0.f;
          acc[j] = __builtin_amdgcn_mfma_f32_16x16x4f32(a, b, acc[j], 0, 0, 0);
        }
      }
    }
#pragma unroll
    for (int j = 0; j < 4; ++j)
#pragma unroll
      for (int r = 0; r < 4; ++r) part[wave][4 * g + r][j * 16 + i] = acc[j][r];
    __syncthreads();
    {
      const int t = threadIdx.x / 64, x = threadIdx.x % 64, e = e0 + x;
      float z = 0.f;
#pragma unroll
      for (int v = 0; v < 16; ++v) z += part[v][t][x];
      if (e < E) logits[t * E + e] = GROUPED ? z : z + bias[e];
    }
    __syncthreads();
  }
  if (t0 + wave < T_) {
    const int t = wave;
    float* z = logits + t * E;
    float* score = &part[wave][0][0];  // plain scores; from 512 on the groups'
    if constexpr (GROUPED) {
      float* gs = score + 512;
      const int n = E / groups;
      auto sync = [] {
        __threadfence_block();
        __builtin_amdgcn_wave_barrier();
      };
      if constexpr (ROUTER == GROUPED_SIGMOID) {
        for (int e = lane; e < E; e += WAVE) {
          score[e] = sigmoid_f(z[e]);
          z[e] = score[e] + bias[e];
        }
      } else {
        float most = -INFINITY, all = 0.f;
        for (int e = lane; e < E; e += WAVE) most = fmaxf(most, z[e]);
        most = wave_max(most);
        for (int e = lane; e < E; e += WAVE) all += score[e] = expf(z[e] - most);
        all = wave_sum(all);
        for (int e = lane; e < E; e += WAVE) score[e] /= all;
      }
      sync();
      for (int x = lane; x < groups; x += WAVE) {
        float a = -INFINITY, b = -INFINITY;  // the two largest
        for (int e = x * n; e < (x + 1) * n; ++e) {
          const float c = z[e];
          b = fmaxf(b, fminf(a, c));
          a = fmaxf(a, c);
        }
        gs[x] = ROUTER == GROUPED_SIGMOID && n > 1 ? a + b : a;
      }
      sync();
      for (int x = lane; x < groups; x += WAVE) {
        int better = 0;
        for (int o = 0; o < groups; ++o)
          better += gs[o] > gs[x] || (gs[o] == gs[x] && o < x);
        if (better >= keep)
          for (int e = x * n; e < (x + 1) * n; ++e) z[e] = -INFINITY;
      }
      sync();
    }
    float first = 0.f, sum = 0.f;
    for (int n = 0; n < top; ++n) {
      float best = -INFINITY;
      int at = 0x7fffffff;
      for (int e = lane; e < E; e += WAVE)
        if (z[e] > best) { best = z[e]; at = e; }
#pragma unroll
      for (int off = 32; off > 0; off >>= 1) {
        const float ob = __shfl_xor(best, off, WAVE);
        const int oa = __shfl_xor(at, off, WAVE);
        if (ob > best || (ob == best && oa < at)) { best = ob; at = oa; }
      }
      at = min(at, E - 1);  // all logits NaN: still a valid expert
      if (n == 0) first = best;
      const float p = GROUPED ? score[at] : expf(best - first);
      sum += p;
      if (lane == n % WAVE) {
        sel[(long)(t0 + t) * top + n] = at;
        gate[(long)(t0 + t) * top + n] = p;
      }
      if (lane == 0) z[at] = -INFINITY;
      __threadfence_block();
      __builtin_amdgcn_wave_barrier();
    }
    // each lane rescales what it wrote
    for (int n = lane; n < top; n += WAVE) {
      float& w = gate[(long)(t0 + t) * top + n];
      w = ROUTER == GROUPED_SIGMOID ? w / (sum + 1e-20f) * scale
          : ROUTER == GROUPED_SOFTMAX ? w * scale : w / sum;
    }
  }
}

template <int ROUTER>
static std::vector<torch::Tensor> route(const torch::Tensor& h, const torch::Tensor& router,
                                        const c10::optional<torch::Tensor>& bias, long top,
                                        long groups, long keep, double scale) {
  TORCH_CHECK(h.is_cuda() && h.dim() == 2 && h.is_contiguous() &&
              router.is_contiguous() && router.dtype() == h.dtype());
  const long T_ = h.size(0), W = h.size(1), E = router.size(0);
  TORCH_CHECK(router.size(1) == W);
  TORCH_CHECK(ROUTER == GROUPED_SOFTMAX ? !bias : bias && bias->numel() == E &&
              bias->dtype() == torch::kFloat32, "router bias");
  TORCH_CHECK(top >= 1 && top <= E && E <= 512, "1 <= top <= experts <= 512");
  auto sel = torch::empty({T_, top}, h.options().dtype(torch::kInt32));
  auto gate = torch::empty({T_, top}, h.options().dtype(torch::kFloat32));
  if (T_ == 0) return {sel, gate};
  DISPATCH_ELEM(h.dtype() == torch::kBFloat16, {
    auto launch = [&](auto kern) {
      hipLaunchKernelGGL(kern, dim3((T_ + 15) / 16), dim3(1024), 16 * E * 4, CUR_STREAM,
                         (const T*)h.data_ptr(), (const T*)router.data_ptr(),
                         bias ? bias->data_ptr<float>() : nullptr, sel.data_ptr<int>(),
                         gate.data_ptr<float>(), (int)T_, (int)W, (int)E, (int)top,
                         (int)groups, (int)keep, (float)scale);
    };
    constexpr bool B16 = sizeof(T) == 2;
    if (B16 && W % 8 == 0) launch(moe_route_kernel<T, B16, ROUTER>);
    else launch(moe_route_kernel<T, false, ROUTER>);
  });
  HIP_CHECK_KERNEL();
  return {sel, gate};
}

std::vector<torch::Tensor> moe_route(torch::Tensor h, torch::Tensor router,
                                     torch::Tensor bias, long top) {
  return route<CHOSEN_SOFTMAX>(h, router, bias, top, 1, 1, 1.0);
}

// sigmoid scores with a correction, softmax scores without
std::vector<torch::Tensor> moe_route_grouped(torch::Tensor h, torch::Tensor router,
                                             c10::optional<torch::Tensor> correction,
                                             long top, long groups, long keep, double scale) {
  const long E = router.size(0);
  TORCH_CHECK(groups >= 1 && E % groups == 0 && keep >= 1 && keep <= groups &&
              top <= keep * (E / groups), "expert groups");
  if (!correction) return route<GROUPED_SOFTMAX>(h, router, correction, top, groups, keep, scale);
  return route<GROUPED_SIGMOID>(h, router, correction, top, groups, keep, scale);
}

// --------------------------------------------------------------------- sort

// place[a]: sorted row of choice a; token[row]: its token; table: (expert, first
// row, rows) of every row tile, then expert -1
__global__ __launch_bounds__(1024) void moe_sort_kernel(
    const int* __restrict__ sel, int A, int E, int top, int TM, int tiles,
    int* __restrict__ place, int* __restrict__ token, int* __restrict__ table) {
  __shared__ int count[MAX_EXPERTS], base[MAX_EXPERTS], tbase[MAX_EXPERTS];
  const int tid = threadIdx.x;
  for (int e = tid; e < E; e += 1024) count[e] = 0;
  __syncthreads();
  for (int a = tid; a < A; a += 1024) atomicAdd(&count[sel[a]], 1);
  __syncthreads();
  if (tid < WAVE) {  // exclusive sums over experts, one wave
    int rows = 0, nt = 0;
    for (int e0 = 0; e0 < E; e0 += WAVE) {
      const int e = e0 + tid;
      const int c = e < E ? count[e] : 0, k = (c + TM - 1) / TM;
      int sc = c, sk = k;
#pragma unroll
      for (int off = 1; off < WAVE; off <<= 1) {
        const int a = __shfl_up(sc, off, WAVE), b = __shfl_up(sk, off, WAVE);
        if (tid >= off) { sc += a; sk += b; }
      }
      if (e < E) { base[e] = rows + sc - c; tbase[e] = nt + sk - k; }
      rows += __shfl(sc, WAVE - 1, WAVE);
      nt += __shfl(sk, WAVE - 1, WAVE);
    }
    for (int t = nt + tid; t < tiles; t += WAVE) table[t * 3] = -1;
  }
  __syncthreads();
  for (int e = tid; e < E; e += 1024) {
    for (int k = 0, r = 0; r < count[e]; ++k, r += TM) {
      int* t = table + (tbase[e] + k) * 3;
      t[0] = e;
      t[1] = base[e] + r;
      t[2] = min(TM, count[e] - r);
    }
  }
  __syncthreads();
  for (int a = tid; a < A; a += 1024) {
    const int row = atomicAdd(&base[sel[a]], 1);
    place[a] = row;
    token[row] = a / top;
  }
}

// ------------------------------------------------------------ grouped product

// what the product's epilogue does
enum { NO_ACT = 0, GLU_ACT = 1, RELU2_ACT = 2 };

struct GroupArgs {
  const void* x;       // rows [*, K]; row r of the sorted batch is x[gather[r]]
  const int* gather;   // null: x itself is sorted
  const void* w;       // [E, N, K]; GLU: [E, 2N, K], gate rows then up rows
  void* y;             // [A, N]
  const int* table;
  int N, K;
  float limit, alpha, shift;
};

DEVINL float clamped_glu(float g, float u, const GroupArgs& p) {
  g = fminf(g, p.limit);
  u = fminf(fmaxf(u, -p.limit), p.limit);
  return g * (u + p.shift) / (1.f + expf(-p.alpha * g));
}

// Any size and float32: 32 rows x 64 columns, 16 of K at a time, through LDS as
// fp32 (GLU: 32 gate and the matching 32 up columns).
template <typename T, int ACT>
__global__ __launch_bounds__(256) void grouped_any_kernel(GroupArgs p) {
  constexpr bool GLU = ACT == GLU_ACT;
  const int* tb = p.table + blockIdx.y * 3;
  const int e = tb[0];
  if (e < 0) return;
  const int row0 = tb[1], cnt = tb[2];
  __shared__ float xs[32][17], ws[64][17], cs[32][65];
  const int tid = threadIdx.x, lane = tid % WAVE, wave = tid / WAVE;
  const int i = lane & 15, g = lane >> 4;
  constexpr int BN = GLU ? 32 : 64;
  const int n0 = blockIdx.x * BN;
  const T* w = (const T*)p.w + (long)e * (GLU ? 2 : 1) * p.N * p.K;
  floatx4 acc[2] = {{0.f, 0.f, 0.f, 0.f}, {0.f, 0.f, 0.f, 0.f}};
  for (int k0 = 0; k0 < p.K; k0 += 16) {
    __syncthreads();
    for (int x = tid; x < 32 * 16; x += 256) {
      const int r = x / 16, k = k0 + x % 16;
      const long src = row0 + min(r, cnt - 1);
      xs[r][x % 16] = k < p.K ? ldf((const T*)p.x + (long)(p.gather ? p.gather[src] : src) *
                                    p.K + k) : 0.f;
    }
    for (int x = tid; x < 64 * 16; x += 256) {
      const int r = x / 16, k = k0 + x % 16;
      const int c = n0 + (GLU ? r % 32 : r);
      const long wr = min(c, p.N - 1) + (GLU && r >= 32 ? p.N : 0);
      ws[r][x % 16] = k < p.K ? ldf(w + wr * p.K + k) : 0.f;
    }
    __syncthreads();
#pragma unroll
    for (int s = 0; s < 16; s += 4) {
      const float b = ws[wave * 16 + i][s + g];
#pragma unroll
      for (int m = 0; m < 2; ++m)
        acc[m] = __builtin_amdgcn_mfma_f32_16x16x4f32(xs[m * 16 + i][s + g], b, acc[m],
                                                      0, 0, 0);
    }
  }
#pragma unroll
  for (int m = 0; m < 2; ++m)
#pragma unroll
    for (int r = 0; r < 4; ++r) cs[m * 16 + 4 * g + r][wave * 16 + i] = acc[m][r];
  __syncthreads();
  for (int x = tid; x < 32 * BN; x += 256) {
    const int r = x / BN, c = x % BN;
    if (r >= cnt || n0 + c >= p.N) continue;
    float v = GLU ? clamped_glu(cs[r][c], cs[r][32 + c], p) : cs[r][c];
    if constexpr (ACT == RELU2_ACT) v = v > 0.f ? v * v : 0.f;
    stf((T*)p.y + (long)(row0 + r) * p.N + n0 + c, v);
  }
}

// bf16, K a multiple of 64: TM rows x TB weight rows (GLU: half gate, half up), K in
// steps of 64 through an NS-deep ring of LDS stages filled by direct-to-LDS
// loads. A stage's 16-byte units are XOR-swizzled by row so that fragment reads
// are free of bank conflicts. A wave's columns hold gate and up of the same
// outputs, so the activation is register to register.
#define GK 64

template <int TM, int TB, int NS, int NTHR, int ACT>
__global__ __launch_bounds__(NTHR) void grouped_bf16_kernel(GroupArgs p) {
  constexpr bool GLU = ACT == GLU_ACT;
  const int* tb = p.table + blockIdx.y * 3;
  const int e = tb[0];
  if (e < 0) return;
  constexpr int MW = TM >= 64 ? 2 : 1;        // waves along rows
  constexpr int NW = NTHR / 64 / MW;          // waves along columns
  constexpr int WM = TM / MW, WN = TB / NW;   // a wave's tile
  constexpr int MI = WM / 16, NI = WN / 16;
  constexpr int LA = TM * 8 / NTHR, LB = TB * 8 / NTHR;  // loads per thread
  constexpr int STAGE = (TM + TB) * GK * 2;
  extern __shared__ __attribute__((aligned(16))) char lds[];
  const int row0 = tb[1], cnt = tb[2];
  const int tid = threadIdx.x, lane = tid % WAVE, wave = tid / WAVE;
  const int i = lane & 15, g = lane >> 4;
  constexpr int BN = GLU ? TB / 2 : TB;
  const int n0 = blockIdx.x * BN;
  const int K = p.K;
  const bf16_t* w = (const bf16_t*)p.w + (long)e * (GLU ? 2 : 1) * p.N * K;

  // source of each 16-byte unit this thread fills (LDS is linear in the lane)
  const bf16_t* as[LA];
  const bf16_t* bs[LB];
#pragma unroll
  for (int x = 0; x < LA; ++x) {
    const int r = (tid + x * NTHR) >> 3, unit = (tid & 7) ^ (r & 7);
    const int src = row0 + min(r, cnt - 1);
    as[x] = (const bf16_t*)p.x + (long)(p.gather ? p.gather[src] : src) * K + unit * 8;
  }
#pragma unroll
  for (int x = 0; x < LB; ++x) {
    const int r = (tid + x * NTHR) >> 3, unit = (tid & 7) ^ (r & 7);
    long wr;
    if constexpr (GLU) {  // within a wave's columns: first half gate, second up
      const int q = r % WN, c = n0 + r / WN * (WN / 2) + q % (WN / 2);
      wr = min(c, p.N - 1) + (q >= WN / 2 ? p.N : 0);
    } else {
      wr = min(n0 + r, p.N - 1);
    }
    bs[x] = w + wr * K + unit * 8;
  }
  auto issue = [&](int c) {
    char* st = lds + (c % NS) * STAGE;
#pragma unroll
    for (int x = 0; x < LA; ++x)
      __builtin_amdgcn_global_load_lds(
          (const __attribute__((address_space(1))) void*)(as[x] + (long)c * GK),
          (__attribute__((address_space(3))) void*)(st + (tid + x * NTHR) * 16), 16, 0, 0);
#pragma unroll
    for (int x = 0; x < LB; ++x)
      __builtin_amdgcn_global_load_lds(
          (const __attribute__((address_space(1))) void*)(bs[x] + (long)c * GK),
          (__attribute__((address_space(3))) void*)(st + TM * GK * 2 + (tid + x * NTHR) * 16),
          16, 0, 0);
  };
  floatx4 acc[MI][NI];
#pragma unroll
  for (int m = 0; m < MI; ++m)
#pragma unroll
    for (int n = 0; n < NI; ++n) acc[m][n] = floatx4{0.f, 0.f, 0.f, 0.f};

  const int nc = K / GK;
  const int wm = wave / NW * WM, wn = wave % NW * WN;
#pragma unroll
  for (int c = 0; c < NS - 1; ++c)
    if (c < nc) issue(c);
  for (int c = 0; c < nc; ++c) {
    // stage c has landed when at most the NS - 2 later ones are in flight. A
    // plain s_barrier: __syncthreads would drain the later stages as well.
    if (c + NS - 1 <= nc)
      asm volatile("s_waitcnt vmcnt(%0) lgkmcnt(0)\n\ts_barrier"
                   ::"n"((NS - 2) * (LA + LB)) : "memory");
    else
      asm volatile("s_waitcnt vmcnt(0) lgkmcnt(0)\n\ts_barrier" ::: "memory");
    if (c + NS - 1 < nc) issue(c + NS - 1);
    const char* xa = lds + (c % NS) * STAGE;
    const char* wb = xa + TM * GK * 2;
#pragma unroll
    for (int s = 0; s < GK / 32; ++s) {
      mfrag a[MI], b[NI];
#pragma unroll
      for (int m = 0; m < MI; ++m) {
        const int r = wm + m * 16 + i;
        a[m].s = *reinterpret_cast<const shortx8*>(xa + r * 128 + (((s * 4 + g) ^ (r & 7)) << 4));
      }
#pragma unroll
      for (int n = 0; n < NI; ++n) {
        const int r = wn + n * 16 + i;
        b[n].s = *reinterpret_cast<const shortx8*>(wb + r * 128 + (((s * 4 + g) ^ (r & 7)) << 4));
      }
#pragma unroll
      for (int m = 0; m < MI; ++m)
#pragma unroll
        for (int n = 0; n < NI; ++n)
          acc[m][n] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(a[m].v, b[n].v, acc[m][n],
                                                              0, 0, 0);
    }
  }
  bf16_t* y = (bf16_t*)p.y;
  constexpr int NO = GLU ? NI / 2 : NI;
#pragma unroll
  for (int m = 0; m < MI; ++m)
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int row = wm + m * 16 + 4 * g + r;
      if (row >= cnt) continue;
#pragma unroll
      for (int n = 0; n < NO; ++n) {
        const int c = n0 + (GLU ? wn / 2 : wn) + n * 16 + i;
        if (c >= p.N) continue;
        float v = GLU ? clamped_glu(acc[m][n][r], acc[m][n + (GLU ? NO : 0)][r], p)
                      : acc[m][n][r];
        if constexpr (ACT == RELU2_ACT) v = v > 0.f ? v * v : 0.f;
        y[(long)(row0 + row) * p.N + c] = f32_to_bf16(v);
      }
    }
}

template <int TM, int TB, int NS, int NTHR, int ACT>
static void grouped_bf16(const GroupArgs& p, int tiles) {
  constexpr int BN = ACT == GLU_ACT ? TB / 2 : TB;
  constexpr int lds = NS * (TM + TB) * GK * 2;
  auto kern = grouped_bf16_kernel<TM, TB, NS, NTHR, ACT>;
  if (lds > 64 * 1024) {
    static const hipError_t once = hipFuncSetAttribute(
        (const void*)kern, hipFuncAttributeMaxDynamicSharedMemorySize, lds);
    (void)once;
  }
  hipLaunchKernelGGL(kern, dim3((p.N + BN - 1) / BN, tiles), dim3(NTHR), lds, CUR_STREAM, p);
}

template <int ACT>
static void grouped(const GroupArgs& p, bool bf16, int tiles, int TM, long busy) {
  constexpr bool GLU = ACT == GLU_ACT;
  if (bf16 && p.K % GK == 0) {
    const long blocks = (p.N + (GLU ? 63 : 127)) / (GLU ? 64 : 128) * busy;
    if (TM == 256) grouped_bf16<256, 256, 2, 512, ACT>(p, tiles);
    else if (TM == 128) grouped_bf16<128, 128, 2, 256, ACT>(p, tiles);
    else if (TM == 64) grouped_bf16<64, 128, 3, 256, ACT>(p, tiles);
    // few rows: the weights' stream counts. Two workgroups per CU with four
    // stages each, or one with seven where there are not enough for two
    else if (blocks >= 512) grouped_bf16<32, 128, 4, 256, ACT>(p, tiles);
    else grouped_bf16<32, 128, 7, 256, ACT>(p, tiles);
    return;
  }
  TORCH_CHECK(TM == 32);
  const dim3 grid((p.N + (GLU ? 31 : 63)) / (GLU ? 32 : 64), tiles);
  if (bf16)
    hipLaunchKernelGGL((grouped_any_kernel<bf16_t, ACT>), grid, dim3(256), 0, CUR_STREAM, p);
  else
    hipLaunchKernelGGL((grouped_any_kernel<float, ACT>), grid, dim3(256), 0, CUR_STREAM, p);
}

template <int ACT>
static std::vector<torch::Tensor> experts(const torch::Tensor& h, const torch::Tensor& sel,
                                          const torch::Tensor& w_up, const torch::Tensor& w_dn,
                                          double limit, double alpha, double shift) {
  TORCH_CHECK(h.is_cuda() && h.dim() == 2 && h.is_contiguous() && sel.is_contiguous() &&
              sel.dtype() == torch::kInt32 && sel.size(0) == h.size(0));
  const long T_ = h.size(0), W = h.size(1), top = sel.size(1), A = T_ * top;
  const long E = w_up.size(0), F = w_up.size(1) / (ACT == GLU_ACT ? 2 : 1);
  TORCH_CHECK(w_up.is_contiguous() && w_dn.is_contiguous() && w_up.dtype() == h.dtype() &&
              w_dn.dtype() == h.dtype() && w_up.size(2) == W && w_dn.size(0) == E &&
              w_dn.size(1) == W && w_dn.size(2) == F && E <= MAX_EXPERTS);
  auto i32 = h.options().dtype(torch::kInt32);
  auto y = torch::empty({A, W}, h.options()), place = torch::empty({T_, top}, i32);
  if (A == 0) return {y, place};
  const bool bf16 = h.dtype() == torch::kBFloat16;
  // row tile: enough rows per weight read when experts are well filled
  const bool matrix = bf16 && W % GK == 0 && F % GK == 0;
  // and the large tile only where it leaves enough blocks for the chip
  const long cols = ACT == GLU_ACT ? 128 : 256;
  const bool large = A >= 512 * E && A / 256 * ((F + cols - 1) / cols) >= 1024;
  const int TM = !matrix || A < 48 * E ? 32 : A < 160 * E ? 64 : large ? 256 : 128;
  const int tiles = (int)(A / TM + std::min(E, A));
  auto token = torch::empty({A}, i32), table = torch::empty({tiles, 3}, i32);
  auto act = torch::empty({A, F}, h.options());
  hipLaunchKernelGGL(moe_sort_kernel, dim3(1), dim3(1024), 0, CUR_STREAM,
                     sel.data_ptr<int>(), (int)A, (int)E, (int)top, TM, tiles,
                     place.data_ptr<int>(), token.data_ptr<int>(), table.data_ptr<int>());
  GroupArgs p = {h.data_ptr(), token.data_ptr<int>(), w_up.data_ptr(), act.data_ptr(),
                 table.data_ptr<int>(), (int)F, (int)W, (float)limit, (float)alpha,
                 (float)shift};
  grouped<ACT>(p, bf16, tiles, TM, std::min(E, A));
  p.x = act.data_ptr();
  p.gather = nullptr;
  p.w = w_dn.data_ptr();
  p.y = y.data_ptr();
  p.N = W;
  p.K = F;
  grouped<NO_ACT>(p, bf16, tiles, TM, std::min(E, A));
  HIP_CHECK_KERNEL();
  return {y, place};
}

std::vector<torch::Tensor> moe_clamped_glu(torch::Tensor h, torch::Tensor sel,
                                           torch::Tensor w_gu, torch::Tensor w_dn,
                                           double limit, double alpha, double shift) {
  return experts<GLU_ACT>(h, sel, w_gu, w_dn, limit, alpha, shift);
}

std::vector<torch::Tensor> moe_relu2(torch::Tensor h, torch::Tensor sel, torch::Tensor w_up,
                                     torch::Tensor w_dn) {
  return experts<RELU2_ACT>(h, sel, w_up, w_dn, 0.0, 0.0, 0.0);
}
