// Latent attention on gfx950: one cached vector c per token and layer, from
// which every head's key and value are linear maps (uk, uv).
//
// A head's score q.(uk c) is (uk' q).c, and its output uv (sum_j p_j c_j), so
// attention can stay in the latents' space: all (token, head) rows of a
// sequence attend to ONE key row that is also the value row. A rotated key part that
// the heads share follows c in that row and scores like the rest of it. That is what
// decoding does (a latent is read once for all heads; 2 R flops per byte and
// head row, so it needs the matrix cores), and short prompt portions on a long
// context. Long portions spell keys and values out and run the flash prefill
// kernel (ops.sequence.expand_latents decides).
//
// latent_attention_kernel: a workgroup holds 16 or 32 rows and walks its
// context in tiles of 64 latents, four waves:
//  * every wave loads its own 16 latents of the next tile straight to LDS while
//    the tile before is computed, and scores them: S^T = C Q^T, the rows'
//    queries live in registers as B fragments;
//  * the bf16 weights go through LDS (one barrier a tile), then every wave owns
//    VR / 4 columns of O += P C, VR the row's width without the key part. The value fragments are columns of the row-major
//    tile: ds_read_b64_tr_b16 transposes on the way to the registers.
//    Contraction slot 8 g + j holds key 4 g + j (j < 4) or 16 + 4 g + j - 4, on
//    both operands;
//  * a wave's 16 latents lie in LDS as R / 32 blocks of [16 rows][64 bytes], so
//    that one load fills a block, a lane's source moves by 64 bytes from load to
//    load, a score fragment is a block read in order, and all reads of a tile
//    are one address plus constants. In rows 4-7 and 12-15 the two halves of the
//    64 bytes change places, which spreads the column reads over all banks;
//  * weights are taken against a reference that need not be the maximum: it only
//    moves, and only then the waves exchange maxima and rescale O, when a score
//    exceeds it by more than LAT_SLACK, so weights stay below 2^LAT_SLACK.
// Few rows: the context is split over blockIdx.y, partial sums are merged by
// latent_combine_kernel. A row's softmax starts from its sink, if there is one (split
// 0 only). A window leaves out the tiles before it. Scores, maxima and sinks are in
// units of log 2.
#include "head_turn.h"
#include <torch/extension.h>
#include <c10/hip/HIPStream.h>

#include <type_traits>

#define CUR_STREAM c10::hip::getCurrentHIPStream().stream()
#define LAT_KEYS 64                    // latents per tile
#define LAT_PSTRIDE (LAT_KEYS + 8)     // row stride of the weights in LDS
#define LAT_SLACK 10.f
#define LAT_SPLITS 128                 // most parts of a context
#define LOG2E 1.44269504f

union lfrag {
  shortx8 s;
  shortx4 h[2];
  bf16x8 v;
};

template <int N, typename F>
DEVINL void static_for(F&& f) {
  if constexpr (N > 0) {
    static_for<N - 1>(f);
    f(std::integral_constant<int, N - 1>{});
  }
}

// Reads of two neighbouring blocks; then wait until the two before have arrived.
template <int AT>
DEVINL void read_blocks(shortx8& a, shortx8& b, shortx8& ready_a, shortx8& ready_b,
                        unsigned addr) {
  asm volatile(
      "ds_read_b128 %0, %4 offset:%5\n\t"
      "ds_read_b128 %1, %4 offset:%6\n\t"
      "s_waitcnt lgkmcnt(2)"
      : "=&v"(a), "=&v"(b), "+v"(ready_a), "+v"(ready_b)
      : "v"(addr), "n"(AT), "n"(AT + 1024)
      : "memory");
}

DEVINL void await_blocks(shortx8& a, shortx8& b) {
  asm volatile("s_waitcnt lgkmcnt(0)" : "+v"(a), "+v"(b)::"memory");
}

// Transposing reads of the four 16-row slices (STEP bytes apart) of one 16-column
// tile; then wait until the slices requested two calls before have arrived.
// Written out because the compiler puts a wait for all global loads in flight,
// the next tile's among them, before the builtin form of these reads.
template <int AT, int STEP>
DEVINL void read_columns(shortx4 (&next)[4], shortx4 (&ready)[4], unsigned addr) {
  asm volatile(
      "ds_read_b64_tr_b16 %0, %8 offset:%9\n\t"
      "ds_read_b64_tr_b16 %1, %8 offset:%10\n\t"
      "ds_read_b64_tr_b16 %2, %8 offset:%11\n\t"
      "ds_read_b64_tr_b16 %3, %8 offset:%12\n\t"
      "s_waitcnt lgkmcnt(8)"
      : "=&v"(next[0]), "=&v"(next[1]), "=&v"(next[2]), "=&v"(next[3]), "+v"(ready[0]),
        "+v"(ready[1]), "+v"(ready[2]), "+v"(ready[3])
      : "v"(addr), "n"(AT), "n"(AT + STEP), "n"(AT + 2 * STEP), "n"(AT + 3 * STEP)
      : "memory");
}

// the slices requested PENDING calls before the last have arrived
template <int PENDING>
DEVINL void await_columns(shortx4 (&ready)[4]) {
  asm volatile("s_waitcnt lgkmcnt(%4)"
               : "+v"(ready[0]), "+v"(ready[1]), "+v"(ready[2]), "+v"(ready[3])
               : "n"(4 * PENDING)
               : "memory");
}

template <int R, int VR, int MT>
__global__ __launch_bounds__(256, 1) void latent_attention_kernel(
    const bf16_t* __restrict__ q,      // [T * H, R]
    const bf16_t* __restrict__ cache,  // [NP, P, R]
    const int* __restrict__ bt, int MP, const int* __restrict__ cu,
    const int* __restrict__ ctx, const int* __restrict__ bseq,
    const int* __restrict__ boff, const float* __restrict__ sink,
    bf16_t* __restrict__ out,          // [T * H, VR] (one split)
    float* __restrict__ part,          // [CS, T * H, VR] (several)
    float* __restrict__ part_ml,       // [CS, T * H, 2]
    int H, int P, long rows_all, float scale, int window) {
  constexpr int NT = VR / 64;          // 16-column tiles of O per wave
  constexpr int ROWS = 16 * MT;
  constexpr int SLICE = 16 * R * 2;    // bytes of a wave's 16 latents
  constexpr int TILE = 4 * SLICE;
  extern __shared__ __attribute__((aligned(16))) char smem[];
  short* pbuf = (short*)(smem + 2 * TILE);  // [2][ROWS][LAT_PSTRIDE]
  float* stat = (float*)(smem + 2 * TILE + 2 * ROWS * LAT_PSTRIDE * 2);  // [4][ROWS]
  float* exceed = stat + 4 * ROWS;          // [2][4]: 1 where a wave saw a score too high

  const int tid = threadIdx.x, lane = tid % WAVE;
  const int wave = __builtin_amdgcn_readfirstlane(tid / WAVE);
  const int col = lane & 15, g = lane >> 4;
  const int tiles_per_seq = (H + ROWS - 1) / ROWS;  // single tokens
  const int nb = gridDim.x - 1 - blockIdx.x;  // a portion's late rows see most: first
  const int seq = cu ? bseq[nb] : nb / tiles_per_seq;
  const int off = cu ? boff[nb] : nb % tiles_per_seq * ROWS;
  const int n = cu ? cu[seq + 1] - cu[seq] : 1;
  const long row0 = (long)(cu ? cu[seq] : seq) * H + off;
  const int nrows = min(ROWS, n * H - off);
  const int start = ctx[seq] - n;
  const int first_pos = start + off / H;
  const int kend = start + (off + nrows - 1) / H + 1;  // keys any row here sees
  const int win = window > 0 ? window : 0x3fffffff;
  const int before = max(0, first_pos - win + 1) / LAT_KEYS;  // tiles nobody here sees
  const int ntiles = (kend + LAT_KEYS - 1) / LAT_KEYS;
  const int per = (ntiles - before + gridDim.y - 1) / gridDim.y;
  const int tile0 = before + blockIdx.y * per, tile1 = min(ntiles, tile0 + per);
  const int* pages = bt + (long)seq * MP;
  const float scale2 = scale * LOG2E;

  // this lane's latent of the next tile to look up (four lanes share one), as
  // page and place; past the end the last one again. Pages are looked up a tile
  // ahead of the loads that need them.
  const int last_pg = (kend - 1) / P, last_in = (kend - 1) % P;
  const int step_pg = LAT_KEYS / P, step_in = LAT_KEYS % P;
  int key = tile0 * LAT_KEYS + wave * 16 + (lane >> 2), pg = key / P, in = key % P;
  int page = 0, in_page = 0;
  auto lookup = [&]() {
    const bool past = key >= kend;
    page = pages[past ? last_pg : pg];
    in_page = past ? last_in : in;
    key += LAT_KEYS;
    pg += step_pg;
    in += step_in;
    if (in >= P) {
      in -= P;
      ++pg;
    }
  };
  const int src_unit = (lane & 3) ^ (((lane >> 4) & 1) << 1);
  // this wave's 16 latents of the tile looked up; the constant offset of a load
  // moves its source and its destination
  auto issue = [&](int tile) {
    const bf16_t* src = cache + ((long)page * P + in_page) * R + src_unit * 8;
    char* dst = smem + (tile & 1) * TILE + wave * SLICE;
    static_for<R / 32>([&](auto I) {
      constexpr int i = decltype(I)::value;
      __builtin_amdgcn_global_load_lds(
          (const __attribute__((address_space(1))) void*)src,
          (__attribute__((address_space(3))) void*)(dst + i * (1024 - 64)), 16, i * 64, 0);
    });
    lookup();
  };
  if (tile0 < tile1) {
    lookup();
    issue(tile0);
  }

  // queries (B operand: lane's row col, contraction 8 g + j), positions, sinks
  lfrag qf[MT][R / 32];
  int pos[MT];
  float m[MT], l[MT];
#pragma unroll
  for (int t = 0; t < MT; ++t) {
    const int r = min(t * 16 + col, nrows - 1);
    const bf16_t* src = q + (row0 + r) * R + g * 8;
#pragma unroll
    for (int k = 0; k < R / 32; ++k) qf[t][k].s = *(const shortx8*)(src + k * 32);
    pos[t] = start + (off + r) / H;
    m[t] = sink && blockIdx.y == 0 ? sink[(off + r) % H] * LOG2E : -1e30f;
    l[t] = sink && blockIdx.y == 0 && wave == 0 && g == 0 ? 1.f : 0.f;
  }
  floatx4 o[MT][NT];
#pragma unroll
  for (int t = 0; t < MT; ++t)
#pragma unroll
    for (int c = 0; c < NT; ++c) o[t][c] = floatx4{0.f, 0.f, 0.f, 0.f};

  // where a lane's score fragments lie, and its pieces of the wave's columns:
  // lane i of a group reads row i / 4 of the group's four, 8 bytes of 32
  const unsigned smem_at = (unsigned)(size_t)(__attribute__((address_space(3))) char*)smem;
  const unsigned score_at = smem_at + wave * SLICE + col * 64 + (g ^ (((col >> 2) & 1) << 1)) * 16;
  unsigned vcol[2];
  {
    const int row = g * 4 + (col >> 2), flip = (row >> 2) & 1, ct = wave * NT;
    const unsigned at = smem_at + ct / 2 * 1024 + row * 64 + (lane & 3) * 8;
    vcol[0] = at + ((ct & 1) ^ flip) * 32;
    vcol[1] = at + ((ct & 1) ^ flip ^ 1) * 32;
  }

  auto score = [&](floatx4 (&st)[MT], shortx8 a, shortx8 b, int k) {
    lfrag fa, fb;
    fa.s = a;
    fb.s = b;
#pragma unroll
    for (int t = 0; t < MT; ++t)
      st[t] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(fa.v, qf[t][k].v, st[t], 0, 0, 0);
#pragma unroll
    for (int t = 0; t < MT; ++t)
      st[t] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(fb.v, qf[t][k + 1].v, st[t], 0, 0, 0);
  };

  for (int tile = tile0; tile < tile1; ++tile) {
    const int buf = (tile & 1) * TILE;
    asm volatile("s_waitcnt vmcnt(0)" : "+v"(page)::"memory");
    // scores of the wave's own keys: S^T rows 4 g + r, columns are query rows
    floatx4 st[MT];
#pragma unroll
    for (int t = 0; t < MT; ++t) st[t] = floatx4{0.f, 0.f, 0.f, 0.f};
    const unsigned krow = score_at + buf;
    shortx8 kf[(R / 64 + 1) * 2];  // block k is kf[k + 2]
    kf[0] = kf[1] = shortx8{};
    static_for<R / 64>([&](auto K) {
      constexpr int k = decltype(K)::value * 2;
      read_blocks<k * 1024>(kf[k + 2], kf[k + 3], kf[k], kf[k + 1], krow);
      if constexpr (k > 0) score(st, kf[k], kf[k + 1], k - 2);
    });
    await_blocks(kf[R / 32], kf[R / 32 + 1]);
    score(st, kf[R / 32], kf[R / 32 + 1], R / 32 - 2);
    const bool some_hidden = tile * LAT_KEYS + LAT_KEYS - 1 > first_pos ||
                             kend - 1 - tile * LAT_KEYS >= win;
    const int key0 = tile * LAT_KEYS + wave * 16 + g * 4;
    short* pb = pbuf + (tile & 1) * (ROWS * LAT_PSTRIDE);
#pragma unroll
    for (int t = 0; t < MT; ++t) {
      st[t] *= scale2;
      if (some_hidden)
#pragma unroll
        for (int r = 0; r < 4; ++r)
          if (key0 + r > pos[t] || pos[t] - key0 - r >= win) st[t][r] = -INFINITY;
    }
    auto weigh = [&](int t) {  // stores the weights, returns their sum
      floatx4 p;
#pragma unroll
      for (int r = 0; r < 4; ++r) p[r] = __builtin_amdgcn_exp2f(st[t][r] - m[t]);
      *(bf16x4*)(pb + (t * 16 + col) * LAT_PSTRIDE + wave * 16 + g * 4) =
          __builtin_convertvector(p, bf16x4);
      return (p[0] + p[1]) + (p[2] + p[3]);
    };
    float mx[MT], sum[MT];
    bool high = false;
#pragma unroll
    for (int t = 0; t < MT; ++t) {
      mx[t] = fmaxf(fmaxf(st[t][0], st[t][1]), fmaxf(st[t][2], st[t][3]));
      high = high || mx[t] > m[t] + LAT_SLACK;
      sum[t] = weigh(t);
    }
    float* flag = exceed + (tile & 1) * 4;
    const float too_high = __any(high) ? 1.f : 0.f;
    if (lane == 0) flag[wave] = too_high;
    // the whole tile and its weights are there, and nobody reads the other buffer
    asm volatile("s_waitcnt lgkmcnt(0)\n\ts_barrier" ::: "memory");
    if (tile + 1 < tile1) issue(tile + 1);
    if (__any((flag[0] + flag[1]) + (flag[2] + flag[3]) > 0.f)) {
      // all waves: move the references to the largest scores so far
#pragma unroll
      for (int t = 0; t < MT; ++t) {
        mx[t] = fmaxf(mx[t], __shfl_xor(mx[t], 16, WAVE));
        mx[t] = fmaxf(mx[t], __shfl_xor(mx[t], 32, WAVE));
        if (g == 0) stat[wave * ROWS + t * 16 + col] = mx[t];
      }
      asm volatile("s_waitcnt lgkmcnt(0)\n\ts_barrier" ::: "memory");
#pragma unroll
      for (int t = 0; t < MT; ++t) {
        float mn = m[t];
#pragma unroll
        for (int w = 0; w < 4; ++w) mn = fmaxf(mn, stat[w * ROWS + t * 16 + col]);
        const float alpha = __builtin_amdgcn_exp2f(m[t] - mn);
        m[t] = mn;
        l[t] *= alpha;
        floatx4 av;
#pragma unroll
        for (int r = 0; r < 4; ++r) av[r] = __shfl(alpha, g * 4 + r, WAVE);
#pragma unroll
        for (int c = 0; c < NT; ++c) o[t][c] *= av;
        sum[t] = weigh(t);
      }
      asm volatile("s_waitcnt lgkmcnt(0)\n\ts_barrier" ::: "memory");
    }
#pragma unroll
    for (int t = 0; t < MT; ++t) l[t] += sum[t];
    lfrag pf[2][MT];
#pragma unroll
    for (int kk = 0; kk < 2; ++kk)
#pragma unroll
      for (int t = 0; t < MT; ++t) {
        const short* pr = pb + (t * 16 + col) * LAT_PSTRIDE + kk * 32 + g * 4;
        pf[kk][t].h[0] = *(const shortx4*)pr;
        pf[kk][t].h[1] = *(const shortx4*)(pr + 16);
      }
    // slice 2 kk + j holds contraction slots 8 g + 4 j ..+3 of step kk
    const unsigned va[2] = {vcol[0] + buf, vcol[1] + buf};
    shortx4 cols[NT + 2][4] = {};  // tile c is cols[c + 2]
    read_columns<0, SLICE>(cols[2], cols[0], va[0]);
    if constexpr (NT > 1) read_columns<0, SLICE>(cols[3], cols[1], va[1]);
    static_for<NT>([&](auto C) {
      constexpr int c = decltype(C)::value;
      if constexpr (c + 2 < NT)
        read_columns<(c + 2) / 2 * 1024, SLICE>(cols[c + 4], cols[c + 2], va[c & 1]);
      else
        await_columns<NT - 1 - c>(cols[c + 2]);
#pragma unroll
      for (int kk = 0; kk < 2; ++kk) {
        lfrag cf;
        cf.h[0] = cols[c + 2][2 * kk];
        cf.h[1] = cols[c + 2][2 * kk + 1];
#pragma unroll
        for (int t = 0; t < MT; ++t)
          o[t][c] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(pf[kk][t].v, cf.v, o[t][c], 0, 0, 0);
      }
    });
  }

  // the waves' sums of weights
  asm volatile("s_waitcnt lgkmcnt(0)\n\ts_barrier" ::: "memory");
#pragma unroll
  for (int t = 0; t < MT; ++t) {
    l[t] += __shfl_xor(l[t], 16, WAVE);
    l[t] += __shfl_xor(l[t], 32, WAVE);
    if (g == 0) stat[wave * ROWS + t * 16 + col] = l[t];
  }
  asm volatile("s_waitcnt lgkmcnt(0)\n\ts_barrier" ::: "memory");
  if (gridDim.y == 1) {
    bf16_t* ob = (bf16_t*)smem;
#pragma unroll
    for (int t = 0; t < MT; ++t)
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int row = t * 16 + g * 4 + r;
        float sum = 0.f;
#pragma unroll
        for (int w = 0; w < 4; ++w) sum += stat[w * ROWS + row];
        const float inv = 1.f / sum;
#pragma unroll
        for (int c = 0; c < NT; ++c)
          stf(ob + row * VR + (wave * NT + c) * 16 + col, o[t][c][r] * inv);
      }
    asm volatile("s_waitcnt lgkmcnt(0)\n\ts_barrier" ::: "memory");
    for (int i = tid; i < nrows * (VR / 8); i += 256)
      *(shortx8*)(out + row0 * VR + (long)i * 8) = *(const shortx8*)(ob + i * 8);
    return;
  }
  // (a split without keys has no sums, and nobody reads any)
  const long prow = blockIdx.y * rows_all + row0;
#pragma unroll
  for (int t = 0; t < MT; ++t)
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int row = t * 16 + g * 4 + r;
      if (row >= nrows || tile0 >= tile1) continue;
#pragma unroll
      for (int c = 0; c < NT; ++c)
        part[(prow + row) * VR + (wave * NT + c) * 16 + col] = o[t][c][r];
    }
  if (wave == 0 && g == 0)
#pragma unroll
    for (int t = 0; t < MT; ++t) {
      const int row = t * 16 + col;
      if (row >= nrows) continue;
      float sum = 0.f;
#pragma unroll
      for (int w = 0; w < 4; ++w) sum += stat[w * ROWS + row];
      part_ml[(prow + row) * 2] = m[t];
      part_ml[(prow + row) * 2 + 1] = sum;
    }
}

// merge the context splits: one workgroup per row, R / 4 threads each on some of
// the splits
__global__ __launch_bounds__(256) void latent_combine_kernel(
    const float* __restrict__ part, const float* __restrict__ part_ml,
    bf16_t* __restrict__ out, long rows, int CS, int R) {
  __shared__ float weight[LAT_SPLITS];
  __shared__ __attribute__((aligned(16))) float sums[1024];
  __shared__ float red[4];
  const long row = blockIdx.x;
  const int tid = threadIdx.x, wave = tid / WAVE;
  float m = -1e30f, l = 0.f;
  if (tid < CS) {
    m = part_ml[(tid * rows + row) * 2];
    l = part_ml[(tid * rows + row) * 2 + 1];
  }
  float M = wave_max(m);
  if (tid % WAVE == 0) red[wave] = M;
  __syncthreads();
  M = fmaxf(fmaxf(red[0], red[1]), fmaxf(red[2], red[3]));
  const float w = __builtin_amdgcn_exp2f(m - M);
  if (tid < CS) weight[tid] = l != 0.f ? w : 0.f;  // a split without keys left no sums
  const float L = block_sum4(w * l, red);
  const int per = R / 4, groups = 256 / per, grp = tid / per, d = tid % per * 4;
  floatx4 a = {0.f, 0.f, 0.f, 0.f};
  if (grp < groups) {
#pragma unroll 4
    for (int s = grp; s < CS; s += groups)
      if (weight[s] != 0.f) a += ld4(part + (s * rows + row) * R + d) * weight[s];
    *(floatx4*)(sums + grp * R + d) = a;
  }
  __syncthreads();
  if (grp != 0) return;
  for (int i = 1; i < groups; ++i) a += *(const floatx4*)(sums + i * R + d);
  st4(out + row * R + d, a * (1.f / L));
}

torch::Tensor latent_attention(torch::Tensor q, torch::Tensor cache, torch::Tensor bt,
                               c10::optional<torch::Tensor> cu, torch::Tensor ctx,
                               c10::optional<torch::Tensor> bseq,
                               c10::optional<torch::Tensor> boff, long rows, double scale,
                               c10::optional<torch::Tensor> sink, long VR, long window) {
  const int T = q.size(0), H = q.size(1), R = q.size(2), S = ctx.numel();
  const int P = cache.size(2), MP = bt.size(1);
  TORCH_CHECK(q.is_cuda() && q.dtype() == torch::kBFloat16 && q.is_contiguous());
  TORCH_CHECK(cache.dtype() == torch::kBFloat16 && cache.is_contiguous() &&
              cache.size(1) == 1 && cache.size(3) == R, "latent cache");
  TORCH_CHECK(cache.size(0) * P < (1L << 31), "cache slots");
  TORCH_CHECK(bt.is_contiguous() && bt.dtype() == torch::kInt32 && bt.size(0) == S &&
              ctx.dtype() == torch::kInt32);
  TORCH_CHECK(!sink || (sink->numel() == H && sink->dtype() == torch::kFloat32));
  TORCH_CHECK(rows == 16 || rows == 32);
  int blocks;
  if (cu) {
    TORCH_CHECK(bseq && boff && bseq->numel() == boff->numel() && cu->numel() == S + 1 &&
                cu->dtype() == torch::kInt32 && bseq->dtype() == torch::kInt32 &&
                boff->dtype() == torch::kInt32);
    blocks = bseq->numel();
  } else {
    TORCH_CHECK(T == S);
    blocks = S * ((H + rows - 1) / rows);
  }
  auto out = torch::empty({T, H, VR}, q.options());
  if (T == 0 || blocks == 0) return out;
  // one workgroup per CU, or as many as its LDS holds
  int CS = std::max(1, std::min(LAT_SPLITS, (R > 256 ? 256 : 512) / blocks));
  // a split of its own for every tile that a window touches, at most
  if (window > 0) CS = std::min<long>(CS, (window + LAT_KEYS - 2) / LAT_KEYS + 1);
  const long all = (long)T * H;
  torch::Tensor part, ml;
  if (CS > 1) {
    part = torch::empty({CS, all, VR}, q.options().dtype(torch::kFloat32));
    ml = torch::empty({CS, all, 2}, q.options().dtype(torch::kFloat32));
  }
#define LATENT(RR, VV, MT)                                                               \
  do {                                                                                   \
    auto kern = latent_attention_kernel<RR, VV, MT>;                                     \
    constexpr int lds = 2 * LAT_KEYS * (RR) * 2 + \
                        2 * 16 * MT * LAT_PSTRIDE * 2 + 4 * 16 * MT * 4 + 32;              \
    static const hipError_t once = hipFuncSetAttribute(                                  \
        (const void*)kern, hipFuncAttributeMaxDynamicSharedMemorySize, lds);             \
    TORCH_CHECK(once == hipSuccess, "LDS of the latent attention kernel");               \
    hipLaunchKernelGGL(kern, dim3(blocks, CS), dim3(256), lds, CUR_STREAM,               \
                       (const bf16_t*)q.data_ptr(), (const bf16_t*)cache.data_ptr(),     \
                       bt.data_ptr<int>(), MP, cu ? cu->data_ptr<int>() : nullptr,       \
                       ctx.data_ptr<int>(), cu ? bseq->data_ptr<int>() : nullptr,        \
                       cu ? boff->data_ptr<int>() : nullptr,                             \
                       sink ? sink->data_ptr<float>() : nullptr,                         \
                       (bf16_t*)out.data_ptr(), CS > 1 ? part.data_ptr<float>() : nullptr, \
                       CS > 1 ? ml.data_ptr<float>() : nullptr, H, P, all, (float)scale,  \
                       (int)window);                                                     \
  } while (0)
#define LATENT_W(RR, VV)                       \
  if (R == RR && VR == VV) {                   \
    if (rows == 16) LATENT(RR, VV, 1);         \
    else LATENT(RR, VV, 2);                    \
  } else
#define LATENT_R(VV) LATENT_W(VV, VV) LATENT_W((VV + 64), VV)
  LATENT_R(64) LATENT_R(128) LATENT_R(256) LATENT_R(384) LATENT_R(512)
  TORCH_CHECK(false, "unsupported latent widths ", R, ", ", VR);
#undef LATENT_R
#undef LATENT_W
#undef LATENT
  if (CS > 1)
    hipLaunchKernelGGL(latent_combine_kernel, dim3(all), dim3(256), 0, CUR_STREAM,
                       part.data_ptr<float>(), ml.data_ptr<float>(), (bf16_t*)out.data_ptr(),
                       all, CS, (int)VR);
  HIP_CHECK_KERNEL();
  return out;
}

// ------------------------------------------------------------------ latents

template <typename T>
struct FrontArgs {
  const T* proj;         // [T, stride]
  long stride;
  int c0, rank;          // latents; c0 < 0: none
  const float* weight;
  int k0, key_at, rot;   // the rotated key part and its place in a row; rot 0: none
  const float* cs;       // [positions, rot]
  const int *pos, *slots;
  T* cache;              // rows of C
  int C;
  int q0, q_rank;        // the queries' latent; q_rank 0: none
  const float* q_weight;
  T* cq;                 // [T, q_rank]
  float eps;
};

// What latent attention does first, one wave per token and part: a token's latent is
// normed in fp32 and goes to its place in the cache with the rotated key part behind
// it; the queries' latent is normed.
template <typename T, int V>
__global__ __launch_bounds__(256) void latent_front_kernel(FrontArgs<T> a, int T_) {
  const int w = blockIdx.x * 4 + threadIdx.x / WAVE, lane = threadIdx.x % WAVE;
  const int parts = (a.c0 >= 0) + (a.q_rank > 0);
  const int t = w / parts;
  if (t >= T_) return;
  const bool query = a.c0 < 0 || w % parts == 1;
  const int slot = query ? 0 : a.slots[t];
  if (slot < 0) return;
  const int rank = query ? a.q_rank : a.rank;
  const T* row = a.proj + t * a.stride;
  const T* src = row + (query ? a.q0 : a.c0);
  const float* weight = query ? a.q_weight : a.weight;
  T* dst = query ? a.cq + (long)t * rank : a.cache + (long)slot * a.C;
  float ss = 0.f;
  for (int i = lane * V; i < rank; i += WAVE * V) {
    if constexpr (V == 4) {
      const floatx4 v = ld4(src + i);
#pragma unroll
      for (int j = 0; j < 4; ++j) ss += v[j] * v[j];
    } else {
      const float v = ldf(src + i);
      ss += v * v;
    }
  }
  const float inv = rsqrtf(wave_sum(ss) / rank + a.eps);
  const int width = query ? rank : a.C;
  const float* cs = a.rot > 0 && !query ? a.cs + (long)a.pos[t] * a.rot : nullptr;
  for (int i = lane * V; i < width; i += WAVE * V) {
    const int k = i - a.key_at;  // within the key part
    const bool key = cs && k >= 0 && k < a.rot;
    if constexpr (V == 4) {
      floatx4 y = {0.f, 0.f, 0.f, 0.f};
      if (i < rank) {
        y = ld4(src + i) * inv * ld4(weight + i);
      } else if (key) {
        y = ld4(row + a.k0 + k);
        float u0 = y[0], v0 = y[1], u1 = y[2], v1 = y[3];
        turn_pair(u0, v0, cs[k / 2], cs[(a.rot + k) / 2]);
        turn_pair(u1, v1, cs[k / 2 + 1], cs[(a.rot + k) / 2 + 1]);
        y = floatx4{u0, v0, u1, v1};
      }
      st4(dst + i, y);
    } else {
      float y = 0.f;
      if (i < rank) {
        y = ldf(src + i) * inv * weight[i];
      } else if (key) {
        float u = ldf(row + a.k0 + (k & ~1)), v = ldf(row + a.k0 + (k | 1));
        turn_pair(u, v, cs[k / 2], cs[a.rot / 2 + k / 2]);
        y = k & 1 ? v : u;
      }
      stf(dst + i, y);
    }
  }
}

// c0 < 0: the latents are another layer's; no cq: queries come without a latent
void latent_front(torch::Tensor proj, long c0, long rank, c10::optional<torch::Tensor> weight,
                  double eps, long k0, long key_at, c10::optional<torch::Tensor> cos_sin,
                  c10::optional<torch::Tensor> pos, torch::Tensor slots, torch::Tensor cache,
                  long q0, c10::optional<torch::Tensor> q_weight,
                  c10::optional<torch::Tensor> cq) {
  const int T_ = proj.size(0), C = cache.size(3);
  TORCH_CHECK(proj.is_cuda() && proj.dim() == 2 && proj.stride(1) == 1);
  TORCH_CHECK(cache.is_contiguous() && cache.size(1) == 1 && cache.dtype() == proj.dtype());
  auto norm = [&](const c10::optional<torch::Tensor>& w, long n) {
    return w && w->numel() == n && w->dtype() == torch::kFloat32 && w->is_contiguous();
  };
  const bool own = c0 >= 0;
  const int rot = own && cos_sin ? (int)cos_sin->size(1) : 0;
  if (own) {
    TORCH_CHECK(c0 + rank <= proj.size(1) && rank <= C && norm(weight, rank), "latents");
    TORCH_CHECK(slots.numel() == T_ && slots.dtype() == torch::kInt32);
  }
  if (rot) {
    TORCH_CHECK(cos_sin->dtype() == torch::kFloat32 && cos_sin->is_contiguous() &&
                cos_sin->dim() == 2 && rot % 2 == 0 && key_at >= rank && key_at + rot <= C &&
                k0 >= 0 && k0 + rot <= proj.size(1), "rotated key part");
    TORCH_CHECK(pos && pos->numel() == T_ && pos->dtype() == torch::kInt32);
  }
  const int q_rank = cq ? (int)cq->size(1) : 0;
  if (cq)
    TORCH_CHECK(cq->is_contiguous() && cq->size(0) == T_ && cq->dtype() == proj.dtype() &&
                q0 >= 0 && q0 + q_rank <= proj.size(1) && norm(q_weight, q_rank),
                "queries' latent");
  const long waves = (long)T_ * (own + (q_rank > 0));
  if (waves == 0) return;
  DISPATCH_ELEM(proj.dtype() == torch::kBFloat16, {
    FrontArgs<T> a = {};
    a.proj = (const T*)proj.data_ptr();
    a.stride = proj.stride(0);
    a.c0 = own ? c0 : -1;
    a.rank = rank;
    if (own) a.weight = weight->data_ptr<float>();
    a.key_at = rot ? key_at : C;
    if (rot) {
      a.k0 = k0;
      a.rot = rot;
      a.cs = cos_sin->data_ptr<float>();
      a.pos = pos->data_ptr<int>();
    }
    if (own) a.slots = slots.data_ptr<int>();
    a.cache = (T*)cache.data_ptr();
    a.C = C;
    if (q_rank) {
      a.q0 = q0;
      a.q_rank = q_rank;
      a.q_weight = q_weight->data_ptr<float>();
      a.cq = (T*)cq->data_ptr();
    }
    a.eps = eps;
    auto launch = [&](auto kern) {
      hipLaunchKernelGGL(kern, dim3((waves + 3) / 4), dim3(256), 0, CUR_STREAM, a, T_);
    };
    const long units = proj.stride(0) | q_rank | (q_rank ? q0 : 0) |
                       (own ? c0 | rank | C | a.key_at : 0) | (rot ? k0 | rot : 0);
    const bool vec = (units & 3) == 0 &&
                     (reinterpret_cast<uintptr_t>(proj.data_ptr()) & 15) == 0;
    if (vec) launch(latent_front_kernel<T, 4>);
    else launch(latent_front_kernel<T, 1>);
  });
  HIP_CHECK_KERNEL();
}

// cached rows, packed: 16 bytes per thread
__global__ __launch_bounds__(256) void gather_latents_kernel(
    const shortx8* __restrict__ cache, const int* __restrict__ rows, shortx8* __restrict__ out,
    long total, int units) {
  const long i = (long)blockIdx.x * 256 + threadIdx.x;
  if (i >= total) return;
  const int n = (int)(i / units);
  out[i] = cache[(long)rows[n] * units + i % units];
}

torch::Tensor gather_latents(torch::Tensor cache, torch::Tensor rows) {
  const long N = rows.numel(), C = cache.size(3);
  TORCH_CHECK(cache.is_cuda() && cache.is_contiguous() && cache.size(1) == 1 &&
              cache.dtype() == torch::kBFloat16 && C % 8 == 0, "latent cache");
  TORCH_CHECK(rows.dtype() == torch::kInt32 && rows.is_contiguous());
  auto out = torch::empty({N, C}, cache.options());
  const long total = N * (C / 8);
  if (total == 0) return out;
  hipLaunchKernelGGL(gather_latents_kernel, dim3((total + 255) / 256), dim3(256), 0, CUR_STREAM,
                     (const shortx8*)cache.data_ptr(), rows.data_ptr<int>(),
                     (shortx8*)out.data_ptr(), total, (int)(C / 8));
  HIP_CHECK_KERNEL();
  return out;
}

// ------------------------------------------------------------- rotated dimensions

// neighbouring pairs of x's first ``rot`` dimensions turn into out, zeros follow
template <typename T>
struct TurnHeads {
  const T* x;
  long xt, xh;
  T* out;
  long ot, oh;
  const float* cs;  // [positions, rot]
  const int* pos;
  int rot, W;       // W: dimensions of out, even
  int unit;         // dimensions per thread: 8 in 16-byte accesses, or 2
  __host__ __device__ int units() const { return W / unit; }
};

template <typename T>
DEVINL void turn_heads(const TurnHeads<T>& a, int t, int h, int i) {
  const int d = i * a.unit;
  const T* p = a.x + t * a.xt + h * a.xh + d;
  T* to = a.out + t * a.ot + h * a.oh + d;
  const float* cs = a.cs + (long)a.pos[t] * a.rot + d / 2;
  const bool turns = d < a.rot;
  if (a.unit == 8) {
    floatx4 y[2] = {{0.f, 0.f, 0.f, 0.f}, {0.f, 0.f, 0.f, 0.f}};
    if (turns) {
      const floatx4 c = ld4(cs), s = ld4(cs + a.rot / 2);
#pragma unroll
      for (int k = 0; k < 2; ++k) {
        const floatx4 x = ld4(p + 4 * k);
        float u0 = x[0], v0 = x[1], u1 = x[2], v1 = x[3];
        turn_pair(u0, v0, c[2 * k], s[2 * k]);
        turn_pair(u1, v1, c[2 * k + 1], s[2 * k + 1]);
        y[k] = floatx4{u0, v0, u1, v1};
      }
    }
    st4(to, y[0]);
    st4(to + 4, y[1]);
    return;
  }
  float u = 0.f, v = 0.f;
  if (turns) {
    u = ldf(p);
    v = ldf(p + 1);
    turn_pair(u, v, cs[0], cs[a.rot / 2]);
  }
  stf(to, u);
  stf(to + 1, v);
}

template <typename T>
__global__ __launch_bounds__(256) void rotate_heads_kernel(TurnHeads<T> a, long total, int H) {
  const long i = (long)blockIdx.x * 256 + threadIdx.x;
  if (i >= total) return;
  const int units = a.units();
  const long th = i / units;
  turn_heads(a, (int)(th / H), (int)(th % H), (int)(i % units));
}

template <typename T>
static TurnHeads<T> turn_args(const torch::Tensor& x, const torch::Tensor& pos,
                              const torch::Tensor& cos_sin, const torch::Tensor& out) {
  TORCH_CHECK(x.is_cuda() && x.dim() == 3 && out.dim() == 3 && out.dtype() == x.dtype() &&
              out.size(0) == x.size(0) && out.size(1) == x.size(1) && x.stride(2) == 1 &&
              out.stride(2) == 1, "rotated heads");
  TORCH_CHECK(cos_sin.dtype() == torch::kFloat32 && cos_sin.is_contiguous() &&
              cos_sin.dim() == 2 && cos_sin.size(1) % 2 == 0 && cos_sin.size(1) <= x.size(2) &&
              cos_sin.size(1) <= out.size(2) && out.size(2) % 2 == 0, "rotation");
  TORCH_CHECK(pos.numel() == x.size(0) && pos.dtype() == torch::kInt32 && pos.is_contiguous());
  TurnHeads<T> a = {(const T*)x.data_ptr(), x.stride(0), x.stride(1), (T*)out.data_ptr(),
                    out.stride(0), out.stride(1), cos_sin.data_ptr<float>(),
                    pos.data_ptr<int>(), (int)cos_sin.size(1), (int)out.size(2), 2};
  const long strides = a.xt | a.xh | a.ot | a.oh | a.rot | a.W;
  const uintptr_t at = reinterpret_cast<uintptr_t>(a.x) | reinterpret_cast<uintptr_t>(a.out);
  if ((strides & 7) == 0 && (at & 15) == 0) a.unit = 8;
  return a;
}

void rotate_heads(torch::Tensor x, torch::Tensor pos, torch::Tensor cos_sin,
                  torch::Tensor out) {
  DISPATCH_ELEM(x.dtype() == torch::kBFloat16, {
    const TurnHeads<T> a = turn_args<T>(x, pos, cos_sin, out);
    const long total = x.size(0) * x.size(1) * a.units();
    if (total == 0) return;
    hipLaunchKernelGGL((rotate_heads_kernel<T>), dim3((total + 255) / 256), dim3(256), 0,
                       CUR_STREAM, a, total, (int)x.size(1));
  });
  HIP_CHECK_KERNEL();
}

// --------------------------------------------------------- per-head products

// out[t, h, n] = sum_k x[t, h, k] w[h, n, k], times sigmoid(gate[t, h]). Waves
// take 16 outputs each (KS 1) or split the contraction (KS 4); TT 16-token
// tiles per workgroup. K and N are multiples of 32; STEPS: 32-wide steps of a
// wave if known, all of whose loads are then in flight at once. With ``turn`` the last
// ``turners`` blocks of a row of blocks turn the rotated dimensions of the same tokens
// and head.
template <int TT, int KS, int STEPS>
__global__ __launch_bounds__(256) void head_linear_kernel(
    const bf16_t* __restrict__ x, long xt, long xh, const bf16_t* __restrict__ w,
    const bf16_t* __restrict__ gate, long gt, bf16_t* __restrict__ out, long ot, long oh,
    int T_, int N, int K, TurnHeads<bf16_t> turn, int turners) {
  __shared__ __attribute__((aligned(16))) float red[KS > 1 ? 4 : 1][TT][WAVE][4];
  const int wave = threadIdx.x / WAVE, lane = threadIdx.x % WAVE;
  const int col = lane & 15, g = lane >> 4;
  const int h = blockIdx.y, t0 = blockIdx.z * 16 * TT;
  const int part = (int)blockIdx.x - (int)(gridDim.x - turners);
  if (part >= 0) {
    const int units = turn.units(), n = min(16 * TT, T_ - t0) * units;
    for (int i = part * 256 + threadIdx.x; i < n; i += turners * 256)
      turn_heads(turn, t0 + i / units, h, i % units);
    return;
  }
  const int n0 = KS > 1 ? blockIdx.x * 16 : (blockIdx.x * 4 + wave) * 16;
  if (n0 >= N) return;  // KS 1 only: whole waves, no barrier follows
  const int steps = K / 32, lo = KS > 1 ? steps * wave / 4 : 0,
            hi = KS > 1 ? steps * (wave + 1) / 4 : steps;
  const bf16_t* wp = w + ((long)h * N + n0 + col) * K + lo * 32 + g * 8;
  const bf16_t* xp[TT];
#pragma unroll
  for (int t = 0; t < TT; ++t)
    xp[t] = x + min(t0 + t * 16 + col, T_ - 1) * xt + h * xh + lo * 32 + g * 8;
  floatx4 acc[TT];
#pragma unroll
  for (int t = 0; t < TT; ++t) acc[t] = floatx4{0.f, 0.f, 0.f, 0.f};
  if constexpr (STEPS > 0) {
    lfrag a[STEPS], b[STEPS][TT];
#pragma unroll
    for (int k = 0; k < STEPS; ++k) {
      a[k].s = *(const shortx8*)(wp + k * 32);
#pragma unroll
      for (int t = 0; t < TT; ++t) b[k][t].s = *(const shortx8*)(xp[t] + k * 32);
    }
#pragma unroll
    for (int k = 0; k < STEPS; ++k)
#pragma unroll
      for (int t = 0; t < TT; ++t)
        acc[t] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(a[k].v, b[k][t].v, acc[t], 0, 0, 0);
  } else {
    for (int k = 0; k < hi - lo; ++k) {
      lfrag a, b;
      a.s = *(const shortx8*)(wp + k * 32);
#pragma unroll
      for (int t = 0; t < TT; ++t) {
        b.s = *(const shortx8*)(xp[t] + k * 32);
        acc[t] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(a.v, b.v, acc[t], 0, 0, 0);
      }
    }
  }
  if constexpr (KS > 1) {
#pragma unroll
    for (int t = 0; t < TT; ++t) *(floatx4*)red[wave][t][lane] = acc[t];
    __syncthreads();
  }
#pragma unroll
  for (int t = 0; t < TT; ++t) {
    if (KS > 1 && (t & 3) != wave) continue;  // the waves share the tiles
    floatx4 y = acc[t];
    if constexpr (KS > 1) {
      y = *(const floatx4*)red[0][t][lane];
#pragma unroll
      for (int s = 1; s < 4; ++s) y += *(const floatx4*)red[s][t][lane];
    }
    const int tok = t0 + t * 16 + col;
    if (tok >= T_) continue;
    if (gate) y *= sigmoid_f(ldf(gate + tok * gt + h));
    st4(out + tok * ot + h * oh + n0 + g * 4, y);
  }
}

void head_linear(torch::Tensor x, torch::Tensor w, c10::optional<torch::Tensor> gate,
                 torch::Tensor out, c10::optional<torch::Tensor> turn_x,
                 c10::optional<torch::Tensor> turn_pos, c10::optional<torch::Tensor> turn_cs,
                 c10::optional<torch::Tensor> turn_out) {
  const int T_ = x.size(0), H = x.size(1), K = x.size(2), N = w.size(1);
  TORCH_CHECK(x.is_cuda() && x.dtype() == torch::kBFloat16 && w.dtype() == x.dtype() &&
              out.dtype() == x.dtype() && w.is_contiguous());
  TORCH_CHECK(w.size(0) == H && w.size(2) == K && K % 32 == 0 && N % 32 == 0);
  auto aligned = [](const torch::Tensor& t, long unit) {
    return t.stride(2) == 1 && t.stride(0) % unit == 0 && t.stride(1) % unit == 0 &&
           (reinterpret_cast<uintptr_t>(t.data_ptr()) & (unit * 2 - 1)) == 0;
  };
  TORCH_CHECK(aligned(x, 8) && aligned(out, 4) && out.size(0) == T_ && out.size(1) == H &&
              out.size(2) == N);
  if (gate)
    TORCH_CHECK(gate->size(0) == T_ && gate->size(1) == H && gate->stride(1) == 1 &&
                gate->dtype() == x.dtype());
  TurnHeads<bf16_t> turn = {};
  if (turn_x) {
    TORCH_CHECK(turn_pos && turn_cs && turn_out && turn_x->size(0) == T_ &&
                turn_x->size(1) == H && turn_x->dtype() == x.dtype());
    turn = turn_args<bf16_t>(*turn_x, *turn_pos, *turn_cs, *turn_out);
  }
  if (T_ == 0) return;
  auto launch = [&](auto kern, int tt, int ks) {
    const int turners = turn.x ? (std::min(16 * tt, T_) * turn.units() + 255) / 256 : 0;
    const dim3 grid((ks > 1 ? N / 16 : (N + 63) / 64) + turners, H,
                    (T_ + 16 * tt - 1) / (16 * tt));
    hipLaunchKernelGGL(kern, grid, dim3(256), 0, CUR_STREAM, (const bf16_t*)x.data_ptr(),
                       x.stride(0), x.stride(1), (const bf16_t*)w.data_ptr(),
                       gate ? (const bf16_t*)gate->data_ptr() : nullptr,
                       gate ? gate->stride(0) : 0, (bf16_t*)out.data_ptr(), out.stride(0),
                       out.stride(1), T_, N, K, turn, turners);
  };
  // a long contraction for few tokens: split it over the waves
  const bool split = K >= 256 && T_ <= 64;
  const int steps = K / 32 % (split ? 4 : 1) ? 0 : K / 32 / (split ? 4 : 1);
#define HEAD_LINEAR(TT, KS)                                            \
  do {                                                                 \
    if (steps == 2) launch(head_linear_kernel<TT, KS, 2>, TT, KS);     \
    else if (steps == 4) launch(head_linear_kernel<TT, KS, 4>, TT, KS); \
    else launch(head_linear_kernel<TT, KS, 0>, TT, KS);                \
  } while (0)
#define HEAD_LINEAR_T(TT) \
  do { if (split) HEAD_LINEAR(TT, 4); else HEAD_LINEAR(TT, 1); } while (0)
  if (T_ <= 16) HEAD_LINEAR_T(1);
  else if (T_ <= 32) HEAD_LINEAR_T(2);
  else HEAD_LINEAR_T(4);
#undef HEAD_LINEAR_T
#undef HEAD_LINEAR
  HIP_CHECK_KERNEL();
}
