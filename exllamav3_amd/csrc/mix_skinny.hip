// Matrix products of few rows (decode steps): y = x W^T with W [out][in] as a checkpoint stores it, bfloat16, float32 accumulation.  Such a product is a stream over the
// weights: one workgroup takes 16 or 32 rows of W, its waves an equal share of the contraction each, every wave with many 16-byte loads in flight.
// v_mfma_f32_16x16x32_bf16: A = 16 rows of W straight from memory (lane (g, c): row c, entries 8g .. 8g + 7 of the step's 32), B = up to 16 rows of x, result lane (g, c):
// rows 4g .. 4g + 3 of W for row c of x.  The waves' partial tiles meet in LDS in a fixed order.
// Several matrices of the same shape with an x of their own (and one last matrix of another height) run as one launch.
#include "mix_common.cuh"

typedef __bf16 bf16x8 __attribute__((ext_vector_type(8)));
typedef float f32x4 __attribute__((ext_vector_type(4)));


// RT: 16-row tiles of W per workgroup; AHEAD: steps of 32 whose loads are in flight together; WAVES: waves per workgroup.  Matrix m of `mats` (rows x k at w + m rows k) reads x + m x_mat and writes out + m out_mat; matrix `mats` (tail rows, behind the
// others) writes out_tail.  K is a multiple of 8; entries beyond it weigh nothing.
template <int RT, int AHEAD, int WAVES>
__global__ __launch_bounds__(64 * WAVES) void skinny_kernel(bf16_t* __restrict__ out, int64_t out_ld, int64_t out_mat, bf16_t* __restrict__ out_tail, int64_t tail_ld,
                                                            const bf16_t* __restrict__ x, int64_t x_ld, int64_t x_mat, const bf16_t* __restrict__ w, int64_t w_ld,
                                                            const bf16_t* __restrict__ bias, int n, int K, int mats, int rows, int tail, int tiles)
{
    __shared__ __attribute__((aligned(16))) float part[WAVES][RT][64][4];
    const int lane = threadIdx.x & 63, wv = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6), g = lane >> 4, c = lane & 15;
    const int m = min((int) blockIdx.x / tiles, mats), r0 = ((int) blockIdx.x - m * tiles) * (16 * RT), mrows = m == mats ? tail : rows;
    const int n0 = blockIdx.y * 16;
    const bf16_t* xr = x + m * x_mat + (int64_t) min(n0 + c, n - 1) * x_ld;             // rows beyond the last: computed and never stored
    const bf16_t* wr[RT];
    #pragma unroll
    for (int t = 0; t < RT; ++t) wr[t] = w + ((int64_t) m * rows + min(r0 + t * 16 + c, mrows - 1)) * w_ld;
    const int steps = (K + 31) / 32, per = (steps + WAVES - 1) / WAVES, s_end = min((wv + 1) * per, steps);
    f32x4 acc[RT];
    #pragma unroll
    for (int t = 0; t < RT; ++t) acc[t] = f32x4{0.f, 0.f, 0.f, 0.f};
    union frag { bf16x8 v; uint4 x; };
    int s = wv * per;
    for (; s + AHEAD <= s_end && (s + AHEAD) * 32 <= K; s += AHEAD)            // whole groups: no bounds inside
    {
        frag a[AHEAD][RT], b[AHEAD];
        #pragma unroll
        for (int u = 0; u < AHEAD; ++u)
        {
            const int k = (s + u) * 32 + g * 8;
            #pragma unroll
            for (int t = 0; t < RT; ++t) a[u][t].x = *(const uint4*) (wr[t] + k);
            b[u].x = *(const uint4*) (xr + k);
        }
        #pragma unroll
        for (int u = 0; u < AHEAD; ++u)
        {
            #pragma unroll
            for (int t = 0; t < RT; ++t) acc[t] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(a[u][t].v, b[u].v, acc[t], 0, 0, 0);
        }
    }
    for (; s < s_end; ++s)
    {
        const int k = s * 32 + g * 8;
        const bool ok = k < K;
        frag b;
        b.x = ok ? *(const uint4*) (xr + k) : uint4{0u, 0u, 0u, 0u};
        #pragma unroll
        for (int t = 0; t < RT; ++t)
        {
            frag a;
            a.x = ok ? *(const uint4*) (wr[t] + k) : uint4{0u, 0u, 0u, 0u};
            acc[t] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(a.v, b.v, acc[t], 0, 0, 0);
        }
    }
    #pragma unroll
    for (int t = 0; t < RT; ++t) *(f32x4*) part[wv][t][lane] = acc[t];
    __syncthreads();
    for (int e = threadIdx.x; e < RT * 256; e += 64 * WAVES)
    {
        const int col = e / (RT * 16), rr = e - col * (RT * 16), t = rr >> 4, i = rr & 15;      // neighbouring threads: neighbouring rows of W
        const int src = (i >> 2) * 16 + col;
        float y = 0.f;
        #pragma unroll
        for (int v = 0; v < WAVES; ++v) y += part[v][t][src][i & 3];
        const int r = r0 + rr;
        if (r >= mrows || n0 + col >= n) continue;
        if (bias) y += to_f(bias[(int64_t) m * rows + r]);
        bf16_t* dst = m == mats ? out_tail + (int64_t) (n0 + col) * tail_ld : out + m * out_mat + (int64_t) (n0 + col) * out_ld;
        dst[r] = from_f<bf16_t>(y);
    }
}

extern "C" int exl3_mix_skinny(void* out, int64_t out_ld, int64_t out_mat, void* out_tail, int64_t tail_ld, const void* x, int64_t x_ld, int64_t x_mat, const void* w, int64_t w_ld,
                               const void* bias, int n, int K, int mats, int rows, int tail, void* stream)
{
    MIX_CHECK(out && x && w && n >= 0 && n <= 16 * 65535 && K > 0 && K % 8 == 0 && mats >= 1 && rows > 0 && tail >= 0 && (tail == 0 || (out_tail && tail_ld >= tail)), "mix_skinny: bad sizes (K a multiple of 8)");
    MIX_CHECK(out_ld >= rows && x_ld >= K && w_ld >= K && x_ld % 8 == 0 && w_ld % 8 == 0 && x_mat % 8 == 0 && (uintptr_t) x % 16 == 0 && (uintptr_t) w % 16 == 0, "mix_skinny: 16-byte aligned rows");
    if (n == 0) return EXL3_MIX_OK;
    // One to four rows: the weights are all there is to read, sixteen waves share a tile's contraction.  More rows: x is read as often as W, so workgroups of few waves and two
    // tiles (one read of x for both) where there are enough of them.
    const int rt = n > 4 && (int64_t) mats * rows >= 8192 ? 2 : 1;
    const int tiles = (rows + 16 * rt - 1) / (16 * rt);
    const int64_t blocks = (int64_t) mats * tiles + (tail + 16 * rt - 1) / (16 * rt);
    MIX_CHECK(blocks < (1 << 30), "mix_skinny: too many rows");
    #define SK_LAUNCH(RTV, AV, WV) hipLaunchKernelGGL((skinny_kernel<RTV, AV, WV>), dim3((unsigned) blocks, (n + 15) / 16), dim3(64 * WV), 0, (hipStream_t) stream, (bf16_t*) out, out_ld, out_mat, \
                                                      (bf16_t*) out_tail, tail_ld, (const bf16_t*) x, x_ld, x_mat, (const bf16_t*) w, w_ld, (const bf16_t*) bias, n, K, mats, rows, tail, tiles)
    if (n <= 4) SK_LAUNCH(1, 4, 16); else if (rt == 2) SK_LAUNCH(2, 4, 4); else SK_LAUNCH(1, 2, 8);
    #undef SK_LAUNCH
    return mix_check_launch("mix_skinny");
}
