// Attention over a sliding window with kept first tokens and a bias by distance (storage type bf16 or fp32, sizes at run time).
//
//   position i sees j <= i with i - j < window or j < keep_first;  score = (q . k) * scale + bias[h][min(i - j, n_dist - 1)]
//
// cache row   [K of every kv head | V of every kv head], each head padded with zeros to a multiple of 8 elements, so that any head size
//             is read in 16-byte (bf16) or 32-byte (fp32) pieces.  Where values are keys (SHARED) a head is there once, as projected: it
//             is read once, is the value, and its score takes 1 / rms of the key as a factor, so no second form of a key exists anywhere.
// keys        a query's visible keys are numbered 0 .. count - 1: first the kept ones in front of the window, then the window
// rows kernel work-group = 4 waves on one (token, kv head, block of query heads, split of the keys); 16 lanes hold one key, eight
//             elements a lane, so a wave takes four keys at a time; every 16-lane group keeps its own running maximum and sum for
//             each of its query heads and they meet once, at the end.  Scores, weights and sums are fp32.
#include "gh_product.h"
#include "gh_window.h"

#include <algorithm>

namespace gh {
namespace {

// cache rows are reached through pointers out of a table: the cast names the address space, so that no flat loads are used
typedef uint32_t u32x4_t __attribute__( ( ext_vector_type( 4 ) ) );
typedef const u32x4_t __attribute__( ( address_space( 1 ) ) ) global_u32x4_t;

// where a row's heads go: heads * vdim columns, rows `stride` elements apart; a factor for each head's output, or NULL
template<typename E>
struct WindowOut
{
  E* out;
  uint64_t stride;
  const float* gates;
  uint32_t heads;
  __device__ __forceinline__ float gate( uint64_t row, uint32_t head ) const { return gates != nullptr ? gates[row * heads + head] : 1.0f; }
};

// ---- q / k norm over the whole projection, cache append ------------------------------------------
// work-group = one token's q, its k or its v (blockIdx.y): columns of the product, normed where there is a norm, to padded heads
struct AppendPart
{
  uint32_t first, cols, dim, pad; // columns of the product; head size and its padded form
  const void* norm;               // (cols) or NULL
};

template<typename E>
__device__ __forceinline__ E* append_target( E* q_out, const WindowRows& wr, const WindowShape& s, uint64_t row )
{
  const uint32_t ctx = (uint32_t)( row / wr.n_tokens ), tok = (uint32_t)( row % wr.n_tokens );
  uint8_t* base = static_cast<uint8_t*>( wr.rows[ctx] );
  if ( base == nullptr ) {
    return nullptr;
  }
  if ( blockIdx.y == 0 ) {
    return q_out + row * s.heads * s.dpad;
  }
  E* cache = reinterpret_cast<E*>( base + wr.offset ) + (uint64_t)( wr.start_pos[ctx] + tok ) * s.row_elems();
  return cache + ( blockIdx.y == 1 ? 0 : s.k_elems() );
}

__device__ __forceinline__ float append_row_sum( float v, float* smem )
{
  v = wave_sum( v );
  if ( ( threadIdx.x & 63 ) == 0 ) {
    smem[threadIdx.x >> 6] = v;
  }
  __syncthreads();
  float total = 0.0f;
  for ( uint32_t w = 0; w < blockDim.x / WAVE; w++ ) {
    total += smem[w];
  }
  return total;
}

// head size, product columns and tables in groups of four; a thread owns NV groups, kept in registers across the norm
template<typename E, typename View, int NV>
__global__ __launch_bounds__( 1024 ) void window_append4_kernel( E* __restrict__ q_out, View y, const E* __restrict__ bias, AppendPart pq, AppendPart pk, AppendPart pv,
                                                                 WindowRows wr, WindowShape s, float eps )
{
  __shared__ float smem[16];
  const uint64_t row = blockIdx.x;
  E* dst = append_target( q_out, wr, s, row );
  if ( dst == nullptr ) {
    return;
  }
  const AppendPart p = blockIdx.y == 0 ? pq : blockIdx.y == 1 ? pk : pv;
  const E* norm = static_cast<const E*>( p.norm );
  float4 v[NV], w[NV];
  float ss = 0.0f;
#pragma unroll
  for ( int g = 0; g < NV; g++ ) {
    const uint32_t c = ( g * blockDim.x + threadIdx.x ) * 4, at = c < p.cols ? c : 0;
    v[g] = y.at4( row, p.first + at );
    w[g] = norm != nullptr ? ProductView<E>::load4( norm + at ) : make_float4( 1.0f, 1.0f, 1.0f, 1.0f );
    if ( bias != nullptr ) {
      const float4 b = ProductView<E>::load4( bias + p.first + at );
      v[g] = make_float4( v[g].x + b.x, v[g].y + b.y, v[g].z + b.z, v[g].w + b.w );
    }
    ss += c < p.cols ? v[g].x * v[g].x + v[g].y * v[g].y + v[g].z * v[g].z + v[g].w * v[g].w : 0.0f;
  }
  const float inv = norm != nullptr ? 1.0f / sqrtf( append_row_sum( ss, smem ) / (float)p.cols + eps ) : 1.0f;
#pragma unroll
  for ( int g = 0; g < NV; g++ ) {
    const uint32_t c = ( g * blockDim.x + threadIdx.x ) * 4;
    if ( c >= p.cols ) {
      continue;
    }
    union
    {
      E e[4];
      uint2 half;
      uint4 full;
    } o;
    o.e[0] = from_f32<E>( v[g].x * inv * w[g].x );
    o.e[1] = from_f32<E>( v[g].y * inv * w[g].y );
    o.e[2] = from_f32<E>( v[g].z * inv * w[g].z );
    o.e[3] = from_f32<E>( v[g].w * inv * w[g].w );
    // (without padding the columns are where they belong already, and the divisions can be saved)
    const bool padded = p.pad != p.dim;
    const uint32_t h = padded ? c / p.dim : 0, e = c - h * p.dim;
    E* at = dst + (uint64_t)h * p.pad + e;
    if constexpr ( sizeof( E ) == 2 ) {
      *reinterpret_cast<uint2*>( at ) = o.half;
    } else {
      *reinterpret_cast<uint4*>( at ) = o.full;
    }
    if ( padded && e + 4 == p.dim ) {
      for ( uint32_t z = p.dim; z < p.pad; z++ ) {
        dst[(uint64_t)h * p.pad + z] = from_f32<E>( 0.0f );
      }
    }
  }
}

// prompts (bias and both norms present): work-group = a token's q, k and v together, the columns of the product in one run; all loads go out
// together and both sums meet at one barrier
template<typename E, typename View, int NV>
__global__ __launch_bounds__( 1024 ) void window_append_row_kernel( E* __restrict__ q_out, View y, const E* __restrict__ bias, AppendPart pq, AppendPart pk, AppendPart pv,
                                                                    WindowRows wr, WindowShape s, float eps )
{
  __shared__ float q_sums[16], k_sums[16];
  const uint64_t row = blockIdx.x;
  const uint32_t ctx = (uint32_t)( row / wr.n_tokens ), tok = (uint32_t)( row % wr.n_tokens );
  uint8_t* base = static_cast<uint8_t*>( wr.rows[ctx] );
  if ( base == nullptr ) {
    return;
  }
  const uint32_t cols = pv.first + pv.cols;
  const E *q_norm = static_cast<const E*>( pq.norm ), *k_norm = static_cast<const E*>( pk.norm );
  float4 v[NV], w[NV];
  float qq = 0.0f, kk = 0.0f;
#pragma unroll
  for ( int g = 0; g < NV; g++ ) {
    const uint32_t c = ( g * blockDim.x + threadIdx.x ) * 4, at = c < cols ? c : 0;
    v[g] = y.at4( row, at );
    const bool is_q = at < pk.first;
    w[g] = ProductView<E>::load4( is_q ? q_norm + at : k_norm + ( at < pv.first ? at - pk.first : 0 ) ); // (v: not used)
    const float4 b = ProductView<E>::load4( bias + at );
    v[g] = make_float4( v[g].x + b.x, v[g].y + b.y, v[g].z + b.z, v[g].w + b.w );
    const float sum = c < pv.first ? v[g].x * v[g].x + v[g].y * v[g].y + v[g].z * v[g].z + v[g].w * v[g].w : 0.0f;
    qq += is_q ? sum : 0.0f;
    kk += is_q ? 0.0f : sum;
  }
  qq = wave_sum( qq );
  kk = wave_sum( kk );
  if ( ( threadIdx.x & 63 ) == 0 ) {
    q_sums[threadIdx.x >> 6] = qq;
    k_sums[threadIdx.x >> 6] = kk;
  }
  __syncthreads();
  qq = kk = 0.0f;
  for ( uint32_t i = 0; i < blockDim.x / WAVE; i++ ) {
    qq += q_sums[i];
    kk += k_sums[i];
  }
  const float q_inv = 1.0f / sqrtf( qq / (float)pq.cols + eps );
  const float k_inv = 1.0f / sqrtf( kk / (float)pk.cols + eps );
  E* q_dst = q_out + row * s.heads * s.dpad;
  E* k_dst = reinterpret_cast<E*>( base + wr.offset ) + (uint64_t)( wr.start_pos[ctx] + tok ) * s.row_elems();
  E* v_dst = k_dst + s.k_elems();
#pragma unroll
  for ( int g = 0; g < NV; g++ ) {
    const uint32_t c = ( g * blockDim.x + threadIdx.x ) * 4;
    if ( c >= cols ) {
      continue;
    }
    const bool is_q = c < pk.first, is_v = c >= pv.first;
    const float inv = is_q ? q_inv : k_inv;
    const uint32_t local = c - ( is_q ? 0 : is_v ? pv.first : pk.first );
    const uint32_t dim = is_v ? pv.dim : pq.dim, pad = is_v ? pv.pad : pq.pad;
    union
    {
      E e[4];
      uint2 half;
      uint4 full;
    } o;
    o.e[0] = from_f32<E>( is_v ? v[g].x : v[g].x * inv * w[g].x );
    o.e[1] = from_f32<E>( is_v ? v[g].y : v[g].y * inv * w[g].y );
    o.e[2] = from_f32<E>( is_v ? v[g].z : v[g].z * inv * w[g].z );
    o.e[3] = from_f32<E>( is_v ? v[g].w : v[g].w * inv * w[g].w );
    const uint32_t h = pad != dim ? local / dim : 0, e = local - h * dim;
    E* at = ( is_q ? q_dst : is_v ? v_dst : k_dst ) + (uint64_t)h * pad + e;
    if constexpr ( sizeof( E ) == 2 ) {
      *reinterpret_cast<uint2*>( at ) = o.half;
    } else {
      *reinterpret_cast<uint4*>( at ) = o.full;
    }
    if ( pad != dim && e + 4 == dim ) {
      for ( uint32_t z = dim; z < pad; z++ ) {
        at[z - e] = from_f32<E>( 0.0f );
      }
    }
  }
}

// any sizes: the columns of the part pass through LDS
template<typename E, typename View>
__global__ __launch_bounds__( 256 ) void window_append_any_kernel( E* __restrict__ q_out, View y, const E* __restrict__ bias, AppendPart pq, AppendPart pk, AppendPart pv,
                                                                   WindowRows wr, WindowShape s, float eps )
{
  extern __shared__ float vals[];
  __shared__ float smem[4];
  const uint64_t row = blockIdx.x;
  E* dst = append_target( q_out, wr, s, row );
  if ( dst == nullptr ) {
    return;
  }
  const AppendPart p = blockIdx.y == 0 ? pq : blockIdx.y == 1 ? pk : pv;
  const E* norm = static_cast<const E*>( p.norm );
  float ss = 0.0f;
  for ( uint32_t c = threadIdx.x; c < p.cols; c += blockDim.x ) {
    const float v = y.at( row, p.first + c ) + ( bias != nullptr ? to_f32( bias[p.first + c] ) : 0.0f );
    vals[c] = v;
    ss += v * v;
  }
  const float total = append_row_sum( ss, smem ); // (also the barrier in front of the reads below)
  const float inv = norm != nullptr ? 1.0f / sqrtf( total / (float)p.cols + eps ) : 1.0f;
  for ( uint32_t c = threadIdx.x; c < p.cols / p.dim * p.pad; c += blockDim.x ) {
    const uint32_t h = c / p.pad, e = c % p.pad, src = h * p.dim + e;
    dst[c] = from_f32<E>( e < p.dim ? vals[src] * inv * ( norm != nullptr ? to_f32( norm[src] ) : 1.0f ) : 0.0f );
  }
}

template<typename E, typename View>
int launch_append( E* q, const View& y, const E* bias, const void* q_norm, const void* k_norm, float eps, const WindowRows& wr, const WindowShape& s, uint64_t rows,
                   hipStream_t st )
{
  const uint32_t nq = s.heads * s.dim, nk = s.kv_heads * s.dim, nv = s.kv_heads * s.vdim;
  const AppendPart pq { 0, nq, s.dim, s.dpad, q_norm }, pk { nq, nk, s.dim, s.dpad, k_norm }, pv { nq + nk, nv, s.vdim, s.vpad, nullptr };
  const uint32_t most = std::max( { nq, nk, nv } );
  const dim3 grid( (unsigned)rows, 3 );
  const uintptr_t tables = reinterpret_cast<uintptr_t>( bias ) | reinterpret_cast<uintptr_t>( q_norm ) | reinterpret_cast<uintptr_t>( k_norm );
  if ( s.dim % 4 == 0 && s.vdim % 4 == 0 && y.stride % 4 == 0 && ( tables & 15u ) == 0 && most <= 32768 ) {
    if ( const uint32_t all = ( nq + nk + nv ) / 4; rows >= 1024 && all <= 4096 && bias != nullptr && q_norm != nullptr && k_norm != nullptr ) {
      const uint32_t threads = std::max<uint32_t>( 64, ( ( all + 3 ) / 4 + 63 ) / 64 * 64 );
      window_append_row_kernel<E, View, 4><<<(unsigned)rows, threads, 0, st>>>( q, y, bias, pq, pk, pv, wr, s, eps );
      GH_LAUNCH_CHECK();
      return GH_OK;
    }
    const uint32_t groups = most / 4;
    const uint32_t want = rows >= 1024 ? ( groups + 3 ) / 4 : groups;
    const uint32_t threads = std::min<uint32_t>( 1024, std::max<uint32_t>( 64, ( want + 63 ) / 64 * 64 ) );
    const uint32_t per = ( groups + threads - 1 ) / threads;
    if ( per <= 1 ) {
      window_append4_kernel<E, View, 1><<<grid, threads, 0, st>>>( q, y, bias, pq, pk, pv, wr, s, eps );
    } else if ( per <= 2 ) {
      window_append4_kernel<E, View, 2><<<grid, threads, 0, st>>>( q, y, bias, pq, pk, pv, wr, s, eps );
    } else if ( per <= 4 ) {
      window_append4_kernel<E, View, 4><<<grid, threads, 0, st>>>( q, y, bias, pq, pk, pv, wr, s, eps );
    } else {
      window_append4_kernel<E, View, 8><<<grid, threads, 0, st>>>( q, y, bias, pq, pk, pv, wr, s, eps );
    }
  } else {
    GH_REQUIRE( most <= 15 * 1024, "gh_matmul_window_append: the heads of a token do not fit in LDS" );
    window_append_any_kernel<E, View><<<grid, 256, most * sizeof( float ), st>>>( q, y, bias, pq, pk, pv, wr, s, eps );
  }
  GH_LAUNCH_CHECK();
  return GH_OK;
}

// ---- visible keys ------------------------------------------------------------------------------
struct Visible
{
  uint32_t kept, first, count; // kept keys in front of the window, first key of the window, all of them
  __device__ __forceinline__ uint32_t key( uint32_t idx ) const { return idx < kept ? idx : first + ( idx - kept ); }
};
__device__ __forceinline__ Visible visible_keys( uint32_t pos, const WindowShape& s )
{
  Visible v;
  v.first = pos + 1 > s.window ? pos + 1 - s.window : 0;
  v.kept = min( s.keep_first, v.first );
  v.count = v.kept + ( pos + 1 - v.first );
  return v;
}

template<typename E>
__device__ __forceinline__ void load8( float out[8], const E* p )
{
  if constexpr ( sizeof( E ) == 2 ) {
    union
    {
      uint4 raw;
      E e[8];
    } u;
    u.raw = __builtin_bit_cast( uint4, *(global_u32x4_t*)( p ) );
#pragma unroll
    for ( int i = 0; i < 8; i++ ) {
      out[i] = to_f32( u.e[i] );
    }
  } else {
    const float4 a = __builtin_bit_cast( float4, *(global_u32x4_t*)( p ) ), b = __builtin_bit_cast( float4, *(global_u32x4_t*)( p + 4 ) );
    out[0] = a.x, out[1] = a.y, out[2] = a.z, out[3] = a.w, out[4] = b.x, out[5] = b.y, out[6] = b.z, out[7] = b.w;
  }
}

constexpr float NO_KEY = -1e30f; // running maximum before the first key: exp(NO_KEY - anything real) is 0

// partial result of one split of one (row, head): vpad weighted sums, then the sum of the weights and the maximum
__host__ __device__ inline uint64_t partial_stride( const WindowShape& s ) { return s.vpad + 2; }

// The results of a work-group's NW waves for the query heads h0 .. h0 + nh - 1 of a row, wave w's for head h at
// lds[(w * hq + h) * (vpad + 2)]: added up and stored, as the output or as the partial result of a split.
template<typename E, int NW>
__device__ __forceinline__ void finish_split( const WindowOut<E>& out, float* partial, const float* lds, uint32_t hq, uint32_t nh, uint64_t row, uint32_t h0, uint32_t split,
                                              uint32_t splits, const WindowShape& s )
{
  const uint32_t stride = s.vpad + 2;
  for ( uint32_t i = threadIdx.x; i < nh * s.vpad; i += 64 * NW ) {
    const uint32_t h = i / s.vpad, e = i % s.vpad;
    float m = NO_KEY;
#pragma unroll
    for ( int w = 0; w < NW; w++ ) {
      m = fmaxf( m, lds[( w * hq + h ) * stride + s.vpad + 1] );
    }
    float a = 0.0f, sm = 0.0f;
#pragma unroll
    for ( int w = 0; w < NW; w++ ) {
      const float* src = lds + ( w * hq + h ) * stride;
      const float f = __expf( src[s.vpad + 1] - m );
      a += src[e] * f;
      sm += src[s.vpad] * f;
    }
    if ( splits == 1 ) {
      if ( e < s.vdim ) {
        out.out[row * out.stride + ( h0 + h ) * s.vdim + e] = from_f32<E>( a / sm * out.gate( row, h0 + h ) );
      }
    } else {
      float* dst = partial + ( ( row * s.heads + h0 + h ) * splits + split ) * stride;
      dst[e] = a;
      if ( e == 0 ) {
        dst[s.vpad] = sm;
        dst[s.vpad + 1] = m;
      }
    }
  }
}

// HQ query heads at a time; NC pieces of 128 elements per head (a lane holds 8 of each)
template<typename E, int HQ, int NC, bool SHARED>
__global__ __launch_bounds__( 256 ) void window_rows_kernel( WindowOut<E> out,
                                                             float* __restrict__ partial,
                                                             const E* __restrict__ q,
                                                             const float* __restrict__ bias,
                                                             WindowRows wr,
                                                             WindowShape s,
                                                             uint32_t keys_per_split,
                                                             uint32_t splits )
{
  extern __shared__ float lds[]; // 4 waves x HQ x (vpad + 2)
  const uint32_t head_blocks = ( s.group + HQ - 1 ) / HQ;
  const uint32_t g = blockIdx.y / head_blocks, hb = blockIdx.y % head_blocks;
  const uint64_t row = blockIdx.x;
  const uint32_t split = blockIdx.z;
  const uint32_t ctx = (uint32_t)( row / wr.n_tokens ), tok = (uint32_t)( row % wr.n_tokens );
  const uint8_t* base = static_cast<const uint8_t*>( wr.rows[ctx] );
  if ( base == nullptr ) {
    return;
  }
  const uint32_t pos = wr.start_pos[ctx] + tok;
  const Visible vis = visible_keys( pos, s );
  const uint32_t wave = threadIdx.x >> 6, lane = threadIdx.x & 63, l16 = lane & 15, g4 = lane >> 4;
  const uint32_t h0 = g * s.group + hb * HQ;
  const uint32_t nh = min( (uint32_t)HQ, s.group - hb * HQ );
  const E* cache = reinterpret_cast<const E*>( base + wr.offset );
  const uint32_t k_begin = split * keys_per_split, k_end = min( vis.count, k_begin + keys_per_split );

  float qv[HQ][NC][8], acc[HQ][NC][8], mx[HQ], sum[HQ];
#pragma unroll
  for ( int h = 0; h < HQ; h++ ) {
    mx[h] = NO_KEY;
    sum[h] = 0.0f;
#pragma unroll
    for ( int c = 0; c < NC; c++ ) {
#pragma unroll
      for ( int e = 0; e < 8; e++ ) {
        qv[h][c][e] = 0.0f;
        acc[h][c][e] = 0.0f;
      }
      const uint32_t at = c * 128 + l16 * 8;
      if ( (uint32_t)h < nh && at < s.dpad ) {
        load8( qv[h][c], q + ( row * s.heads + h0 + h ) * s.dpad + at );
      }
    }
  }
  // U keys per 16-lane group and step: all their loads go out before the first is used.  A key past the end reads the step's first again
  // and gets no weight.
  constexpr uint32_t U = HQ * NC >= 4 ? 2 : 4;
  const uint32_t at_k = g * s.dpad, at_v = s.k_elems() + g * s.vpad;
  const float* factors = reinterpret_cast<const float*>( base + wr.factors );
  for ( uint32_t i0 = k_begin + wave * 4 * U; i0 < k_end; i0 += 16 * U ) {
    float kv[U][NC][8], vv[SHARED ? 1 : U][NC][8], factor[U];
    uint32_t dist[U];
    bool live[U];
#pragma unroll
    for ( uint32_t u = 0; u < U; u++ ) {
      const uint32_t idx = i0 + 4 * u + g4;
      live[u] = idx < k_end;
      const uint32_t j = vis.key( live[u] ? idx : i0 );
      dist[u] = min( pos - j, s.n_dist - 1 );
      factor[u] = SHARED ? s.scale * factors[factor_index( j, g, s.kv_heads )] : s.scale;
      const E* row_j = cache + (uint64_t)j * s.row_elems();
#pragma unroll
      for ( int c = 0; c < NC; c++ ) {
        const uint32_t at = c * 128 + l16 * 8;
#pragma unroll
        for ( int e = 0; e < 8; e++ ) {
          kv[u][c][e] = 0.0f;
        }
        if ( at < s.dpad ) {
          load8( kv[u][c], row_j + at_k + at );
        }
        if constexpr ( !SHARED ) {
#pragma unroll
          for ( int e = 0; e < 8; e++ ) {
            vv[u][c][e] = 0.0f;
          }
          if ( at < s.vpad ) {
            load8( vv[u][c], row_j + at_v + at );
          }
        }
      }
    }
#pragma unroll
    for ( int h = 0; h < HQ; h++ ) {
      float score[U];
      float m_new = mx[h];
#pragma unroll
      for ( uint32_t u = 0; u < U; u++ ) {
        float dot = 0.0f;
#pragma unroll
        for ( int c = 0; c < NC; c++ ) {
#pragma unroll
          for ( int e = 0; e < 8; e++ ) {
            dot += qv[h][c][e] * kv[u][c][e];
          }
        }
        const float b = bias != nullptr && (uint32_t)h < nh ? bias[(uint64_t)( h0 + h ) * s.n_dist + dist[u]] : 0.0f;
        score[u] = live[u] ? row16_sum( dot ) * factor[u] + b : NO_KEY;
        m_new = fmaxf( m_new, score[u] );
      }
      const float old = __expf( mx[h] - m_new );
      mx[h] = m_new;
      float p[U], p_sum = 0.0f;
#pragma unroll
      for ( uint32_t u = 0; u < U; u++ ) {
        p[u] = live[u] ? __expf( score[u] - m_new ) : 0.0f;
        p_sum += p[u];
      }
      sum[h] = sum[h] * old + p_sum;
#pragma unroll
      for ( int c = 0; c < NC; c++ ) {
#pragma unroll
        for ( int e = 0; e < 8; e++ ) {
          float a = acc[h][c][e] * old;
#pragma unroll
          for ( uint32_t u = 0; u < U; u++ ) {
            a += p[u] * ( SHARED ? kv[u][c][e] : vv[SHARED ? 0 : u][c][e] );
          }
          acc[h][c][e] = a;
        }
      }
    }
  }
  // the four 16-lane groups of the wave, then the four waves
  const uint32_t stride = s.vpad + 2;
#pragma unroll
  for ( int h = 0; h < HQ; h++ ) {
    float m = fmaxf( mx[h], __shfl_xor( mx[h], 16 ) );
    m = fmaxf( m, __shfl_xor( m, 32 ) );
    const float f = __expf( mx[h] - m );
    float sm = sum[h] * f;
    sm += __shfl_xor( sm, 16 );
    sm += __shfl_xor( sm, 32 );
    float* mine = lds + ( wave * HQ + h ) * stride;
#pragma unroll
    for ( int c = 0; c < NC; c++ ) {
      const uint32_t at = c * 128 + l16 * 8;
#pragma unroll
      for ( int e = 0; e < 8; e++ ) {
        float a = acc[h][c][e] * f;
        a += __shfl_xor( a, 16 );
        a += __shfl_xor( a, 32 );
        if ( g4 == 0 && at + e < s.vpad ) {
          mine[at + e] = a;
        }
      }
    }
    if ( lane == 0 ) {
      mine[s.vpad] = sm;
      mine[s.vpad + 1] = m;
    }
  }
  __syncthreads();
  finish_split<E, 4>( out, partial, lds, HQ, nh, row, h0, split, splits, s );
}

// one wave per (row, head)
template<typename E>
__global__ __launch_bounds__( 256 ) void window_merge_kernel( WindowOut<E> out, const float* __restrict__ partial, WindowRows wr, WindowShape s, uint32_t splits,
                                                              uint64_t pairs )
{
  const uint64_t pair = (uint64_t)blockIdx.x * 4 + ( threadIdx.x >> 6 );
  if ( pair >= pairs || wr.rows[pair / s.heads / wr.n_tokens] == nullptr ) {
    return;
  }
  const uint32_t lane = threadIdx.x & 63, stride = s.vpad + 2;
  const float* src = partial + pair * splits * stride;
  float m = NO_KEY;
  for ( uint32_t k = 0; k < splits; k++ ) {
    m = fmaxf( m, src[k * stride + s.vpad + 1] );
  }
  const uint64_t row = pair / s.heads;
  const uint32_t head = (uint32_t)( pair % s.heads );
  const float gate = out.gate( row, head );
  float sm = 0.0f;
  for ( uint32_t k = 0; k < splits; k++ ) {
    sm += src[k * stride + s.vpad] * __expf( src[k * stride + s.vpad + 1] - m );
  }
  for ( uint32_t e = lane; e < s.vdim; e += 64 ) {
    float a = 0.0f;
    for ( uint32_t k = 0; k < splits; k++ ) {
      a += src[k * stride + e] * __expf( src[k * stride + s.vpad + 1] - m );
    }
    out.out[row * out.stride + head * s.vdim + e] = from_f32<E>( a / sm * gate );
  }
}

// ---- many tokens: key tiles on the matrix cores (bf16, head sizes up to 128) -----------------------------------------------------
//
// work-group  4 waves on one (context, kv head), 32 query columns a wave; a column is (token, query head) with the query heads of a group side
//             by side where their number is a power of two, else one query head per work-group
// keys        64 at a time: the tiles of the kept first tokens in front of the window, then those of the window of the work-group's
//             tokens.  A tile that every column sees whole takes no mask, one farther away than the bias table is long a constant bias.
// scores^T    K Q^T by v_mfma_f32_32x32x16_bf16 (K out of LDS, Q in registers): a lane holds 32 of the tile's 64 scores of ITS column, the
//             lane 32 further on the others, so maximum and sum stay in the lane but for one exchange
// values      O^T += V^T P^T: the weights are, as they lie, the right operand; V^T comes out of LDS by transposing reads.  The weights
//             are fp32: they enter as two bf16 terms (16 bits of mantissa), their sum is taken in fp32.
// LDS         rows of 256 bytes whatever the head size (the rest is zero), 16-byte chunks XORed with bits of the row; the next tile's
//             rows are in registers while this one is multiplied, and two work-groups share a CU.  Where values are keys both products
//             read one tile: the low four bits of the row, pairs exchanged, keep the plain reads (16 rows, one chunk) and the
//             transposing ones (4 rows, 4 chunks) apart.
constexpr float LOG2E = 1.4426950408889634f;
constexpr float LAZY = 8.0f; // the reference point of a column's exponentials moves when its maximum has grown by 2^LAZY
constexpr uint32_t TILE_KEYS = 64;
constexpr uint32_t BIAS_LDS = 8192; // floats of bias table a work-group can hold
typedef __attribute__( ( address_space( 3 ) ) ) char lds_char;
typedef short v4s __attribute__( ( ext_vector_type( 4 ) ) );
typedef __attribute__( ( address_space( 3 ) ) ) v4s* lds_v4s;
typedef Mfma<__bf16>::x8 bf16x8;

__device__ __forceinline__ uint32_t shared_swizzle( uint32_t row ) { return ( ( row & 3 ) << 2 ) | ( ( row >> 2 ) & 3 ); }

// KS: steps of 16 of the query/key size; VB: blocks of 32 of the value size
template<int KS, int VB, bool SHARED>
__global__ __launch_bounds__( 256, 2 ) void window_tiles_kernel( WindowOut<__bf16> out,
                                                                 const __bf16* __restrict__ q,
                                                                 const float* __restrict__ bias,
                                                                 WindowRows wr,
                                                                 WindowShape s,
                                                                 uint32_t head_cols,  // query heads side by side in the columns
                                                                 uint32_t col_blocks, // work-groups along the tokens of a pair
                                                                 uint32_t n_pairs,    // contexts x kv heads x (query heads of a group / head_cols)
                                                                 uint32_t bias_floats )
{
  extern __shared__ uint4 lds16[];
  uint4* s_k = lds16;
  uint4* s_v = SHARED ? s_k : s_k + TILE_KEYS * 16;
  float* s_factor = reinterpret_cast<float*>( s_v + TILE_KEYS * 16 );  // SHARED: of the tile's keys, times scale and log2(e)
  float* s_bias = s_factor + ( SHARED ? TILE_KEYS : 0 );               // (head_cols, n_dist), times log2(e)

  // all column blocks of a pair on one XCD, next to each other in time: its keys come into one L2 once; the longest first
  const uint32_t xcd = blockIdx.x & 7, slot = blockIdx.x >> 3;
  const uint32_t cb = col_blocks - 1 - slot % col_blocks;
  const uint32_t pair = ( slot / col_blocks ) * 8 + xcd;
  if ( pair >= n_pairs ) {
    return;
  }
  const uint32_t per_group = s.group / head_cols;
  const uint32_t ctx = pair / ( s.kv_heads * per_group );
  const uint32_t g = pair / per_group % s.kv_heads;
  const uint32_t h0 = g * s.group + pair % per_group * head_cols;
  const uint8_t* base = static_cast<const uint8_t*>( wr.rows[ctx] );
  if ( base == nullptr ) {
    return;
  }
  const __bf16* cache = reinterpret_cast<const __bf16*>( base + wr.offset );
  const uint32_t start = wr.start_pos[ctx];
  const uint32_t wave = threadIdx.x >> 6, lane = threadIdx.x & 63, r = lane & 31, g2 = lane >> 5;
  const uint32_t tok_wg = cb * ( 128 / head_cols );
  const uint32_t tok_last = min( wr.n_tokens, tok_wg + 128 / head_cols ) - 1;
  const uint32_t colnum = wave * 32 + r;
  const uint32_t tok = tok_wg + colnum / head_cols, hc = colnum % head_cols;
  const bool col_ok = tok < wr.n_tokens;
  const uint32_t pos = start + ( col_ok ? tok : tok_last ); // a column without a query does as the last one and is not stored
  const uint32_t pos_first = start + tok_wg, pos_last = start + tok_last;

  for ( uint32_t i = threadIdx.x; i < bias_floats; i += 256 ) {
    s_bias[i] = bias[(uint64_t)h0 * s.n_dist + i] * LOG2E;
  }

  bf16x8 qb[KS];
  {
    const __bf16* qp = q + ( ( (uint64_t)ctx * wr.n_tokens + ( col_ok ? tok : tok_last ) ) * s.heads + h0 + hc ) * s.dpad;
#pragma unroll
    for ( int k = 0; k < KS; k++ ) {
      const uint32_t ch = 2 * k + g2;
      u32x4_t v = { 0, 0, 0, 0 };
      if ( ch * 8 < s.dpad ) {
        v = *(global_u32x4_t*)( qp + ch * 8 );
      }
      qb[k] = __builtin_bit_cast( bf16x8, v );
    }
  }

  // tiles: kept keys [0, kept), then [first, pos_last]
  const uint32_t first = pos_first + 1 > s.window ? pos_first + 1 - s.window : 0;
  const uint32_t kept = min( s.keep_first, first );
  const uint32_t kept_tiles = ( kept + TILE_KEYS - 1 ) / TILE_KEYS;
  const uint32_t tiles = kept_tiles + ( pos_last + 1 - first + TILE_KEYS - 1 ) / TILE_KEYS;
  auto tile_at = [&]( uint32_t i ) { return i < kept_tiles ? i * TILE_KEYS : first + ( i - kept_tiles ) * TILE_KEYS; };

  // a thread's four 16-byte pieces of a tile of K and of V: row threadIdx / 16 + 16 i, chunk threadIdx % 16
  const uint32_t ld_chunk = threadIdx.x & 15, ld_row = threadIdx.x >> 4;
  u32x4_t rk[4], rv[SHARED ? 1 : 4];
  const float* factors = reinterpret_cast<const float*>( base + wr.factors );
  float rf = 0.0f;
  auto load = [&]( uint32_t i ) {
    const uint32_t t0 = tile_at( i ), end = i < kept_tiles ? kept : pos_last + 1;
    if ( SHARED && threadIdx.x < TILE_KEYS ) {
      rf = factors[factor_index( min( t0 + threadIdx.x, end - 1 ), g, s.kv_heads )];
    }
#pragma unroll
    for ( int k = 0; k < 4; k++ ) {
      const uint32_t key = t0 + ld_row + 16 * k;
      rk[k] = u32x4_t { 0, 0, 0, 0 };
      const __bf16* row = cache + (uint64_t)min( key, end - 1 ) * s.row_elems();
      if ( key < end && ld_chunk * 8 < s.dpad && ld_chunk < 2 * KS ) {
        rk[k] = *(global_u32x4_t*)( row + g * s.dpad + ld_chunk * 8 );
      }
      if constexpr ( !SHARED ) {
        rv[k] = u32x4_t { 0, 0, 0, 0 };
        if ( key < end && ld_chunk * 8 < s.vpad && ld_chunk < 4 * VB ) {
          rv[k] = *(global_u32x4_t*)( row + s.k_elems() + g * s.vpad + ld_chunk * 8 );
        }
      }
    }
  };
  const float scale_log2e = s.scale * LOG2E;
  auto store = [&] {
#pragma unroll
    for ( int k = 0; k < 4; k++ ) {
      const uint32_t row = ld_row + 16 * k;
      s_k[row * 16 + ( ld_chunk ^ ( SHARED ? shared_swizzle( row ) : row & 15 ) )] = __builtin_bit_cast( uint4, rk[k] );
      if constexpr ( !SHARED ) {
        s_v[row * 16 + ( ld_chunk ^ ( 4 * ( row & 3 ) ) )] = __builtin_bit_cast( uint4, rv[k] );
      }
    }
    if ( SHARED && threadIdx.x < TILE_KEYS ) {
      s_factor[threadIdx.x] = rf * scale_log2e;
    }
  };
  const uint32_t tr_e = ( lane & 15 ) >> 2, tr_q = lane & 3, tr_grp = ( lane >> 4 ) & 1;
  const uint32_t v_lane = ( 4 * g2 + tr_e ) * 256 + ( ( ( 2 * tr_grp + ( tr_q >> 1 ) ) ^ ( 4 * tr_e ) ^ ( SHARED ? g2 : 0 ) ) * 16 ) + ( tr_q & 1 ) * 8;

  mfma_f32x16 acc[VB];
#pragma unroll
  for ( int vb = 0; vb < VB; vb++ ) {
#pragma unroll
    for ( int v = 0; v < 16; v++ ) {
      acc[vb][v] = 0.0f;
    }
  }
  float m = NO_KEY, l = 0.0f;
  const float* my_bias = s_bias + hc * s.n_dist;

  load( 0 );
  for ( uint32_t i = 0; i < tiles; i++ ) {
    __syncthreads(); // the last tile's readers are done (and the bias table is written)
    store();
    __syncthreads();
    if ( i + 1 < tiles ) {
      load( i + 1 );
    }
    const uint32_t t0 = tile_at( i );
    mfma_f32x16 st[2];
#pragma unroll
    for ( int sub = 0; sub < 2; sub++ ) {
#pragma unroll
      for ( int v = 0; v < 16; v++ ) {
        st[sub][v] = 0.0f;
      }
#pragma unroll
      for ( int k = 0; k < KS; k++ ) {
        const uint32_t row = 32 * sub + r;
        const bf16x8 a = __builtin_bit_cast( bf16x8, s_k[row * 16 + ( ( 2 * k + g2 ) ^ ( SHARED ? shared_swizzle( row ) : row & 15 ) )] );
        st[sub] = Mfma<__bf16>::k16( a, qb[k], st[sub] );
      }
    }
    // what a score is multiplied with: one number, or that of its key
    float factor[2][16];
#pragma unroll
    for ( int sub = 0; sub < 2; sub++ ) {
#pragma unroll
      for ( int q4 = 0; q4 < 4; q4++ ) {
        float4 f = make_float4( scale_log2e, scale_log2e, scale_log2e, scale_log2e );
        if constexpr ( SHARED ) {
          f = *reinterpret_cast<const float4*>( s_factor + 32 * sub + 8 * q4 + 4 * g2 );
        }
        factor[sub][4 * q4] = f.x, factor[sub][4 * q4 + 1] = f.y, factor[sub][4 * q4 + 2] = f.z, factor[sub][4 * q4 + 3] = f.w;
      }
    }
    // ---- scale, bias by distance, mask (log2 domain)
    const uint32_t key_l = t0 + 4 * g2; // key of register v: key_l + 32 sub + 8 (v / 4) + v % 4
    const uint32_t last_key = t0 + TILE_KEYS - 1;
    if ( bias_floats == 0 || ( last_key <= pos_first && pos_first - last_key >= s.n_dist - 1 ) ) { // every distance in the table's last row
      const float b = bias_floats == 0 ? 0.0f : my_bias[s.n_dist - 1];
#pragma unroll
      for ( int sub = 0; sub < 2; sub++ ) {
#pragma unroll
        for ( int v = 0; v < 16; v++ ) {
          st[sub][v] = st[sub][v] * factor[sub][v] + b;
        }
      }
    } else {
#pragma unroll
      for ( int sub = 0; sub < 2; sub++ ) {
#pragma unroll
        for ( int v = 0; v < 16; v++ ) {
          const uint32_t key = key_l + 32 * sub + 8 * ( v / 4 ) + v % 4;
          st[sub][v] = st[sub][v] * factor[sub][v] + my_bias[min( pos - min( key, pos ), s.n_dist - 1 )];
        }
      }
    }
    const bool in_window = i >= kept_tiles;
    const bool whole = in_window ? last_key <= pos_first && ( pos_last - t0 < s.window || last_key < s.keep_first ) : last_key < kept;
    if ( !whole ) {
      const uint32_t end = in_window ? 0xffffffffu : kept;
#pragma unroll
      for ( int sub = 0; sub < 2; sub++ ) {
#pragma unroll
        for ( int v = 0; v < 16; v++ ) {
          const uint32_t key = key_l + 32 * sub + 8 * ( v / 4 ) + v % 4;
          const bool seen = key <= pos && key < end && ( pos - key < s.window || key < s.keep_first );
          st[sub][v] = seen ? st[sub][v] : -INFINITY;
        }
      }
    }
    // ---- online softmax
    float mx4[4];
#pragma unroll
    for ( int c = 0; c < 4; c++ ) {
      mx4[c] = st[c >> 1][8 * ( c & 1 )];
#pragma unroll
      for ( int e = 1; e < 8; e++ ) {
        mx4[c] = fmaxf( mx4[c], st[c >> 1][8 * ( c & 1 ) + e] );
      }
    }
    const float mx = half_wave_max( fmaxf( fmaxf( mx4[0], mx4[1] ), fmaxf( mx4[2], mx4[3] ) ) );
    if ( __builtin_amdgcn_ballot_w64( mx > m + LAZY ) != 0 ) {
      const float m_new = fmaxf( m, mx );
      const float alpha = __builtin_amdgcn_exp2f( m - m_new );
      m = m_new;
      l *= alpha;
#pragma unroll
      for ( int vb = 0; vb < VB; vb++ ) {
#pragma unroll
        for ( int v = 0; v < 16; v++ ) {
          acc[vb][v] *= alpha;
        }
      }
    }
#pragma unroll
    for ( int kk = 0; kk < 4; kk++ ) { // 16 keys
      bf16x8 hi, lo;
#pragma unroll
      for ( int e = 0; e < 8; e++ ) {
        const float p = __builtin_amdgcn_exp2f( st[kk >> 1][8 * ( kk & 1 ) + e] - m );
        l += p;
        hi[e] = (__bf16)p;
        lo[e] = (__bf16)( p - (float)hi[e] );
      }
#pragma unroll
      for ( int vb = 0; vb < VB; vb++ ) {
        union
        {
          v4s half[2];
          bf16x8 x;
        } a;
#pragma unroll
        for ( int hf = 0; hf < 2; hf++ ) {
          a.half[hf] = __builtin_amdgcn_ds_read_tr16_b64_v4i16( (lds_v4s)( (lds_char*)s_v + ( v_lane ^ ( 64 * vb ) ^ ( SHARED ? 32 * hf : 0 ) ) + ( 16 * kk + 8 * hf ) * 256 ) );
        }
        acc[vb] = Mfma<__bf16>::k16( a.x, lo, acc[vb] );
        acc[vb] = Mfma<__bf16>::k16( a.x, hi, acc[vb] );
      }
    }
  }
  l += __shfl_xor( l, 32 );
  if ( !col_ok ) {
    return;
  }
  const uint64_t row = (uint64_t)ctx * wr.n_tokens + tok;
  const float inv = 1.0f / l * out.gate( row, h0 + hc );
  __bf16* o = out.out + row * out.stride + ( h0 + hc ) * s.vdim;
  const bool wide = s.vdim % 4 == 0 && out.stride % 4 == 0;
#pragma unroll
  for ( int vb = 0; vb < VB; vb++ ) {
#pragma unroll
    for ( int q4 = 0; q4 < 4; q4++ ) {
      const uint32_t d = 32 * vb + 8 * q4 + 4 * g2;
      union
      {
        __bf16 e[4];
        uint2 raw;
      } y;
#pragma unroll
      for ( int e = 0; e < 4; e++ ) {
        y.e[e] = (__bf16)( acc[vb][4 * q4 + e] * inv );
      }
      if ( wide && d < s.vdim ) {
        *reinterpret_cast<uint2*>( o + d ) = y.raw;
      } else if ( !wide ) {
        for ( int e = 0; e < 4; e++ ) {
          if ( d + e < s.vdim ) {
            o[d + e] = y.e[e];
          }
        }
      }
    }
  }
}

// ---- few tokens: one query row at a time on the matrix cores (bf16, head sizes up to 128) ---------------------------------------
//
// The products of the tile kernel in 16 x 16 blocks, with the query heads of a group as the columns (where the group is small most of them
// stay empty: the kernel streams keys, and the matrix cores keep up with that many times over).  A wave takes every NW-th tile of 32 of the
// row's visible keys, numbered as in the rows kernel, so nothing needs a mask but the end; its tiles pass through LDS of its own, the next
// one's rows on their way into registers meanwhile, without a barrier.  Two blocks of scores are, as they lie, the right operand of
// the product with the values: slot 8 g + e of its 32 keys is key 4 g + e for e < 4, else key 16 + 4 g + e - 4 (g = lane / 16).
constexpr uint32_t STEP_KEYS = 32;
constexpr uint32_t STEP_COLS = 16; // query heads of a work-group
// LDS of a work-group in 16-byte units: the waves' tiles, and the factors of their keys behind them; the results of the waves take its place
// at the end
constexpr uint32_t step_lds( int waves, bool shared ) { return waves * ( STEP_KEYS * ( shared ? 16 : 32 ) + ( shared ? STEP_KEYS / 4 : 0 ) ); }
static_assert( step_lds( 1, true ) * 16 >= STEP_COLS * ( 128 + 2 ) * sizeof( float ), "the results of a wave, heads of up to 128" );
// 16-byte chunks of a key's 256 bytes are XORed with this: 16 rows at one chunk (plain reads) and 8 rows at one pair of chunks (transposing
// reads) lie in different banks
__device__ __forceinline__ uint32_t step_swizzle( uint32_t row ) { return ( ( row & 7 ) << 1 ) | ( ( row >> 3 ) & 1 ); }

// maximum over the four lanes of a column (lane, lane ^ 16, lane ^ 32, lane ^ 48), in all of them
__device__ __forceinline__ float column_max( float v )
{
  const unsigned bits = __builtin_bit_cast( unsigned, v );
  const auto rows = __builtin_amdgcn_permlane16_swap( bits, bits, false, false );
  const unsigned even = rows[0], odd = rows[1];
  return half_wave_max( fmaxf( __builtin_bit_cast( float, even ), __builtin_bit_cast( float, odd ) ) );
}

// D: head size up to which the kernel goes; NW waves
template<int D, bool SHARED, int NW>
__global__ __launch_bounds__( 64 * NW, SHARED ? 4 : 2 ) void window_decode_kernel( WindowOut<__bf16> out,
                                                                                         float* __restrict__ partial,
                                                                                         const __bf16* __restrict__ q,
                                                                                         const float* __restrict__ bias,
                                                                                         WindowRows wr,
                                                                                         WindowShape s,
                                                                                         uint32_t head_cols,
                                                                                         uint32_t keys_per_split,
                                                                                         uint32_t splits )
{
  constexpr int KS = D / 32, VB = D / 16; // steps of 32 of the query/key size, blocks of 16 of the value size
  __shared__ uint4 tiles[step_lds( NW, SHARED )]; // K and V of each wave, 256 bytes a key
  const uint32_t head_blocks = s.heads / head_cols;
  const uint32_t hb = blockIdx.x % head_blocks, split = blockIdx.x / head_blocks % splits;
  const uint64_t row = blockIdx.x / head_blocks / splits;
  const uint32_t ctx = (uint32_t)( row / wr.n_tokens ), tok = (uint32_t)( row % wr.n_tokens );
  const uint8_t* base = static_cast<const uint8_t*>( wr.rows[ctx] );
  if ( base == nullptr ) {
    return;
  }
  const __bf16* cache = reinterpret_cast<const __bf16*>( base + wr.offset );
  const uint32_t h0 = hb * head_cols, g = h0 / s.group;
  const uint32_t pos = wr.start_pos[ctx] + tok;
  const Visible vis = visible_keys( pos, s );
  const uint32_t k_begin = split * keys_per_split, k_end = min( vis.count, k_begin + keys_per_split );
  const uint32_t wave = __builtin_amdgcn_readfirstlane( threadIdx.x >> 6 );
  const uint32_t lane = threadIdx.x & 63, r = lane & 15, g4 = lane >> 4;
  const uint32_t hc = min( r, head_cols - 1 ); // columns beyond do as the last one and are not stored
  uint4* s_k = tiles + wave * STEP_KEYS * ( SHARED ? 16 : 32 );
  uint4* s_v = SHARED ? s_k : s_k + STEP_KEYS * 16;
  float* s_factor = reinterpret_cast<float*>( tiles + NW * STEP_KEYS * ( SHARED ? 16 : 32 ) ) + wave * STEP_KEYS; // times scale and log2(e)

  bf16x8 qb[KS];
#pragma unroll
  for ( int k = 0; k < KS; k++ ) {
    const uint32_t ch = 4 * k + g4;
    u32x4_t v = { 0, 0, 0, 0 };
    if ( ch * 8 < s.dpad ) {
      v = *(global_u32x4_t*)( q + ( row * s.heads + h0 + hc ) * s.dpad + ch * 8 );
    }
    qb[k] = __builtin_bit_cast( bf16x8, v );
  }
  const bool k_chunk = r * 8 < s.dpad && r < D / 8, v_chunk = r * 8 < s.vpad && r < D / 8;
  const uint32_t row_bytes = s.row_elems() * sizeof( __bf16 );
  const uint32_t at_k = ( g * s.dpad + r * 8 ) * sizeof( __bf16 ), at_v = ( s.k_elems() + g * s.vpad + r * 8 ) * sizeof( __bf16 );
  u32x4_t rk[8], rv[SHARED ? 1 : 8]; // chunks beyond a head's size stay zero
#pragma unroll
  for ( int k = 0; k < 8; k++ ) {
    rk[k] = u32x4_t { 0, 0, 0, 0 };
    rv[SHARED ? 0 : k] = u32x4_t { 0, 0, 0, 0 };
  }
  const float* factors = reinterpret_cast<const float*>( base + wr.factors );
  float rf = 0.0f;
  auto load_row = [&]( int k, const char* row_k, uint32_t off ) {
    if ( k_chunk ) {
      rk[k] = __builtin_nontemporal_load( (global_u32x4_t*)( row_k + ( off + at_k ) ) );
    }
    if constexpr ( !SHARED ) {
      if ( v_chunk ) {
        rv[k] = __builtin_nontemporal_load( (global_u32x4_t*)( row_k + ( off + at_v ) ) );
      }
    }
  };
  auto load = [&]( uint32_t i0 ) {
    if constexpr ( SHARED ) {
      rf = factors[factor_index( vis.key( min( i0 + ( lane & 31 ), k_end - 1 ) ), g, s.kv_heads )];
    }
    if ( i0 + STEP_KEYS <= k_end && ( i0 >= vis.kept || i0 + STEP_KEYS <= vis.kept ) ) { // neighbouring rows: one address for the wave
      const char* tile = reinterpret_cast<const char*>( cache ) + (uint64_t)vis.key( i0 ) * row_bytes;
#pragma unroll
      for ( int k = 0; k < 8; k++ ) {
        load_row( k, tile + 4 * k * row_bytes, g4 * row_bytes );
      }
    } else {
#pragma unroll
      for ( int k = 0; k < 8; k++ ) {
        const uint32_t j = vis.key( min( i0 + g4 + 4 * k, k_end - 1 ) ); // past the end: the last key again, without weight
        load_row( k, reinterpret_cast<const char*>( cache ) + (uint64_t)j * row_bytes, 0 );
      }
    }
  };
  // a lane's bytes in a tile: of the row it writes first, of the key it reads for the scores, and of the transposing reads (16 lanes bring
  // 4 keys of 16 value columns, lane i gets column i).  The other places are a few bits and rows away.
  const uint32_t w_home = g4 * 256 + ( r ^ step_swizzle( g4 ) ) * 16;
  const uint32_t k_home = r * 256 + ( g4 ^ step_swizzle( r ) ) * 16;
  const uint32_t v_row = 4 * g4 + ( r >> 2 );
  const uint32_t v_home = v_row * 256 + ( ( ( ( r & 3 ) >> 1 ) ^ step_swizzle( v_row ) ) * 16 ) + ( r & 1 ) * 8;
  const float scale_log2e = s.scale * LOG2E;
  const float* my_bias = bias != nullptr ? bias + (uint64_t)( h0 + hc ) * s.n_dist : nullptr;
  const float far_bias = bias != nullptr ? my_bias[s.n_dist - 1] * LOG2E : 0.0f;

  mfma_f32x4 acc[VB];
#pragma unroll
  for ( int vb = 0; vb < VB; vb++ ) {
    acc[vb] = mfma_f32x4 { 0.0f, 0.0f, 0.0f, 0.0f };
  }
  float m = NO_KEY, l = 0.0f;
  uint32_t i0 = k_begin + wave * STEP_KEYS;
  if ( i0 < k_end ) {
    load( i0 );
  }
  for ( ; i0 < k_end; i0 += NW * STEP_KEYS ) {
    uint32_t w_lane = w_home, k_lane = k_home, v_lane = v_home;
    asm( "" : "+v"( w_lane ), "+v"( k_lane ), "+v"( v_lane ) ); // the addresses beside these are made where they are used, not kept in registers
#pragma unroll
    for ( int k = 0; k < 8; k++ ) {
      const uint32_t at = ( w_lane ^ ( 16 * step_swizzle( 4 * k ) ) ) + 4 * k * 256;
      *reinterpret_cast<uint4*>( reinterpret_cast<char*>( s_k ) + at ) = __builtin_bit_cast( uint4, rk[k] );
      if constexpr ( !SHARED ) {
        *reinterpret_cast<uint4*>( reinterpret_cast<char*>( s_v ) + at ) = __builtin_bit_cast( uint4, rv[k] );
      }
    }
    if ( SHARED && lane < STEP_KEYS ) {
      s_factor[lane] = rf * scale_log2e;
    }
    if ( i0 + NW * STEP_KEYS < k_end ) {
      load( i0 + NW * STEP_KEYS );
    }
    __builtin_amdgcn_fence( __ATOMIC_RELEASE, "wavefront" );
    float st[8]; // of key i0 + 16 (e / 4) + 4 g4 + e % 4
#pragma unroll
    for ( int t = 0; t < 2; t++ ) {
      mfma_f32x4 d = { 0.0f, 0.0f, 0.0f, 0.0f };
#pragma unroll
      for ( int k = 0; k < KS; k++ ) {
        const uint4 a = *reinterpret_cast<const uint4*>( reinterpret_cast<const char*>( s_k ) + ( k_lane ^ ( 64 * k ) ) + 16 * t * 256 );
        d = Mfma<__bf16>::k32( __builtin_bit_cast( bf16x8, a ), qb[k], d );
      }
      float4 f = make_float4( scale_log2e, scale_log2e, scale_log2e, scale_log2e );
      if constexpr ( SHARED ) {
        f = *reinterpret_cast<const float4*>( s_factor + 16 * t + 4 * g4 );
      }
      st[4 * t] = d[0] * f.x, st[4 * t + 1] = d[1] * f.y, st[4 * t + 2] = d[2] * f.z, st[4 * t + 3] = d[3] * f.w;
    }
    if ( bias != nullptr ) {
      // every distance of the tile in the bias table's last row?
      const uint32_t nearest = vis.key( min( i0 + STEP_KEYS, k_end ) - 1 );
      if ( pos - nearest >= s.n_dist - 1 ) {
#pragma unroll
        for ( int e = 0; e < 8; e++ ) {
          st[e] += far_bias;
        }
      } else {
#pragma unroll
        for ( int e = 0; e < 8; e++ ) {
          const uint32_t j = vis.key( min( i0 + 16 * ( e / 4 ) + 4 * g4 + e % 4, k_end - 1 ) );
          st[e] += my_bias[min( pos - j, s.n_dist - 1 )] * LOG2E;
        }
      }
    }
    if ( i0 + STEP_KEYS > k_end ) {
#pragma unroll
      for ( int e = 0; e < 8; e++ ) {
        st[e] = i0 + 16 * ( e / 4 ) + 4 * g4 + e % 4 < k_end ? st[e] : -INFINITY;
      }
    }
    const float mx = column_max( fmaxf( fmaxf( fmaxf( st[0], st[1] ), fmaxf( st[2], st[3] ) ), fmaxf( fmaxf( st[4], st[5] ), fmaxf( st[6], st[7] ) ) ) );
    if ( __builtin_amdgcn_ballot_w64( mx > m + LAZY ) != 0 ) {
      const float m_new = fmaxf( m, mx );
      const float alpha = __builtin_amdgcn_exp2f( m - m_new );
      m = m_new;
      l *= alpha;
#pragma unroll
      for ( int vb = 0; vb < VB; vb++ ) {
#pragma unroll
        for ( int v = 0; v < 4; v++ ) {
          acc[vb][v] *= alpha;
        }
      }
    }
    bf16x8 hi, lo;
#pragma unroll
    for ( int e = 0; e < 8; e++ ) {
      const float p = __builtin_amdgcn_exp2f( st[e] - m );
      l += p;
      hi[e] = (__bf16)p;
      lo[e] = (__bf16)( p - (float)hi[e] );
    }
#pragma unroll
    for ( int vb = 0; vb < VB; vb++ ) {
      union
      {
        v4s half[2];
        bf16x8 x;
      } a;
#pragma unroll
      for ( int t = 0; t < 2; t++ ) {
        a.half[t] = __builtin_amdgcn_ds_read_tr16_b64_v4i16( (lds_v4s)( (lds_char*)s_v + ( v_lane ^ ( 32 * vb ) ) + 16 * t * 256 ) );
      }
      acc[vb] = Mfma<__bf16>::k32( a.x, lo, acc[vb] );
      acc[vb] = Mfma<__bf16>::k32( a.x, hi, acc[vb] );
    }
    __builtin_amdgcn_fence( __ATOMIC_ACQUIRE, "wavefront" );
  }
  l += __shfl_xor( l, 16 );
  l += __shfl_xor( l, 32 );
  __syncthreads(); // the tiles' LDS takes the waves' results
  float* results = reinterpret_cast<float*>( tiles );
  if ( r < head_cols ) {
    float* mine = results + ( wave * head_cols + r ) * ( s.vpad + 2 );
#pragma unroll
    for ( int vb = 0; vb < VB; vb++ ) {
#pragma unroll
      for ( int v = 0; v < 4; v++ ) {
        const uint32_t d = 16 * vb + 4 * g4 + v;
        if ( d < s.vpad ) {
          mine[d] = acc[vb][v];
        }
      }
    }
    if ( g4 == 0 ) {
      mine[s.vpad] = l;
      mine[s.vpad + 1] = m * ( 1.0f / LOG2E ); // the sums are joined in natural units
    }
  }
  __syncthreads();
  finish_split<__bf16, NW>( out, partial, results, head_cols, head_cols, row, h0, split, splits, s );
}

template<typename E, int NC, bool SHARED>
void launch_rows( int hq, dim3 grid, hipStream_t st, const WindowOut<E>& out, float* partial, const E* q, const float* bias, const WindowRows& wr, const WindowShape& s,
                  uint32_t keys_per_split, uint32_t splits )
{
  const size_t lds = 4ull * hq * ( s.vpad + 2 ) * sizeof( float );
  if constexpr ( NC <= 1 ) {
    if ( hq == 8 ) {
      window_rows_kernel<E, 8, NC, SHARED><<<grid, 256, lds, st>>>( out, partial, q, bias, wr, s, keys_per_split, splits );
      return;
    }
  }
  if constexpr ( NC <= 2 ) {
    if ( hq == 4 ) {
      window_rows_kernel<E, 4, NC, SHARED><<<grid, 256, lds, st>>>( out, partial, q, bias, wr, s, keys_per_split, splits );
      return;
    }
    if ( hq == 2 ) {
      window_rows_kernel<E, 2, NC, SHARED><<<grid, 256, lds, st>>>( out, partial, q, bias, wr, s, keys_per_split, splits );
      return;
    }
  }
  window_rows_kernel<E, 1, NC, SHARED><<<grid, 256, lds, st>>>( out, partial, q, bias, wr, s, keys_per_split, splits );
}

// Splits of the visible keys of a call's rows, and room for their partial results: as many as give every CU two work-groups, of at
// least `least` keys each.
struct SplitPlan
{
  uint32_t keys { 0 }, splits { 1 };
  float* partial { nullptr };
};
int plan_splits( const WindowShape& s, uint64_t rows, uint64_t head_blocks, uint32_t max_pos, uint64_t least, hipStream_t st, SplitPlan* plan )
{
  const uint64_t most = std::min<uint64_t>( (uint64_t)max_pos + 1, (uint64_t)s.window + s.keep_first );
  uint64_t splits = std::max<uint64_t>( 1, 2ull * cu_count() / std::max<uint64_t>( 1, rows * head_blocks ) );
  splits = std::min( { splits, std::max<uint64_t>( 1, most / least ), (uint64_t)64 } );
  plan->keys = (uint32_t)( ( ( most + splits - 1 ) / splits + 31 ) / 32 * 32 );
  plan->splits = (uint32_t)( ( most + plan->keys - 1 ) / plan->keys );
  if ( plan->splits > 1 ) {
    void* p = nullptr;
    if ( int rc = stream_scratch( st, SCRATCH_MIXER, rows * s.heads * plan->splits * partial_stride( s ) * sizeof( float ), 1ull << 20, &p ) ) {
      return rc;
    }
    plan->partial = static_cast<float*>( p );
  }
  return GH_OK;
}
template<typename E>
int merge_splits( const WindowOut<E>& out, const SplitPlan& plan, const WindowRows& wr, const WindowShape& s, uint64_t rows, hipStream_t st )
{
  if ( plan.splits > 1 ) {
    const uint64_t pairs = rows * s.heads;
    window_merge_kernel<E><<<(unsigned)( ( pairs + 3 ) / 4 ), 256, 0, st>>>( out, plan.partial, wr, s, plan.splits, pairs );
    GH_LAUNCH_CHECK();
  }
  return GH_OK;
}

// few rows of bf16 with heads of up to 128
int attend_decode( const WindowOut<__bf16>& out, const __bf16* q, const float* bias, const WindowRows& wr, const WindowShape& s, uint64_t rows, uint32_t max_pos, hipStream_t st )
{
  uint32_t head_cols = s.group; // the largest divisor of the group that fits
  while ( head_cols > STEP_COLS || s.group % head_cols != 0 ) {
    head_cols--;
  }
  const uint64_t head_blocks = s.heads / head_cols;
  // keys of a row over eight waves where work-groups of four would leave room on the CUs and each wave still has a few tiles
  const bool wide = s.values_are_keys && rows * head_blocks < 4ull * cu_count() && max_pos >= 16 * STEP_KEYS;
  SplitPlan plan;
  if ( int rc = plan_splits( s, rows, head_blocks, max_pos, ( wide ? 8 : 4 ) * STEP_KEYS, st, &plan ) ) {
    return rc;
  }
  const uint64_t grid = rows * head_blocks * plan.splits;
  GH_REQUIRE( grid < ( 1ull << 31 ), "gh_attn_window: grid too large" );
#define GH_WINDOW_DECODE( D, SHARED, NW ) \
  window_decode_kernel<D, SHARED, NW><<<(unsigned)grid, 64 * NW, 0, st>>>( out, plan.partial, q, bias, wr, s, head_cols, plan.keys, plan.splits )
  const bool small = s.dpad <= 64 && s.vpad <= 64;
  if ( !s.values_are_keys && small ) {
    GH_WINDOW_DECODE( 64, false, 4 );
  } else if ( !s.values_are_keys ) {
    GH_WINDOW_DECODE( 128, false, 4 );
  } else if ( small && wide ) {
    GH_WINDOW_DECODE( 64, true, 8 );
  } else if ( small ) {
    GH_WINDOW_DECODE( 64, true, 4 );
  } else if ( wide ) {
    GH_WINDOW_DECODE( 128, true, 8 );
  } else {
    GH_WINDOW_DECODE( 128, true, 4 );
  }
#undef GH_WINDOW_DECODE
  GH_LAUNCH_CHECK();
  return merge_splits( out, plan, wr, s, rows, st );
}

template<typename E, bool SHARED>
int attend_rows( const WindowOut<E>& out, const E* q, const float* bias, const WindowRows& wr, const WindowShape& s, uint64_t rows, uint32_t max_pos, hipStream_t st )
{
  const uint32_t widest = std::max( s.dpad, s.vpad );
  const int max_hq = widest <= 128 ? 8 : widest <= 256 ? 4 : 1;
  int hq = 1;
  while ( hq < max_hq && hq < (int)s.group ) {
    hq *= 2;
  }
  const uint32_t head_blocks = s.kv_heads * ( ( s.group + hq - 1 ) / hq );
  GH_REQUIRE( head_blocks <= 65535, "gh_attn_window: too many heads" );
  SplitPlan plan;
  if ( int rc = plan_splits( s, rows, head_blocks, max_pos, 64, st, &plan ) ) {
    return rc;
  }
  const uint32_t per = plan.keys;
  const uint32_t splits = plan.splits;
  float* partial = plan.partial;
  const dim3 grid( (unsigned)rows, head_blocks, (unsigned)splits );
  if ( widest <= 128 ) {
    launch_rows<E, 1, SHARED>( hq, grid, st, out, partial, q, bias, wr, s, per, (uint32_t)splits );
  } else if ( widest <= 256 ) {
    launch_rows<E, 2, SHARED>( hq, grid, st, out, partial, q, bias, wr, s, per, (uint32_t)splits );
  } else {
    launch_rows<E, 4, SHARED>( hq, grid, st, out, partial, q, bias, wr, s, per, (uint32_t)splits );
  }
  GH_LAUNCH_CHECK();
  return merge_splits( out, plan, wr, s, rows, st );
}

// Whether the tile kernel serves a call; its launch.
uint32_t tile_head_cols( const WindowShape& s )
{
  uint32_t cols = s.group <= 32 && ( s.group & ( s.group - 1 ) ) == 0 ? s.group : 1;
  while ( cols > 1 && (uint64_t)cols * s.n_dist > BIAS_LDS ) { // as many as have their bias tables fit
    cols /= 2;
  }
  return cols;
}
bool tiles_applicable( const WindowShape& s, const float* bias, uint32_t n_tokens )
{
  return n_tokens >= 16 && s.dpad <= 128 && s.vpad <= 128 && ( bias == nullptr || (uint64_t)tile_head_cols( s ) * s.n_dist <= BIAS_LDS );
}
int attend_tiles( const WindowOut<__bf16>& out, const __bf16* q, const float* bias, const WindowRows& wr, const WindowShape& s, uint64_t batch, hipStream_t st )
{
  const uint32_t head_cols = tile_head_cols( s );
  const uint32_t col_blocks = ( wr.n_tokens + 128 / head_cols - 1 ) / ( 128 / head_cols );
  const uint64_t n_pairs = batch * s.kv_heads * ( s.group / head_cols );
  const uint64_t grid = ( n_pairs + 7 ) / 8 * 8 * col_blocks;
  GH_REQUIRE( grid < ( 1ull << 31 ), "gh_attn_window: grid too large" );
  const uint32_t bias_floats = bias == nullptr ? 0 : head_cols * s.n_dist;
  const size_t lds = ( s.values_are_keys ? TILE_KEYS * ( 256 + sizeof( float ) ) : 2 * TILE_KEYS * 256 ) + bias_floats * sizeof( float );
#define GH_WINDOW_TILES( KS, VB, SHARED ) \
  window_tiles_kernel<KS, VB, SHARED><<<(unsigned)grid, 256, lds, st>>>( out, q, bias, wr, s, head_cols, col_blocks, (uint32_t)n_pairs, bias_floats )
  if ( s.values_are_keys ) {
    if ( s.dpad <= 64 ) {
      GH_WINDOW_TILES( 4, 2, true );
    } else if ( s.dpad <= 96 ) {
      GH_WINDOW_TILES( 6, 3, true );
    } else {
      GH_WINDOW_TILES( 8, 4, true );
    }
  } else if ( s.dpad <= 64 && s.vpad <= 64 ) {
    GH_WINDOW_TILES( 4, 2, false );
  } else if ( s.vpad <= 64 ) {
    GH_WINDOW_TILES( 8, 2, false );
  } else {
    GH_WINDOW_TILES( 8, 4, false );
  }
#undef GH_WINDOW_TILES
  GH_LAUNCH_CHECK();
  return GH_OK;
}

} // namespace
} // namespace gh

using namespace gh;

extern "C" {

uint64_t gh_window_row_bytes( const gh_window_attn* a, gh_dtype dt ) { return (uint64_t)window_shape( a ).row_elems() * dtype_size( dt ); }

uint64_t gh_window_factor_bytes( const gh_window_attn* a ) { return a->values_are_keys ? (uint64_t)a->kv_heads * sizeof( float ) : 0; }

uint64_t gh_window_query_elements( const gh_window_attn* a ) { return (uint64_t)a->heads * window_shape( a ).dpad; }

int gh_matmul_window_append( void* q, const void* x, const void* wqkv, const void* bias, uint64_t width, const gh_window_attn* a, const void* q_norm,
                             const void* k_norm, float eps, void* const* context_rows_dev, uint64_t cache_offset, const uint32_t* start_pos_dev, uint64_t batch,
                             uint32_t n_tokens, gh_dtype dt, gh_stream stream )
{
  if ( int rc = ensure_init() ) {
    return rc;
  }
  const uint64_t rows = batch * n_tokens;
  if ( rows == 0 ) {
    return GH_OK;
  }
  GH_REQUIRE( q && x && wqkv && a && context_rows_dev && start_pos_dev, "gh_matmul_window_append: NULL pointer" );
  GH_REQUIRE( dt == GH_BF16 || dt == GH_F32, "gh_matmul_window_append: unsupported dtype %d", (int)dt );
  GH_REQUIRE( window_shape_ok( a ) && rows < ( 1ull << 31 ) && cache_offset % 16 == 0 && !a->values_are_keys, "gh_matmul_window_append: bad shape" );
  const WindowShape s = window_shape( a );
  const uint64_t r = (uint64_t)s.heads * s.dim + (uint64_t)s.kv_heads * ( s.dim + s.vdim );
  hipStream_t st = as_stream( stream );
  Product y;
  if ( int rc = make_product( x, wqkv, width, r, rows, dt, false, st, &y ) ) {
    return rc;
  }
  const WindowRows wr { context_rows_dev, cache_offset, 0, start_pos_dev, n_tokens };
  return with_product( dt, y, [&]( auto tag, auto view ) -> int {
    using E = decltype( tag );
    return launch_append<E>( static_cast<E*>( q ), view, static_cast<const E*>( bias ), q_norm, k_norm, eps, wr, s, rows, st );
  } );
}

int gh_attn_window( void* out, uint64_t out_stride, const float* head_gates, const void* q, const gh_window_attn* a, const float* distance_bias_dev,
                    void* const* context_rows_dev, uint64_t cache_offset, uint64_t factor_offset, const uint32_t* start_pos_dev, uint64_t batch, uint32_t n_tokens,
                    uint32_t max_start_pos, gh_dtype dt, gh_stream stream )
{
  if ( int rc = ensure_init() ) {
    return rc;
  }
  const uint64_t rows = batch * n_tokens;
  if ( rows == 0 ) {
    return GH_OK;
  }
  GH_REQUIRE( out && q && a && context_rows_dev && start_pos_dev, "gh_attn_window: NULL pointer" );
  GH_REQUIRE( dt == GH_BF16 || dt == GH_F32, "gh_attn_window: unsupported dtype %d", (int)dt );
  GH_REQUIRE( window_shape_ok( a ) && rows < ( 1ull << 31 ) && cache_offset % 16 == 0, "gh_attn_window: bad shape" );
  const WindowShape s = window_shape( a );
  GH_REQUIRE( out_stride >= (uint64_t)s.heads * s.vdim && factor_offset % 16 == 0, "gh_attn_window: bad stride or offset" );
  const WindowRows wr { context_rows_dev, cache_offset, factor_offset, start_pos_dev, n_tokens };
  const uint32_t max_pos = max_start_pos + n_tokens - 1;
  hipStream_t st = as_stream( stream );
  if ( dt == GH_F32 ) {
    const WindowOut<float> to { static_cast<float*>( out ), out_stride, head_gates, s.heads };
    const float* qf = static_cast<const float*>( q );
    return s.values_are_keys ? attend_rows<float, true>( to, qf, distance_bias_dev, wr, s, rows, max_pos, st )
                             : attend_rows<float, false>( to, qf, distance_bias_dev, wr, s, rows, max_pos, st );
  }
  const WindowOut<__bf16> to { static_cast<__bf16*>( out ), out_stride, head_gates, s.heads };
  const __bf16* qb = static_cast<const __bf16*>( q );
  if ( tiles_applicable( s, distance_bias_dev, n_tokens ) ) {
    return attend_tiles( to, qb, distance_bias_dev, wr, s, batch, st );
  }
  if ( s.dpad <= 128 && s.vpad <= 128 ) {
    return attend_decode( to, qb, distance_bias_dev, wr, s, rows, max_pos, st );
  }
  return s.values_are_keys ? attend_rows<__bf16, true>( to, qb, distance_bias_dev, wr, s, rows, max_pos, st )
                           : attend_rows<__bf16, false>( to, qb, distance_bias_dev, wr, s, rows, max_pos, st );
}

} // extern "C"
