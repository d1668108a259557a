// Driver of the Famidra design for the hip target: weights, scratch, and the ops of one step.  A step is `n_tokens` consecutive tokens
// of every context of a batch; decode is a step of one token, prefill a step of many, over the same ops:
//
//   embedding        x = embed[token] + pos[position]
//   pass of the loop x = W_in [x; x0] + step[t], in front of the first layer of every pass
//   mixer            h = norm1(x); mLSTM or windowed attention on h; x += norm1b( W_o . )
//   feed-forward     h = norm2(x); x += norm2b( W_down (gelu(W_gate h) * (W_up h)) ), biases on all three
//   output           logits = embed . final_norm(x) * logit_scale (fp32) -> (Gumbel noise if temperature > 0) -> argmax
//
// The residual stream x is fp32.  Every projection is fused with what follows it up to the next product's input (see gh_stream_step), so
// a layer is a handful of launches in either dtype.  The design is hosted whole: a pass needs the embedding output again, so a cut
// between nodes would carry two rows a token.
#pragma once

#include <algorithm>
#include <cstdio>
#include <filesystem>
#include <functional>
#include <memory>
#include <string>
#include <vector>

#include "glint/famidra_config.hh"
#include "glint/hip/ops.hh"
#include "glint/layered_context.hh"
#include "glint/model_options.hh"
#include "glint/safetensors.hh"
#include "glint/span_timer.hh"
#include "glint/state.hh"

namespace glint {

template<typename DType, typename Context = hip::LayeredContext>
class Famidra
{
public:
  using ConfigType = configs::Famidra;
  using DataTypeT = DType;
  using ContextType = Context;
  using SettingsType = DesignSettings;
  using StateType = BatchedInferenceState<ConfigType>;
  using ContextVector = std::vector<std::shared_ptr<Context>>;
  using Operations = hip::Operations<DType>;
  static constexpr gh_dtype DT = hip::gh_type<DType>();

  // weights are left for load(), or drawn N(0, weight_std) with norm weights 1 when settings.randomize_parameters
  Famidra( const FamidraConfig& config, SettingsType settings, const ModelOptions options = {} )
    : config_( config )
    , settings_( std::move( settings ) )
    , options_( options )
    , runs_( config_.runs() )
  {
    GLINT_CHECK( settings_.concurrency_limit > 0 && settings_.concurrency_limit <= MAX_BATCH_SIZE );
    settings_.plan = std::make_shared<const ContextPlan>( plan( config_ ) );
    describe_layers();
    describe_tensors();
    allocate_weights();
    allocate_tables();
    if ( settings_.randomize_parameters ) {
      randomize_weights();
    }
  }
  ~Famidra()
  {
    if ( tables_host_ != nullptr ) {
      (void)gh_host_free( tables_host_ );
    }
  }
  Famidra( const Famidra& ) = delete;
  Famidra& operator=( const Famidra& ) = delete;

  static ContextPlan plan( const FamidraConfig& config )
  {
    ContextPlan p( config.max_positions );
    for ( const auto& run : config.runs() ) {
      const auto& layer = config.layers[run.layer];
      if ( layer.mlstm ) {
        const gh_mlstm m = mlstm_shape( *layer.mlstm, config.eps );
        p.add_state( gh_mlstm_state_bytes( &m ) );
      } else {
        const gh_window_attn a = window_shape( *layer.attention );
        p.add_rows( gh_window_row_bytes( &a, DT ) );
      }
    }
    return p;
  }

  const FamidraConfig& config() const { return config_; }
  const SettingsType& settings() const { return settings_; }
  Operations& ops() { return ops_; }
  uint32_t vocab_size() const { return config_.vocab; }
  uint32_t max_positions() const { return config_.max_positions; }

  void time_device_spans( const bool on ) { spans_.enable( on ); }
  std::pair<double, uint64_t> device_spans() { return spans_.take(); }

  // every tensor of the design out of a safetensors file; empty string on success
  std::string load( const std::filesystem::path& model_dir )
  {
    SafeTensors file;
    if ( auto err = file.open( model_dir / "model.safetensors" ); !err.empty() ) {
      return err;
    }
    std::vector<DType> host;
    for ( const auto& t : tensors_ ) {
      const auto* src = file.find( t.name );
      if ( src == nullptr ) {
        return "tensor " + t.name + " is missing";
      }
      if ( src->shape != t.shape || src->dtype == "I32" ) {
        return "tensor " + t.name + " has another shape or type than config.json implies";
      }
      host.resize( src->elements() );
      for ( uint64_t i = 0; i < host.size(); i++ ) {
        host[i] = static_cast<DType>( SafeTensors::value( *src, i ) );
      }
      ops_.copy( t.dst, host.data(), host.size() * sizeof( DType ), CopyType::HostToDevice );
    }
    for ( size_t l = 0; l < layers_.size(); l++ ) {
      if ( !config_.layers[l].attention ) {
        continue;
      }
      const std::string name = prefix( l ) + "mix.rel";
      const auto* rel = file.find( name );
      const uint32_t heads = config_.layers[l].attention->heads;
      if ( rel == nullptr || rel->shape.size() != 2 || rel->shape[0] == 0 || rel->shape[1] != heads || rel->dtype == "I32" ) {
        return "tensor " + name + " is missing or does not have a column per head";
      }
      std::vector<float> table( rel->elements() );
      for ( uint64_t i = 0; i < table.size(); i++ ) {
        table[i] = SafeTensors::value( *rel, i );
      }
      set_distance_bias( l, table, static_cast<uint32_t>( rel->shape[0] ) );
    }
    return {};
  }

  // Whether a batch can be run at these positions: inside the model's positions, every context at the length it has, and none twice
  // (a recurrent state takes its tokens one after the other).
  bool positions_fit( const ContextVector& contexts, const uint32_t* start_pos, const uint32_t n_tokens ) const
  {
    std::vector<const void*> seen;
    for ( const auto& c : contexts ) {
      if ( !c->empty() ) {
        seen.push_back( c->data() );
      }
    }
    std::sort( seen.begin(), seen.end() );
    if ( std::adjacent_find( seen.begin(), seen.end() ) != seen.end() ) {
      return false;
    }
    for ( size_t i = 0; i < contexts.size(); i++ ) {
      if ( !contexts[i]->empty() && ( (uint64_t)start_pos[i] + n_tokens > config_.max_positions || !contexts[i]->takes( start_pos[i] ) ) ) {
        return false;
      }
    }
    return true;
  }
  bool positions_fit( const StateType& states, const ContextVector& contexts ) const
  {
    std::vector<uint32_t> pos( states.batch_size() );
    for ( size_t i = 0; i < pos.size(); i++ ) {
      pos[i] = states.token_pos( i );
    }
    return contexts.size() == pos.size() && positions_fit( contexts, pos.data(), 1 );
  }

  // one token of every active row: the next token of each is sampled into the state
  void forward( StateType& states, const ContextVector& contexts )
  {
    const size_t batch = states.batch_size();
    GLINT_CHECK( batch > 0 && batch <= settings_.concurrency_limit && contexts.size() == batch );
    GLINT_CHECK( states.next_stage() == InferenceStage::PreAttention && states.next_layer() == 0 );
    GLINT_CHECK( states.dtype() == dtype_of<DType>() );
    GLINT_CHECK( positions_fit( states, contexts ) );
    ensure_scratch( batch, batch );
    begin_tables( batch, batch, 0 );
    for ( size_t i = 0; i < batch; i++ ) {
      const bool live = states.active( i );
      GLINT_CHECK( !live || states.token( i ) < config_.vocab );
      put_context( i, *contexts[i], live ? states.token_pos( i ) : 0, 1 );
      table_tokens()[i] = live ? states.token( i ) : 0;
    }
    upload_tables();
    spans_.mark( 0, ops_.stream() );
    run_layers( batch, 1, true );
    classify( batch );
    spans_.mark( 1, ops_.stream() );

    std::vector<float> temperatures;
    for ( size_t i = 0; i < batch; i++ ) {
      temperatures.push_back( states.temperature( i ) );
    }
    if ( std::any_of( temperatures.begin(), temperatures.end(), []( float t ) { return t > 0; } ) ) {
      logit_ops_.soft_sample( logits_.get(), temperatures, config_.vocab );
    }
    sample( batch );
    spans_.close();
    states.set_next_layer( 0 );
    states.set_next_stage( InferenceStage::PreAttention );
    for ( size_t i = 0; i < batch; i++ ) {
      if ( !contexts[i]->empty() ) {
        contexts[i]->set_length( states.token_pos( i ) + 1 );
      }
      if ( states.active( i ) ) {
        states.set_token( i, argmax_[i] );
        states.set_token_pos( i, states.token_pos( i ) + 1 );
        if ( states.check_finished( i ) || states.token_pos( i ) >= config_.max_positions ) {
          states.set_finished( i );
        }
      }
    }
  }

  // `n_tokens` consecutive tokens per context, context i from start_pos[i] on (row = context * n_tokens + token).
  //   want          rows whose logits are asked for, ascending; they go to logits_out (host, (want.size(), vocab) fp32)
  //   next_tokens   (batch) greedy token behind each context's last row, or nullptr
  //   residuals_out the residual stream behind every layer run (host, (runs, rows, width) fp32), or nullptr: for tests
  void prefill( const ContextVector& contexts,
                const uint32_t* start_pos,
                const uint32_t n_tokens,
                const uint32_t* token_ids,
                const std::vector<uint32_t>& want,
                float* logits_out,
                uint32_t* next_tokens,
                float* residuals_out = nullptr )
  {
    const size_t batch = contexts.size();
    const uint64_t rows = (uint64_t)batch * n_tokens;
    GLINT_CHECK( batch > 0 && batch <= settings_.concurrency_limit && n_tokens > 0 && rows <= 0x7fffffffull );
    GLINT_CHECK( positions_fit( contexts, start_pos, n_tokens ) );
    std::vector<uint32_t> picked = want;
    if ( next_tokens != nullptr ) {
      for ( size_t i = 0; i < batch; i++ ) {
        picked.push_back( static_cast<uint32_t>( ( i + 1 ) * n_tokens - 1 ) );
      }
    }
    ensure_scratch( rows, std::max<uint64_t>( 1, std::min<uint64_t>( picked.size(), LOGIT_ROWS ) ) );
    begin_tables( batch, rows, picked.size() );
    for ( size_t i = 0; i < batch; i++ ) {
      put_context( i, *contexts[i], start_pos[i], n_tokens );
    }
    for ( uint64_t r = 0; r < rows; r++ ) {
      GLINT_CHECK( token_ids[r] < config_.vocab );
      table_tokens()[r] = token_ids[r];
    }
    for ( size_t k = 0; k < picked.size(); k++ ) {
      GLINT_CHECK( picked[k] < rows );
      table_picked()[k] = picked[k];
    }
    upload_tables();
    run_layers( batch, n_tokens, false, residuals_out );
    // the wanted rows, at most LOGIT_ROWS of them at a time
    for ( size_t k = 0; k < picked.size(); k += LOGIT_ROWS ) {
      const size_t n = std::min<size_t>( LOGIT_ROWS, picked.size() - k );
      GLINT_GH( gh_gather_rows( picked_x_.get(), x_.get(), picked_dev() + k, n, rows, config_.width, ops_.stream() ) );
      gh_stream_step step = no_step();
      step.next_norm = final_norm_;
      step.out = h_.get();
      step.out_stride = config_.width;
      GLINT_GH( gh_stream_out( picked_x_.get(), config_.width, n, &step, DT, ops_.stream() ) );
      classify( n );
      const size_t plain = k < want.size() ? std::min( n, want.size() - k ) : 0;
      if ( plain > 0 ) {
        logit_ops_.copy( logits_out + k * config_.vocab, logits_.get(), plain * config_.vocab * sizeof( float ), CopyType::DeviceToHost );
      }
      if ( plain < n ) {
        sample( n );
        for ( size_t j = plain; j < n; j++ ) {
          next_tokens[k + j - want.size()] = argmax_[j];
        }
      }
    }
    ops_.synchronize();
    for ( size_t i = 0; i < batch; i++ ) {
      if ( !contexts[i]->empty() ) {
        contexts[i]->set_length( start_pos[i] + n_tokens );
      }
    }
  }

  // logits of the last forward(): (batch, vocab) fp32, on the device
  float* logits() const { return logits_.get(); }
  void copy_logits( float* host, const uint64_t rows )
  {
    logit_ops_.copy( host, logits_.get(), rows * config_.vocab * sizeof( float ), CopyType::DeviceToHost );
  }
  size_t n_runs() const { return runs_.size(); }

private:
  static constexpr uint64_t LOGIT_ROWS = 256;

  struct Layer
  {
    DType *norm1 {}, *norm1b {}, *norm2 {}, *norm2b {};
    DType *mix_in {}, *mix_bias {}, *mix_out {}; // projections in front of and behind the mixer
    DType *q_norm {}, *k_norm {}, *head_norm {}, *bias_i {}, *bias_f {};
    DType *gate_up {}, *gate_up_bias {}, *down {}, *down_bias {};
    float* distance_bias {};
    uint64_t mixed_cols {};       // columns of the mixer's output
    gh_mlstm mlstm {};
    gh_window_attn attention {};
  };

  struct Tensor
  {
    std::string name;
    std::vector<uint64_t> shape;
    DType* dst;
    uint64_t elements() const
    {
      uint64_t n = 1;
      for ( const uint64_t d : shape ) {
        n *= d;
      }
      return n;
    }
    bool is_norm() const { return name.ends_with( "norm" ) || name.find( ".norm" ) != std::string::npos; }
  };

  static gh_mlstm mlstm_shape( const MlstmConfig& m, const float eps ) { return { m.heads, m.dim, m.vdim, m.gate_cap, eps }; }
  static gh_window_attn window_shape( const WindowAttentionConfig& a )
  {
    // distances beyond the table's last row all have its bias
    const uint32_t n_dist = static_cast<uint32_t>( std::ceil( a.bias_max ) ) + 1;
    return { a.heads, a.kv_heads, a.dim, a.vdim, a.window, a.keep_first, n_dist, a.scale };
  }
  static std::string prefix( const size_t layer ) { return "l" + std::to_string( layer ) + "."; }

  void describe_layers()
  {
    layers_.resize( config_.layers.size() );
    for ( size_t l = 0; l < layers_.size(); l++ ) {
      const auto& c = config_.layers[l];
      if ( c.mlstm ) {
        layers_[l].mlstm = mlstm_shape( *c.mlstm, config_.eps );
        layers_[l].mixed_cols = (uint64_t)c.mlstm->heads * c.mlstm->vdim;
        mixed_max_ = std::max( mixed_max_, layers_[l].mixed_cols );
      } else {
        layers_[l].attention = window_shape( *c.attention );
        layers_[l].mixed_cols = (uint64_t)c.attention->heads * c.attention->vdim;
        mixed_max_ = std::max( mixed_max_, layers_[l].mixed_cols );
        query_max_ = std::max( query_max_, gh_window_query_elements( &layers_[l].attention ) );
      }
      ff_max_ = std::max<uint64_t>( ff_max_, c.ff );
    }
  }

  // One pass over every tensor of the design.  Tensors that form one matrix for a product lie behind one another; `pad` leaves a
  // multiple of that many rows of zeros behind a group.  Run twice: first with no memory behind it, to size it.
  uint64_t lay_out( DType* base )
  {
    uint64_t at = 0;
    tensors_.clear();
    const uint64_t width = config_.width;
    auto take = [&]( const uint64_t n ) {
      DType* p = base == nullptr ? nullptr : base + at;
      at += n;
      return p;
    };
    auto align = [&] { at = ( at + 127 ) / 128 * 128; };
    auto tensor = [&]( std::string name, std::vector<uint64_t> shape ) {
      tensors_.push_back( { std::move( name ), std::move( shape ), nullptr } );
      tensors_.back().dst = take( tensors_.back().elements() );
      return tensors_.back().dst;
    };
    auto alone = [&]( std::string name, std::vector<uint64_t> shape ) {
      align();
      return tensor( std::move( name ), std::move( shape ) );
    };

    embed_ = alone( "embed", { config_.vocab, width } );
    pos_ = alone( "pos", { config_.max_positions, width } );
    final_norm_ = alone( "final.norm", { width } );
    if ( config_.looped ) {
      loop_in_ = alone( "loop.in", { width, 2 * width } );
      loop_step_ = alone( "loop.step", { config_.loop_times, width } );
    }
    for ( size_t l = 0; l < layers_.size(); l++ ) {
      auto& w = layers_[l];
      const auto& c = config_.layers[l];
      const std::string p = prefix( l );
      w.norm1 = alone( p + "norm1", { width } );
      w.norm1b = alone( p + "norm1b", { width } );
      if ( c.mlstm ) {
        const uint64_t hd = (uint64_t)c.mlstm->heads * c.mlstm->dim, hv = (uint64_t)c.mlstm->heads * c.mlstm->vdim, h = c.mlstm->heads;
        uint64_t gate_row = 0;
        const uint64_t rows = gh_mlstm_weight_rows( &w.mlstm, &gate_row );
        w.mix_in = alone( p + "mix.q", { hd, width } );
        tensor( p + "mix.k", { hd, width } );
        tensor( p + "mix.v", { hv, width } );
        tensor( p + "mix.g", { hv, width } );
        take( ( gate_row - 2 * hd - 2 * hv ) * width );
        tensor( p + "mix.i", { h, width } );
        tensor( p + "mix.f", { h, width } );
        take( ( rows - gate_row - 2 * h ) * width );
        w.bias_i = alone( p + "mix.i.b", { h } );
        w.bias_f = alone( p + "mix.f.b", { h } );
        w.head_norm = alone( p + "mix.norm", { hv } );
        w.mix_out = alone( p + "mix.o", { width, hv } );
      } else {
        const auto& a = *c.attention;
        const uint64_t q = (uint64_t)a.heads * a.dim, k = (uint64_t)a.kv_heads * a.dim, v = (uint64_t)a.kv_heads * a.vdim;
        w.mix_in = alone( p + "mix.q", { q, width } );
        tensor( p + "mix.k", { k, width } );
        tensor( p + "mix.v", { v, width } );
        w.mix_bias = alone( p + "mix.q.b", { q } );
        tensor( p + "mix.k.b", { k } );
        tensor( p + "mix.v.b", { v } );
        w.q_norm = alone( p + "mix.q.norm", { q } );
        w.k_norm = alone( p + "mix.k.norm", { k } );
        w.mix_out = alone( p + "mix.o", { width, (uint64_t)a.heads * a.vdim } );
        align();
        // the bias of every distance up to the table's end, fp32, one row a head
        w.distance_bias = reinterpret_cast<float*>( take( (uint64_t)w.attention.heads * w.attention.n_dist * sizeof( float ) / sizeof( DType ) ) );
      }
      if ( c.ff > 0 ) {
        w.norm2 = alone( p + "norm2", { width } );
        w.norm2b = alone( p + "norm2b", { width } );
        w.gate_up = alone( p + "mlp.gate", { c.ff, width } );
        tensor( p + "mlp.up", { c.ff, width } );
        w.gate_up_bias = alone( p + "mlp.gate.b", { c.ff } );
        tensor( p + "mlp.up.b", { c.ff } );
        w.down = alone( p + "mlp.down", { width, c.ff } );
        w.down_bias = alone( p + "mlp.down.b", { width } );
      }
    }
    align();
    return at;
  }

  void describe_tensors() { weight_elements_ = lay_out( nullptr ); }

  void allocate_weights()
  {
    weights_ = ops_.device_allocate( weight_elements_ * sizeof( DType ) );
    GLINT_GH( gh_memset_zero( weights_.get(), weight_elements_ * sizeof( DType ), ops_.stream() ) );
    (void)lay_out( weights_.get() );
  }

  void set_distance_bias( const size_t l, const std::vector<float>& table, const uint32_t table_rows )
  {
    const auto& a = layers_[l].attention;
    std::vector<float> by_distance( (uint64_t)a.heads * a.n_dist );
    for ( uint32_t n = 0; n < a.n_dist; n++ ) {
      const uint32_t row = distance_bucket( n, table_rows, config_.layers[l].attention->bias_max );
      for ( uint32_t h = 0; h < a.heads; h++ ) {
        by_distance[(uint64_t)h * a.n_dist + n] = table[(uint64_t)row * a.heads + h];
      }
    }
    GLINT_GH( gh_memcpy( layers_[l].distance_bias, by_distance.data(), by_distance.size() * sizeof( float ), GH_HOST_TO_DEVICE, 0, ops_.stream() ) );
  }

  void randomize_weights()
  {
    uint64_t seed = options_.seed * 1000003ull;
    for ( const auto& t : tensors_ ) {
      GLINT_GH( gh_fill_normal( t.dst, t.elements(), t.is_norm() ? 1.0f : 0.0f, options_.weight_std, seed++, DT, ops_.stream() ) );
    }
    for ( size_t l = 0; l < layers_.size(); l++ ) {
      if ( config_.layers[l].attention ) {
        const auto& a = layers_[l].attention;
        GLINT_GH( gh_fill_normal( layers_[l].distance_bias, (uint64_t)a.heads * a.n_dist, 0.0f, options_.weight_std, seed++, GH_F32, ops_.stream() ) );
      }
    }
    ops_.synchronize();
  }

  // ---- scratch and tables --------------------------------------------------------------------
  // grows to the largest step seen
  void ensure_scratch( const uint64_t rows, const uint64_t logit_rows )
  {
    if ( rows > rows_ ) {
      ops_.synchronize();
      const uint64_t w = config_.width;
      x_ = logit_ops_.device_allocate( rows * w * sizeof( float ) );
      h_ = ops_.device_allocate( std::max( rows, LOGIT_ROWS ) * w * sizeof( DType ) );
      mixed_ = ops_.device_allocate( rows * mixed_max_ * sizeof( DType ) );
      q_ = ops_.device_allocate( std::max<uint64_t>( rows * query_max_, 8 ) * sizeof( DType ) );
      hidden_ = ops_.device_allocate( std::max<uint64_t>( rows * ff_max_, 8 ) * sizeof( DType ) );
      if ( config_.looped ) {
        cat_ = ops_.device_allocate( rows * 2 * w * sizeof( DType ) );
      }
      rows_ = rows;
    }
    if ( logit_rows > logit_rows_ ) {
      ops_.synchronize();
      logits_ = logit_ops_.device_allocate( logit_rows * config_.vocab * sizeof( float ) );
      picked_x_ = logit_ops_.device_allocate( logit_rows * config_.width * sizeof( float ) );
      argmax_dev_ = logit_ops_.device_allocate( logit_rows * sizeof( uint32_t ) );
      argmax_.resize( logit_rows );
      logit_rows_ = logit_rows;
    }
  }

  // one upload per step: [context base | start position | token | picked row], page-locked on the host
  void allocate_tables() { grow_tables( settings_.concurrency_limit, settings_.concurrency_limit, 0 ); }
  void grow_tables( const uint64_t batch, const uint64_t rows, const uint64_t picked )
  {
    const uint64_t bytes = batch * ( sizeof( void* ) + sizeof( uint32_t ) ) + ( rows + picked ) * sizeof( uint32_t ) + 64;
    if ( bytes <= tables_bytes_ ) {
      return;
    }
    ops_.synchronize();
    if ( tables_host_ != nullptr ) {
      GLINT_GH( gh_host_free( tables_host_ ) );
    }
    tables_dev_ = ops_.device_allocate( bytes );
    void* pinned = nullptr;
    GLINT_GH( gh_host_malloc( &pinned, bytes ) );
    tables_host_ = static_cast<uint8_t*>( pinned );
    tables_bytes_ = bytes;
  }
  void begin_tables( const uint64_t batch, const uint64_t rows, const uint64_t picked )
  {
    // the last step ended with a wait for its results, so its upload has been read
    grow_tables( batch, rows, picked );
    t_batch_ = batch;
    t_rows_ = rows;
    t_picked_ = picked;
    max_start_ = 0;
  }
  uint64_t pos_off() const { return t_batch_ * sizeof( void* ); }
  uint64_t tokens_off() const { return pos_off() + t_batch_ * sizeof( uint32_t ); }
  uint64_t picked_off() const { return tokens_off() + t_rows_ * sizeof( uint32_t ); }
  uint32_t* table_tokens() { return reinterpret_cast<uint32_t*>( tables_host_ + tokens_off() ); }
  uint32_t* table_picked() { return reinterpret_cast<uint32_t*>( tables_host_ + picked_off() ); }
  void put_context( const size_t i, Context& ctx, const uint32_t pos, const uint32_t n_tokens )
  {
    GLINT_CHECK( ctx.prepare( pos, n_tokens ) );
    reinterpret_cast<void**>( tables_host_ )[i] = ctx.data();
    reinterpret_cast<uint32_t*>( tables_host_ + pos_off() )[i] = pos;
    max_start_ = std::max( max_start_, pos );
  }
  void upload_tables()
  {
    GLINT_GH( gh_memcpy( tables_dev_.get(), tables_host_, picked_off() + t_picked_ * sizeof( uint32_t ), GH_HOST_TO_DEVICE, 1, ops_.stream() ) );
  }
  const uint8_t* dev() const { return reinterpret_cast<const uint8_t*>( tables_dev_.get() ); }
  void* const* contexts_dev() const { return reinterpret_cast<void* const*>( tables_dev_.get() ); }
  const uint32_t* pos_dev() const { return reinterpret_cast<const uint32_t*>( dev() + pos_off() ); }
  const uint32_t* tokens_dev() const { return reinterpret_cast<const uint32_t*>( dev() + tokens_off() ); }
  const uint32_t* picked_dev() const { return reinterpret_cast<const uint32_t*>( dev() + picked_off() ); }

  // ---- ops -------------------------------------------------------------------------------------
  gh_stream_step no_step() const
  {
    gh_stream_step s {};
    s.eps = config_.eps;
    return s;
  }
  // what run k (or the output behind the last run) reads: the next product's input leaves with the residual update in front of it
  void lead_into( gh_stream_step& step, const size_t k, const bool all_rows_classified ) const
  {
    if ( k == runs_.size() ) {
      if ( all_rows_classified ) {
        step.next_norm = final_norm_;
        step.out = h_.get();
        step.out_stride = config_.width;
      }
    } else if ( runs_[k].first_of_pass ) {
      step.out = cat_.get();
      step.out_stride = 2ull * config_.width;
    } else {
      step.next_norm = layers_[runs_[k].layer].norm1;
      step.out = h_.get();
      step.out_stride = config_.width;
    }
  }

  void run_layers( const uint64_t batch, const uint32_t n_tokens, const bool all_rows_classified, float* residuals_out = nullptr )
  {
    const uint64_t rows = batch * n_tokens, width = config_.width;
    const gh_stream stream = ops_.stream();
    DType* x0 = config_.looped ? cat_.get() + width : nullptr;
    GLINT_GH( gh_embed_positions( x_.get(), tokens_dev(), pos_dev(), batch, n_tokens, embed_, pos_, width, config_.vocab, config_.max_positions, x0, 2 * width, DT,
                                  stream ) );
    {
      gh_stream_step first = no_step();
      lead_into( first, 0, all_rows_classified );
      GLINT_GH( gh_stream_out( x_.get(), width, rows, &first, DT, stream ) );
    }
    for ( size_t k = 0; k < runs_.size(); k++ ) {
      const auto& run = runs_[k];
      const auto& w = layers_[run.layer];
      const auto& part = settings_.plan->parts[k];
      if ( run.first_of_pass ) {
        gh_stream_step s = no_step();
        s.add = loop_step_ + (uint64_t)run.pass * width;
        s.next_norm = w.norm1;
        s.out = h_.get();
        s.out_stride = width;
        GLINT_GH( gh_matmul_stream( x_.get(), cat_.get(), loop_in_, 2 * width, width, rows, &s, DT, stream ) );
      }
      if ( config_.layers[run.layer].mlstm ) {
        GLINT_GH( gh_mlstm_forward( mixed_.get(), h_.get(), w.mix_in, width, &w.mlstm, w.bias_i, w.bias_f, w.head_norm, contexts_dev(), part.offset, pos_dev(), batch,
                                    n_tokens, DT, stream ) );
      } else {
        GLINT_GH( gh_matmul_window_append( q_.get(), h_.get(), w.mix_in, w.mix_bias, width, &w.attention, w.q_norm, w.k_norm, config_.eps, contexts_dev(),
                                           part.offset, pos_dev(), batch, n_tokens, DT, stream ) );
        GLINT_GH( gh_attn_window( mixed_.get(), q_.get(), &w.attention, w.distance_bias, contexts_dev(), part.offset, pos_dev(), batch, n_tokens, max_start_, DT,
                                  stream ) );
      }
      const bool ff = config_.layers[run.layer].ff > 0;
      gh_stream_step s = no_step();
      s.post_norm = w.norm1b;
      s.accumulate = 1;
      if ( ff ) {
        s.next_norm = w.norm2;
        s.out = h_.get();
        s.out_stride = width;
      } else {
        lead_into( s, k + 1, all_rows_classified );
      }
      GLINT_GH( gh_matmul_stream( x_.get(), mixed_.get(), w.mix_out, w.mixed_cols, width, rows, &s, DT, stream ) );
      if ( ff ) {
        const uint64_t hidden = config_.layers[run.layer].ff;
        GLINT_GH( gh_matmul_gate( hidden_.get(), h_.get(), w.gate_up, w.gate_up_bias, width, hidden, rows, GH_ACT_GELU_TANH, DT, stream ) );
        gh_stream_step d = no_step();
        d.bias = w.down_bias;
        d.post_norm = w.norm2b;
        d.accumulate = 1;
        lead_into( d, k + 1, all_rows_classified );
        GLINT_GH( gh_matmul_stream( x_.get(), hidden_.get(), w.down, hidden, width, rows, &d, DT, stream ) );
      }
      if ( residuals_out != nullptr ) {
        logit_ops_.copy( residuals_out + k * rows * width, x_.get(), rows * width * sizeof( float ), CopyType::DeviceToHost );
      }
    }
  }

  // logits of the first n rows of h
  void classify( const uint64_t n )
  {
    GLINT_GH( gh_matmul_scaled( logits_.get(), h_.get(), embed_, config_.width, config_.vocab, n, config_.logit_scale, DT, ops_.stream() ) );
  }
  // greedy token of the first n rows of the logits, on the host
  void sample( const uint64_t n )
  {
    GLINT_GH( gh_argmax( argmax_.data(), reinterpret_cast<uint32_t*>( argmax_dev_.get() ), logits_.get(), config_.vocab, n, GH_F32, ops_.stream() ) );
  }

  FamidraConfig config_;
  SettingsType settings_;
  ModelOptions options_;
  std::vector<FamidraConfig::Run> runs_;
  Operations ops_ {};
  hip::Operations<float> logit_ops_ {};
  DeviceSpans spans_ {};

  std::vector<Layer> layers_ {};
  std::vector<Tensor> tensors_ {};
  uint64_t weight_elements_ { 0 }, mixed_max_ { 0 }, query_max_ { 0 }, ff_max_ { 0 };
  typename Operations::DeviceUniquePtr weights_ {};
  DType *embed_ {}, *pos_ {}, *final_norm_ {}, *loop_in_ {}, *loop_step_ {};

  typename Operations::DeviceUniquePtr h_ {}, mixed_ {}, q_ {}, hidden_ {}, cat_ {}, tables_dev_ {};
  hip::Operations<float>::DeviceUniquePtr x_ {}, logits_ {}, picked_x_ {}, argmax_dev_ {};
  uint64_t rows_ { 0 }, logit_rows_ { 0 };
  std::vector<uint32_t> argmax_ {};
  uint8_t* tables_host_ { nullptr };
  uint64_t tables_bytes_ { 0 }, t_batch_ { 0 }, t_rows_ { 0 }, t_picked_ { 0 };
  uint32_t max_start_ { 0 };
};

} // namespace glint
